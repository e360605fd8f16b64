// What a gated feed-forward makes of its two projections, by kind, in 32-bit:
//   GATE_SILU       silu(gate) * up
//   GATE_GELU_TANH  gelu(gate) * up with the tanh form, 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))
//   GATE_LIMITED    g sigmoid(alpha g) (u + 1) with g = min(gate, limit) and u = up held within -limit .. limit
#pragma once
#include "common.h"

enum { GATE_SILU = 0, GATE_GELU_TANH = 1, GATE_LIMITED = 2 };

template <int ACT>
__device__ __forceinline__ float gate_up(float gate, float up, float alpha, float limit) {
    if (ACT == GATE_GELU_TANH) return 0.5f * gate * (1.0f + tanhf(0.7978845608028654f * (gate + 0.044715f * gate * gate * gate))) * up;
    if (ACT == GATE_LIMITED) {
        const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
        return g * (1.0f / (1.0f + expf(-alpha * g))) * (u + 1.0f);
    }
    return gate * (1.0f / (1.0f + expf(-gate))) * up;
}

// The same where the kind is known at run time only (the epilogues of the matrix products): limit > 0 says GATE_LIMITED.
__device__ __forceinline__ float gate_up_of(float gate, float up, float alpha, float limit) {
    return limit > 0.f ? gate_up<GATE_LIMITED>(gate, up, alpha, limit) : gate_up<GATE_SILU>(gate, up, alpha, limit);
}
