#pragma once
#include "common.h"

// Moves between the lanes of a group of sixteen inside the vector unit (no trip through LDS): the neighbour, the lane two
// away, the mirror image within eight and within sixteen.  After the first two every lane of a quad holds the quad's sum,
// so the mirror image within eight brings the other quad's, and the one within sixteen the other eight's.
__device__ __forceinline__ float lane_xor1(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, true));     // quad_perm [1, 0, 3, 2]
}
__device__ __forceinline__ float lane_xor2(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), 0x4E, 0xF, 0xF, true));     // quad_perm [2, 3, 0, 1]
}
__device__ __forceinline__ float lane_mirror8(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), 0x141, 0xF, 0xF, true));    // row_half_mirror
}
__device__ __forceinline__ float lane_mirror16(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), 0x140, 0xF, 0xF, true));    // row_mirror
}
// The sum over the sixteen lanes of a group, in all of them, always added in the same order.
__device__ __forceinline__ float sum_over_16(float v) {
    v += lane_xor1(v);
    v += lane_xor2(v);
    v += lane_mirror8(v);
    v += lane_mirror16(v);
    return v;
}

// The sum over a wave, in all lanes: within sixteen as above, then across the rows of sixteen by exchanging them in the vector unit.
__device__ __forceinline__ float wave_sum_in_place(float v) {
    const unsigned u = __float_as_uint(sum_over_16(v));
    const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);     // (rows 0 0 2 2, rows 1 1 3 3)
    const unsigned w = __float_as_uint(__uint_as_float(a[0]) + __uint_as_float(a[1]));
    const auto b = __builtin_amdgcn_permlane32_swap(w, w, false, false);     // (lower half twice, upper half twice)
    return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}
