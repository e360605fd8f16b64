// What stands between attention over the cache and its output product, head by head, in 32-bit with one rounding:
//
//   element gate     out[t, c] = x[t, c] * sigmoid(gate[t, c])                                   a gate of its own for every element
//   two maps         every head was attended twice over the same values; with a1, a2 the two outputs
//                    o = a1 - lambda a2,  o <- o / sqrt(mean(o^2) + eps) * factor,  o <- o * sigmoid(gate)   (the gate optional)
//
// The heads of x may stand further apart than their true size (dims of zeros behind it); out is [n, heads * dv].
#include "common.h"

__device__ __forceinline__ float sigmoid_of(float z) { return 1.0f / (1.0f + expf(-z)); }

template <class TG, class T>
__global__ void element_gate_kernel(const T *__restrict__ x, int head_stride, int row_stride, const TG *__restrict__ gate, int gate_stride,
                                    T *__restrict__ out, int nh, int dv) {
    const int t = blockIdx.x;
    for (int c = threadIdx.x; c < nh * dv; c += blockDim.x) {
        const float v = to_f32(x[(size_t)t * row_stride + (size_t)(c / dv) * head_stride + c % dv]);
        out[(size_t)t * nh * dv + c] = from_f32<T>(v * sigmoid_of(to_f32(gate[(size_t)t * gate_stride + c])));
    }
}

// x: [n, row_stride] of type, head h's dv dims from column h * head_stride; gate: [n, gate_stride] of gate_type, nh * dv columns;
// out: [n, nh * dv] of type.
LCU_API int lcu_element_gate(const void *x, int type, int head_stride, int row_stride, const void *gate, int gate_type, int gate_stride,
                             void *out, int n, int nh, int dv, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (nh <= 0 || dv <= 0 || head_stride < dv || row_stride < (nh - 1) * head_stride + dv || gate_stride < nh * dv || !x || !gate || !out)
        return LCU_BAD_ARGUMENT;
    dim3 grid(n), block(256);
#define GO(TG, T) element_gate_kernel<TG, T><<<grid, block, 0, stream>>>((const T *)x, head_stride, row_stride, (const TG *)gate, gate_stride, (T *)out, nh, dv)
    if (gate_type == LCU_F32 && type == LCU_F32) GO(float, float);
    else if (gate_type == LCU_F32 && type == LCU_BF16) GO(float, bf16_t);
    else if (gate_type == LCU_BF16 && type == LCU_BF16) GO(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// One wave per (token, head).  Head h's map m stands at column (2 * (h / map_group * map_group) + m * map_group + h %
// map_group) * head_stride: map_group 1: the two maps of a head side by side; the heads of a group g: first the
// group's first maps, then its second ones.
constexpr int MM_ITEMS = 10;                     // up to 640 dims a head

template <class TG, class T>
__global__ void __launch_bounds__(WAVE)
two_maps_kernel(const T *__restrict__ x, int head_stride, int row_stride, int map_group, float lambda, float eps, float factor,
                const TG *__restrict__ gate, int gate_stride, T *__restrict__ out, int nh, int dv) {
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const int first = 2 * (h / map_group * map_group) + h % map_group;
    const T *a1 = x + (size_t)t * row_stride + (size_t)first * head_stride, *a2 = a1 + (size_t)map_group * head_stride;
    float o[MM_ITEMS], ss = 0.f;
#pragma unroll
    for (int i = 0; i < MM_ITEMS; ++i) {
        const int c = lane + WAVE * i;
        o[i] = c < dv ? to_f32(a1[c]) - lambda * to_f32(a2[c]) : 0.f;
        ss += o[i] * o[i];
    }
    const float f = factor / sqrtf(wave_sum(ss) / (float)dv + eps);
#pragma unroll
    for (int i = 0; i < MM_ITEMS; ++i) {
        const int c = lane + WAVE * i;
        if (c >= dv) break;
        const float g = gate ? sigmoid_of(to_f32(gate[(size_t)t * gate_stride + (size_t)h * dv + c])) : 1.0f;
        out[((size_t)t * nh + h) * dv + c] = from_f32<T>(o[i] * f * g);
    }
}

// x: [n, row_stride] of type, 2 * nh heads head_stride apart; gate: null or [n, gate_stride] of gate_type; out: [n, nh * dv] of type.
LCU_API int lcu_two_maps(const void *x, int type, int head_stride, int row_stride, int map_group, float lambda, float eps, float factor,
                         const void *gate, int gate_type, int gate_stride, void *out, int n, int nh, int dv, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (nh <= 0 || nh > 65535 || dv <= 0 || dv > WAVE * MM_ITEMS || head_stride < dv || row_stride < 2 * nh * head_stride || map_group <= 0 ||
        nh % map_group || (gate && gate_stride < nh * dv) || !x || !out)
        return LCU_BAD_ARGUMENT;
    dim3 grid(n, nh), block(WAVE);
#define GO(TG, T) two_maps_kernel<TG, T><<<grid, block, 0, stream>>>((const T *)x, head_stride, row_stride, map_group, lambda, eps, factor, (const TG *)gate, gate_stride, (T *)out, nh, dv)
    if (gate_type == LCU_F32 && type == LCU_F32) GO(float, float);
    else if (gate_type == LCU_F32 && type == LCU_BF16) GO(float, bf16_t);
    else if (gate_type == LCU_BF16 && type == LCU_BF16) GO(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}
