// What stands between attention over the cache and its output product, head by head, in 32-bit with one rounding:
//
//   element gate     out[t, c] = x[t, c] * sigmoid(gate[t, c])                                   a gate of its own for every element
//   two maps         every head was attended twice over the same values; with a1, a2 the two outputs
//                    o = a1 - lambda a2,  o <- o / sqrt(mean(o^2) + eps) * factor,  o <- o * sigmoid(gate)   (the gate optional)
//
// The heads of x may stand further apart than their true size (dims of zeros behind it); out is [n, heads * dv].
#include "common.h"
#include "lane_moves.h"

__device__ __forceinline__ float sigmoid_of(float z) { return 1.0f / (1.0f + expf(-z)); }

template <class T, int V> struct alignas(V * sizeof(T)) MixVec { T v[V]; };

// V neighbouring columns a thread (V > 1: dv and every stride a multiple of V).
template <class TG, class T, int V>
__global__ void __launch_bounds__(256)
element_gate_kernel(const T *__restrict__ x, int head_stride, int row_stride, const TG *__restrict__ gate, int gate_stride, T *__restrict__ out,
                    int nh, int dv) {
    const int t = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * V;
    if (c >= nh * dv) return;
    const MixVec<T, V> a = *(const MixVec<T, V> *)(x + (size_t)t * row_stride + (size_t)(c / dv) * head_stride + c % dv);
    const MixVec<TG, V> g = *(const MixVec<TG, V> *)(gate + (size_t)t * gate_stride + c);
    MixVec<T, V> o;
#pragma unroll
    for (int e = 0; e < V; ++e) o.v[e] = from_f32<T>(to_f32(a.v[e]) * sigmoid_of(to_f32(g.v[e])));
    *(MixVec<T, V> *)(out + (size_t)t * nh * dv + c) = o;
}

// x: [n, row_stride] of type, head h's dv dims from column h * head_stride; gate: [n, gate_stride] of gate_type, nh * dv columns;
// out: [n, nh * dv] of type.
LCU_API int lcu_element_gate(const void *x, int type, int head_stride, int row_stride, const void *gate, int gate_type, int gate_stride,
                             void *out, int n, int nh, int dv, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (nh <= 0 || dv <= 0 || head_stride < dv || row_stride < (nh - 1) * head_stride + dv || gate_stride < nh * dv || !x || !gate || !out)
        return LCU_BAD_ARGUMENT;
    const int v = dv % 8 == 0 && head_stride % 8 == 0 && row_stride % 8 == 0 && gate_stride % 8 == 0 && (uintptr_t)x % 32 == 0 &&
                  (uintptr_t)gate % 32 == 0 && (uintptr_t)out % 32 == 0 ? 8 : 1;
    dim3 grid(n, (nh * dv + 256 * v - 1) / (256 * v)), block(256);
#define GO_V(TG, T, V) element_gate_kernel<TG, T, V><<<grid, block, 0, stream>>>((const T *)x, head_stride, row_stride, (const TG *)gate, gate_stride, (T *)out, nh, dv)
#define GO(TG, T)                   \
    do {                            \
        if (v == 8) GO_V(TG, T, 8); \
        else GO_V(TG, T, 1);        \
    } while (0)
    if (gate_type == LCU_F32 && type == LCU_F32) GO(float, float);
    else if (gate_type == LCU_F32 && type == LCU_BF16) GO(float, bf16_t);
    else if (gate_type == LCU_BF16 && type == LCU_BF16) GO(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
#undef GO_V
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// One wave per (token, head), four to a workgroup.  Head h's map m stands at column (2 * (h / map_group * map_group) + m *
// map_group + h % map_group) * head_stride: map_group 1: the two maps of a head side by side; the heads of a group g: first the
// group's first maps, then its second ones.  V neighbouring dims a lane at a time (V > 1: dv and every stride a multiple of
// V), ITEMS such: up to 640 dims a head.
template <class TG, class T, int V, int ITEMS>
__global__ void __launch_bounds__(256)
two_maps_kernel(const T *__restrict__ x, int head_stride, int row_stride, int map_group, float lambda, float eps, float factor,
                const TG *__restrict__ gate, int gate_stride, T *__restrict__ out, int nh, int dv) {
    const int t = blockIdx.x, h = blockIdx.y * 4 + threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
    if (h >= nh) return;
    const int first = 2 * (h / map_group * map_group) + h % map_group;
    const T *a1 = x + (size_t)t * row_stride + (size_t)first * head_stride, *a2 = a1 + (size_t)map_group * head_stride;
    const TG *gr = gate ? gate + (size_t)t * gate_stride + (size_t)h * dv : nullptr;
    float o[ITEMS][V], ss = 0.f;
#pragma unroll
    for (int i = 0; i < ITEMS; ++i) {
        const int c = (lane + WAVE * i) * V;
        MixVec<T, V> p = {}, q = {};
        if (c < dv) {
            p = *(const MixVec<T, V> *)(a1 + c);
            q = *(const MixVec<T, V> *)(a2 + c);
        }
#pragma unroll
        for (int e = 0; e < V; ++e) {
            o[i][e] = to_f32(p.v[e]) - lambda * to_f32(q.v[e]);
            ss += o[i][e] * o[i][e];
        }
    }
    const float f = factor / sqrtf(wave_sum_in_place(ss) / (float)dv + eps);
#pragma unroll
    for (int i = 0; i < ITEMS; ++i) {
        const int c = (lane + WAVE * i) * V;
        if (c >= dv) break;
        MixVec<TG, V> g = {};
        if (gr) g = *(const MixVec<TG, V> *)(gr + c);
        MixVec<T, V> w;
#pragma unroll
        for (int e = 0; e < V; ++e) w.v[e] = from_f32<T>(o[i][e] * f * (gr ? sigmoid_of(to_f32(g.v[e])) : 1.0f));
        *(MixVec<T, V> *)(out + ((size_t)t * nh + h) * dv + c) = w;
    }
}

// x: [n, row_stride] of type, 2 * nh heads head_stride apart; gate: null or [n, gate_stride] of gate_type; out: [n, nh * dv] of type.
LCU_API int lcu_two_maps(const void *x, int type, int head_stride, int row_stride, int map_group, float lambda, float eps, float factor,
                         const void *gate, int gate_type, int gate_stride, void *out, int n, int nh, int dv, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (nh <= 0 || nh > 65535 || dv <= 0 || dv > 640 || head_stride < dv || row_stride < 2 * nh * head_stride || map_group <= 0 ||
        nh % map_group || (gate && gate_stride < nh * dv) || !x || !out)
        return LCU_BAD_ARGUMENT;
    const bool two = dv % 2 == 0 && head_stride % 2 == 0 && row_stride % 2 == 0 && gate_stride % 2 == 0 && (uintptr_t)x % 8 == 0 &&
                     (uintptr_t)gate % 8 == 0 && (uintptr_t)out % 8 == 0;
    dim3 grid(n, (nh + 3) / 4), block(256);
#define GO(TG, T)                                \
    do {                                         \
        if (two && dv <= 128) GO_V(TG, T, 2, 1); \
        else if (two) GO_V(TG, T, 2, 5);         \
        else GO_V(TG, T, 1, 10);                 \
    } while (0)
#define GO_V(TG, T, V, I) two_maps_kernel<TG, T, V, I><<<grid, block, 0, stream>>>((const T *)x, head_stride, row_stride, map_group, lambda, eps, factor, (const TG *)gate, gate_stride, (T *)out, nh, dv)
    if (gate_type == LCU_F32 && type == LCU_F32) GO(float, float);
    else if (gate_type == LCU_F32 && type == LCU_BF16) GO(float, bf16_t);
    else if (gate_type == LCU_BF16 && type == LCU_BF16) GO(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
#undef GO_V
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}
