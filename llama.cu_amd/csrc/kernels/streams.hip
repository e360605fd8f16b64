// Several residual streams side by side: between two sublayers, in one pass over a row,
//
//   x_t <- sum_s mix[s, t] x_s + out[t] y          all t at once from the old x; y: the last sublayer's output
//   u    = sum_s read[s] x_s                       what the next sublayer reads
//   h    = u * rsqrt(mean(u^2) + eps) * w          its norm
//
// x: [n, S, d] 32-bit, updated in place.  Every part is optional but the norm: no y (the streams stay as they are), no `read` (all
// ones: the sum of the streams, behind the last sublayer).  y may be float32 planes of partial sums, added one after the other.
// One block per row; all of it is 32-bit with one rounding where h is stored.  Several streams are several times the bytes of one:
// the kernel reads and writes each once, V neighbouring columns of all streams a thread, and keeps u in registers for the norm.
#include "common.h"

template <class T, int V> struct alignas(V * sizeof(T)) StVec { T v[V]; };

constexpr int ST_MAX = 8;           // streams

// SMAX: room for so many streams (`streams` <= SMAX are there); ITEMS: pieces of V columns a thread takes.
template <int SMAX, int V, int ITEMS, class TY, class TO>
__global__ void __launch_bounds__(1024)
streams_norm_kernel(float *__restrict__ x, int streams, const TY *__restrict__ y, int planes, size_t plane_stride,
                    const float *__restrict__ mix, const float *__restrict__ out_w, const float *__restrict__ read,
                    const float *__restrict__ w, TO *__restrict__ h, int d, float eps, int write_back) {
    constexpr bool EXACT = SMAX <= 4;
    __shared__ float scratch[16];
    const int S = EXACT ? SMAX : streams, threads = blockDim.x;
    float *xr = x + (size_t)blockIdx.x * S * d;
    const TY *yr = y ? y + (size_t)blockIdx.x * d : nullptr;
    float u[ITEMS][V];
    float acc = 0.f;
#pragma unroll
    for (int k = 0; k < ITEMS; ++k) {
        const int c = (k * threads + threadIdx.x) * V;
#pragma unroll
        for (int e = 0; e < V; ++e) u[k][e] = 0.f;
        if (c >= d) continue;
        StVec<float, V> xs[SMAX];
#pragma unroll
        for (int s = 0; s < SMAX; ++s)
            if (EXACT || s < S) xs[s] = *(const StVec<float, V> *)(xr + (size_t)s * d + c);
        if (yr) {
            float yv[V];
#pragma unroll
            for (int e = 0; e < V; ++e) yv[e] = 0.f;
            for (int p0 = 0; p0 < planes; p0 += 4) {
                StVec<TY, V> q[4];
#pragma unroll
                for (int p = 0; p < 4; ++p) q[p] = *(const StVec<TY, V> *)(yr + (p0 + p < planes ? p0 + p : p0) * plane_stride + c);
#pragma unroll
                for (int p = 0; p < 4; ++p)
                    if (p0 + p < planes)
#pragma unroll
                        for (int e = 0; e < V; ++e) yv[e] += to_f32(q[p].v[e]);
            }
#pragma unroll
            for (int t = 0; t < SMAX; ++t) {
                if (!EXACT && t >= S) break;
                StVec<float, V> n;
#pragma unroll
                for (int e = 0; e < V; ++e) n.v[e] = out_w[t] * yv[e];
#pragma unroll
                for (int s = 0; s < SMAX; ++s)
                    if (EXACT || s < S)
#pragma unroll
                        for (int e = 0; e < V; ++e) n.v[e] = fmaf(mix[s * S + t], xs[s].v[e], n.v[e]);
                if (write_back) *(StVec<float, V> *)(xr + (size_t)t * d + c) = n;
                const float f = read ? read[t] : 1.f;
#pragma unroll
                for (int e = 0; e < V; ++e) u[k][e] = fmaf(f, n.v[e], u[k][e]);
            }
        } else {
#pragma unroll
            for (int s = 0; s < SMAX; ++s) {
                if (!EXACT && s >= S) break;
                const float f = read ? read[s] : 1.f;
#pragma unroll
                for (int e = 0; e < V; ++e) u[k][e] = fmaf(f, xs[s].v[e], u[k][e]);
            }
        }
#pragma unroll
        for (int e = 0; e < V; ++e) acc += u[k][e] * u[k][e];
    }
    const float f = rsqrtf(block_sum(acc, scratch) / (float)d + eps);
    TO *o = h + (size_t)blockIdx.x * d;
#pragma unroll
    for (int k = 0; k < ITEMS; ++k) {
        const int c = (k * threads + threadIdx.x) * V;
        if (c >= d) continue;
        const StVec<float, V> wv = *(const StVec<float, V> *)(w + c);
        StVec<TO, V> ov;
#pragma unroll
        for (int e = 0; e < V; ++e) ov.v[e] = from_f32<TO>(u[k][e] * f * wv.v[e]);
        *(StVec<TO, V> *)(o + c) = ov;
    }
}

// x: [n, streams, d] float32.  y: null, or `planes` arrays [n, d] of y_type, one after the other.  mix: [streams, streams] (from, to),
// out_w: [streams] (with y); read: [streams] or null; w: [d]; all float32.  h: [n, d] of h_type.
LCU_API int lcu_streams_norm(float *x, int streams, const void *y, int y_type, int planes, const float *mix, const float *out_w, const float *read,
                             const float *w, void *h, int h_type, int n, int d, float eps, int write_back, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (d <= 0 || streams < 1 || streams > ST_MAX || !x || !w || !h || planes < 1 || (y && (!mix || !out_w))) return LCU_BAD_ARGUMENT;
    const bool four = d % 4 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)h % 16 == 0;
    const int pieces = four ? d / 4 : d, most = n <= 192 ? 1024 : 256;
    int threads = (pieces + WAVE - 1) / WAVE * WAVE;
    if (threads > most) threads = most;
    int items = (pieces + threads - 1) / threads;
    if (items > (four ? 4 : 8)) {
        threads = 1024;
        items = (pieces + threads - 1) / threads;
        if (items > (four ? 4 : 8)) return LCU_UNSUPPORTED;
    }
    const size_t stride = (size_t)n * d;
#define GO(S, V, I, TY, TO) streams_norm_kernel<S, V, I, TY, TO><<<dim3(n), dim3(threads), 0, stream>>>(x, streams, (const TY *)y, planes, stride, mix, out_w, read, w, (TO *)h, d, eps, write_back)
#define SIZES(S, TY, TO)                              \
    do {                                              \
        if (!four) GO(S, 1, 8, TY, TO);               \
        else if (items == 1) GO(S, 4, 1, TY, TO);     \
        else if (items == 2) GO(S, 4, 2, TY, TO);     \
        else GO(S, 4, 4, TY, TO);                     \
    } while (0)
#define STREAMS(TY, TO)                               \
    do {                                              \
        if (streams == 1) SIZES(1, TY, TO);           \
        else if (streams == 2) SIZES(2, TY, TO);      \
        else if (streams == 3) SIZES(3, TY, TO);      \
        else if (streams == 4) SIZES(4, TY, TO);      \
        else SIZES(8, TY, TO);                        \
    } while (0)
    if (h_type == LCU_F32 && (!y || y_type == LCU_F32)) STREAMS(float, float);
    else if (h_type == LCU_BF16 && (!y || y_type == LCU_BF16)) STREAMS(bf16_t, bf16_t);
    else if (h_type == LCU_BF16 && y_type == LCU_F32) STREAMS(float, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef STREAMS
#undef SIZES
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}
