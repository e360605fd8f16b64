// Row-wise kernels: embedding gather, row gather, RMS norm fused with the residual
// sum, SwiGLU, residual add.  Sums, the norm and the activation are computed in
// 32-bit whatever the storage type.
#include "common.h"
#include "gate_act.h"

// ---------------------------------------------------------------- embedding gather
// out[i, k, :] = table[ids[i], :] * scale for k < copies (the product in 32-bit).  An id outside the table writes NaN into the row
// (the host checks ids before; this keeps a bad id from reading out of bounds).
template <class TT, class TO>
__global__ void embedding_gather_kernel(TO *__restrict__ out, const TT *__restrict__ table,
                                        const int *__restrict__ ids, int d, int vocab, float scale, int copies) {
    const int row = blockIdx.x;
    const int id = ids[row / copies];
    TO *o = out + (size_t)row * d;
    if (id < 0 || id >= vocab) {
        for (int c = threadIdx.x; c < d; c += blockDim.x) o[c] = from_f32<TO>(__uint_as_float(0x7fc00000u));
        return;
    }
    const TT *t = table + (size_t)id * d;
    if (d % 8 == 0 && ((size_t)t % (8 * sizeof(TT))) == 0 && ((size_t)o % (8 * sizeof(TO))) == 0) {
        // eight neighbouring elements per load (a row is read once, from memory: few, wide loads)
        struct alignas(8 * sizeof(TT)) In8 { TT v[8]; };
        struct alignas(8 * sizeof(TO)) Out8 { TO v[8]; };
        for (int c = threadIdx.x * 8; c < d; c += blockDim.x * 8) {
            const In8 in = *(const In8 *)(t + c);
            Out8 res;
#pragma unroll
            for (int e = 0; e < 8; ++e) res.v[e] = from_f32<TO>(to_f32(in.v[e]) * scale);
            *(Out8 *)(o + c) = res;
        }
        return;
    }
    for (int c = threadIdx.x; c < d; c += blockDim.x) o[c] = from_f32<TO>(to_f32(t[c]) * scale);
}

LCU_API int lcu_embedding_gather(void *out, int out_type, const void *table, int table_type,
                                 const int *ids, int n, int d, int vocab, float scale, int copies, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (d <= 0 || vocab <= 0 || copies <= 0) return LCU_BAD_ARGUMENT;
    dim3 grid((unsigned)n * copies), block(256);
#define GO(TT, TO) embedding_gather_kernel<TT, TO><<<grid, block, 0, stream>>>((TO *)out, (const TT *)table, ids, d, vocab, scale, copies)
    if (table_type == LCU_F32 && out_type == LCU_F32) GO(float, float);
    else if (table_type == LCU_BF16 && out_type == LCU_F32) GO(bf16_t, float);
    else if (table_type == LCU_BF16 && out_type == LCU_BF16) GO(bf16_t, bf16_t);
    else if (table_type == LCU_F32 && out_type == LCU_BF16) GO(float, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// ---------------------------------------------------------------- row gather
// V neighbouring elements a thread, the row shared out over blockIdx.y (few rows are gathered, often one: what counts is that all of
// it is on its way at once).
template <class T, int V>
__global__ void __launch_bounds__(256)
gather_rows_kernel(T *__restrict__ out, const T *__restrict__ x, const int *__restrict__ rows, int d, int n_src) {
    struct alignas(V * sizeof(T)) Piece { T v[V]; };
    const int r = rows[blockIdx.x], c = (blockIdx.y * 256 + threadIdx.x) * V;
    if (c >= d) return;
    Piece p;
    if (r < 0 || r >= n_src) {
#pragma unroll
        for (int e = 0; e < V; ++e) p.v[e] = from_f32<T>(__uint_as_float(0x7fc00000u));
    } else {
        p = *(const Piece *)(x + (size_t)r * d + c);
    }
    *(Piece *)(out + (size_t)blockIdx.x * d + c) = p;
}

LCU_API int lcu_gather_rows(void *out, const void *x, int type, const int *rows, int n_out, int d,
                            int n_src, hipStream_t stream) {
    if (n_out <= 0) return LCU_OK;
    if (d <= 0) return LCU_BAD_ARGUMENT;
    const bool four = d % 4 == 0 && (uintptr_t)out % 16 == 0 && (uintptr_t)x % 16 == 0;
    const int per = four ? 1024 : 256;
    if ((d + per - 1) / per > 65535) return LCU_BAD_ARGUMENT;
    dim3 grid(n_out, (d + per - 1) / per), block(256);
#define GO(T)                                                                                                             \
    do {                                                                                                                  \
        if (four) gather_rows_kernel<T, 4><<<grid, block, 0, stream>>>((T *)out, (const T *)x, rows, d, n_src);           \
        else gather_rows_kernel<T, 1><<<grid, block, 0, stream>>>((T *)out, (const T *)x, rows, d, n_src);                \
    } while (0)
    if (type == LCU_F32) GO(float);
    else if (type == LCU_BF16) GO(bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// ---------------------------------------------------------------- RMS norm (+ residual sum)
// One block per row.  If `delta` is given: x += delta first (in 32-bit, written back
// when x is 32-bit: x is then the residual stream); delta may be `planes` planes [n, d],
// `plane_stride` elements apart (a product's partial sums over slices of K), which are added
// one after the other in the order of the planes; every element of the branch's output enters
// times `delta_scale` (1: as it is).  Then
//   y = x * rsqrt(sum(x^2)/d + eps) * w        (32-bit, one rounding at the store)
// The order of the sum depends on d and the block size only, not on the batch.
template <class TX, class TD, class TW, class TO>
__global__ void rmsnorm_kernel(TX *__restrict__ x, const TD *__restrict__ delta, const TW *__restrict__ w,
                               TO *__restrict__ out, int d, float eps, int write_back, int planes, size_t plane_stride, float delta_scale) {
    __shared__ float scratch[16];
    TX *xr = x + (size_t)blockIdx.x * d;
    const TD *dr = delta ? delta + (size_t)blockIdx.x * d : nullptr;
    float acc = 0.f;
    for (int c = threadIdx.x; c < d; c += blockDim.x) {
        float v = to_f32(xr[c]);
        if (dr) {
            for (int p = 0; p < planes; ++p) v = fmaf(delta_scale, to_f32(dr[p * plane_stride + c]), v);
            if (write_back) xr[c] = from_f32<TX>(v);
        }
        acc += v * v;
    }
    const float total = block_sum(acc, scratch);
    const float rms = rsqrtf(total / (float)d + eps);
    TO *o = out + (size_t)blockIdx.x * d;
    for (int c = threadIdx.x; c < d; c += blockDim.x) {
        float v = to_f32(xr[c]);
        if (dr && !write_back)
            for (int p = 0; p < planes; ++p) v = fmaf(delta_scale, to_f32(dr[p * plane_stride + c]), v);
        o[c] = from_f32<TO>(rms * v * to_f32(w[c]));
    }
}

// The same for rows of up to 8192 elements whose width is a multiple of 4: one read of
// the row (four elements per load), the row kept in registers between the sum and the
// scaling.  The row is dealt to 1024 virtual threads, two loads each; a block has 1024
// threads (few rows leave most of the chip idle: what counts then is how many loads a row has
// in flight) or 256 that play four virtual threads each (many rows: fewer, longer-lived waves
// stream faster).  The sums are added as the 1024 threads would add them, wave by wave, so
// the result does not depend on the block's size, only on d.  The planes are loaded four at
// a time.
constexpr int NORM_VTHREADS = 1024, NORM_ITEMS = 2;

template <class T> struct alignas(4 * sizeof(T)) Vec4 { T v[4]; };

template <int THREADS, class TX, class TD, class TW, class TO>
__global__ void __launch_bounds__(THREADS)
rmsnorm_fast_kernel(TX *__restrict__ x, const TD *__restrict__ delta, const TW *__restrict__ w, TO *__restrict__ out,
                    int d, float eps, int write_back, int planes, size_t plane_stride, float delta_scale) {
    constexpr int PLAY = NORM_VTHREADS / THREADS;           // virtual threads per thread
    __shared__ float scratch[NORM_VTHREADS / WAVE];
    TX *xr = x + (size_t)blockIdx.x * d;
    const TD *dr = delta ? delta + (size_t)blockIdx.x * d : nullptr;
    float v[PLAY][NORM_ITEMS][4];
#pragma unroll
    for (int j = 0; j < PLAY; ++j) {
        float acc = 0.f;
#pragma unroll
        for (int i = 0; i < NORM_ITEMS; ++i) {
            const int c = (i * NORM_VTHREADS + j * THREADS + threadIdx.x) * 4;
            if (c < d) {
                const Vec4<TX> xv = *(const Vec4<TX> *)(xr + c);
#pragma unroll
                for (int e = 0; e < 4; ++e) v[j][i][e] = to_f32(xv.v[e]);
                if (dr) {
                    for (int p0 = 0; p0 < planes; p0 += 4) {
                        Vec4<TD> dv[4];
#pragma unroll
                        for (int q = 0; q < 4; ++q) dv[q] = *(const Vec4<TD> *)(dr + (p0 + q < planes ? p0 + q : p0) * plane_stride + c);
#pragma unroll
                        for (int q = 0; q < 4; ++q)
                            if (p0 + q < planes) {
#pragma unroll
                                for (int e = 0; e < 4; ++e) v[j][i][e] = fmaf(delta_scale, to_f32(dv[q].v[e]), v[j][i][e]);
                            }
                    }
                    Vec4<TX> back;
#pragma unroll
                    for (int e = 0; e < 4; ++e) back.v[e] = from_f32<TX>(v[j][i][e]);
                    if (write_back) *(Vec4<TX> *)(xr + c) = back;
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) acc += v[j][i][e] * v[j][i][e];
            }
        }
        // the wave of the 1024 threads that these virtual threads are
        acc = wave_sum(acc);
        if ((threadIdx.x & (WAVE - 1)) == 0) scratch[j * (THREADS / WAVE) + threadIdx.x / WAVE] = acc;
    }
    __syncthreads();
    float total = 0.f;
#pragma unroll
    for (int k = 0; k < NORM_VTHREADS / WAVE; ++k) total += scratch[k];
    const float rms = rsqrtf(total / (float)d + eps);
    TO *o = out + (size_t)blockIdx.x * d;
#pragma unroll
    for (int j = 0; j < PLAY; ++j)
#pragma unroll
        for (int i = 0; i < NORM_ITEMS; ++i) {
            const int c = (i * NORM_VTHREADS + j * THREADS + threadIdx.x) * 4;
            if (c < d) {
                const Vec4<TW> wv = *(const Vec4<TW> *)(w + c);
                Vec4<TO> ov;
#pragma unroll
                for (int e = 0; e < 4; ++e) ov.v[e] = from_f32<TO>(rms * v[j][i][e] * to_f32(wv.v[e]));
                *(Vec4<TO> *)(o + c) = ov;
            }
        }
}

template <class TX, class TD, class TO>
static int rmsnorm_w(void *x, const void *delta, const void *w, int w_type, void *out, int n, int d, float eps,
                     int write_back, float delta_scale, hipStream_t stream, int planes = 1, size_t plane_stride = 0) {
    dim3 grid(n), block(d >= 2048 ? 512 : 256);
    if (d % 4 == 0 && d <= NORM_VTHREADS * NORM_ITEMS * 4) {
#define FAST(T_, TW_) rmsnorm_fast_kernel<T_, TX, TD, TW_, TO><<<grid, dim3(T_), 0, stream>>>((TX *)x, (const TD *)delta, (const TW_ *)w, (TO *)out, d, eps, write_back, planes, plane_stride, delta_scale)
        const bool few = n <= 192;        // (measured with four planes: steps of 160 and 192 rows 2 % faster with 1024 threads, of 256 rows 1 % slower)
        if (w_type == LCU_F32) {
            if (few) FAST(1024, float); else FAST(256, float);
        } else if (w_type == LCU_BF16) {
            if (few) FAST(1024, bf16_t); else FAST(256, bf16_t);
        } else {
            return LCU_BAD_ARGUMENT;
        }
#undef FAST
        LCU_LAUNCH_CHECK();
        return LCU_OK;
    }
    if (w_type == LCU_F32)
        rmsnorm_kernel<TX, TD, float, TO><<<grid, block, 0, stream>>>((TX *)x, (const TD *)delta, (const float *)w, (TO *)out, d, eps, write_back, planes, plane_stride, delta_scale);
    else if (w_type == LCU_BF16)
        rmsnorm_kernel<TX, TD, bf16_t, TO><<<grid, block, 0, stream>>>((TX *)x, (const TD *)delta, (const bf16_t *)w, (TO *)out, d, eps, write_back, planes, plane_stride, delta_scale);
    else
        return LCU_BAD_ARGUMENT;
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// x: [n, d] of x_type (read; written when write_back and delta are set), delta: [n, d] of
// delta_type or null, out: [n, d] of act_type.  delta enters times delta_scale.
LCU_API int lcu_rmsnorm(void *x, int x_type, const void *delta, int delta_type, const void *w, int w_type, void *out,
                        int act_type, int n, int d, float eps, int write_back, float delta_scale, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (d <= 0) return LCU_BAD_ARGUMENT;
#define GO(TX, TD, TO) return rmsnorm_w<TX, TD, TO>(x, delta, w, w_type, out, n, d, eps, write_back, delta_scale, stream)
    if (x_type == LCU_F32 && act_type == LCU_F32 && delta_type == LCU_F32) GO(float, float, float);
    if (x_type == LCU_F32 && act_type == LCU_F32 && delta_type == LCU_BF16) GO(float, bf16_t, float);
    if (x_type == LCU_F32 && act_type == LCU_BF16 && delta_type == LCU_BF16) GO(float, bf16_t, bf16_t);
    if (x_type == LCU_BF16 && act_type == LCU_BF16 && delta_type == LCU_BF16) GO(bf16_t, bf16_t, bf16_t);
#undef GO
    return LCU_BAD_ARGUMENT;
}

// The same with the branch's output as `planes` float32 planes [n, d], one after the other:
// x (float32) += delta_scale * (plane 0, plane 1, ... in this order), then the norm.  d a multiple of 4.
LCU_API int lcu_rmsnorm_planes(float *x, const float *planes_ptr, int planes, const void *w, int w_type, void *out,
                               int act_type, int n, int d, float eps, int write_back, float delta_scale, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (d <= 0 || d % 4 || planes <= 0 || !planes_ptr) return LCU_BAD_ARGUMENT;
    const size_t stride = (size_t)n * d;
    if (act_type == LCU_F32) return rmsnorm_w<float, float, float>(x, planes_ptr, w, w_type, out, n, d, eps, write_back, delta_scale, stream, planes, stride);
    if (act_type == LCU_BF16) return rmsnorm_w<float, float, bf16_t>(x, planes_ptr, w, w_type, out, n, d, eps, write_back, delta_scale, stream, planes, stride);
    return LCU_BAD_ARGUMENT;
}

// ---------------------------------------------------------------- the residual stream as a product's operand
// x (f32) += delta_scale * delta (planes as above; null: nothing), written back; out[r, c] = x[r, c] in the compute type, rows ldo
// apart: the stream (or, with no delta, a copy of it) as columns of a wider operand.
// V neighbouring columns a thread, all loads of a thread's planes (four at a time) before it waits for one.
template <class T, int V> struct alignas(V * sizeof(T)) VecN { T v[V]; };

template <class TD, class TO, int V>
__global__ void __launch_bounds__(256)
stream_rows_kernel(float *__restrict__ x, const TD *__restrict__ delta, int planes, size_t plane_stride, float delta_scale,
                   TO *__restrict__ out, int ldo, int d) {
    const int c = (blockIdx.y * 256 + threadIdx.x) * V;
    if (c >= d) return;
    const size_t at = (size_t)blockIdx.x * d + c;
    VecN<float, V> v = *(const VecN<float, V> *)(x + at);
    if (delta) {
        for (int p0 = 0; p0 < planes; p0 += 4) {
            VecN<TD, V> q[4];
#pragma unroll
            for (int p = 0; p < 4; ++p) q[p] = *(const VecN<TD, V> *)(delta + (p0 + p < planes ? p0 + p : p0) * plane_stride + at);
#pragma unroll
            for (int p = 0; p < 4; ++p)
                if (p0 + p < planes)
#pragma unroll
                    for (int e = 0; e < V; ++e) v.v[e] = fmaf(delta_scale, to_f32(q[p].v[e]), v.v[e]);
        }
        *(VecN<float, V> *)(x + at) = v;
    }
    VecN<TO, V> o;
#pragma unroll
    for (int e = 0; e < V; ++e) o.v[e] = from_f32<TO>(v.v[e]);
    *(VecN<TO, V> *)(out + (size_t)blockIdx.x * ldo + c) = o;
}

LCU_API int lcu_stream_rows(float *x, const void *delta, int delta_type, int planes, float delta_scale, void *out, int out_type, int ldo,
                            int n, int d, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (d <= 0 || ldo < d || planes < 1 || !x || !out) return LCU_BAD_ARGUMENT;
    const size_t stride = (size_t)n * d;
    const int v = d % 4 == 0 && ldo % 4 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)delta % 16 == 0 && (uintptr_t)out % 16 == 0 ? 4 : 1;
    dim3 grid(n, (d + 256 * v - 1) / (256 * v)), block(256);
#define GO(TD, TO)                                                                                                                              \
    do {                                                                                                                                        \
        if (v == 4) stream_rows_kernel<TD, TO, 4><<<grid, block, 0, stream>>>(x, (const TD *)delta, planes, stride, delta_scale, (TO *)out, ldo, d); \
        else stream_rows_kernel<TD, TO, 1><<<grid, block, 0, stream>>>(x, (const TD *)delta, planes, stride, delta_scale, (TO *)out, ldo, d);   \
    } while (0)
    if (delta_type == LCU_F32 && out_type == LCU_F32) GO(float, float);
    else if (delta_type == LCU_F32 && out_type == LCU_BF16) GO(float, bf16_t);
    else if (delta_type == LCU_BF16 && out_type == LCU_BF16) GO(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// ---------------------------------------------------------------- residual add: x (f32) += scale * delta
template <class TD>
__global__ void residual_add_kernel(float *__restrict__ x, const TD *__restrict__ delta, size_t total, float scale) {
    size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < total) x[i] = fmaf(scale, to_f32(delta[i]), x[i]);
}

LCU_API int lcu_residual_add(float *x, const void *delta, int delta_type, long long total, float scale, hipStream_t stream) {
    if (total <= 0) return LCU_OK;
    dim3 block(256), grid((unsigned)((total + 255) / 256));
    if (delta_type == LCU_F32) residual_add_kernel<float><<<grid, block, 0, stream>>>(x, (const float *)delta, (size_t)total, scale);
    else if (delta_type == LCU_BF16) residual_add_kernel<bf16_t><<<grid, block, 0, stream>>>(x, (const bf16_t *)delta, (size_t)total, scale);
    else return LCU_BAD_ARGUMENT;
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// ---------------------------------------------------------------- SwiGLU and its kin
// out[r, c] = gate_up(gate, up) with gate = gu[r, c], up = gu[r, di + c] (gate_act.h).
template <class T, int ACT>
__global__ void swiglu_kernel(T *__restrict__ out, const T *__restrict__ gu, int di, float alpha, float limit) {
    const int c = blockIdx.x * blockDim.x + threadIdx.x;
    if (c >= di) return;
    const size_t r = blockIdx.y;
    const float gate = to_f32(gu[r * 2 * di + c]);
    const float up = to_f32(gu[r * 2 * di + di + c]);
    out[r * di + c] = from_f32<T>(gate_up<ACT>(gate, up, alpha, limit));
}

// The same, eight neighbouring columns per thread (16-byte loads of bfloat16, 32-byte of
// float32); for widths that are multiples of 8.
template <class T> struct alignas(8 * sizeof(T)) Vec8 { T v[8]; };

template <class T, int ACT>
__global__ void swiglu_vec8_kernel(T *__restrict__ out, const T *__restrict__ gu, int di, float alpha, float limit) {
    const int c = (blockIdx.x * blockDim.x + threadIdx.x) * 8;
    if (c >= di) return;
    const size_t r = blockIdx.y;
    const Vec8<T> g = *(const Vec8<T> *)(gu + r * 2 * di + c);
    const Vec8<T> u = *(const Vec8<T> *)(gu + r * 2 * di + di + c);
    Vec8<T> o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o.v[e] = from_f32<T>(gate_up<ACT>(to_f32(g.v[e]), to_f32(u.v[e]), alpha, limit));
    *(Vec8<T> *)(out + r * di + c) = o;
}

template <class T, int ACT>
static void swiglu_launch(T *out, const T *gate_up, int rows, int di, float alpha, float limit, hipStream_t stream) {
    const dim3 block(256);
    if (di % 8 == 0)
        swiglu_vec8_kernel<T, ACT><<<dim3((di / 8 + 255) / 256, rows), block, 0, stream>>>(out, gate_up, di, alpha, limit);
    else
        swiglu_kernel<T, ACT><<<dim3((di + 255) / 256, rows), block, 0, stream>>>(out, gate_up, di, alpha, limit);
}

template <class T>
static int swiglu_t(T *out, const T *gu, int n, int di, int act, float alpha, float limit, hipStream_t stream) {
    // grid.y is limited to 65535 rows: larger batches go in slices
    for (int r0 = 0; r0 < n; r0 += 65535) {
        const int rows = (n - r0) < 65535 ? (n - r0) : 65535;
        T *o = out + (size_t)r0 * di;
        const T *g = gu + (size_t)r0 * 2 * di;
        if (act == GATE_SILU) swiglu_launch<T, GATE_SILU>(o, g, rows, di, alpha, limit, stream);
        else if (act == GATE_GELU_TANH) swiglu_launch<T, GATE_GELU_TANH>(o, g, rows, di, alpha, limit, stream);
        else swiglu_launch<T, GATE_LIMITED>(o, g, rows, di, alpha, limit, stream);
    }
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// act: 0 silu, 1 the tanh form of gelu, 2 the limited form with alpha and limit (gate_act.h).
LCU_API int lcu_swiglu(void *out, const void *gate_up, int type, int n, int di, int act, float alpha, float limit, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (di <= 0 || act < GATE_SILU || act > GATE_LIMITED || (act == GATE_LIMITED && !(limit > 0.f))) return LCU_BAD_ARGUMENT;
    if (type == LCU_F32) return swiglu_t<float>((float *)out, (const float *)gate_up, n, di, act, alpha, limit, stream);
    if (type == LCU_BF16) return swiglu_t<bf16_t>((bf16_t *)out, (const bf16_t *)gate_up, n, di, act, alpha, limit, stream);
    return LCU_BAD_ARGUMENT;
}

// ---------------------------------------------------------------- a cap on the logits
// x <- cap * tanh(x / cap), in place, 32-bit.
__global__ void softcap_kernel(float *__restrict__ x, size_t total, float cap) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < total) x[i] = cap * tanhf(x[i] / cap);
}

LCU_API int lcu_softcap(float *x, long long total, float cap, hipStream_t stream) {
    if (total <= 0) return LCU_OK;
    if (!(cap > 0.f)) return LCU_BAD_ARGUMENT;
    softcap_kernel<<<dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream>>>(x, (size_t)total, cap);
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// ---------------------------------------------------------------- token feedback
// tokens[dst[i]] = sampled[src[i]]: the ids that the last step sampled become this step's
// inputs on the device, so the host need not wait for them before it launches
// (llama.cu/src/op/fast_embedding.cuh:1-15 does the same from its sampled pairs).
__global__ void feed_tokens_kernel(int *__restrict__ tokens, const int *__restrict__ sampled,
                                   const int *__restrict__ src, const int *__restrict__ dst, int n, int n_tokens,
                                   int n_sampled) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const int s = src[i], d = dst[i];
    if (s >= 0 && s < n_sampled && d >= 0 && d < n_tokens) tokens[d] = sampled[s];
}

LCU_API int lcu_feed_tokens(int *tokens, int n_tokens, const int *sampled, int n_sampled, const int *src, const int *dst,
                            int n, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    feed_tokens_kernel<<<dim3((n + 255) / 256), dim3(256), 0, stream>>>(tokens, sampled, src, dst, n, n_tokens, n_sampled);
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}
