// Everything between the q, k, v product and the attention, for attention whose queries, keys and values take more
// than a rotation of whole heads: each step is optional and a parameter.
//
//   q, k, v <- product + bias                                           (bias: one vector over the row's columns)
//   q, k    <- x * rsqrt(mean over the head's dims of x^2 + eps) * w     (w [dh], shared by all heads; one for q, one for k)
//              or x * rsqrt(mean over all heads' dims of x^2 + eps) * w   (w [heads * dh]; a kernel of its own)
//   q, k    <- the first rot_dim dims of every head turned by the angle of the token's position (tables
//              [max_pos, rot_dim / 2]; pairing 0: (i, i + rot_dim/2), 1: (2i, 2i + 1)); the other dims pass
//   q -> q_out [n, nh * dhp]; k, v -> the token's place in its page
//
// Maps (maps > 1): every query head and every key head is `maps` vectors of dh dims side by side in the rows, each normed and
// rotated by itself, over the head's one set of values (attention that is several attentions over the same values).  The
// kernels behind this one see plain attention heads, one per (head, map), in one of two layouts:
//   joint   a key head is its maps' keys side by side (maps * dh dims); the query of map m has its dims at m * dh and zeros
//           elsewhere, so its score is that of map m alone; query heads in the order (head, map);
//   split   a key head for every (key head, map), each with a copy of the values; query heads in the order (key head, map,
//           head of the group).
//
// The head sizes of the rows (dh, dv) may be any; what is stored has dhp >= dh and dvp >= dv dims per head, the
// dims beyond the true ones zeros (dhp a multiple of 8, as the pages' layout wants; zeros change no score and no
// output).  All arithmetic is 32-bit, one rounding at each store.  One wave per (token, head), four to a workgroup.
#include "common.h"
#include "kv_layout.h"

constexpr int QP_MAX_DIM = 640;

constexpr int QP_WAVES = 4;

// Between a wave's writes to LDS that is its own and its lanes' reads of one another's: a wave's LDS accesses are carried out
// in order, so only the compiler has to keep them so.
__device__ __forceinline__ void own_lds_fence() {
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
}

// two neighbouring elements in one store (p + c on a boundary of two elements)
__device__ __forceinline__ void store_two(float *p, float a, float b) { *(float2 *)p = make_float2(a, b); }
__device__ __forceinline__ void store_two(bf16_t *p, float a, float b) { *(uint32_t *)p = pack2_bf16(a, b); }

template <class TI, class T>
__global__ void __launch_bounds__(QP_WAVES *WAVE)
qkv_prepare_kernel(const TI *__restrict__ rows, int row_stride, int q_off, int k_off, int v_off,
                   const float *__restrict__ bias, const float *__restrict__ q_norm, const float *__restrict__ k_norm,
                   float eps, const int *__restrict__ positions, const float *__restrict__ cos_t,
                   const float *__restrict__ sin_t, int max_pos, int rot_dim, int pairing, T *__restrict__ q_out,
                   const int *__restrict__ slots, T *__restrict__ cache, int nh, int nkvh, int dh, int dhp, int dv,
                   int dvp, int page, int store_kv, int maps, int joint) {
    // nh and nkvh count (head, map) pairs; stored_kvh: key/value heads in the cache
    const int wave = threadIdx.x / WAVE, t = blockIdx.x, head = blockIdx.y * QP_WAVES + wave, lane = threadIdx.x & (WAVE - 1);
    const int stored_kvh = joint ? nkvh / maps : nkvh;
    if (head >= (store_kv ? nh + nkvh + stored_kvh : nh)) return;         // (no barrier below: a wave's LDS is its own)
    const TI *row = rows + (size_t)t * row_stride;
    extern __shared__ float xs_all[];                                     // a wave's dh numbers, rounded up to whole words of its own
    float *xs = xs_all + wave * ((dh + 3) / 4 * 4);
    int slot = -1;
    T *pg = nullptr;
    int tok = 0;
    if (head >= nh) {
        slot = store_kv ? slots[t] : -1;
        if (slot < 0) return;
        pg = cache + (size_t)(slot / page) * kv_page_elems(stored_kvh, dhp, dvp, page);
        tok = slot % page;
    }
    if (head >= nh + nkvh) {                                  // a value head: product + bias, as it is
        const int kvh = head - nh - nkvh, col0 = v_off + (joint ? kvh : kvh / maps) * dv;
        for (int c = lane; c < dvp; c += WAVE) {
            float v = 0.f;
            if (c < dv) v = to_f32(row[col0 + c]) + (bias ? bias[col0 + c] : 0.f);
            pg[kv_value_offset(stored_kvh, kvh, tok, c, dhp, dvp, page)] = from_f32<T>(v);
        }
        return;
    }
    const bool is_key = head >= nh;
    const int col0 = is_key ? k_off + (head - nh) * dh : q_off + head * dh;
    const float *nw = is_key ? k_norm : q_norm;
    float sq = 0.f;
    for (int c = lane; c < dh; c += WAVE) {
        const float v = to_f32(row[col0 + c]) + (bias ? bias[col0 + c] : 0.f);
        xs[c] = v;
        sq += v * v;
    }
    if (nw) {
        const float f = rsqrtf(wave_sum(sq) / (float)dh + eps);
        for (int c = lane; c < dh; c += WAVE) xs[c] = xs[c] * f * nw[c];
    }
    own_lds_fence();
    if (cos_t) {
        const int pos = positions[t], half = rot_dim / 2;
        const bool in_table = pos >= 0 && pos < max_pos;
        for (int i = lane; i < half; i += WAVE) {
            const int ia = pairing == 0 ? i : 2 * i, ib = pairing == 0 ? i + half : 2 * i + 1;
            float ra = __uint_as_float(0x7fc00000u), rb = ra;      // a position outside the table gives NaN, not a wrong value
            if (in_table) rotate_pair(xs[ia], xs[ib], cos_t[(size_t)pos * half + i], sin_t[(size_t)pos * half + i], ra, rb);
            xs[ia] = ra;
            xs[ib] = rb;
        }
        own_lds_fence();
    }
    // where the vector's first dim goes among the stored head's dims; a joint head's other dims are zeros in a query and the
    // other maps' in a key, whose last map also writes the zeros behind them
    const int map = maps > 1 ? (is_key ? head - nh : head) % maps : 0, at = joint ? map * dh : 0;
    if (!is_key) {
        int place = head;
        if (maps > 1 && !joint) {
            const int group = nh / nkvh, qh = head / maps;            // query heads of a key head
            place = (qh / group * maps + map) * group + qh % group;
        }
        T *o = q_out + (size_t)t * nh * dhp + (size_t)place * dhp;
        auto dim = [&](int c) { return c >= at && c < at + dh ? xs[c - at] : 0.f; };
        for (int c = 2 * lane; c < dhp; c += 2 * WAVE) store_two(o + c, dim(c), dim(c + 1));
    } else {
        const int kvh = joint ? (head - nh) / maps : head - nh;
        const int end = !joint || map == maps - 1 ? dhp : at + dh;
        auto dim = [&](int c) { return c < at + dh ? xs[c - at] : 0.f; };
        if (at % 2 == 0 && end % 2 == 0) {
            for (int c = at + 2 * lane; c < end; c += 2 * WAVE) store_two(pg + kv_key_offset(kvh, tok, c, dhp, page), dim(c), dim(c + 1));
        } else {
            for (int c = at + lane; c < end; c += WAVE) pg[kv_key_offset(kvh, tok, c, dhp, page)] = from_f32<T>(dim(c));
        }
    }
}

// The common case in one pass with wide accesses: no bias, no norm, pairs (i, i + rot_dim/2) or no rotation, every size and column
// a multiple of 8 (rot_dim of 16).  A thread takes eight neighbouring dims of what is stored for one head of one token (and, of a
// turned part, the eight that they are paired with), or eight dims of a value.  The same roundings as above.
template <class T> struct alignas(8 * sizeof(T)) QpRow8 { T v[8]; };

template <class TI, class T>
__global__ void __launch_bounds__(256)
qkv_prepare_wide_kernel(const TI *__restrict__ rows, int row_stride, int q_off, int k_off, int v_off, const int *__restrict__ positions,
                        const float *__restrict__ cos_t, const float *__restrict__ sin_t, int max_pos, int rot_dim, T *__restrict__ q_out,
                        const int *__restrict__ slots, T *__restrict__ cache, int nh, int nkvh, int dh, int dhp, int dv, int dvp, int page,
                        int store_kv, int maps, int joint) {
    const int t = blockIdx.x, half8 = rot_dim / 16, stored_kvh = joint ? nkvh / maps : nkvh;
    // the work items of a stored query head: its turned pairs, its other dims, its zeros; of a (key head, map): the same without
    // zeros (a joint head has them once, at its last map)
    const int turned = half8 + (dh - rot_dim) / 8, q_items = turned + (dhp - dh) / 8, k_zeros = joint ? (dhp - maps * dh) / 8 : (dhp - dh) / 8;
    const int k_items = turned + k_zeros, n_q = nh * q_items, n_k = store_kv ? nkvh * k_items : 0, n_v = store_kv ? stored_kvh * (dvp / 8) : 0;
    const int w = blockIdx.y * 256 + threadIdx.x;
    if (w >= n_q + n_k + n_v) return;
    const TI *row = rows + (size_t)t * row_stride;
    T *pg = nullptr;
    int tok = 0;
    if (w >= n_q) {
        const int slot = slots[t];
        if (slot < 0) return;
        pg = cache + (size_t)(slot / page) * kv_page_elems(stored_kvh, dhp, dvp, page);
        tok = slot % page;
    }
    if (w >= n_q + n_k) {
        const int kvh = (w - n_q - n_k) / (dvp / 8), c0 = (w - n_q - n_k) % (dvp / 8) * 8;
        QpRow8<TI> a = {};
        if (c0 < dv) a = *(const QpRow8<TI> *)(row + v_off + (joint ? kvh : kvh / maps) * dv + c0);
#pragma unroll
        for (int e = 0; e < 8; ++e) pg[kv_value_offset(stored_kvh, kvh, tok, c0 + e, dhp, dvp, page)] = from_f32<T>(to_f32(a.v[e]));
        return;
    }
    const bool is_key = w >= n_q;
    const int head = is_key ? (w - n_q) / k_items : w / q_items, item = is_key ? (w - n_q) % k_items : w % q_items;
    const int map = maps > 1 ? head % maps : 0, at = joint ? map * dh : 0;
    int place = joint && is_key ? head / maps : head;
    if (!is_key && maps > 1 && !joint) {
        const int group = nh / nkvh, qh = head / maps;
        place = (qh / group * maps + map) * group + qh % group;
    }
    // where eight dims of the stored head lie
    auto at_dim = [&](int c) -> QpRow8<T> * {
        return (QpRow8<T> *)(is_key ? pg + kv_key_offset(place, tok, c, dhp, page) : q_out + (size_t)t * nh * dhp + (size_t)place * dhp + c);
    };
    if (item >= turned) {
        // zeros: of a query every dim that is not its map's, of a key the dims behind the true ones
        const int z = (item - turned) * 8;
        if (is_key && joint && map != maps - 1) return;
        const int c = is_key ? (joint ? maps * dh : dh) + z : (z < at ? z : z + dh);
        QpRow8<T> o;
#pragma unroll
        for (int e = 0; e < 8; ++e) o.v[e] = from_f32<T>(0.f);
        *at_dim(c) = o;
        return;
    }
    const TI *x = row + (is_key ? k_off : q_off) + head * dh;
    if (item >= half8) {
        const int c = rot_dim + (item - half8) * 8;
        const QpRow8<TI> a = *(const QpRow8<TI> *)(x + c);
        QpRow8<T> o;
#pragma unroll
        for (int e = 0; e < 8; ++e) o.v[e] = from_f32<T>(to_f32(a.v[e]));
        *at_dim(at + c) = o;
        return;
    }
    const int i0 = item * 8, half = rot_dim / 2, pos = positions[t];
    const bool in_table = pos >= 0 && pos < max_pos;
    const size_t tab = (size_t)(in_table ? pos : 0) * half + i0;
    const QpRow8<TI> a = *(const QpRow8<TI> *)(x + i0), b = *(const QpRow8<TI> *)(x + half + i0);
    const QpRow8<float> cs = *(const QpRow8<float> *)(cos_t + tab), sn = *(const QpRow8<float> *)(sin_t + tab);
    QpRow8<T> oa, ob;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        float ra, rb;
        rotate_pair(to_f32(a.v[e]), to_f32(b.v[e]), cs.v[e], sn.v[e], ra, rb);
        if (!in_table) ra = rb = __uint_as_float(0x7fc00000u);        // a position outside the table gives NaN, not a wrong value
        oa.v[e] = from_f32<T>(ra);
        ob.v[e] = from_f32<T>(rb);
    }
    *at_dim(at + i0) = oa;
    *at_dim(at + half + i0) = ob;
}

// rows: [n, row_stride] of in_type, a token's q heads at column q_off (nh * dh), k heads at k_off (nkvh * dh), v heads
// at v_off (nkvh * dv); bias: null or float32 over the row's columns; q_norm, k_norm: null or float32 [dh].
// q_out: [n, nh * dhp] of type; cache: this layer's pages of type, kv_page_elems(nkvh, dhp, dvp, page) each;
// slots[t] = page * page_size + place, or -1 to store nothing for token t.  store_kv 0: queries only.  maps > 1: nh and nkvh count
// (head, map) pairs; the cache's pages hold nkvh / maps (joint) or nkvh (split) key/value heads, dhp >= maps * dh (joint) or dh.
LCU_API int lcu_qkv_prepare(const void *rows, int in_type, int n, int row_stride, int q_off, int k_off, int v_off,
                            const float *bias, const float *q_norm, const float *k_norm, float eps, const int *positions,
                            const float *cos_t, const float *sin_t, int max_pos, int rot_dim, int pairing, void *q_out,
                            int type, const int *slots, void *cache, int nh, int nkvh, int dh, int dhp, int dv, int dvp,
                            int page, int store_kv, int maps, int joint, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (nh <= 0 || nkvh < 0 || dh <= 0 || dh > QP_MAX_DIM || dhp < dh || dhp % 8 || dhp > QP_MAX_DIM || dv <= 0 || dvp < dv ||
        dvp > QP_MAX_DIM || page <= 0 || page % 8 || rot_dim < 0 || rot_dim % 2 || rot_dim > dh || (pairing != 0 && pairing != 1) ||
        !rows || !q_out || (cos_t && (!sin_t || !positions || rot_dim == 0)) || nh + 2 * nkvh > 65535 ||
        maps < 1 || nh % maps || nkvh % maps || (joint && (maps < 2 || dhp < maps * dh)) || (maps > 1 && !store_kv))
        return LCU_BAD_ARGUMENT;
    if (store_kv && (!cache || !slots || nkvh <= 0)) return LCU_BAD_ARGUMENT;
    const int stored_kvh = joint ? nkvh / maps : nkvh;
    if (!bias && !q_norm && !k_norm && (!cos_t || (pairing == 0 && rot_dim % 16 == 0)) && dh % 8 == 0 && dv % 8 == 0 && dvp % 8 == 0 &&
        row_stride % 8 == 0 && q_off % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && (uintptr_t)rows % 32 == 0 && (uintptr_t)q_out % 32 == 0 &&
        (uintptr_t)cache % 32 == 0 && (uintptr_t)cos_t % 32 == 0 && (uintptr_t)sin_t % 32 == 0) {
        const int rot = cos_t ? rot_dim : 0, turned = rot / 16 + (dh - rot) / 8;
        const int items = nh * (turned + (dhp - dh) / 8) +
                          (store_kv ? nkvh * (turned + (joint ? dhp - maps * dh : dhp - dh) / 8) + stored_kvh * (dvp / 8) : 0);
        dim3 wgrid(n, (items + 255) / 256), wblock(256);
#define WIDE(TI, T) qkv_prepare_wide_kernel<TI, T><<<wgrid, wblock, 0, stream>>>((const TI *)rows, row_stride, q_off, k_off, v_off, positions, cos_t, sin_t, max_pos, rot, (T *)q_out, slots, (T *)cache, nh, nkvh, dh, dhp, dv, dvp, page, store_kv ? 1 : 0, maps, joint)
        if (in_type == LCU_F32 && type == LCU_F32) WIDE(float, float);
        else if (in_type == LCU_F32 && type == LCU_BF16) WIDE(float, bf16_t);
        else if (in_type == LCU_BF16 && type == LCU_BF16) WIDE(bf16_t, bf16_t);
        else return LCU_BAD_ARGUMENT;
#undef WIDE
        LCU_LAUNCH_CHECK();
        return LCU_OK;
    }
    const int heads = store_kv ? nh + nkvh + stored_kvh : nh;
    dim3 grid(n, (heads + QP_WAVES - 1) / QP_WAVES), block(QP_WAVES * WAVE);
    const size_t lds = (size_t)QP_WAVES * ((dh + 3) / 4 * 4) * sizeof(float);
#define GO(TI, T) qkv_prepare_kernel<TI, T><<<grid, block, lds, stream>>>((const TI *)rows, row_stride, q_off, k_off, v_off, bias, q_norm, k_norm, eps, positions, cos_t, sin_t, max_pos, rot_dim, pairing, (T *)q_out, slots, (T *)cache, nh, nkvh, dh, dhp, dv, dvp, page, store_kv, maps, joint)
    if (in_type == LCU_F32 && type == LCU_F32) GO(float, float);
    else if (in_type == LCU_F32 && type == LCU_BF16) GO(float, bf16_t);
    else if (in_type == LCU_BF16 && type == LCU_BF16) GO(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// A norm over the whole projection of the queries, and one over that of the keys, needs a token's whole row: a workgroup per token.
// The row is read twice, the second time from the caches.  V dims a piece (1: any sizes, either pairing).
template <class TI, class T, int V>
__global__ void __launch_bounds__(512)
qkv_prepare_rows_kernel(const TI *__restrict__ rows, int row_stride, int q_off, int k_off, int v_off, const float *__restrict__ q_norm,
                        const float *__restrict__ k_norm, float eps, const int *__restrict__ positions, const float *__restrict__ cos_t,
                        const float *__restrict__ sin_t, int max_pos, int rot_dim, int pairing, T *__restrict__ q_out,
                        const int *__restrict__ slots, T *__restrict__ cache, int nh, int nkvh, int dh, int dhp, int dv, int dvp, int page,
                        int store_kv) {
    struct alignas(V * sizeof(TI)) In { TI v[V]; };
    struct alignas(V * sizeof(T)) Out { T v[V]; };
    struct alignas(V * sizeof(float)) F32 { float v[V]; };
    __shared__ float sums[2][16];
    const int t = blockIdx.x, threads = blockDim.x, nq = nh * dh, nk = store_kv ? nkvh * dh : 0;
    const TI *row = rows + (size_t)t * row_stride;
    float sq = 0.f, sk = 0.f;
    for (int c = threadIdx.x * V; c < nq + nk; c += threads * V) {
        const In a = *(const In *)(row + (c < nq ? q_off + c : k_off + c - nq));
        float part = 0.f;
#pragma unroll
        for (int e = 0; e < V; ++e) part += to_f32(a.v[e]) * to_f32(a.v[e]);
        if (c < nq) sq += part;
        else sk += part;
    }
    sq = wave_sum(sq);                            // both sums behind one barrier
    sk = wave_sum(sk);
    if (threadIdx.x % WAVE == 0) { sums[0][threadIdx.x / WAVE] = sq; sums[1][threadIdx.x / WAVE] = sk; }
    __syncthreads();
    sq = sk = 0.f;
    for (int i = 0; i < threads / WAVE; ++i) { sq += sums[0][i]; sk += sums[1][i]; }
    const float fq = rsqrtf(sq / (float)nq + eps), fk = nk ? rsqrtf(sk / (float)nk + eps) : 0.f;
    const int slot = store_kv ? slots[t] : -1, tok = slot < 0 ? 0 : slot % page;
    T *pg = slot < 0 ? nullptr : cache + (size_t)(slot / page) * kv_page_elems(nkvh, dhp, dvp, page);
    const int pos = cos_t ? positions[t] : 0, half = rot_dim / 2;
    const bool in_table = pos >= 0 && pos < max_pos;
    // the pieces of a stored head: its turned pairs, its other dims, its zeros; of a value head: its dims with zeros behind them
    const int turned = half / V, passed = (dh - rot_dim) / V, items = turned + passed + (dhp - dh) / V;
    const int n_q = nh * items, n_k = slot < 0 ? 0 : nkvh * items, n_v = slot < 0 ? 0 : nkvh * ((dvp + V - 1) / V);
    for (int i = threadIdx.x; i < n_q + n_k + n_v; i += threads) {
        if (i >= n_q + n_k) {
            const int per = (dvp + V - 1) / V, kvh = (i - n_q - n_k) / per, c = (i - n_q - n_k) % per * V;
            In a = {};
            if (c < dv) a = *(const In *)(row + v_off + kvh * dv + c);
#pragma unroll
            for (int e = 0; e < V; ++e) pg[kv_value_offset(nkvh, kvh, tok, c + e, dhp, dvp, page)] = from_f32<T>(to_f32(a.v[e]));
            continue;
        }
        const bool is_key = i >= n_q;
        const int head = (is_key ? i - n_q : i) / items, item = (is_key ? i - n_q : i) % items;
        const TI *x = row + (is_key ? k_off : q_off) + head * dh;
        const float *w = (is_key ? k_norm : q_norm) + head * dh;
        const float f = is_key ? fk : fq;
        auto at_dim = [&](int c) -> Out * { return (Out *)(is_key ? pg + kv_key_offset(head, tok, c, dhp, page) : q_out + (size_t)t * nh * dhp + (size_t)head * dhp + c); };
        auto normed = [&](int c, float *o) {
            const In a = *(const In *)(x + c);
            const F32 wv = *(const F32 *)(w + c);
#pragma unroll
            for (int e = 0; e < V; ++e) o[e] = to_f32(a.v[e]) * f * wv.v[e];
        };
        float a[V], b[V];
        Out oa, ob;
        if (item < turned) {
            const int i0 = item * V, ca = pairing == 0 ? i0 : 2 * i0, cb = pairing == 0 ? half + i0 : 2 * i0 + 1;      // (neighbours: V is 1)
            normed(ca, a);
            normed(cb, b);
            const size_t tab = (size_t)(in_table ? pos : 0) * half + i0;
            const F32 cs = *(const F32 *)(cos_t + tab), sn = *(const F32 *)(sin_t + tab);
#pragma unroll
            for (int e = 0; e < V; ++e) {
                float ra, rb;
                rotate_pair(a[e], b[e], cs.v[e], sn.v[e], ra, rb);
                if (!in_table) ra = rb = __uint_as_float(0x7fc00000u);        // a position outside the table gives NaN, not a wrong value
                oa.v[e] = from_f32<T>(ra);
                ob.v[e] = from_f32<T>(rb);
            }
            *at_dim(ca) = oa;
            *at_dim(cb) = ob;
        } else {
            const int c = rot_dim + (item - turned) * V;
            if (c < dh) normed(c, a);
#pragma unroll
            for (int e = 0; e < V; ++e) oa.v[e] = from_f32<T>(c < dh ? a[e] : 0.f);
            *at_dim(c) = oa;
        }
    }
}

// rows, q_out, cache and the rest as lcu_qkv_prepare (no bias, no maps); q_norm [nh * dh], k_norm [nkvh * dh].
LCU_API int lcu_qkv_prepare_rows(const void *rows, int in_type, int n, int row_stride, int q_off, int k_off, int v_off, const float *q_norm,
                                 const float *k_norm, float eps, const int *positions, const float *cos_t, const float *sin_t, int max_pos,
                                 int rot_dim, int pairing, void *q_out, int type, const int *slots, void *cache, int nh, int nkvh, int dh,
                                 int dhp, int dv, int dvp, int page, int store_kv, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (nh <= 0 || nkvh <= 0 || dh <= 0 || dhp < dh || dhp % 8 || dhp > QP_MAX_DIM || dv <= 0 || dvp < dv || dvp > QP_MAX_DIM || page <= 0 ||
        page % 8 || rot_dim < 0 || rot_dim % 2 || rot_dim > dh || (pairing != 0 && pairing != 1) || !rows || !q_out || !q_norm || !k_norm ||
        (cos_t && (!sin_t || !positions || rot_dim == 0)) || (store_kv && (!cache || !slots)))
        return LCU_BAD_ARGUMENT;
    const int rot = cos_t ? rot_dim : 0;
    const bool four = (pairing == 0 || !rot) && dh % 4 == 0 && rot % 8 == 0 && dv % 4 == 0 && dvp % 4 == 0 && row_stride % 4 == 0 && q_off % 4 == 0 &&
                      k_off % 4 == 0 && v_off % 4 == 0 && (uintptr_t)rows % 16 == 0 && (uintptr_t)q_out % 16 == 0 && (uintptr_t)cache % 16 == 0 &&
                      (uintptr_t)cos_t % 16 == 0 && (uintptr_t)sin_t % 16 == 0 && (uintptr_t)q_norm % 16 == 0 && (uintptr_t)k_norm % 16 == 0;
    dim3 grid(n), block(n <= 192 ? 512 : 256);
#define GO(TI, T, V) qkv_prepare_rows_kernel<TI, T, V><<<grid, block, 0, stream>>>((const TI *)rows, row_stride, q_off, k_off, v_off, q_norm, k_norm, eps, positions, cos_t, sin_t, max_pos, rot, pairing, (T *)q_out, slots, (T *)cache, nh, nkvh, dh, dhp, dv, dvp, page, store_kv)
#define EITHER(TI, T) do { if (four) GO(TI, T, 4); else GO(TI, T, 1); } while (0)
    if (in_type == LCU_F32 && type == LCU_F32) EITHER(float, float);
    else if (in_type == LCU_F32 && type == LCU_BF16) EITHER(float, bf16_t);
    else if (in_type == LCU_BF16 && type == LCU_BF16) EITHER(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef EITHER
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// The output of every head times sigmoid of the head's gate: out[t, h, :] = factor * sigmoid(gate[t, h]) * x[t, h, :], the gate's rows
// [n, gate_stride] with the heads' numbers from column g_off, out's rows out_stride apart (out may be x).  The factor is 32-bit.
template <class TG, class T, int V>
__global__ void __launch_bounds__(256)
head_gate_kernel(T *out, int out_stride, const T *x, const TG *__restrict__ gate, int gate_stride, int g_off, int nh, int dv, float factor) {
    struct alignas(V * sizeof(T)) Piece { T v[V]; };
    const int t = blockIdx.x;
    for (int c = threadIdx.x * V; c < nh * dv; c += blockDim.x * V) {
        const float g = to_f32(gate[(size_t)t * gate_stride + g_off + c / dv]);
        const float f = factor / (1.0f + expf(-g));
        Piece p = *(const Piece *)(x + (size_t)t * nh * dv + c);
#pragma unroll
        for (int e = 0; e < V; ++e) p.v[e] = from_f32<T>(to_f32(p.v[e]) * f);
        *(Piece *)(out + (size_t)t * out_stride + c) = p;
    }
}

LCU_API int lcu_head_gate(void *out, int out_stride, const void *x, int type, const void *gate, int gate_type, int gate_stride, int g_off, int n,
                          int nh, int dv, float factor, hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (nh <= 0 || dv <= 0 || !out || !x || !gate || out_stride < nh * dv) return LCU_BAD_ARGUMENT;
    dim3 grid(n), block(256);
    const bool four = dv % 4 == 0 && out_stride % 4 == 0 && (uintptr_t)out % 16 == 0 && (uintptr_t)x % 16 == 0;
#define GO(TG, T)                                                                                                                                      \
    do {                                                                                                                                               \
        if (four) head_gate_kernel<TG, T, 4><<<grid, block, 0, stream>>>((T *)out, out_stride, (const T *)x, (const TG *)gate, gate_stride, g_off, nh, dv, factor); \
        else head_gate_kernel<TG, T, 1><<<grid, block, 0, stream>>>((T *)out, out_stride, (const T *)x, (const TG *)gate, gate_stride, g_off, nh, dv, factor);     \
    } while (0)
    if (gate_type == LCU_F32 && type == LCU_F32) GO(float, float);
    else if (gate_type == LCU_F32 && type == LCU_BF16) GO(float, bf16_t);
    else if (gate_type == LCU_BF16 && type == LCU_BF16) GO(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}
