// Linear attention with one decay per head and token, in chunks on the matrix cores.  Per head, with key channels i and
// value columns j, a state S [d, dv] in 32-bit:
//
//   S_t = a_t S_(t-1) + b_t k_t v_t^T          o_t = scale * S_t^T q_t
//
// Two ways to make a and b:
//   fixed   a = decay[h], b = 1;
//   gated   from the projections of two gates with a cap c:  i = c tanh((z_i + bias_i) / c), f = log sigmoid(c tanh((z_f + bias_f) / c)),
//           a running maximum m_t = max(f + m_(t-1), i) (0 before the first token), a = exp(f + m_(t-1) - m_t), b = exp(i - m_t).
//           A normaliser n_t = a n_(t-1) + b k goes along with S (here: one more value column, of ones), and so does m.
// q, k and v may pass through silu on their way in.  The outputs:
//   joint     the heads side by side divided by their root mean square, times a weight, times sigmoid(gate);
//   per head  o / (max(|scale n . q|, exp(-m)) + 1e-6), divided by its root mean square, times a weight, times sigmoid(gate).
//
// A step that is not all single tokens.  With L_t the sum of log a over the chunk's tokens up to t, a chunk of C tokens is
//   o_t = exp(L_t) S^T q_t + sum_(s <= t) (q_t . k_s) exp(L_t - L_s) b_s v_s       S <- exp(L_C) S + sum_s k_s (exp(L_C - L_s) b_s v_s)^T
// four matrix products.  A wave owns 16 value columns and all key channels of them: its part of S stays in registers as the
// accumulators of the last product, and accumulators are laid out as the next product's operand wants them if the order of
// the summed index is permuted alike on both sides, so neither S nor the scores ever go through LDS; q and k do (k also
// transposed), shared by the workgroup's waves.  Products of 32-bit operands (S, the weighted scores, the weighted values)
// with bfloat16 ones are made of three bfloat16 products, of the operand's upper, middle and lower eight bits, which loses
// nothing of its 24; in float32 all products run on the 32-bit matrix instruction.  L is summed in 64-bit and kept in two parts.
// The weights exp(L_t - L_s) b_s are made once a chunk for all waves, few of them: those of a tile's own 16 tokens one by one, those of
// tokens in an earlier tile as exp(L_t - L_e) times exp(L_e - L_s) b_s, e that tile's last token (neither factor exceeds 1 where
// no decay does).
// A request that feeds DS_LONG tokens or more is cut into up to DS_RUNS runs that are walked side by side, twice: first
// from zeros, which gives what a run adds to any state; a small kernel chains the runs' starts; the second walk gives the outputs.
//
// A step of single tokens: one workgroup per (request, head) streams the head's state through its registers.
//
// The state of a request, one flat slot: S [heads, d, dv], then (gated) n [heads, d] and m [heads].  It is taken as zero where a
// request's first token of the step stands at position 0.  A token's result depends on the tokens before it in its request
// only; how a request was cut into steps changes roundings.
#include "common.h"
#include "lane_moves.h"

constexpr int DS_RUNS = 16;
constexpr int DS_LONG = 256;                     // (not fewer: steps of up to 256 tokens are captured into graphs by their sizes, and of those only a
                                                  // lone request's may be long)
constexpr int DS_WAVES = 8;                       // waves of a chunk workgroup at most

typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
typedef __attribute__((ext_vector_type(2))) uint32_t u32x2;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float log_sigmoid_f(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// silu of a value that is rounded to T next: to bfloat16 with the hardware's exponential and reciprocal (an error of 2^-20 or so)
template <class T> __device__ __forceinline__ float silu_for(float z);
template <> __device__ __forceinline__ float silu_for<float>(float z) { return silu_f(z); }
template <> __device__ __forceinline__ float silu_for<bf16_t>(float z) {
    return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.44269504f * z));
}

template <class T, int V> struct alignas(V * sizeof(T)) DsVec { T v[V]; };

// A product's operand of `PER` elements of the summed index a lane (TILES tiles of 16 a step).  Element j of a lane in group g (of
// 16 lanes) is index 16 * (j / 4) + 4 g + j % 4 of the step: the order in which accumulators hold their rows.
template <class T> struct DsMma;
template <> struct DsMma<bf16_t> {
    static constexpr int PER = 8, KSTEP = 32, SPLITS = 3;
    typedef u32x4 frag;
    // two pieces of four neighbours, 16 elements apart
    static __device__ __forceinline__ frag load(const bf16_t *p) {
        const u32x2 a = *(const u32x2 *)p, b = *(const u32x2 *)(p + 16);
        return frag{a[0], a[1], b[0], b[1]};
    }
    static __device__ __forceinline__ frag exact(const float *v) {             // values that bfloat16 holds
        return frag{pack2_bf16(v[0], v[1]), pack2_bf16(v[2], v[3]), pack2_bf16(v[4], v[5]), pack2_bf16(v[6], v[7])};
    }
    static __device__ __forceinline__ uint32_t upper(float lo, float hi) {      // the upper halves, side by side
        return (__float_as_uint(lo) >> 16) | (__float_as_uint(hi) & 0xffff0000u);
    }
    static __device__ __forceinline__ void split(const float *v, frag *o) {
        float r[8], s[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            r[j] = v[j] - __uint_as_float(__float_as_uint(v[j]) & 0xffff0000u);
            s[j] = r[j] - __uint_as_float(__float_as_uint(r[j]) & 0xffff0000u);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            o[0][j] = upper(v[2 * j], v[2 * j + 1]);
            o[1][j] = upper(r[2 * j], r[2 * j + 1]);
            o[2][j] = pack2_bf16(s[2 * j], s[2 * j + 1]);
        }
    }
    static __device__ __forceinline__ f32x4 mma(frag a, frag b, f32x4 c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
    }
};
template <> struct DsMma<float> {
    static constexpr int PER = 4, KSTEP = 16, SPLITS = 1;
    typedef f32x4 frag;
    static __device__ __forceinline__ frag load(const float *p) { return *(const frag *)p; }
    static __device__ __forceinline__ frag exact(const float *v) { return frag{v[0], v[1], v[2], v[3]}; }
    static __device__ __forceinline__ void split(const float *v, frag *o) { o[0] = frag{v[0], v[1], v[2], v[3]}; }
    static __device__ __forceinline__ f32x4 mma(frag a, frag b, f32x4 c) {
#pragma unroll
        for (int e = 0; e < 4; ++e) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], c, 0, 0, 0);
        return c;
    }
};

// how many of the requests before r feed at least DS_LONG tokens: r's place among those in the runs' arrays
__device__ __forceinline__ int ds_long_index(const int *__restrict__ q_start, int r) {
    int li = 0;
    for (int i = 0; i < r; ++i) li += (q_start[i + 1] - q_start[i] >= DS_LONG);
    return li;
}
__device__ __forceinline__ int ds_run_len(int q) {          // a multiple of 64 tokens
    const int len = (q + DS_RUNS - 1) / DS_RUNS;
    return (len + 63) / 64 * 64;
}

// ---------------------------------------------------------------- the gates
// z: [n, ld] 32-bit with the input gates' projections at z[., h] and the forget gates' at z[., heads + h].  To log_a, b, m: [heads][n].
// A workgroup per (head, request): THREADS tokens at a time, (F, M) = (sum of f, the maximum that tokens alone would leave) composed
// across the threads.
template <int THREADS>
__global__ void __launch_bounds__(THREADS)
ds_gates_kernel(const float *__restrict__ z, int ld, const float *__restrict__ bias_i, const float *__restrict__ bias_f, float cap,
                float *__restrict__ state, size_t slot_stride, size_t m_off, float *__restrict__ log_a, float *__restrict__ b_out,
                float *__restrict__ m_out, const int *__restrict__ q_start, const int *__restrict__ ctx_len,
                const int *__restrict__ state_slot, int n, int heads) {
    constexpr int WAVES = THREADS / WAVE;
    __shared__ float wf[WAVES], wm[WAVES];
    const int h = blockIdx.x, r = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int t0 = q_start[r], t1 = q_start[r + 1];
    if (t1 <= t0) return;
    float *m_slot = state + (size_t)state_slot[r] * slot_stride + m_off + h;
    float m = ctx_len[r] - (t1 - t0) > 0 ? *m_slot : 0.f;
    const float bi = bias_i[h], bf = bias_f[h];
    for (int base = t0; base < t1; base += THREADS) {
        const int t = base + tid;
        float gi = -INFINITY, f = 0.f;                     // beyond the last token: nothing changes
        if (t < t1) {
            gi = cap * tanhf((z[(size_t)t * ld + h] + bi) / cap);
            f = log_sigmoid_f(cap * tanhf((z[(size_t)t * ld + heads + h] + bf) / cap));
        }
        float F = f, M = gi;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float pf = __shfl_up(F, off, WAVE), pm = __shfl_up(M, off, WAVE);
            if (lane >= off) { M = fmaxf(pm + F, M); F += pf; }
        }
        __syncthreads();
        if (lane == 63) { wf[wave] = F; wm[wave] = M; }
        __syncthreads();
        float start = m;                                   // the maximum in front of this wave's tokens, and behind all
#pragma unroll
        for (int w = 0; w < WAVES; ++w) {
            if (w < wave) start = fmaxf(start + wf[w], wm[w]);
            m = fmaxf(m + wf[w], wm[w]);
        }
        const float pf = __shfl_up(F, 1, WAVE), pm = __shfl_up(M, 1, WAVE);
        const float before = lane == 0 ? start : fmaxf(start + pf, pm);
        if (t < t1) {
            const float now = fmaxf(f + before, gi);
            const size_t at = (size_t)h * n + t;
            log_a[at] = f + before - now;
            b_out[at] = expf(gi - now);
            m_out[at] = now;
            if (t == t1 - 1) *m_slot = now;
        }
    }
}

// ---------------------------------------------------------------- chunks
struct DsArgs {
    const void *rows;                             // [n, row_stride]: q, k (heads * d), v (heads * dv) at their columns
    int row_stride, q_off, k_off, v_off;
    const float *log_decay;                       // fixed: [heads][2], the logarithm in two parts (null: gated)
    const float *log_a, *b;                       // gated: [heads][n]
    float *state;
    size_t slot_stride, n_off;                    // where a slot's normalisers begin
    float *o;                                     // [heads][n][tiles * 16]
    float *run_b, *run_in, *run_l;                // [long request][run][heads][d][dvx], the same, [long request][run][heads]
    const int *q_start, *ctx_len, *state_slot;
    int n, heads, d, dv, dvx, tiles;              // dvx: value columns with the normaliser's
    float scale;
    int silu, four;                               // four: rows may be loaded four elements at a time
};

template <class T> struct DsChunk {
    // tokens of a chunk, by the padded key size: what LDS holds (q, k, k transposed) stays within 64 KB
    static constexpr int tokens(int D) { return sizeof(T) == 2 ? (D <= 128 ? 64 : 32) : (D <= 128 ? 32 : 16); }
};

// MODE 0: a request of fewer than DS_LONG tokens.  1: a run from zeros, leaves its own sum in run_b and the sum of its log a in run_l.
// 2: a run from run_in, with outputs; the last one leaves the request's state.
template <class T, int D, int MODE>
__global__ void __launch_bounds__(DS_WAVES *WAVE, 1)
ds_chunk_kernel(DsArgs p) {
    typedef DsMma<T> M;
    typedef typename M::frag frag;
    constexpr int C = DsChunk<T>::tokens(D), PAD = 16 / sizeof(T), LDK = D + PAD, LDT = C + PAD;
    constexpr int TT = C / 16, KT = D / 16, TPS = M::PER / 4;                // tiles of tokens, of key channels; tiles a step of a product
    __shared__ __attribute__((aligned(16))) T qs[C * LDK], ks[C * LDK], kt[D * LDT];
    // weights: [t][s % 16] of a tile's own tokens (rows of 20: no bank twice); t behind the end of each earlier tile; s up to the end of its tile; t from the chunk's
    // start; s up to the chunk's end, and the whole chunk
    __shared__ __attribute__((aligned(16))) float w_own[MODE == 1 ? 1 : C * 20], w_tile[MODE == 1 ? 1 : C], w_end[C];
    __shared__ float w_behind[MODE == 1 ? 1 : TT * C], w_start[MODE == 1 ? 1 : C], w_all;
    __shared__ float l_hi[C], l_lo[C], b_s[C];
    const int r = MODE == 0 ? blockIdx.z : blockIdx.z / DS_RUNS, run = MODE == 0 ? 0 : blockIdx.z % DS_RUNS, h = blockIdx.y;
    int t0 = p.q_start[r], t1 = p.q_start[r + 1];
    const int q_len = t1 - t0;
    if (q_len <= 0 || (MODE != 0) != (q_len >= DS_LONG)) return;
    const bool fresh = p.ctx_len[r] - q_len == 0;
    const int tid = threadIdx.x, threads = blockDim.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, l16 = lane & 15;
    size_t run_no = 0;
    bool last = true;
    if (MODE != 0) {
        const int len = ds_run_len(q_len), end = t1;
        t0 += run * len;
        if (t0 >= end) return;
        t1 = min(end, t0 + len);
        last = t1 == end;
        if (MODE == 1 && last) return;                                        // nothing starts behind the last run
        run_no = ((size_t)ds_long_index(p.q_start, r) * DS_RUNS + run) * p.heads + h;
    }
    const int d = p.d, dv = p.dv, tile = blockIdx.x * (threads >> 6) + wave, col = tile * 16 + l16;
    const bool active = tile < p.tiles;                                        // (an idle wave still helps to stage)
    float *slot = p.state + (size_t)p.state_slot[r] * p.slot_stride;
    // the state's element (key channel i, this lane's column) in a slot; the normaliser is the column dv
    auto in_slot = [&](int i) -> float * { return col < dv ? slot + ((size_t)h * d + i) * dv + col : slot + p.n_off + (size_t)h * d + i; };
    f32x4 s[KT];
#pragma unroll
    for (int x = 0; x < KT; ++x)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int key = 16 * x + 4 * g + i;
            float v = 0.f;
            if (key < d && col < p.dvx) {
                if (MODE == 0 && !fresh) v = *in_slot(key);
                if (MODE == 2) v = p.run_in[(run_no * d + key) * p.dvx + col];
            }
            s[x][i] = v;
        }
    const T *rows = (const T *)p.rows;
    double l_run = 0.0;
    for (int base = t0; base < t1; base += C) {
        const int nt = min(C, t1 - base);
        if (base > t0) __syncthreads();                                        // the chunk before has been read
        // ---- q and k of the chunk's tokens; two tokens and four channels a thread, so that k can be written transposed in pairs
        {
            constexpr int GROUPS = D / 4;
            for (int w = tid; w < C / 2 * GROUPS; w += threads) {
                // eight groups of channels, then eight pairs of tokens, then the rest: whole pieces of rows from memory, few banks hit twice
                constexpr int GW = GROUPS < 8 ? GROUPS : 8, PW = 64 / GW < C / 2 ? 64 / GW : C / 2, BLK = GW * PW;
                const int blk = w / BLK, in = w % BLK, pair = blk / (GROUPS / GW) * PW + in / GW, c0 = (blk % (GROUPS / GW) * GW + in % GW) * 4;
                float qv[2][4], kv[2][4];
#pragma unroll
                for (int a = 0; a < 2; ++a) {
                    const int t = 2 * pair + a;
                    const T *row = rows + (size_t)(base + min(t, nt - 1)) * p.row_stride + h * d;
                    if (p.four) {
                        const int c = min(c0, d - 4);
                        const DsVec<T, 4> kk = *(const DsVec<T, 4> *)(row + p.k_off + c), qq = *(const DsVec<T, 4> *)(row + p.q_off + c);
#pragma unroll
                        for (int e = 0; e < 4; ++e) { kv[a][e] = to_f32(kk.v[e]); qv[a][e] = to_f32(qq.v[e]); }
                    } else {
#pragma unroll
                        for (int e = 0; e < 4; ++e) {
                            const int c = min(c0 + e, d - 1);
                            kv[a][e] = to_f32(row[p.k_off + c]);
                            qv[a][e] = to_f32(row[p.q_off + c]);
                        }
                    }
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        const bool in_row = t < nt && c0 + e < d;
                        if (p.silu) { kv[a][e] = silu_for<T>(kv[a][e]); qv[a][e] = silu_for<T>(qv[a][e]); }
                        if (!in_row) kv[a][e] = qv[a][e] = 0.f;
                    }
                    DsVec<T, 4> ko, qo;
#pragma unroll
                    for (int e = 0; e < 4; ++e) { ko.v[e] = from_f32<T>(kv[a][e]); qo.v[e] = from_f32<T>(qv[a][e]); }
                    if (MODE != 1) {
                        *(DsVec<T, 4> *)(ks + t * LDK + c0) = ko;
                        *(DsVec<T, 4> *)(qs + t * LDK + c0) = qo;
                    }
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    DsVec<T, 2> both;
                    both.v[0] = from_f32<T>(kv[0][e]);
                    both.v[1] = from_f32<T>(kv[1][e]);
                    *(DsVec<T, 2> *)(kt + (c0 + e) * LDT + 2 * pair) = both;
                }
            }
        }
        // ---- the sums of log a, in 64-bit, by the first wave
        if (wave == 0) {
            double l = 0.0;
            float b = 0.f;
            if (p.log_decay) {
                l = (double)min(lane + 1, nt) * ((double)p.log_decay[2 * h] + (double)p.log_decay[2 * h + 1]);
                b = lane < nt ? 1.f : 0.f;
            } else {
                if (lane < nt) {
                    l = (double)p.log_a[(size_t)h * p.n + base + lane];
                    b = p.b[(size_t)h * p.n + base + lane];
                }
#pragma unroll
                for (int off = 1; off < C; off <<= 1) {
                    const double before = __shfl_up(l, off, WAVE);
                    if (lane >= off) l += before;
                }
            }
            if (lane < C) {
                const float hi = (float)l;
                l_hi[lane] = hi;
                l_lo[lane] = (float)(l - (double)hi);
                b_s[lane] = b;
            }
        }
        // ---- this lane's column of v, the tokens in the order of the products
        float v[C / 16][4];
#pragma unroll
        for (int x = 0; x < C / 16; ++x)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * x + 4 * g + i;
                float e = to_f32(rows[(size_t)(base + min(t, nt - 1)) * p.row_stride + p.v_off + h * dv + min(col, dv - 1)]);
                if (p.silu) e = silu_for<T>(e);
                v[x][i] = to_f32(from_f32<T>(t >= nt || col >= p.dvx ? 0.f : col < dv ? e : 1.f));
            }
        __syncthreads();
        // ---- the weights
        {
            auto between = [&](int t, int u) { return expf((l_hi[t] - l_hi[u]) + (l_lo[t] - l_lo[u])); };
            if (MODE != 1) {
                for (int x = tid; x < C * 16; x += threads) {
                    const int t = x / 16, u = t / 16 * 16 + x % 16;
                    w_own[t * 20 + x % 16] = u <= t ? between(t, u) * b_s[u] : 0.f;
                }
                for (int x = tid; x < TT * C; x += threads) {
                    const int c = x / C, t = x % C;
                    if (t / 16 > c) w_behind[x] = between(t, 16 * c + 15);
                }
                for (int t = tid; t < C; t += threads) {
                    w_tile[t] = between(t | 15, t) * b_s[t];
                    w_start[t] = expf(l_hi[t] + l_lo[t]);
                }
            }
            for (int t = tid; t < C; t += threads) w_end[t] = between(C - 1, t) * b_s[t];
            if (tid == 0) w_all = expf(l_hi[C - 1] + l_lo[C - 1]);
        }
        __syncthreads();
        if (!active) continue;
        if (MODE != 1) {
            // ---- what the chunk found in the state, and the scores
            f32x4 o[TT], sc[TT][TT];
#pragma unroll
            for (int a = 0; a < TT; ++a) {
                o[a] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int c = 0; c < TT; ++c) sc[a][c] = f32x4{0.f, 0.f, 0.f, 0.f};
            }
#pragma unroll
            for (int x = 0; x < KT; x += TPS) {
                float sv[M::PER];
#pragma unroll
                for (int j = 0; j < M::PER; ++j) sv[j] = s[x + j / 4][j % 4];
                frag sf[M::SPLITS], kf[TT];
                M::split(sv, sf);
#pragma unroll
                for (int c = 0; c < TT; ++c) kf[c] = M::load(ks + (16 * c + l16) * LDK + 16 * x + 4 * g);
#pragma unroll
                for (int a = 0; a < TT; ++a) {
                    const frag qf = M::load(qs + (16 * a + l16) * LDK + 16 * x + 4 * g);
#pragma unroll
                    for (int e = M::SPLITS - 1; e >= 0; --e) o[a] = M::mma(sf[e], qf, o[a]);
#pragma unroll
                    for (int c = 0; c <= a; ++c) sc[a][c] = M::mma(kf[c], qf, sc[a][c]);
                }
            }
            // ---- the chunk's own tokens: the lane's scores are those of token t (its column) with the tokens 16 c + 4 g + i
#pragma unroll
            for (int a = 0; a < TT; ++a) {
                const int t = 16 * a + l16;
                o[a] *= w_start[t];
#pragma unroll
                for (int c0 = 0; c0 < TT; c0 += TPS) {
                    if (c0 > a) continue;
                    float w[M::PER], vv[M::PER];
#pragma unroll
                    for (int j = 0; j < M::PER; ++j) {
                        const int c = c0 + j / 4;
                        const float own = c == a ? w_own[t * 20 + 4 * g + j % 4] : 0.f;
                        w[j] = c < a ? sc[a][c][j % 4] * (w_behind[c * C + t] * w_tile[16 * c + 4 * g + j % 4]) : c == a ? sc[a][c][j % 4] * own : 0.f;
                        vv[j] = v[c][j % 4];
                    }
                    frag wf[M::SPLITS];
                    M::split(w, wf);
                    const frag vf = M::exact(vv);
#pragma unroll
                    for (int e = M::SPLITS - 1; e >= 0; --e) o[a] = M::mma(vf, wf[e], o[a]);
                }
                if (t < nt) {
                    float *out = p.o + ((size_t)h * p.n + base + t) * (p.tiles * 16) + tile * 16 + 4 * g;
                    *(float4 *)out = make_float4(p.scale * o[a][0], p.scale * o[a][1], p.scale * o[a][2], p.scale * o[a][3]);
                }
            }
        }
        l_run += (double)l_hi[C - 1] + (double)l_lo[C - 1];
        if (MODE == 2 && !last && base + C >= t1) break;                       // nobody reads the state behind this run
        // ---- the state behind the chunk
        const float keep = w_all;
#pragma unroll
        for (int x = 0; x < KT; ++x) s[x] *= keep;
#pragma unroll
        for (int c0 = 0; c0 < C / 16; c0 += TPS) {
            float w[M::PER];
#pragma unroll
            for (int j = 0; j < M::PER; ++j) {
                const int c = c0 + j / 4, u = 16 * c + 4 * g + j % 4;
                w[j] = v[c][j % 4] * w_end[u];
            }
            frag wf[M::SPLITS];
            M::split(w, wf);
#pragma unroll
            for (int x = 0; x < KT; ++x) {
                const frag kf = M::load(kt + (16 * x + l16) * LDT + 16 * c0 + 4 * g);
#pragma unroll
                for (int e = M::SPLITS - 1; e >= 0; --e) s[x] = M::mma(kf, wf[e], s[x]);
            }
        }
    }
    if (!active || (MODE == 2 && !last)) return;
#pragma unroll
    for (int x = 0; x < KT; ++x)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int key = 16 * x + 4 * g + i;
            if (key < d && col < p.dvx) {
                if (MODE == 1) p.run_b[(run_no * d + key) * p.dvx + col] = s[x][i];
                else *in_slot(key) = s[x][i];
            }
        }
    if (MODE == 1 && tile == 0 && lane == 0) p.run_l[run_no] = (float)l_run;
}

// The state that every run of a long request starts from: run 0 from the request's state (zeros at position 0), the next from exp(sum of
// log a) times the run's start plus the run's own sum.  A thread per element.
__global__ void __launch_bounds__(256)
ds_chain_kernel(DsArgs p) {
    const int h = blockIdx.y, r = blockIdx.z, t0 = p.q_start[r], q_len = p.q_start[r + 1] - t0;
    if (q_len < DS_LONG) return;
    const int e = blockIdx.x * 256 + threadIdx.x, per = p.d * p.dvx;
    if (e >= per) return;
    const int key = e / p.dvx, col = e % p.dvx, runs = (q_len + ds_run_len(q_len) - 1) / ds_run_len(q_len);
    const float *slot = p.state + (size_t)p.state_slot[r] * p.slot_stride;
    float at = 0.f;
    if (p.ctx_len[r] > q_len) at = col < p.dv ? slot[((size_t)h * p.d + key) * p.dv + col] : slot[p.n_off + (size_t)h * p.d + key];
    const size_t first = ((size_t)ds_long_index(p.q_start, r) * DS_RUNS) * p.heads + h;
    float b[DS_RUNS];                             // (all loads are on their way before the first is needed)
#pragma unroll
    for (int k = 0; k < DS_RUNS; ++k) b[k] = p.run_b[(first + (size_t)min(k, runs - 2) * p.heads) * per + e];
#pragma unroll
    for (int k = 0; k < DS_RUNS; ++k) {
        if (k >= runs) break;
        const size_t no = first + (size_t)k * p.heads;
        p.run_in[no * per + e] = at;
        if (k + 1 < runs) at = fmaf(expf(p.run_l[no]), at, b[k]);
    }
}

// ---------------------------------------------------------------- outputs
// joint: out[t, :] = o / rms(o) over all heads * weight * sigmoid(gate) * factor.  A workgroup per token, V columns a thread.
template <class T, int V>
__global__ void __launch_bounds__(256)
ds_out_joint_kernel(const float *__restrict__ o, int ldo, const T *__restrict__ rows, int row_stride, int g_off, const float *__restrict__ weight,
                    T *__restrict__ out, int out_stride, int n, int heads, int dv, float eps, float factor) {
    __shared__ float scratch[16];
    const int t = blockIdx.x, hv = heads * dv;
    float sq = 0.f;
    for (int c = threadIdx.x * V; c < hv; c += 256 * V) {
        const DsVec<float, V> x = *(const DsVec<float, V> *)(o + ((size_t)(c / dv) * n + t) * ldo + c % dv);
#pragma unroll
        for (int e = 0; e < V; ++e) sq += x.v[e] * x.v[e];
    }
    const float f = factor * rsqrtf(block_sum(sq, scratch) / (float)hv + eps);
    for (int c = threadIdx.x * V; c < hv; c += 256 * V) {
        const DsVec<float, V> x = *(const DsVec<float, V> *)(o + ((size_t)(c / dv) * n + t) * ldo + c % dv);
        const DsVec<float, V> w = *(const DsVec<float, V> *)(weight + c);
        const DsVec<T, V> z = *(const DsVec<T, V> *)(rows + (size_t)t * row_stride + g_off + c);
        DsVec<T, V> y;
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] = from_f32<T>(x.v[e] * f * w.v[e] * sigmoid_f(to_f32(z.v[e])));
        *(DsVec<T, V> *)(out + (size_t)t * out_stride + c) = y;
    }
}

// per head: one wave per (token, head), four to a workgroup; column dv of o is the normaliser's.
template <class T, int V>
__global__ void __launch_bounds__(256)
ds_out_heads_kernel(const float *__restrict__ o, int ldo, const float *__restrict__ m, const T *__restrict__ rows, int row_stride, int g_off,
                    const float *__restrict__ weight, T *__restrict__ out, int out_stride, int n, int heads, int dv, float eps, float factor) {
    const int t = blockIdx.x, h = blockIdx.y * 4 + threadIdx.x / WAVE, lane = threadIdx.x & 63;
    if (h >= heads) return;
    const float *x = o + ((size_t)h * n + t) * ldo;
    const float inv = 1.0f / (fmaxf(fabsf(x[dv]), expf(-m[(size_t)h * n + t])) + 1e-6f);
    float sq = 0.f;
    for (int c = lane * V; c < dv; c += WAVE * V) {
        const DsVec<float, V> a = *(const DsVec<float, V> *)(x + c);
#pragma unroll
        for (int e = 0; e < V; ++e) sq += (a.v[e] * inv) * (a.v[e] * inv);
    }
    const float f = factor * inv * rsqrtf(wave_sum_in_place(sq) / (float)dv + eps);
    for (int c = lane * V; c < dv; c += WAVE * V) {
        const DsVec<float, V> a = *(const DsVec<float, V> *)(x + c), w = *(const DsVec<float, V> *)(weight + h * dv + c);
        const DsVec<T, V> z = *(const DsVec<T, V> *)(rows + (size_t)t * row_stride + g_off + h * dv + c);
        DsVec<T, V> y;
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] = from_f32<T>(a.v[e] * f * w.v[e] * sigmoid_f(to_f32(z.v[e])));
        *(DsVec<T, V> *)(out + (size_t)t * out_stride + h * dv + c) = y;
    }
}

// ---------------------------------------------------------------- single tokens
// A workgroup per (request, head), every request one token.  A thread keeps V neighbouring value columns of every ROWS-th key
// channel; the state's loads go out before anything else is made.  FINISH: gated: the finished output; fixed: the rows times weight
// and gate, the norm's factor still to come, and the head's share of the row's sum of squares.
struct DsSingle {
    const void *rows;
    int row_stride, q_off, k_off, v_off, g_off;
    const float *decay;                           // fixed: [heads] (null: gated)
    const float *z, *bias_i, *bias_f;             // gated: as ds_gates_kernel
    int ldz;
    float cap;
    float *state;
    size_t slot_stride, n_off, m_off;
    const float *weight;
    void *out;                                    // [n, out_stride]
    int out_stride;
    float *sumsq;                                 // fixed: [n, heads]
    const int *q_start, *ctx_len, *state_slot;
    int heads, d, dv;
    float scale, eps, factor;
    int silu;
};

template <class TI, class T, int V>
__global__ void __launch_bounds__(256)
ds_single_kernel(DsSingle p) {
    constexpr int KEEP = 16;                      // pieces of the state a thread loads at a time
    __shared__ float qk[2][256];
    __shared__ float vs[512], scratch[16];
    __shared__ float4 red4[256];                  // the rows' partial sums, V of each thread
    float *red = (float *)red4;
    const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, t = p.q_start[r], d = p.d, dv = p.dv;
    const bool fresh = p.ctx_len[r] == 1;
    const TI *row = (const TI *)p.rows + (size_t)t * p.row_stride;
    float *slot = p.state + (size_t)p.state_slot[r] * p.slot_stride, *S = slot + (size_t)h * d * dv;
    const int groups = (dv + V - 1) / V;          // of V columns
    const int cols = min(groups, 256), nrows = 256 / cols, my_row = tid / cols, my_col = tid % cols;
    const bool works = my_row < nrows;
    float a, b, m_now = 0.f;
    if (p.decay) {
        a = p.decay[h];
        b = 1.f;
    } else {
        const float m = fresh ? 0.f : slot[p.m_off + h];
        const float gi = p.cap * tanhf((p.z[(size_t)t * p.ldz + h] + p.bias_i[h]) / p.cap);
        const float f = log_sigmoid_f(p.cap * tanhf((p.z[(size_t)t * p.ldz + p.heads + h] + p.bias_f[h]) / p.cap));
        m_now = fmaxf(f + m, gi);
        a = expf(f + m - m_now);
        b = expf(gi - m_now);
    }
    if (fresh) a = 0.f;                           // the state is zero: what the slot held is not used (it is not read either)
    for (int c = tid; c < d; c += 256) {
        float q = to_f32(row[p.q_off + h * d + c]), k = to_f32(row[p.k_off + h * d + c]);
        if (p.silu) { q = silu_for<T>(q); k = silu_for<T>(k); }
        qk[0][c] = to_f32(from_f32<T>(q));
        qk[1][c] = to_f32(from_f32<T>(k));
    }
    for (int c = tid; c < dv; c += 256) {
        float v = to_f32(row[p.v_off + h * dv + c]);
        if (p.silu) v = silu_for<T>(v);
        vs[c] = to_f32(from_f32<T>(v));
    }
    __syncthreads();                              // (every thread has read m)
    float inv = 1.f;
    if (!p.decay) {
        float den = 0.f;
        if (tid < d) {
            float *N = slot + p.n_off + (size_t)h * d + tid;
            const float n_new = fmaf(b, qk[1][tid], fresh ? 0.f : a * *N);
            *N = n_new;
            den = n_new * qk[0][tid];
        }
        den = p.scale * block_sum(den, scratch);
        inv = 1.0f / (fmaxf(fabsf(den), expf(-m_now)) + 1e-6f);
        if (tid == 0) slot[p.m_off + h] = m_now;
    }
    float sq = 0.f;
    for (int c0 = 0; c0 < groups; c0 += 256) {    // (once, unless a head has more than 256 groups of columns)
        const int cg = c0 + my_col, c = cg * V;
        const bool on = works && cg < groups;
        float acc[V], v[V];
#pragma unroll
        for (int e = 0; e < V; ++e) { acc[e] = 0.f; v[e] = on && c + e < dv ? b * vs[c + e] : 0.f; }
        for (int i0 = my_row; on && i0 < d; i0 += KEEP * nrows) {
            DsVec<float, V> s[KEEP];
#pragma unroll
            for (int x = 0; x < KEEP; ++x) {
                const int i = i0 + x * nrows;
                if (fresh) {
#pragma unroll
                    for (int e = 0; e < V; ++e) s[x].v[e] = 0.f;
                } else {
                    s[x] = *(const DsVec<float, V> *)(S + (size_t)min(i, d - 1) * dv + c);
                }
            }
#pragma unroll
            for (int x = 0; x < KEEP; ++x) {
                const int i = i0 + x * nrows;
                if (i >= d) break;
                const float k = qk[1][i], q = qk[0][i];
#pragma unroll
                for (int e = 0; e < V; ++e) {
                    s[x].v[e] = fmaf(a, s[x].v[e], k * v[e]);
                    acc[e] = fmaf(q, s[x].v[e], acc[e]);
                }
                *(DsVec<float, V> *)(S + (size_t)i * dv + c) = s[x];
            }
        }
        __syncthreads();                          // (red is free again)
#pragma unroll
        for (int e = 0; e < V; ++e) red[tid * V + e] = acc[e];
        __syncthreads();
        for (int x = tid; x < cols * V; x += 256) {
            const int cc = c0 * V + x;
            if (cc >= dv) continue;
            float o = 0.f;
            for (int w = 0; w < nrows; ++w) o += red[w * cols * V + x];
            o *= p.scale * inv;
            vs[cc] = o;                           // (v of these columns has been used)
            sq += o * o;
        }
    }
    const float total = block_sum(sq, scratch);   // (its barriers make vs visible)
    const float f = p.factor * (p.decay ? 1.f : rsqrtf(total / (float)dv + p.eps));
    if (p.decay && tid == 0) p.sumsq[(size_t)t * p.heads + h] = total;
    T *out = (T *)p.out + (size_t)t * p.out_stride + h * dv;
    for (int c = tid; c < dv; c += 256) {
        const float z = to_f32(row[p.g_off + h * dv + c]);
        out[c] = from_f32<T>(vs[c] * f * p.weight[h * dv + c] * sigmoid_f(z));
    }
}

// rows[t, :] times rsqrt(sum of the token's shares / width + eps): the norm that ds_single_kernel leaves to whoever reads its rows.
template <class T>
__global__ void __launch_bounds__(256)
ds_row_factor_kernel(T *__restrict__ rows, int stride, const float *__restrict__ sumsq, int parts, int width, float eps) {
    const int t = blockIdx.x;
    float s = 0.f;
    for (int i = 0; i < parts; ++i) s += sumsq[(size_t)t * parts + i];
    const float f = rsqrtf(s / (float)width + eps);
    for (int c = threadIdx.x; c < width; c += 256) rows[(size_t)t * stride + c] = from_f32<T>(to_f32(rows[(size_t)t * stride + c]) * f);
}

LCU_API int lcu_decay_scan_long(void) { return DS_LONG; }
// the value columns of a head in the scratch array of outputs
LCU_API int lcu_decay_scan_out_cols(int dv, int gated) { return (dv + (gated ? 1 : 0) + 15) / 16 * 16; }
LCU_API long long lcu_decay_scan_run_floats(int n_long, int heads, int d, int dv, int gated) {
    return (long long)n_long * DS_RUNS * heads * (2ll * d * (dv + (gated ? 1 : 0)) + 1);
}

static bool ds_sizes_ok(int heads, int d, int dv, long long slot_stride, int gated) {
    return heads > 0 && heads <= 65535 && d > 0 && d <= 256 && dv > 0 && dv <= 512 &&
           slot_stride >= (long long)heads * d * dv + (gated ? (long long)heads * (d + 1) : 0);
}

template <class T>
static int ds_launch(DsArgs &p, int n_req, int n_long, hipStream_t stream) {
    const int blocks = (p.tiles + DS_WAVES - 1) / DS_WAVES, waves = (p.tiles + blocks - 1) / blocks;
    const dim3 block(waves * WAVE);
#define MODES(D)                                                                                                              \
    do {                                                                                                                      \
        if (n_long < n_req) ds_chunk_kernel<T, D, 0><<<dim3(blocks, p.heads, n_req), block, 0, stream>>>(p);                  \
        if (n_long > 0) {                                                                                                     \
            ds_chunk_kernel<T, D, 1><<<dim3(blocks, p.heads, n_req * DS_RUNS), block, 0, stream>>>(p);                        \
            ds_chain_kernel<<<dim3((p.d * p.dvx + 255) / 256, p.heads, n_req), dim3(256), 0, stream>>>(p);                    \
            ds_chunk_kernel<T, D, 2><<<dim3(blocks, p.heads, n_req * DS_RUNS), block, 0, stream>>>(p);                        \
        }                                                                                                                     \
    } while (0)
    if (p.d <= 32) MODES(32);
    else if (p.d <= 64) MODES(64);
    else if (p.d <= 96) MODES(96);
    else if (p.d <= 128) MODES(128);
    else MODES(256);
#undef MODES
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// rows: [n, row_stride] of `type` with q, k (heads * d) and v, gate (heads * dv) at their columns.  Fixed: log_decay [heads][2].  Gated
// (log_decay null): z [n, ldz], bias_i, bias_f [heads], gates: scratch of 3 * heads * n floats.  o: scratch [heads, n,
// lcu_decay_scan_out_cols]; runs: scratch of lcu_decay_scan_run_floats (null if n_long is 0).  state: slot s at state + s * slot_stride.
// out: [n, out_stride] of `type`, heads * dv columns.
LCU_API int lcu_decay_scan(const void *rows, int type, int row_stride, int q_off, int k_off, int v_off, int g_off, int silu,
                           const float *log_decay, const float *z, int ldz, const float *bias_i, const float *bias_f, float cap, float *gates,
                           float *o, float *runs, int n_long, float *state, long long slot_stride, const float *weight, void *out,
                           int out_stride, const int *q_start, const int *ctx_len, const int *state_slot, int n, int n_req, int heads, int d,
                           int dv, float scale, float eps, float factor, hipStream_t stream) {
    if (n <= 0 || n_req <= 0) return LCU_OK;
    const int gated = log_decay == nullptr;
    if (!ds_sizes_ok(heads, d, dv, slot_stride, gated) || !rows || !o || !state || !weight || !out || out_stride < heads * dv || n_long < 0 ||
        (n_long > 0 && !runs) || n_req * DS_RUNS > 65535 || (gated && (!z || !bias_i || !bias_f || !gates || !(cap > 0.f))))
        return LCU_BAD_ARGUMENT;
    DsArgs p = {};
    p.rows = rows; p.row_stride = row_stride; p.q_off = q_off; p.k_off = k_off; p.v_off = v_off;
    p.log_decay = log_decay;
    p.state = state; p.slot_stride = (size_t)slot_stride; p.n_off = (size_t)heads * d * dv;
    p.o = o;
    p.q_start = q_start; p.ctx_len = ctx_len; p.state_slot = state_slot;
    p.n = n; p.heads = heads; p.d = d; p.dv = dv; p.dvx = dv + gated; p.tiles = (p.dvx + 15) / 16;
    p.scale = scale;
    p.silu = silu;
    p.four = d % 4 == 0 && row_stride % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0 && (uintptr_t)rows % 16 == 0;
    const size_t one = (size_t)n_long * DS_RUNS * heads;
    if (n_long) { p.run_b = runs; p.run_in = runs + one * d * p.dvx; p.run_l = p.run_in + one * d * p.dvx; }
    float *m = nullptr;
    if (gated) {
        float *la = gates, *b = gates + (size_t)heads * n;
        m = b + (size_t)heads * n;
#define GATES(THREADS) ds_gates_kernel<THREADS><<<dim3(heads, n_req), dim3(THREADS), 0, stream>>>(z, ldz, bias_i, bias_f, cap, state, (size_t)slot_stride, \
                                                                  p.n_off + (size_t)heads * d, la, b, m, q_start, ctx_len, state_slot, n, heads)
        if (n > 256) GATES(1024);
        else GATES(256);
#undef GATES
        LCU_LAUNCH_CHECK();
        p.log_a = la;
        p.b = b;
    }
    int rc = type == LCU_F32 ? ds_launch<float>(p, n_req, n_long, stream) : type == LCU_BF16 ? ds_launch<bf16_t>(p, n_req, n_long, stream) : LCU_BAD_ARGUMENT;
    if (rc) return rc;
    const int ldo = p.tiles * 16;
    const bool wide = dv % 4 == 0 && row_stride % 4 == 0 && g_off % 4 == 0 && out_stride % 4 == 0 && (uintptr_t)rows % 16 == 0 &&
                      (uintptr_t)out % 16 == 0 && (uintptr_t)weight % 16 == 0;
#define OUT(T, V)                                                                                                                                 \
    do {                                                                                                                                        \
        if (gated) ds_out_heads_kernel<T, V><<<dim3(n, (heads + 3) / 4), dim3(256), 0, stream>>>(o, ldo, m, (const T *)rows, row_stride, g_off, weight, (T *)out, out_stride, n, heads, dv, eps, factor); \
        else ds_out_joint_kernel<T, V><<<dim3(n), dim3(256), 0, stream>>>(o, ldo, (const T *)rows, row_stride, g_off, weight, (T *)out, out_stride, n, heads, dv, eps, factor); \
    } while (0)
    if (type == LCU_F32) { if (wide) OUT(float, 4); else OUT(float, 1); }
    else { if (wide) OUT(bf16_t, 4); else OUT(bf16_t, 1); }
#undef OUT
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// The same for a step in which every request feeds one token (n == n_req; the rows may be float32 beside a bfloat16 output).  Fixed (decay [heads] given): `sumsq` [n, heads] takes the
// heads' shares of the rows' sums of squares, and the rows in `out` are not yet normed; with apply they are, by one more kernel.
LCU_API int lcu_decay_scan_single(const void *rows, int type, int row_stride, int q_off, int k_off, int v_off, int g_off, int silu,
                                  const float *decay, const float *z, int ldz, const float *bias_i, const float *bias_f, float cap, float *state,
                                  long long slot_stride, const float *weight, void *out, int out_type, int out_stride, float *sumsq, int apply,
                                  const int *q_start, const int *ctx_len, const int *state_slot, int n_req, int heads, int d, int dv, float scale,
                                  float eps, float factor, hipStream_t stream) {
    if (n_req <= 0) return LCU_OK;
    const int gated = decay == nullptr;
    if (!ds_sizes_ok(heads, d, dv, slot_stride, gated) || !rows || !state || !weight || !out || out_stride < heads * dv || (!gated && !sumsq) ||
        (gated && (!z || !bias_i || !bias_f || !(cap > 0.f))))
        return LCU_BAD_ARGUMENT;
    DsSingle p = {};
    p.rows = rows; p.row_stride = row_stride; p.q_off = q_off; p.k_off = k_off; p.v_off = v_off; p.g_off = g_off;
    p.decay = decay; p.z = z; p.bias_i = bias_i; p.bias_f = bias_f; p.ldz = ldz; p.cap = cap;
    p.state = state; p.slot_stride = (size_t)slot_stride; p.n_off = (size_t)heads * d * dv; p.m_off = p.n_off + (size_t)heads * d;
    p.weight = weight; p.out = out; p.out_stride = out_stride; p.sumsq = sumsq;
    p.q_start = q_start; p.ctx_len = ctx_len; p.state_slot = state_slot;
    p.heads = heads; p.d = d; p.dv = dv; p.scale = scale; p.eps = eps; p.factor = factor; p.silu = silu;
    const bool wide = dv % 4 == 0 && slot_stride % 4 == 0 && (uintptr_t)state % 16 == 0;
    const dim3 grid(n_req, heads), block(256);
#define GO(TI, T)                                                                 \
    do {                                                                          \
        if (wide) ds_single_kernel<TI, T, 4><<<grid, block, 0, stream>>>(p);      \
        else ds_single_kernel<TI, T, 1><<<grid, block, 0, stream>>>(p);           \
    } while (0)
    if (type == LCU_F32 && out_type == LCU_F32) GO(float, float);
    else if (type == LCU_F32 && out_type == LCU_BF16) GO(float, bf16_t);
    else if (type == LCU_BF16 && out_type == LCU_BF16) GO(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    if (!gated && apply) {
        if (out_type == LCU_F32) ds_row_factor_kernel<float><<<dim3(n_req), block, 0, stream>>>((float *)out, out_stride, sumsq, heads, heads * dv, eps);
        else ds_row_factor_kernel<bf16_t><<<dim3(n_req), block, 0, stream>>>((bf16_t *)out, out_stride, sumsq, heads, heads * dv, eps);
        LCU_LAUNCH_CHECK();
    }
    return LCU_OK;
}
