// A time mixer with a matrix state per head, a decay per key channel that is a function of the token, and a bonus for
// the token's own key.  Per head, with key channels i and value channels j, S [d, dv] in 32-bit:
//
//   w   = exp(-exp(z)),  z = W2 tanh(l) + w0                        (l: a low-rank projection of the token)
//   o_j = sum_i r_i (S_ij + u_i k_i v_j)  =  sum_i r_i S_ij + b v_j,  b = sum_i r_i u_i k_i
//   S  <- diag(w) S + k v^T                                         (o reads the state as the token found it)
//
// What the projections read is mixed with the token before: token_shift_kernel makes, for every projection s, the rows
// h + (h' - h) mu_s, h' the token before's h (zeros in front of a request's first token; the last h of a step is state).
//
// A step of single tokens: one kernel per layer, a workgroup per (request, head), which streams the head's state through
// its registers and makes everything between the projections and the output product.
// Any other step: prep (parallel over tokens and heads: w and b, 32-bit, a head's tokens one after the other), scan, out.  The
// scan (r, k and v as the projections left them go through LDS beside w, a stage of tokens at a time, the next stage on its way): column j of S depends on column j alone; a
// workgroup keeps 64 columns of one head in registers, a lane four columns of a sixteenth of the key channels; the sum over
// key channels crosses sixteen lanes after a stage of tokens.  A request that feeds at least WK_LONG tokens is cut into
// WK_RUNS runs that are walked at once, twice: first from zeros, which gives what a run adds to any state it starts from
// (S_end = diag(product of its w) S_start + B); a small kernel chains the runs' starts; the second walk gives the outputs.
//
// The state is taken as zero where a request's first token of the step stands at position 0.  A token's result depends on
// the tokens before it in its request only; how a request was cut into steps changes roundings.
#include "common.h"
#include "lane_moves.h"

constexpr int WK_MAX_RANK = 512;
constexpr int WK_THREADS = 256;
constexpr int WK_LANES = 16;                               // lanes that share a column
constexpr int WK_CPL = 4;                                  // columns of a lane
constexpr int WK_COLS = WK_THREADS / WK_LANES * WK_CPL;    // columns of a workgroup
constexpr int WK_TOK = 8;                                  // tokens of a stage
constexpr int WK_RUNS = 16;
constexpr int WK_LONG = 512;
constexpr int WK_PREP_TOK = 16;                            // tokens of a prep workgroup

// ---------------------------------------------------------------- the mix with the token before
// h: [n, d] 32-bit; mu: [sets, d]; out: [sets, n, d].  The previous token's h of a request's first token of the step lies at
// prev + slot * slot_stride (d floats); that token's workgroup also leaves the step's last h there (each thread reads an
// element before it writes it, so nothing races).
// V neighbouring channels a thread, TB tokens one after the other (the weights are loaded once for them, and a token's own row is
// the next one's row before).
template <class T, int V> struct alignas(V * sizeof(T)) WkVec { T v[V]; };

template <class T, int V, int TB>
__global__ void __launch_bounds__(256)
token_shift_kernel(const float *__restrict__ h, const float *__restrict__ mu, int sets, float *__restrict__ prev, size_t slot_stride,
                   const int *__restrict__ req_of_token, const int *__restrict__ q_start, const int *__restrict__ ctx_len,
                   const int *__restrict__ state_slot, T *__restrict__ out, int n, int d) {
    constexpr int SETS = 8;                                    // weights kept in registers; more sets are walked in turn
    const int c = (blockIdx.y * 256 + threadIdx.x) * V, t_first = blockIdx.x * TB, t_end = min(n, t_first + TB);
    if (c >= d) return;
    for (int s0 = 0; s0 < sets; s0 += SETS) {
        WkVec<float, V> m[SETS];
#pragma unroll
        for (int s = 0; s < SETS; ++s)
            if (s0 + s < sets) m[s] = *(const WkVec<float, V> *)(mu + (size_t)(s0 + s) * d + c);
        WkVec<float, V> before = {};
#pragma unroll
        for (int b = 0; b < TB; ++b) {
            const int t = t_first + b;
            if (t >= t_end) break;
            const int r = req_of_token[t], t0 = q_start[r], t1 = q_start[r + 1];
            const WkVec<float, V> x = *(const WkVec<float, V> *)(h + (size_t)t * d + c);
            if (t == t0) {
                WkVec<float, V> *ps = (WkVec<float, V> *)(prev + (size_t)state_slot[r] * slot_stride + c);
                before = *ps;
                if (ctx_len[r] - (t1 - t0) == 0)
#pragma unroll
                    for (int e = 0; e < V; ++e) before.v[e] = 0.f;
                if (s0 + SETS >= sets) *ps = *(const WkVec<float, V> *)(h + (size_t)(t1 - 1) * d + c);
            } else if (b == 0) {
                before = *(const WkVec<float, V> *)(h + (size_t)(t - 1) * d + c);
            }
#pragma unroll
            for (int s = 0; s < SETS; ++s) {
                if (s0 + s >= sets) break;
                WkVec<T, V> o;
#pragma unroll
                for (int e = 0; e < V; ++e) o.v[e] = from_f32<T>(fmaf(before.v[e] - x.v[e], m[s].v[e], x.v[e]));
                *(WkVec<T, V> *)(out + ((size_t)(s0 + s) * n + t) * d + c) = o;
            }
            before = x;
        }
    }
}

LCU_API int lcu_token_shift(const float *h, const float *mu, int sets, float *prev, long long slot_stride, const int *req_of_token,
                            const int *q_start, const int *ctx_len, const int *state_slot, void *out, int out_type, int n, int d,
                            hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (d <= 0 || sets <= 0 || slot_stride < d || !h || !mu || !prev || !out) return LCU_BAD_ARGUMENT;
    const bool four = d % 4 == 0 && slot_stride % 4 == 0 && (uintptr_t)h % 16 == 0 && (uintptr_t)mu % 16 == 0 && (uintptr_t)prev % 16 == 0 &&
                      (uintptr_t)out % 16 == 0;
    const int v = four ? 4 : 1, tb = n >= 512 ? 4 : 1;
    const dim3 grid((n + tb - 1) / tb, (d + 256 * v - 1) / (256 * v)), block(256);
#define GO(T, V, TB) token_shift_kernel<T, V, TB><<<grid, block, 0, stream>>>(h, mu, sets, prev, (size_t)slot_stride, req_of_token, q_start, ctx_len, state_slot, (T *)out, n, d)
#define SIZES(T)                          \
    do {                                  \
        if (four && tb == 4) GO(T, 4, 4); \
        else if (four) GO(T, 4, 1);       \
        else if (tb == 4) GO(T, 1, 4);    \
        else GO(T, 1, 1);                 \
    } while (0)
    if (out_type == LCU_F32) SIZES(float);
    else if (out_type == LCU_BF16) SIZES(bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef SIZES
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// ---------------------------------------------------------------- prep
__host__ __device__ constexpr int wk_pad_keys(int d) { return d <= 64 ? 64 : d <= 128 ? 128 : 256; }      // key channels of a row of w (zeros behind the true ones)
__host__ __device__ constexpr int wk_pad_cols(int dv) { return (dv + WK_COLS - 1) / WK_COLS * WK_COLS; }

// rows: [n, row_stride] with r and k (heads * d) at their columns; low: [n, ld_low] 32-bit; w2t: [rank, heads * d].  To w: [heads][n][D]
// and bonus: [heads][n].
// A workgroup has 256 threads, D of them a head: 256 / D heads of WK_PREP_TOK tokens, a thread per key channel.  The rank's numbers
// lie in LDS with the tokens side by side: every thread reads the same four at a time.
template <class T>
__global__ void __launch_bounds__(256)
wkv_prep_kernel(const T *__restrict__ rows, int row_stride, int r_off, int k_off, const float *__restrict__ low, int ld_low,
                const float *__restrict__ w2t, const float *__restrict__ w0, const float *__restrict__ u, float *__restrict__ w_out,
                float *__restrict__ bonus, int n, int heads, int d, int rank, int D) {
    constexpr int TB = WK_PREP_TOK;
    extern __shared__ float4 th4[];                            // [rank][TB]
    __shared__ float part[TB][4];
    float *th = (float *)th4;
    const int t0 = blockIdx.x * TB, nt = min(TB, n - t0);
    for (int x = threadIdx.x; x < TB * rank; x += 256) {
        const int b = x / rank, j = x % rank;                  // (neighbouring threads, neighbouring addresses in memory)
        th[j * TB + b] = b < nt ? tanhf(low[(size_t)(t0 + b) * ld_low + j]) : 0.f;
    }
    __syncthreads();
    const int h = blockIdx.y * (256 / D) + threadIdx.x / D, i = threadIdx.x % D, c = h * d + i;
    const bool live = i < d && h < heads;
    float z[TB];
#pragma unroll
    for (int b = 0; b < TB; ++b) z[b] = live ? w0[c] : 0.f;
    if (live) {
#pragma unroll 4
        for (int j = 0; j < rank; ++j) {
            const float w = w2t[(size_t)j * heads * d + c];
#pragma unroll
            for (int b = 0; b < TB; b += 4) {
                const float4 q = th4[(j * TB + b) / 4];
                z[b] = fmaf(w, q.x, z[b]);
                z[b + 1] = fmaf(w, q.y, z[b + 1]);
                z[b + 2] = fmaf(w, q.z, z[b + 2]);
                z[b + 3] = fmaf(w, q.w, z[b + 3]);
            }
        }
    }
    const float uu = live ? u[c] : 0.f;
    float own[TB];                                             // r u k of the thread's channel
#pragma unroll
    for (int b = 0; b < TB; ++b) {
        const T *row = rows + (size_t)(t0 + min(b, nt - 1)) * row_stride + (live ? c : 0);       // (no branch around a load)
        own[b] = to_f32(row[r_off]) * uu * to_f32(row[k_off]);
    }
#pragma unroll
    for (int b = 0; b < TB; ++b) {
        const float s = wave_sum_in_place(own[b]);
        if ((threadIdx.x & (WAVE - 1)) == 0) part[b][threadIdx.x / WAVE] = s;
        if (h < heads && b < nt) w_out[((size_t)h * n + t0 + b) * D + i] = live ? expf(-expf(z[b])) : 0.f;
    }
    __syncthreads();
    if (i < nt && h < heads) {
        float s = 0.f;
        for (int w = 0; w < D / WAVE; ++w) s += part[i][threadIdx.x / D * (D / WAVE) + w];
        bonus[(size_t)h * n + t0 + i] = s;
    }
}

// ---------------------------------------------------------------- scan
// how many of the requests before r feed at least WK_LONG tokens: r's place among those in the runs' arrays
__device__ __forceinline__ int wk_long_index(const int *__restrict__ q_start, int r) {
    int li = 0;
    for (int i = 0; i < r; ++i) li += (q_start[i + 1] - q_start[i] >= WK_LONG);
    return li;
}

// MODE 0: a request of fewer than WK_LONG tokens in one chain; 1: a run from zeros, leaves B in run_b and the product of its w in
// run_p; 2: a run from run_in, with outputs.  o: [heads][n][DV].  run_b, run_in: [long request][run][heads][d][dv], run_p: [..][heads][d].
// FOUR: d, dv and every column and stride are multiples of 4 (r, k and v are loaded four at a time).
template <class T> struct alignas(4 * sizeof(T)) WkQuad { T v[4]; };

template <class T, int DPL, int MODE, bool FOUR>
__global__ void __launch_bounds__(WK_THREADS)
wkv_scan_kernel(const T *__restrict__ rows, int row_stride, int r_off, int k_off, int v_off, const float *__restrict__ w_in,
                const float *__restrict__ bonus, float *__restrict__ state, size_t slot_stride, float *__restrict__ o_out,
                const int *__restrict__ q_start, const int *__restrict__ ctx_len, const int *__restrict__ state_slot,
                float *__restrict__ run_b, float *__restrict__ run_p, const float *__restrict__ run_in, int n, int nh, int d, int dv, int DV) {
    constexpr int D = WK_LANES * DPL, TOK = WK_TOK;
    constexpr int G = (2 * D + WK_COLS) / 4;                   // groups of four of a token: r, k, the workgroup's columns of v
    constexpr int PER = (TOK * G + WK_THREADS - 1) / WK_THREADS, PER_W = (TOK * D / 4 + WK_THREADS - 1) / WK_THREADS;
    __shared__ float4 lds[2][TOK][G], lds_w[2][TOK][D / 4];
    __shared__ float lds_b[2][TOK];
    const int r = MODE == 0 ? blockIdx.z : blockIdx.z / WK_RUNS, run = MODE == 0 ? 0 : blockIdx.z % WK_RUNS;
    const int h = blockIdx.y, col0 = blockIdx.x * WK_COLS;
    int t0 = q_start[r], t1 = q_start[r + 1];
    if (t1 <= t0 || (MODE != 0) != (t1 - t0 >= WK_LONG)) return;
    const bool fresh = ctx_len[r] - (t1 - t0) == 0;
    const int sub = threadIdx.x % WK_LANES, cg = threadIdx.x / WK_LANES, col = col0 + cg * WK_CPL;
    float *S = state + (size_t)state_slot[r] * slot_stride + (size_t)h * d * dv;
    size_t run_no = 0;
    if (MODE != 0) {
        const int len = (t1 - t0 + WK_RUNS - 1) / WK_RUNS, end = t1;
        t0 = min(end, t0 + run * len);
        t1 = min(end, t0 + len);
        run_no = ((size_t)wk_long_index(q_start, r) * WK_RUNS + run) * nh + h;
    }
    const float *from = MODE == 0 ? (fresh ? nullptr : S) : MODE == 2 ? run_in + run_no * d * dv : nullptr;
    float s[DPL][WK_CPL], pw[DPL];
#pragma unroll
    for (int e = 0; e < DPL; ++e) {
        const int i = sub * DPL + e;
        pw[e] = 1.f;
#pragma unroll
        for (int c = 0; c < WK_CPL; ++c) s[e][c] = (from && i < d && col + c < dv) ? from[(size_t)i * dv + col + c] : 0.f;
    }
    // a stage's numbers on their way: the loads stand under no branch (a place beyond the last token or channel is clamped), and
    // what they brought is converted when it goes to LDS.  Beyond the last token r, k and v are zero and w is 1, which leaves
    // the state.
    WkQuad<T> next[PER];
    float4 next_w[PER_W];
    float next_b = 0.f;
    auto fetch = [&](int base) {
#pragma unroll
        for (int p = 0; p < PER; ++p) {
            const int x = threadIdx.x + p * WK_THREADS, t = min(base + x / G, t1 - 1), g = x % G;
            const bool is_r = g < D / 4, is_v = g >= D / 2;
            const int at = is_r ? 4 * g : is_v ? col0 + 4 * g - 2 * D : 4 * g - D, limit = is_v ? dv : d;
            const T *from_row = rows + (size_t)t * row_stride + (is_r ? r_off + h * d : is_v ? v_off + h * dv : k_off + h * d);
            if (FOUR) next[p] = *(const WkQuad<T> *)(from_row + min(at, limit - 4));
            else
#pragma unroll
                for (int e = 0; e < 4; ++e) next[p].v[e] = from_row[min(at + e, limit - 1)];
        }
#pragma unroll
        for (int p = 0; p < PER_W; ++p) {
            const int x = threadIdx.x + p * WK_THREADS, t = min(base + x / (D / 4), t1 - 1);
            next_w[p] = *(const float4 *)(w_in + ((size_t)h * n + t) * D + x % (D / 4) * 4);
        }
        next_b = bonus[(size_t)h * n + min(base + (int)threadIdx.x, t1 - 1)];
    };
    auto put = [&](int base, int to) {
#pragma unroll
        for (int p = 0; p < PER; ++p) {
            const int x = threadIdx.x + p * WK_THREADS, tt = x / G, g = x % G;
            const bool is_r = g < D / 4, is_v = g >= D / 2;
            const int at = is_r ? 4 * g : is_v ? col0 + 4 * g - 2 * D : 4 * g - D, limit = base + tt < t1 ? (is_v ? dv : d) : 0;
            if (TOK * G % WK_THREADS && x >= TOK * G) break;
            lds[to][tt][g] = make_float4(at < limit ? to_f32(next[p].v[0]) : 0.f, at + 1 < limit ? to_f32(next[p].v[1]) : 0.f,
                                         at + 2 < limit ? to_f32(next[p].v[2]) : 0.f, at + 3 < limit ? to_f32(next[p].v[3]) : 0.f);
        }
#pragma unroll
        for (int p = 0; p < PER_W; ++p) {
            const int x = threadIdx.x + p * WK_THREADS, tt = x / (D / 4);
            if (TOK * D / 4 % WK_THREADS && x >= TOK * D / 4) break;
            lds_w[to][tt][x % (D / 4)] = base + tt < t1 ? next_w[p] : make_float4(1.f, 1.f, 1.f, 1.f);
        }
        if (threadIdx.x < TOK) lds_b[to][threadIdx.x] = next_b;
    };
    fetch(t0);
    put(t0, 0);
    __syncthreads();
    int buf = 0;
    for (int base = t0; base < t1; base += TOK, buf ^= 1) {
        const int nt = min(TOK, t1 - base);
        const bool more = base + TOK < t1;
        if (more) fetch(base + TOK);
        float acc[TOK][WK_CPL];
#pragma unroll
        for (int tt = 0; tt < TOK; ++tt) {
            const float4 *row = lds[buf][tt] + sub * (DPL / 4), *w_row = lds_w[buf][tt] + sub * (DPL / 4);
            const float4 v4 = lds[buf][tt][D / 2 + cg];
            const float v[4] = {v4.x, v4.y, v4.z, v4.w};
#pragma unroll
            for (int c = 0; c < WK_CPL; ++c) acc[tt][c] = 0.f;
#pragma unroll
            for (int e4 = 0; e4 < DPL / 4; ++e4) {
                const float4 k4 = row[D / 4 + e4], w4 = w_row[e4];
                const float4 r4 = MODE == 1 ? make_float4(0.f, 0.f, 0.f, 0.f) : row[e4];
                const float kk[4] = {k4.x, k4.y, k4.z, k4.w}, ww[4] = {w4.x, w4.y, w4.z, w4.w}, rr[4] = {r4.x, r4.y, r4.z, r4.w};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    if (MODE == 1) pw[4 * e4 + e] *= ww[e];
#pragma unroll
                    for (int c = 0; c < WK_CPL; ++c) {
                        float &x = s[4 * e4 + e][c];
                        if (MODE != 1) acc[tt][c] = fmaf(rr[e], x, acc[tt][c]);
                        x = fmaf(ww[e], x, kk[e] * v[c]);
                    }
                }
            }
        }
        if (MODE != 1) {
            // lane tt of a column group's sixteen keeps token tt's four sums, and the stage's outputs leave in one store
            float mine[WK_CPL] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int tt = 0; tt < TOK; ++tt)
#pragma unroll
                for (int c = 0; c < WK_CPL; ++c) {
                    const float a = sum_over_16(acc[tt][c]);
                    if (sub == tt) mine[c] = a;
                }
            if (sub < nt) {
                const float b = lds_b[buf][sub];
                const float4 v4 = lds[buf][sub][D / 2 + cg];
                *(float4 *)(o_out + ((size_t)h * n + base + sub) * DV + col) =
                    make_float4(fmaf(b, v4.x, mine[0]), fmaf(b, v4.y, mine[1]), fmaf(b, v4.z, mine[2]), fmaf(b, v4.w, mine[3]));
            }
        }
        if (more) put(base + TOK, buf ^ 1);
        __syncthreads();
    }
    if (MODE == 2 && run != WK_RUNS - 1) return;
    float *to = MODE == 1 ? run_b + run_no * d * dv : S;
#pragma unroll
    for (int e = 0; e < DPL; ++e) {
        const int i = sub * DPL + e;
        if (MODE == 1 && i < d && blockIdx.x == 0 && cg == 0) run_p[run_no * d + i] = pw[e];
#pragma unroll
        for (int c = 0; c < WK_CPL; ++c)
            if (i < d && col + c < dv) to[(size_t)i * dv + col + c] = s[e][c];
    }
}

// The state that every run of a long request starts from.
__global__ void wkv_chain_kernel(const float *__restrict__ state, size_t slot_stride, const float *__restrict__ run_b,
                                 const float *__restrict__ run_p, float *__restrict__ run_in, const int *__restrict__ q_start,
                                 const int *__restrict__ ctx_len, const int *__restrict__ state_slot, int nh, int d, int dv) {
    const int r = blockIdx.z, h = blockIdx.y, x = blockIdx.x * blockDim.x + threadIdx.x;
    const int tokens = q_start[r + 1] - q_start[r];
    if (tokens < WK_LONG || x >= d * dv) return;
    const size_t first = (size_t)wk_long_index(q_start, r) * WK_RUNS * nh + h;
    float b[WK_RUNS], p[WK_RUNS];
#pragma unroll
    for (int run = 0; run < WK_RUNS; ++run) {
        b[run] = run_b[(first + (size_t)run * nh) * d * dv + x];
        p[run] = run_p[(first + (size_t)run * nh) * d + x / dv];
    }
    float s = ctx_len[r] - tokens == 0 ? 0.f : state[(size_t)state_slot[r] * slot_stride + (size_t)h * d * dv + x];
#pragma unroll
    for (int run = 0; run < WK_RUNS; ++run) {
        run_in[(first + (size_t)run * nh) * d * dv + x] = s;
        s = fmaf(p[run], s, b[run]);
    }
}

// ---------------------------------------------------------------- out
// One wave per (token, head), four to a workgroup: o / rms(o) * weight * silu(gate).
template <class TG, class T>
__global__ void __launch_bounds__(256)
wkv_out_kernel(const float *__restrict__ o, int DV, const TG *__restrict__ rows, int row_stride, int g_off, const float *__restrict__ weight,
               T *__restrict__ out, int n, int nh, int dv, float eps) {
    const int t = blockIdx.x, h = blockIdx.y * 4 + threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
    if (h >= nh) return;
    const float *oh = o + ((size_t)h * n + t) * DV;
    float x[4], z[4], ss = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int j = lane + WAVE * i;
        x[i] = j < dv ? oh[j] : 0.f;
        z[i] = j < dv ? to_f32(rows[(size_t)t * row_stride + g_off + h * dv + j]) : 0.f;
        ss += x[i] * x[i];
    }
    const float f = 1.0f / sqrtf(wave_sum_in_place(ss) / (float)dv + eps);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int j = lane + WAVE * i, c = h * dv + j;
        if (j < dv) out[(size_t)t * nh * dv + c] = from_f32<T>(x[i] * f * weight[c] * (z[i] / (1.0f + expf(-z[i]))));
    }
}

// ---------------------------------------------------------------- a step of single tokens
// A workgroup per (request, head).  Wave w walks the key channels w, w + 4, ..: a lane holds the columns lane, lane + 64, .. of a
// row, so a row of the state is read and written in whole lines.  The first rows are on their way while the decay is made.
template <int D, class TG, class T>
__global__ void __launch_bounds__(WK_THREADS)
wkv_single_kernel(const TG *__restrict__ rows, int row_stride, int r_off, int k_off, int v_off, int g_off, const float *__restrict__ low,
                  int ld_low, const float *__restrict__ w2t, const float *__restrict__ w0, const float *__restrict__ u,
                  const float *__restrict__ weight, float *__restrict__ state, size_t slot_stride, T *__restrict__ out,
                  const int *__restrict__ ctx_len, const int *__restrict__ q_start, const int *__restrict__ state_slot, int nh, int d, int dv,
                  int rank, float eps) {
    constexpr int WAVES = WK_THREADS / WAVE, RW = D / WAVES, NV = D / 64, CH = RW * NV > 64 ? 64 / NV : RW;   // rows of a wave, columns of a lane, rows at a time
    constexpr int PARTS = WK_THREADS / D;                      // threads that share a channel's sum over the rank
    __shared__ float th[WK_MAX_RANK], rs[D], ks[D], ws[D], zs[PARTS][D], red[WAVES][D], scratch[16];
    const int req = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & (WAVE - 1), wave = tid / WAVE;
    const int t = q_start[req];
    const bool fresh = ctx_len[req] == 1;
    float *S = state + (size_t)state_slot[req] * slot_stride + (size_t)h * d * dv;
    const TG *row = rows + (size_t)t * row_stride;
    float s[CH][NV];
    auto load = [&](int first) {
#pragma unroll
        for (int a = 0; a < CH; ++a)
#pragma unroll
            for (int e = 0; e < NV; ++e) {
                const int i = (first + a) * WAVES + wave, j = lane + 64 * e;
                s[a][e] = (!fresh && i < d && j < dv) ? S[(size_t)i * dv + j] : 0.f;
            }
    };
    load(0);
    float v[NV];
#pragma unroll
    for (int e = 0; e < NV; ++e) v[e] = lane + 64 * e < dv ? to_f32(row[v_off + h * dv + lane + 64 * e]) : 0.f;
    for (int x = tid; x < rank; x += WK_THREADS) th[x] = tanhf(low[(size_t)t * ld_low + x]);
    float own = 0.f;
    if (tid < D) {
        const bool live = tid < d;
        const float rr = live ? to_f32(row[r_off + h * d + tid]) : 0.f, kk = live ? to_f32(row[k_off + h * d + tid]) : 0.f;
        rs[tid] = rr;
        ks[tid] = kk;
        own = live ? rr * u[h * d + tid] * kk : 0.f;
    }
    const float bonus = block_sum(own, scratch);               // (its barriers make th, rs and ks visible)
    {
        const int c = tid % D, p = tid / D, per = (rank + PARTS - 1) / PARTS, j1 = min(rank, (p + 1) * per);
        float z = 0.f;
        if (c < d) {
#pragma unroll 8
            for (int j = p * per; j < j1; ++j) z = fmaf(w2t[(size_t)j * nh * d + h * d + c], th[j], z);
        }
        zs[p][c] = z;
    }
    __syncthreads();
    if (tid < D) {
        float z = tid < d ? w0[h * d + tid] : 0.f;
#pragma unroll
        for (int p = 0; p < PARTS; ++p) z += zs[p][tid];
        ws[tid] = expf(-expf(z));
    }
    __syncthreads();
    float acc[NV];
#pragma unroll
    for (int e = 0; e < NV; ++e) acc[e] = 0.f;
#pragma unroll
    for (int first = 0; first < RW; first += CH) {
        if (first > 0) load(first);
#pragma unroll
        for (int a = 0; a < CH; ++a) {
            const int i = (first + a) * WAVES + wave;
            const float rr = rs[i], kk = ks[i], ww = ws[i];
#pragma unroll
            for (int e = 0; e < NV; ++e) {
                acc[e] = fmaf(rr, s[a][e], acc[e]);
                if (i < d && lane + 64 * e < dv) S[(size_t)i * dv + lane + 64 * e] = fmaf(ww, s[a][e], kk * v[e]);
            }
        }
    }
#pragma unroll
    for (int e = 0; e < NV; ++e) red[wave][lane + 64 * e] = acc[e];
    __syncthreads();
    float o = 0.f;
    if (tid < dv) {
#pragma unroll
        for (int w = 0; w < WAVES; ++w) o += red[w][tid];
        o = fmaf(bonus, to_f32(row[v_off + h * dv + tid]), o);
    }
    const float f = 1.0f / sqrtf(block_sum(tid < dv ? o * o : 0.f, scratch) / (float)dv + eps);
    if (tid < dv) {
        const int c = h * dv + tid;
        const float z = to_f32(row[g_off + c]);
        out[(size_t)t * nh * dv + c] = from_f32<T>(o * f * weight[c] * (z / (1.0f + expf(-z))));
    }
}

// The floats of the scratch arrays for a step of n tokens whose `n_long` requests feed at least WK_LONG of them.
LCU_API long long lcu_wkv_prep_floats(int n, int heads, int d) { return (long long)n * heads * (wk_pad_keys(d) + 1); }
LCU_API long long lcu_wkv_out_floats(int n, int heads, int dv) { return (long long)n * heads * wk_pad_cols(dv); }
LCU_API long long lcu_wkv_run_floats(int n_long, int heads, int d, int dv) {
    return (long long)n_long * WK_RUNS * heads * d * (2ll * dv + 1);
}
LCU_API int lcu_wkv_long(void) { return WK_LONG; }

static bool wkv_sizes_ok(int heads, int d, int dv, int rank, long long slot_stride) {
    return heads > 0 && heads <= 65535 && d > 0 && d <= 256 && dv > 0 && dv <= wk_pad_keys(d) && rank > 0 && rank <= WK_MAX_RANK &&
           slot_stride >= (long long)heads * d * dv;
}

// rows: [n, row_stride] of rows_type; r, k [heads * d] and v, g [heads * dv] at their columns.  low: [n, ld_low] 32-bit.
// w2t: [rank, heads * d], w0, u: [heads * d], weight: [heads * dv], all 32-bit.  prep, o, runs: scratch (sizes above; runs may be
// null where no request feeds WK_LONG tokens).  state: slot s at state + s * slot_stride, [heads, d, dv].  out: [n, heads * dv].
LCU_API int lcu_wkv(const void *rows, int rows_type, int row_stride, int r_off, int k_off, int v_off, int g_off, const float *low, int ld_low,
                    const float *w2t, const float *w0, const float *u, const float *weight, float *prep, float *o, float *runs, int n_long,
                    float *state, long long slot_stride, void *out, int out_type, const int *q_start, const int *ctx_len,
                    const int *state_slot, int n, int n_req, int heads, int d, int dv, int rank, float eps, hipStream_t stream) {
    if (n <= 0 || n_req <= 0) return LCU_OK;
    if (!wkv_sizes_ok(heads, d, dv, rank, slot_stride) || !prep || !o || n_long < 0 || (n_long > 0 && !runs) || n_req * WK_RUNS > 65535)
        return LCU_BAD_ARGUMENT;
    const int D = wk_pad_keys(d), DV = wk_pad_cols(dv);
    const dim3 pg((n + WK_PREP_TOK - 1) / WK_PREP_TOK, (heads + 256 / D - 1) / (256 / D));
    const size_t plds = (size_t)rank * WK_PREP_TOK * sizeof(float);
    float *w_buf = prep, *bonus = prep + (size_t)n * heads * D;
    const size_t one = (size_t)n_long * WK_RUNS * heads * d;
    float *run_b = runs, *run_in = runs ? runs + one * dv : nullptr, *run_p = runs ? run_in + one * dv : nullptr;
    const bool four = d % 4 == 0 && dv % 4 == 0 && row_stride % 4 == 0 && r_off % 4 == 0 && k_off % 4 == 0 && v_off % 4 == 0 && (uintptr_t)rows % 16 == 0;
#define SCAN(T, DPL, MODE, Z)                                                                                                                     \
    do {                                                                                                                                        \
        if (four) SCAN_AS(T, DPL, MODE, true, Z);                                                                                               \
        else SCAN_AS(T, DPL, MODE, false, Z);                                                                                                   \
    } while (0)
#define SCAN_AS(T, DPL, MODE, FOUR, Z)                                                                                                            \
    wkv_scan_kernel<T, DPL, MODE, FOUR><<<dim3(DV / WK_COLS, heads, Z), dim3(WK_THREADS), 0, stream>>>((const T *)rows, row_stride, r_off, k_off, \
        v_off, w_buf, bonus, state, (size_t)slot_stride, o, q_start, ctx_len, state_slot, run_b, run_p, run_in, n, heads, d, dv, DV)
#define MODES(T, DPL)                                                                                                           \
    do {                                                                                                                        \
        if (n_long < n_req) SCAN(T, DPL, 0, n_req);                                                                             \
        if (n_long > 0) {                                                                                                       \
            SCAN(T, DPL, 1, n_req * WK_RUNS);                                                                                   \
            wkv_chain_kernel<<<dim3((d * dv + 255) / 256, heads, n_req), dim3(256), 0, stream>>>(state, (size_t)slot_stride,   \
                run_b, run_p, run_in, q_start, ctx_len, state_slot, heads, d, dv);                                              \
            SCAN(T, DPL, 2, n_req * WK_RUNS);                                                                                   \
        }                                                                                                                       \
    } while (0)
#define ALL(T)                                                                                                                                  \
    do {                                                                                                                                        \
        wkv_prep_kernel<T><<<pg, dim3(256), plds, stream>>>((const T *)rows, row_stride, r_off, k_off, low, ld_low, w2t, w0, u, w_buf, bonus, n, \
                                                            heads, d, rank, D);                                                                 \
        if (D == 64) MODES(T, 4);                                                                                                               \
        else if (D == 128) MODES(T, 8);                                                                                                         \
        else MODES(T, 16);                                                                                                                      \
    } while (0)
    if (rows_type == LCU_F32) ALL(float);
    else if (rows_type == LCU_BF16) ALL(bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef ALL
#undef MODES
#undef SCAN
#undef SCAN_AS
    LCU_LAUNCH_CHECK();
#define OUT(TG, T) wkv_out_kernel<TG, T><<<dim3(n, (heads + 3) / 4), dim3(256), 0, stream>>>(o, DV, (const TG *)rows, row_stride, g_off, weight, (T *)out, n, heads, dv, eps)
    if (rows_type == LCU_F32 && out_type == LCU_F32) OUT(float, float);
    else if (rows_type == LCU_F32 && out_type == LCU_BF16) OUT(float, bf16_t);
    else if (rows_type == LCU_BF16 && out_type == LCU_BF16) OUT(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef OUT
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// The same for a step in which every request feeds one token (n == n_req), in one kernel without scratch.
LCU_API int lcu_wkv_single(const void *rows, int rows_type, int row_stride, int r_off, int k_off, int v_off, int g_off, const float *low,
                           int ld_low, const float *w2t, const float *w0, const float *u, const float *weight, float *state,
                           long long slot_stride, void *out, int out_type, const int *q_start, const int *ctx_len, const int *state_slot,
                           int n_req, int heads, int d, int dv, int rank, float eps, hipStream_t stream) {
    if (n_req <= 0) return LCU_OK;
    if (!wkv_sizes_ok(heads, d, dv, rank, slot_stride)) return LCU_BAD_ARGUMENT;
    const int D = wk_pad_keys(d);
#define GO(D_, TG, T) wkv_single_kernel<D_, TG, T><<<dim3(n_req, heads), dim3(WK_THREADS), 0, stream>>>((const TG *)rows, row_stride, r_off, k_off, v_off, g_off, low, ld_low, w2t, w0, u, weight, state, (size_t)slot_stride, (T *)out, ctx_len, q_start, state_slot, heads, d, dv, rank, eps)
#define SIZES(TG, T)                  \
    do {                              \
        if (D == 64) GO(64, TG, T);   \
        else if (D == 128) GO(128, TG, T); \
        else GO(256, TG, T);          \
    } while (0)
    if (rows_type == LCU_F32 && out_type == LCU_F32) SIZES(float, float);
    else if (rows_type == LCU_F32 && out_type == LCU_BF16) SIZES(float, bf16_t);
    else if (rows_type == LCU_BF16 && out_type == LCU_BF16) SIZES(bf16_t, bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef SIZES
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}
