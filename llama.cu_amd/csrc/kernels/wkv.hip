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
// Any other step: prep (parallel over tokens and heads; rows r, k, w, b, v of a head one after the other, so that the
// scan's workgroups each stream a run of memory), scan, out.  The scan: column j of S depends on column j alone; a
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
constexpr int WK_PREP_TOK = 8;                             // tokens of a prep workgroup

// ---------------------------------------------------------------- the mix with the token before
// h: [n, d] 32-bit; mu: [sets, d]; out: [sets, n, d].  The previous token's h of a request's first token of the step lies at
// prev + slot * slot_stride (d floats); that token's workgroup also leaves the step's last h there (each thread reads an
// element before it writes it, so nothing races).
template <class T>
__global__ void token_shift_kernel(const float *__restrict__ h, const float *__restrict__ mu, int sets, float *__restrict__ prev,
                                   size_t slot_stride, const int *__restrict__ req_of_token, const int *__restrict__ q_start,
                                   const int *__restrict__ ctx_len, const int *__restrict__ state_slot, T *__restrict__ out, int n, int d) {
    const int t = blockIdx.x, r = req_of_token[t], t0 = q_start[r], t1 = q_start[r + 1];
    const bool first = t == t0, fresh = ctx_len[r] - (t1 - t0) == 0;
    float *ps = prev + (size_t)state_slot[r] * slot_stride;
    const float *row = h + (size_t)t * d, *last = h + (size_t)(t1 - 1) * d;
    for (int c = threadIdx.x; c < d; c += blockDim.x) {
        const float x = row[c];
        float before;
        if (first) {
            before = fresh ? 0.f : ps[c];
            ps[c] = last[c];
        } else {
            before = row[c - d];
        }
        const float diff = before - x;
        for (int s = 0; s < sets; ++s) out[((size_t)s * n + t) * d + c] = from_f32<T>(fmaf(diff, mu[(size_t)s * d + c], x));
    }
}

LCU_API int lcu_token_shift(const float *h, const float *mu, int sets, float *prev, long long slot_stride, const int *req_of_token,
                            const int *q_start, const int *ctx_len, const int *state_slot, void *out, int out_type, int n, int d,
                            hipStream_t stream) {
    if (n <= 0) return LCU_OK;
    if (d <= 0 || sets <= 0 || slot_stride < d || !h || !mu || !prev || !out) return LCU_BAD_ARGUMENT;
    int threads = (d + 63) / 64 * 64;
    if (threads > 512) threads = 512;
#define GO(T) token_shift_kernel<T><<<dim3(n), dim3(threads), 0, stream>>>(h, mu, sets, prev, (size_t)slot_stride, req_of_token, q_start, ctx_len, state_slot, (T *)out, n, d)
    if (out_type == LCU_F32) GO(float);
    else if (out_type == LCU_BF16) GO(bf16_t);
    else return LCU_BAD_ARGUMENT;
#undef GO
    LCU_LAUNCH_CHECK();
    return LCU_OK;
}

// ---------------------------------------------------------------- prep
__host__ __device__ constexpr int wk_pad_keys(int d) { return d <= 64 ? 64 : d <= 128 ? 128 : 256; }      // key channels in a row: r, k and w each
__host__ __device__ constexpr int wk_pad_cols(int dv) { return (dv + WK_COLS - 1) / WK_COLS * WK_COLS; }
// a row: r, k, w (D each, zeros behind the true channels), b and three zeros, v (padded to whole workgroups' columns)
__host__ __device__ constexpr int wk_row(int D, int DV) { return 3 * D + 4 + DV; }

// rows: [n, row_stride] with r, k (heads * d) and v (heads * dv) at their columns; low: [n, ld_low] 32-bit; w2t: [rank, heads * d].
template <class T>
__global__ void wkv_prep_kernel(const T *__restrict__ rows, int row_stride, int r_off, int k_off, int v_off, const float *__restrict__ low,
                                int ld_low, const float *__restrict__ w2t, const float *__restrict__ w0, const float *__restrict__ u,
                                float *__restrict__ prep, int n, int heads, int d, int dv, int rank, int D, int DV) {
    __shared__ float th[WK_PREP_TOK * WK_MAX_RANK];
    __shared__ float part[WK_PREP_TOK][4];
    const int t0 = blockIdx.x * WK_PREP_TOK, h = blockIdx.y, nt = min(WK_PREP_TOK, n - t0);
    for (int x = threadIdx.x; x < nt * rank; x += blockDim.x) th[x] = tanhf(low[(size_t)(t0 + x / rank) * ld_low + x % rank]);
    __syncthreads();
    const int i = threadIdx.x, c = h * d + i;                  // blockDim.x == D: a thread per key channel
    const bool live = i < d;
    float z[WK_PREP_TOK];
#pragma unroll
    for (int b = 0; b < WK_PREP_TOK; ++b) z[b] = live ? w0[c] : 0.f;
    if (live) {
#pragma unroll 4
        for (int j = 0; j < rank; ++j) {
            const float w = w2t[(size_t)j * heads * d + c];
#pragma unroll
            for (int b = 0; b < WK_PREP_TOK; ++b) z[b] = fmaf(w, b < nt ? th[b * rank + j] : 0.f, z[b]);
        }
    }
    const int R = wk_row(D, DV);
    const float uu = live ? u[c] : 0.f;
#pragma unroll
    for (int b = 0; b < WK_PREP_TOK; ++b) {
        if (b >= nt) break;
        const T *row = rows + (size_t)(t0 + b) * row_stride;
        float *o = prep + ((size_t)h * n + t0 + b) * R;
        const float rr = live ? to_f32(row[r_off + c]) : 0.f, kk = live ? to_f32(row[k_off + c]) : 0.f;
        o[i] = rr;
        o[D + i] = kk;
        o[2 * D + i] = live ? expf(-expf(z[b])) : 0.f;
        for (int j = i; j < DV; j += D) o[3 * D + 4 + j] = j < dv ? to_f32(row[v_off + h * dv + j]) : 0.f;
        const float s = wave_sum(rr * uu * kk);
        if ((i & (WAVE - 1)) == 0) part[b][i / WAVE] = s;
    }
    __syncthreads();
    if (i < 4 * nt) {
        const int b = i / 4;
        float s = 0.f;
        if (i % 4 == 0)
            for (int w = 0; w < D / WAVE; ++w) s += part[b][w];
        prep[((size_t)h * n + t0 + b) * R + 3 * D + i % 4] = s;
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
template <int DPL, int MODE>
__global__ void __launch_bounds__(WK_THREADS)
wkv_scan_kernel(const float *__restrict__ prep, float *__restrict__ state, size_t slot_stride, float *__restrict__ o_out,
                const int *__restrict__ q_start, const int *__restrict__ ctx_len, const int *__restrict__ state_slot,
                float *__restrict__ run_b, float *__restrict__ run_p, const float *__restrict__ run_in, int n, int nh, int d, int dv, int DV) {
    constexpr int D = WK_LANES * DPL, TOK = WK_TOK;
    constexpr int HEAD = 3 * D + 4;                            // floats of a token's row in front of v
    constexpr int V4 = TOK * HEAD / 4;                         // float4s of a stage before its values
    constexpr int STAGE4 = V4 + TOK * WK_COLS / 4;
    constexpr int PER = (STAGE4 + WK_THREADS - 1) / WK_THREADS;
    __shared__ float4 lds[2][STAGE4];
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
    const int R4 = (HEAD + DV) / 4;
    const float4 *src = (const float4 *)prep + (size_t)h * n * R4;
    // element x of a stage: the rows of its tokens up to their values, then the workgroup's columns of the values.  Beyond the
    // last token everything is zero and w is 1, which leaves the state.
    auto fetch = [&](int base, int x) -> float4 {
        const bool is_v = x >= V4;
        const int tt = is_v ? (x - V4) / (WK_COLS / 4) : x / (HEAD / 4), at = is_v ? (x - V4) % (WK_COLS / 4) : x % (HEAD / 4);
        const int t = base + tt;
        if (x >= STAGE4 || t >= t1) {
            const float fill = !is_v && at >= D / 2 && at < 3 * D / 4 ? 1.f : 0.f;
            return make_float4(fill, fill, fill, fill);
        }
        return src[(size_t)t * R4 + (is_v ? HEAD / 4 + col0 / 4 + at : at)];
    };
    float4 next[PER];
#pragma unroll
    for (int k = 0; k < PER; ++k) next[k] = fetch(t0, threadIdx.x + k * WK_THREADS);
#pragma unroll
    for (int k = 0; k < PER; ++k)
        if (threadIdx.x + k * WK_THREADS < STAGE4) lds[0][threadIdx.x + k * WK_THREADS] = next[k];
    __syncthreads();
    int buf = 0;
    for (int base = t0; base < t1; base += TOK, buf ^= 1) {
        const int nt = min(TOK, t1 - base);
        const bool more = base + TOK < t1;
        if (more) {
#pragma unroll
            for (int k = 0; k < PER; ++k) next[k] = fetch(base + TOK, threadIdx.x + k * WK_THREADS);
        }
        const float4 *cur = lds[buf];
        float acc[TOK][WK_CPL];
#pragma unroll
        for (int tt = 0; tt < TOK; ++tt) {
            const float4 *row = cur + tt * (HEAD / 4) + sub * (DPL / 4);
            const float4 v4 = cur[V4 + tt * (WK_COLS / 4) + cg];
            const float v[4] = {v4.x, v4.y, v4.z, v4.w};
#pragma unroll
            for (int c = 0; c < WK_CPL; ++c) acc[tt][c] = 0.f;
#pragma unroll
            for (int e4 = 0; e4 < DPL / 4; ++e4) {
                const float4 k4 = row[D / 4 + e4], w4 = row[D / 2 + e4];
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
                const float b = cur[sub * (HEAD / 4) + 3 * D / 4].x;
                const float4 v4 = cur[V4 + sub * (WK_COLS / 4) + cg];
                *(float4 *)(o_out + ((size_t)h * n + base + sub) * DV + col) =
                    make_float4(fmaf(b, v4.x, mine[0]), fmaf(b, v4.y, mine[1]), fmaf(b, v4.z, mine[2]), fmaf(b, v4.w, mine[3]));
            }
        }
        if (more) {
#pragma unroll
            for (int k = 0; k < PER; ++k)
                if (threadIdx.x + k * WK_THREADS < STAGE4) lds[buf ^ 1][threadIdx.x + k * WK_THREADS] = next[k];
        }
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
// One wave per (token, head): o / rms(o) * weight * silu(gate).
template <class TG, class T>
__global__ void __launch_bounds__(WAVE)
wkv_out_kernel(const float *__restrict__ o, int DV, const TG *__restrict__ rows, int row_stride, int g_off, const float *__restrict__ weight,
               T *__restrict__ out, int n, int nh, int dv, float eps) {
    const int t = blockIdx.x, h = blockIdx.y;
    const float *oh = o + ((size_t)h * n + t) * DV;
    float x[4], ss = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int j = threadIdx.x + WAVE * i;
        x[i] = j < dv ? oh[j] : 0.f;
        ss += x[i] * x[i];
    }
    const float f = 1.0f / sqrtf(wave_sum(ss) / (float)dv + eps);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int j = threadIdx.x + WAVE * i, c = h * dv + j;
        if (j >= dv) break;
        const float z = to_f32(rows[(size_t)t * row_stride + g_off + c]);
        out[(size_t)t * nh * dv + c] = from_f32<T>(x[i] * f * weight[c] * (z / (1.0f + expf(-z))));
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
LCU_API long long lcu_wkv_prep_floats(int n, int heads, int d, int dv) {
    return (long long)n * heads * wk_row(wk_pad_keys(d), wk_pad_cols(dv));
}
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
    const dim3 pg((n + WK_PREP_TOK - 1) / WK_PREP_TOK, heads);
    if (rows_type == LCU_F32)
        wkv_prep_kernel<float><<<pg, dim3(D), 0, stream>>>((const float *)rows, row_stride, r_off, k_off, v_off, low, ld_low, w2t, w0, u, prep, n, heads, d, dv, rank, D, DV);
    else if (rows_type == LCU_BF16)
        wkv_prep_kernel<bf16_t><<<pg, dim3(D), 0, stream>>>((const bf16_t *)rows, row_stride, r_off, k_off, v_off, low, ld_low, w2t, w0, u, prep, n, heads, d, dv, rank, D, DV);
    else
        return LCU_BAD_ARGUMENT;
    LCU_LAUNCH_CHECK();
    const size_t one = (size_t)n_long * WK_RUNS * heads * d;
    float *run_b = runs, *run_in = runs ? runs + one * dv : nullptr, *run_p = runs ? run_in + one * dv : nullptr;
#define SCAN(DPL, MODE, Z) wkv_scan_kernel<DPL, MODE><<<dim3(DV / WK_COLS, heads, Z), dim3(WK_THREADS), 0, stream>>>(prep, state, (size_t)slot_stride, o, q_start, ctx_len, state_slot, run_b, run_p, run_in, n, heads, d, dv, DV)
#define MODES(DPL)                                                                                                              \
    do {                                                                                                                        \
        if (n_long < n_req) SCAN(DPL, 0, n_req);                                                                                \
        if (n_long > 0) {                                                                                                       \
            SCAN(DPL, 1, n_req * WK_RUNS);                                                                                      \
            wkv_chain_kernel<<<dim3((d * dv + 255) / 256, heads, n_req), dim3(256), 0, stream>>>(state, (size_t)slot_stride,   \
                run_b, run_p, run_in, q_start, ctx_len, state_slot, heads, d, dv);                                              \
            SCAN(DPL, 2, n_req * WK_RUNS);                                                                                      \
        }                                                                                                                       \
    } while (0)
    if (D == 64) MODES(4);
    else if (D == 128) MODES(8);
    else MODES(16);
#undef MODES
#undef SCAN
    LCU_LAUNCH_CHECK();
#define OUT(TG, T) wkv_out_kernel<TG, T><<<dim3(n, heads), dim3(WAVE), 0, stream>>>(o, DV, (const TG *)rows, row_stride, g_off, weight, (T *)out, n, heads, dv, eps)
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
