// Token mixers that carry a matrix per head from token to token, and the small steps in front of them:
//   - short causal convolution over time per channel (optional bias, optional silu), its last inputs kept per sequence;
//   - token shift: every token's row mixed with its predecessor's by per-channel weights, the last row kept per sequence;
//   - recurrences over a (key size x value size) memory per head:
//       mlstm   exponential input gate and sigmoid forget gate stabilised by a running maximum, normaliser vector;
//       delta   per-head decay, then a rank-one correction of the memory towards the new value along the key;
//       rwkv    per-key-channel decay, the current token read with a bonus before it is written;
//       decay   one constant decay per head, the token written before it is read (linear attention with a fixed decay; queries and keys may
//               be rotated by position as they are staged: retention); steps of one token per sequence have a form of their own that
//               walks the memory once and ends in the norm and gate of the read-out;
//       gla     a decay per key channel and token, the token written before it is read (gated linear attention).
// Long portions of mlstm, decay and gla are cut into chunks that run side by side, in three phases (see decay).
// One kernel per recurrence serves prompts, portions of prompts and single decoded tokens: a workgroup takes one head of
// one sequence and a block of value columns, a thread keeps KR rows of one column in registers, P neighbouring lanes
// share a column and add their partial read-outs by lane exchange.  The tokens' keys, queries and values are staged
// through LDS TB tokens at a time (converted to float32, unit-normed where the design asks for it), so the sequential
// loop touches no global memory but its output.  Memory, normaliser, maximum, gates and decays are float32.
// A batch is ragged (see seq_mix.hip): qo_indptr / pos0 / state_slot; a sequence at position 0 takes zeros for its state.
#include "fmt_dev.h"

namespace NVX_NS {

// ---- short convolution (+ bias, + silu) ------------------------------------------------------------------------------------
// out[t][c] = act(bias[c] + sum_j w[j][c] * in[t - (taps_n - 1) + j][c]) over the tokens of t's own sequence (bias may be null; act 0:
// none, 1: silu); inputs before this step come from state[slot] (taps_n - 1 rows, oldest first), inputs before the sequence's
// start are zero.
template <typename A>
__global__ __launch_bounds__(256) void short_conv_kernel(const A* __restrict__ x, int64_t x_stride, const float* __restrict__ w,
                                                        const float* __restrict__ bias, int act, int taps_n, const float* __restrict__ state, const int32_t* __restrict__ tok_seq,
                                                             const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                             const int32_t* __restrict__ state_slot, A* __restrict__ out, int channels) {
    const int64_t t = blockIdx.y;
    const int b = tok_seq ? tok_seq[t] : (int)t;
    const SeqSpan s = seq_span(b, qo_indptr, pos0, state_slot);
    const int64_t j = t - s.q0;
    const int hist_n = taps_n - 1;
    const bool has_state = s.pos0 > 0 && s.slot >= 0;
    for (int c = blockIdx.x * 256 + threadIdx.x; c < channels; c += gridDim.x * 256) {
        float acc = bias ? bias[c] : 0.f;
        for (int i = 0; i < taps_n; ++i) {
            const int64_t src = j - (hist_n - i);
            float v = 0.f;
            if (src >= 0) v = ld_f(x, (s.q0 + src) * x_stride + c);
            else if (has_state) v = state[((int64_t)s.slot * hist_n + (hist_n + src)) * channels + c];
            acc += w[(int64_t)i * channels + c] * v;
        }
        st_f(out, t * (int64_t)channels + c, act == 1 ? acc * sigmoid_f(acc) : acc);
    }
}

// state[slot] <- the sequence's last hist_n inputs (older rows of the state move up where the step brought fewer).
template <typename A>
__global__ __launch_bounds__(256) void tail_rows_kernel(const A* __restrict__ x, int64_t x_stride, int hist_n, float* __restrict__ state,
                                                       const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                       const int32_t* __restrict__ state_slot, int channels) {
    const SeqSpan s = seq_span(blockIdx.y, qo_indptr, pos0, state_slot);
    if (s.slot < 0 || s.n <= 0) return;
    const bool has_state = s.pos0 > 0;
    for (int c = blockIdx.x * 256 + threadIdx.x; c < channels; c += gridDim.x * 256) {
        float* st = state + (int64_t)s.slot * hist_n * channels + c;
        for (int r = 0; r < hist_n; ++r) {        // ascending: row r takes old row r + n, which is not yet overwritten
            const int64_t src = s.n - hist_n + r;
            float v;
            if (src >= 0) v = ld_f(x, (s.q0 + src) * x_stride + c);
            else v = has_state ? st[(int64_t)(r + s.n) * channels] : 0.f;
            st[(int64_t)r * channels] = v;
        }
    }
}

// out[m][t][c] = h[t][c] + (h[t-1][c] - h[t][c]) * mu[m][c]; the predecessor of a step's first token is state[slot].
template <typename A>
__global__ __launch_bounds__(256) void token_shift_mix_kernel(const A* __restrict__ h, int64_t h_stride, const float* __restrict__ mu,
                                                             int n_mix, const float* __restrict__ state, const int32_t* __restrict__ tok_seq,
                                                             const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                             const int32_t* __restrict__ state_slot, A* __restrict__ out, int64_t n_tok,
                                                             int width) {
    const int64_t t = blockIdx.y;
    const int b = tok_seq ? tok_seq[t] : (int)t;
    const SeqSpan s = seq_span(b, qo_indptr, pos0, state_slot);
    for (int c = blockIdx.x * 256 + threadIdx.x; c < width; c += gridDim.x * 256) {
        const float cur = ld_f(h, t * h_stride + c);
        float prev = 0.f;
        if (t > s.q0) prev = ld_f(h, (t - 1) * h_stride + c);
        else if (s.pos0 > 0 && s.slot >= 0) prev = state[(int64_t)s.slot * width + c];
        for (int m = 0; m < n_mix; ++m)
            st_f(out, ((int64_t)m * n_tok + t) * width + c, cur + (prev - cur) * mu[(int64_t)m * width + c]);
    }
}

// ---- matrix-memory recurrences ---------------------------------------------------------------------------------------------
constexpr int KR = 32;        // rows of a column that one thread keeps
constexpr int KS = KR + 4;    // LDS stride of such a group of rows (keeps 16-byte alignment, spreads the groups over banks)
constexpr int TB = 8;         // tokens staged at a time

__device__ __forceinline__ int lds_row(int d) { return (d / KR) * KS + (d % KR); }
__device__ __forceinline__ float lanes_sum(float v, int p_lanes) {
    for (int m = 1; m < p_lanes; m <<= 1) v += __shfl_xor(v, m, 64);
    return v;
}

struct ScanThread { int col, p, e, r0; bool active; };
__device__ __forceinline__ ScanThread scan_thread(int p_lanes, int vdim) {
    ScanThread th;
    const int cb = blockDim.x / p_lanes;
    th.col = threadIdx.x / p_lanes;
    th.p = threadIdx.x % p_lanes;
    th.e = blockIdx.x * cb + th.col;
    th.r0 = th.p * KR;
    th.active = th.e < vdim;
    return th;
}

// stage `nt` tokens' rows of `dim` elements starting at column `off` of x into dst (row stride p_lanes * KS), times `mul`
template <typename A>
__device__ __forceinline__ void stage_rows(float* dst, const A* x, int64_t x_stride, int64_t tok0, int nt, int off, int dim, int p_lanes,
                                           float mul) {
    for (int i = threadIdx.x; i < nt * dim; i += blockDim.x) {
        const int tt = i / dim, d = i % dim;
        dst[tt * p_lanes * KS + lds_row(d)] = ld_f(x, (tok0 + tt) * x_stride + off + d) * mul;
    }
}
template <typename A>
__device__ __forceinline__ void stage_cols(float* dst, const A* x, int64_t x_stride, int64_t tok0, int nt, int off, int vdim, int cb) {
    for (int i = threadIdx.x; i < nt * cb; i += blockDim.x) {
        const int tt = i / cb, c = i % cb;
        const int e = blockIdx.x * cb + c;
        dst[i] = e < vdim ? ld_f(x, (tok0 + tt) * x_stride + off + e) : 0.f;
    }
}
// The same for the chunked recurrences, `V` neighbouring elements of a row at a time (V = 4: dim, off and the rows' stride are multiples
// of four and x starts on such a border) and STAGE_U pieces of a thread in flight together before the first is written: a stage is one
// or two memory round trips instead of one per piece.  act 1: silu; times mul.
constexpr int STAGE_U = 8;
__device__ __forceinline__ float scan_act(float z, int act) { return act == 1 ? z * sigmoid_f(z) : z; }
template <typename A, int V, bool ROWS>
__device__ __forceinline__ void stage_pieces(float* dst, int rs, const A* __restrict__ x, int64_t x_stride, int nt, int n, int n_zero, int act, float mul) {
    typedef A veca __attribute__((ext_vector_type(V)));
    typedef float vecf __attribute__((ext_vector_type(V)));
    const int per = n_zero / V, pieces = nt * per;            // n elements of a row are there, those up to n_zero are zeros
    for (int i0 = threadIdx.x; i0 < pieces; i0 += blockDim.x * STAGE_U) {
        veca v[STAGE_U];
#pragma unroll
        for (int u = 0; u < STAGE_U; ++u) {
            const int i = i0 + u * (int)blockDim.x, tt = i / per, d = (i - tt * per) * V;
            if (i < pieces && d < n) v[u] = *reinterpret_cast<const veca*>(x + tt * x_stride + d);
        }
#pragma unroll
        for (int u = 0; u < STAGE_U; ++u) {
            const int i = i0 + u * (int)blockDim.x, tt = i / per, d = (i - tt * per) * V;
            if (i >= pieces) continue;
            vecf f;
#pragma unroll
            for (int k = 0; k < V; ++k) f[k] = d < n ? scan_act((float)v[u][k], act) * mul : 0.f;
            *reinterpret_cast<vecf*>(dst + tt * rs + (ROWS ? lds_row(d) : d)) = f;
        }
    }
}
// key rows (dst: rs floats a token, lds_row inside), and value columns (dst: `width` floats a token, of which `n` are within the head)
template <typename A>
__device__ __forceinline__ void stage_key_rows(float* dst, int rs, const A* x, int64_t x_stride, int nt, int dim, bool vec, int act = 0, float mul = 1.0f) {
    if (vec) stage_pieces<A, 4, true>(dst, rs, x, x_stride, nt, dim, dim, act, mul);
    else stage_pieces<A, 1, true>(dst, rs, x, x_stride, nt, dim, dim, act, mul);
}
template <typename A>
__device__ __forceinline__ void stage_value_cols(float* dst, int width, const A* x, int64_t x_stride, int nt, int n, bool vec, int act = 0) {
    if (vec) stage_pieces<A, 4, false>(dst, width, x, x_stride, nt, n < width ? n : width, width, act, 1.0f);
    else stage_pieces<A, 1, false>(dst, width, x, x_stride, nt, n < width ? n : width, width, act, 1.0f);
}
// whether a launch may stage four elements at a time
template <typename A>
static bool stage_vec_ok(const void* x, int64_t x_stride, int64_t q_off, int64_t k_off, int64_t v_off, int64_t dim, int64_t vdim, int64_t cols) {
    return (reinterpret_cast<uintptr_t>(x) & (4 * sizeof(A) - 1)) == 0 && ((x_stride | q_off | k_off | v_off | dim | vdim | cols) & 3) == 0;
}
__device__ __forceinline__ void zero_rows(float* dst, int n) {
    for (int i = threadIdx.x; i < n; i += blockDim.x) dst[i] = 0.f;
}
// rows of dst (nt of them, `dim` used elements each) scaled to unit length: x / sqrt(sum x^2 + 1e-6) * mul; a wave per row
__device__ __forceinline__ void unit_rows(float* dst, int nt, int dim, int p_lanes, float mul) {
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, n_waves = blockDim.x >> 6;
    for (int tt = wave; tt < nt; tt += n_waves) {
        float* r = dst + tt * p_lanes * KS;
        float ss = 0.f;
        for (int d = lane; d < dim; d += 64) { const float v = r[lds_row(d)]; ss += v * v; }
        const float sc = mul / sqrtf(wave_sum(ss) + 1e-6f);
        for (int d = lane; d < dim; d += 64) r[lds_row(d)] *= sc;
    }
}

// mLSTM.  x[t] holds q at q_off, k at k_off (heads * dim each) and v at v_off (heads * vdim); gates[t] = [i | f] pre-activations
// (heads each, float32), gate_bias likewise.  i = cap tanh(. / cap), f = logsigmoid(cap tanh(. / cap));
//   m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n likewise with k;  o = S^T q / (max(|n.q|, e^(-m')) + 1e-6)
// with q scaled by dim^(-1/2); m starts at 0.  S: (slots, heads, dim, vdim), n: (slots, heads, dim), m: (slots, heads).
// Every column block of a head reads n and m (N_in, M_in) and the first one writes them (N, M): where a head has more than one
// column block the caller hands in copies to read from, since a block that starts late must not see the new values.
// PHASE 0: one workgroup walks a whole portion.  PHASE 1 and 3: chunks of `chunk` tokens side by side (blockIdx.z = sequence * n_chunk_max +
// chunk).  Phase 1 builds a chunk's own memory from nothing (maximum -inf, so the chunk's maximum is that of its own terms) into ws and
// also keeps its sum of forget gates; phase 3 starts from what the carry made of ws and writes the read-out only.
struct MlstmChunks { float* S; float* N; float* M; float* F; int chunk; int n_max; };
template <typename A, int PHASE>
__global__ __launch_bounds__(256) void mlstm_scan_kernel(const A* __restrict__ x, int64_t x_stride, int q_off, int k_off, int v_off,
                                                        const float* __restrict__ gates, const float* __restrict__ gate_bias, float cap,
                                                        float* __restrict__ S, const float* __restrict__ N_in, const float* __restrict__ M_in,
                                                        float* __restrict__ N, float* __restrict__ M,
                                                        const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                        const int32_t* __restrict__ state_slot, float* __restrict__ out, int heads, int dim,
                                                        int vdim, int p_lanes, int tb, int vec, MlstmChunks ck) {
    extern __shared__ float sm[];
    const int cb = blockDim.x / p_lanes, rs = p_lanes * KS;
    float* sq = sm;
    float* sk = sq + tb * rs;
    float* sv = sk + tb * rs;
    float* si = sv + tb * cb;
    float* sf = si + tb;
    const int hd = blockIdx.y;
    SeqSpan sp = seq_span(PHASE ? blockIdx.z / ck.n_max : blockIdx.z, qo_indptr, pos0, state_slot);
    if (sp.slot < 0 || sp.n <= 0) return;
    if (PHASE) {
        const int64_t first = (int64_t)(blockIdx.z % ck.n_max) * ck.chunk;
        if (first >= sp.n) return;
        sp.q0 += first;
        sp.n = sp.n - first < ck.chunk ? sp.n - first : ck.chunk;
    }
    const ScanThread th = scan_thread(p_lanes, vdim);
    const int64_t at = (int64_t)(PHASE ? (int)blockIdx.z : sp.slot) * heads + hd;
    float* Sp = (PHASE ? ck.S : S) + at * dim * vdim;
    float* Np = (PHASE ? ck.N : N) + at * dim;
    const float* Np_in = PHASE ? Np : N_in + at * dim;
    // phase 1 has no use for the normaliser but in the one wave that hands it on
    const bool norm_here = PHASE != 1 || (blockIdx.x == 0 && threadIdx.x < 64);
    float s[KR], nn[KR];
    float m = PHASE == 1 ? -INFINITY : 0.f, f_sum = 0.f;
    const bool cont = PHASE == 3 || (PHASE == 0 && sp.pos0 > 0);
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
        const bool in = cont && row < dim;
        s[r] = (in && th.active) ? Sp[(int64_t)row * vdim + th.e] : 0.f;
        nn[r] = in ? Np_in[row] : 0.f;
    }
    if (cont) m = PHASE ? ck.M[at] : M_in[at];
    zero_rows(sq, 2 * tb * rs);
    const float q_mul = 1.0f / sqrtf((float)dim);
    for (int64_t t0 = 0; t0 < sp.n; t0 += tb) {
        const int nt = (int)(sp.n - t0 < tb ? sp.n - t0 : tb);
        __syncthreads();
        const A* xr = x + (sp.q0 + t0) * x_stride;
        if (PHASE != 1) stage_key_rows(sq, rs, xr + q_off + hd * dim, x_stride, nt, dim, vec, 0, q_mul);
        stage_key_rows(sk, rs, xr + k_off + hd * dim, x_stride, nt, dim, vec);
        stage_value_cols(sv, cb, xr + v_off + hd * vdim + blockIdx.x * cb, x_stride, nt, vdim - (int)blockIdx.x * cb, vec);
        if ((int)threadIdx.x < nt) {
            const float* g = gates + (sp.q0 + t0 + threadIdx.x) * 2 * heads;
            si[threadIdx.x] = cap * tanhf((g[hd] + gate_bias[hd]) / cap);
            sf[threadIdx.x] = logsigmoid_f(cap * tanhf((g[heads + hd] + gate_bias[heads + hd]) / cap));
        }
        __syncthreads();
        for (int tt = 0; tt < nt; ++tt) {
            const float gi = si[tt], gf = sf[tt];
            const float m_new = fmaxf(gf + m, gi);
            const float keep = expf(gf + m - m_new), put = expf(gi - m_new);
            m = m_new;
            if (PHASE == 1) f_sum += gf;
            const float v = sv[tt * cb + th.col];
            const float* kk = sk + tt * rs + th.p * KS;
            const float* qq = sq + tt * rs + th.p * KS;
            if (PHASE == 1) {
#pragma unroll
                for (int r = 0; r < KR; ++r) s[r] = keep * s[r] + put * kk[r] * v;
                if (norm_here) {
#pragma unroll
                    for (int r = 0; r < KR; ++r) nn[r] = keep * nn[r] + put * kk[r];
                }
                continue;
            }
            float num = 0.f, nq = 0.f;
#pragma unroll
            for (int r = 0; r < KR; ++r) {
                const float kp = put * kk[r];
                s[r] = keep * s[r] + kp * v;
                nn[r] = keep * nn[r] + kp;
                num += s[r] * qq[r];
                nq += nn[r] * qq[r];
            }
            num = lanes_sum(num, p_lanes);
            nq = lanes_sum(nq, p_lanes);
            if (th.p == 0 && th.active)
                out[(sp.q0 + t0 + tt) * (int64_t)heads * vdim + (int64_t)hd * vdim + th.e] = num / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
        }
    }
    if (PHASE == 3) return;
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
        if (row < dim && th.active) Sp[(int64_t)row * vdim + th.e] = s[r];
        if (row < dim && blockIdx.x == 0 && th.col == 0) Np[row] = nn[r];
    }
    if (blockIdx.x == 0 && threadIdx.x == 0) {
        (PHASE ? ck.M : M)[at] = m;
        if (PHASE) ck.F[at] = f_sum;
    }
}

// Between the phases, the scalars: with F the sum of a chunk's forget gates and m_own its maximum, the maximum after the chunk is
// max(F + m, m_own) (the same number as step by step), the memory in front is kept with e^(F + m - m') and the chunk's own enters with
// e^(m_own - m').  M becomes the maximum at every chunk's start, F the factor `keep`, put the other; one thread per (sequence, head).
__global__ __launch_bounds__(64) void mlstm_chunk_scalars_kernel(float* __restrict__ M_pool, float* __restrict__ M, float* __restrict__ F,
                                                                float* __restrict__ put, const int32_t* __restrict__ qo_indptr,
                                                                const int64_t* __restrict__ pos0, const int32_t* __restrict__ state_slot, int heads,
                                                                int chunk, int n_chunk_max, int n_seq) {
    const int i = blockIdx.x * 64 + threadIdx.x;
    if (i >= n_seq * heads) return;
    const int seq = i / heads, hd = i % heads;
    const SeqSpan sp = seq_span(seq, qo_indptr, pos0, state_slot);
    if (sp.slot < 0 || sp.n <= 0) return;
    float run = sp.pos0 > 0 ? M_pool[(int64_t)sp.slot * heads + hd] : 0.f;
    for (int ck = 0; (int64_t)ck * chunk < sp.n; ++ck) {
        const int64_t at = ((int64_t)seq * n_chunk_max + ck) * heads + hd;
        const float own = M[at], f = F[at], next = fmaxf(f + run, own);
        M[at] = run;
        F[at] = expf(f + run - next);
        put[at] = expf(own - next);
        run = next;
    }
    M_pool[(int64_t)sp.slot * heads + hd] = run;
}

// Between the phases, a memory of `rows` x `cols` per head: ws[sequence][chunk] holds every chunk's own contribution and is replaced by
// the memory at the chunk's start; what is there after the last chunk goes to the pool.  One chunk further: keep * memory + put * own,
// keep one number per head or (keep_rows) per head and row, put one per head or (null) 1.  One thread per element.
__global__ __launch_bounds__(256) void chunk_carry_kernel(float* __restrict__ pool, float* __restrict__ ws, const float* __restrict__ keep, int keep_rows,
                                                         const float* __restrict__ put, const int32_t* __restrict__ qo_indptr,
                                                         const int64_t* __restrict__ pos0, const int32_t* __restrict__ state_slot, int heads, int rows,
                                                         int cols, int chunk, int n_chunk_max) {
    const SeqSpan sp = seq_span(blockIdx.y, qo_indptr, pos0, state_slot);
    if (sp.slot < 0 || sp.n <= 0) return;
    const int64_t per = (int64_t)heads * rows * cols, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= per) return;
    const int hd = (int)(i / ((int64_t)rows * cols)), row = (int)(i / cols % rows);
    const int n_ck = (int)((sp.n + chunk - 1) / chunk);
    float run = sp.pos0 > 0 ? pool[(int64_t)sp.slot * per + i] : 0.f;
    float* w = ws + (int64_t)blockIdx.y * n_chunk_max * per + i;
    const float* kp = keep + (int64_t)blockIdx.y * n_chunk_max * heads * (keep_rows ? rows : 1) + (keep_rows ? hd * rows + row : hd);
    const float* pp = put ? put + (int64_t)blockIdx.y * n_chunk_max * heads + hd : nullptr;
    const int64_t k_step = (int64_t)heads * (keep_rows ? rows : 1);
    for (int ck = 0; ck < n_ck; ++ck) {
        const float own = w[ck * per];
        w[ck * per] = run;
        run = kp[ck * k_step] * run + (pp ? pp[(int64_t)ck * heads] * own : own);
    }
    pool[(int64_t)sp.slot * per + i] = run;
}


// Gated delta rule.  x[t] holds q at q_off, k at k_off (kv_heads * dim each, after convolution and silu) and v at v_off (heads *
// vdim); ab[t] = [a | b] pre-activations (heads each, float32).  q and k are scaled to unit length per head (q also by
// dim^(-1/2)); g = exp(-exp(A_log) softplus(a + dt_bias)), beta = sigmoid(b);
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.          S: (slots, heads, dim, vdim).
template <typename A>
__global__ __launch_bounds__(256) void delta_scan_kernel(const A* __restrict__ x, int64_t x_stride, int q_off, int k_off, int v_off,
                                                        const float* __restrict__ ab, const float* __restrict__ a_log,
                                                        const float* __restrict__ dt_bias, float* __restrict__ S,
                                                        const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                        const int32_t* __restrict__ state_slot, float* __restrict__ out, int heads,
                                                        int kv_heads, int dim, int vdim, int p_lanes) {
    extern __shared__ float sm[];
    const int cb = blockDim.x / p_lanes, rs = p_lanes * KS;
    float* sq = sm;
    float* sk = sq + TB * rs;
    float* sv = sk + TB * rs;
    float* sg = sv + TB * cb;
    float* sb = sg + TB;
    const int hd = blockIdx.y, kvh = hd / (heads / kv_heads);
    const SeqSpan sp = seq_span(blockIdx.z, qo_indptr, pos0, state_slot);
    if (sp.slot < 0 || sp.n <= 0) return;
    const ScanThread th = scan_thread(p_lanes, vdim);
    float* Sp = S + ((int64_t)sp.slot * heads + hd) * dim * vdim;
    float s[KR];
    const bool cont = sp.pos0 > 0;
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
        s[r] = (cont && row < dim && th.active) ? Sp[(int64_t)row * vdim + th.e] : 0.f;
    }
    zero_rows(sq, 2 * TB * rs);
    const float rate = expf(a_log[hd]), bias = dt_bias[hd];
    const float q_mul = 1.0f / sqrtf((float)dim);
    for (int64_t t0 = 0; t0 < sp.n; t0 += TB) {
        const int nt = (int)(sp.n - t0 < TB ? sp.n - t0 : TB);
        __syncthreads();
        stage_rows(sq, x, x_stride, sp.q0 + t0, nt, q_off + kvh * dim, dim, p_lanes, 1.0f);
        stage_rows(sk, x, x_stride, sp.q0 + t0, nt, k_off + kvh * dim, dim, p_lanes, 1.0f);
        stage_cols(sv, x, x_stride, sp.q0 + t0, nt, v_off + hd * vdim, vdim, cb);
        if ((int)threadIdx.x < nt) {
            const float* g = ab + (sp.q0 + t0 + threadIdx.x) * 2 * heads;
            sg[threadIdx.x] = expf(-rate * softplus_f(g[hd] + bias));
            sb[threadIdx.x] = sigmoid_f(g[heads + hd]);
        }
        __syncthreads();
        unit_rows(sq, nt, dim, p_lanes, q_mul);
        unit_rows(sk, nt, dim, p_lanes, 1.0f);
        __syncthreads();
        for (int tt = 0; tt < nt; ++tt) {
            const float g = sg[tt], beta = sb[tt];
            const float* kk = sk + tt * rs + th.p * KS;
            const float* qq = sq + tt * rs + th.p * KS;
            float kdot = 0.f;
#pragma unroll
            for (int r = 0; r < KR; ++r) {
                s[r] *= g;
                kdot += s[r] * kk[r];
            }
            kdot = lanes_sum(kdot, p_lanes);
            const float u = beta * (sv[tt * cb + th.col] - kdot);
            float o = 0.f;
#pragma unroll
            for (int r = 0; r < KR; ++r) {
                s[r] += kk[r] * u;
                o += s[r] * qq[r];
            }
            o = lanes_sum(o, p_lanes);
            if (th.p == 0 && th.active) out[(sp.q0 + t0 + tt) * (int64_t)heads * vdim + (int64_t)hd * vdim + th.e] = o;
        }
    }
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
        if (row < dim && th.active) Sp[(int64_t)row * vdim + th.e] = s[r];
    }
}

// RWKV-style time mixing.  r, k, v: (n_tok, heads * dim) each (rows rkv_stride apart); wlog (n_tok, heads * dim) float32 and w0
// (heads * dim): the decay of key channel c is w = exp(-exp(wlog + w0)); bonus (heads, dim).
//   o = (S + diag(bonus) k v^T)^T r;  S <- diag(w) S + k v^T.          S: (slots, heads, dim, dim).
template <typename A>
__global__ __launch_bounds__(256) void rwkv_scan_kernel(const A* __restrict__ rx, const A* __restrict__ kx, const A* __restrict__ vx,
                                                       int64_t rkv_stride, const float* __restrict__ wlog, const float* __restrict__ w0,
                                                       const float* __restrict__ bonus, float* __restrict__ S,
                                                       const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                       const int32_t* __restrict__ state_slot, float* __restrict__ out, int heads, int dim,
                                                       int p_lanes) {
    extern __shared__ float sm[];
    const int cb = blockDim.x / p_lanes, rs = p_lanes * KS;
    float* sr = sm;
    float* sk = sr + TB * rs;
    float* sw = sk + TB * rs;
    float* sv = sw + TB * rs;
    const int hd = blockIdx.y;
    const SeqSpan sp = seq_span(blockIdx.z, qo_indptr, pos0, state_slot);
    if (sp.slot < 0 || sp.n <= 0) return;
    const ScanThread th = scan_thread(p_lanes, dim);
    float* Sp = S + ((int64_t)sp.slot * heads + hd) * dim * dim;
    float s[KR], uu[KR];
    const bool cont = sp.pos0 > 0;
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
        s[r] = (cont && row < dim && th.active) ? Sp[(int64_t)row * dim + th.e] : 0.f;
        uu[r] = row < dim ? bonus[hd * dim + row] : 0.f;
    }
    zero_rows(sr, 3 * TB * rs);
    for (int64_t t0 = 0; t0 < sp.n; t0 += TB) {
        const int nt = (int)(sp.n - t0 < TB ? sp.n - t0 : TB);
        __syncthreads();
        stage_rows(sr, rx, rkv_stride, sp.q0 + t0, nt, hd * dim, dim, p_lanes, 1.0f);
        stage_rows(sk, kx, rkv_stride, sp.q0 + t0, nt, hd * dim, dim, p_lanes, 1.0f);
        stage_cols(sv, vx, rkv_stride, sp.q0 + t0, nt, hd * dim, dim, cb);
        for (int i = threadIdx.x; i < nt * dim; i += blockDim.x) {
            const int tt = i / dim, d = i % dim;
            sw[tt * rs + lds_row(d)] = expf(-expf(wlog[(sp.q0 + t0 + tt) * (int64_t)heads * dim + hd * dim + d] + w0[hd * dim + d]));
        }
        __syncthreads();
        for (int tt = 0; tt < nt; ++tt) {
            const float v = sv[tt * cb + th.col];
            const float* rr = sr + tt * rs + th.p * KS;
            const float* kk = sk + tt * rs + th.p * KS;
            const float* ww = sw + tt * rs + th.p * KS;
            float o = 0.f;
#pragma unroll
            for (int r = 0; r < KR; ++r) {
                const float kv = kk[r] * v;
                o += rr[r] * (s[r] + uu[r] * kv);
                s[r] = ww[r] * s[r] + kv;
            }
            o = lanes_sum(o, p_lanes);
            if (th.p == 0 && th.active) out[(sp.q0 + t0 + tt) * (int64_t)heads * dim + (int64_t)hd * dim + th.e] = o;
        }
    }
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
        if (row < dim && th.active) Sp[(int64_t)row * dim + th.e] = s[r];
    }
}

// Linear attention with a constant decay per head.  x[t] holds q at q_off, k at k_off (heads * dim each) and v at v_off (heads *
// vdim), pre-activations if act == 1 (silu is applied to all three as they are staged), values as they are if act == 0.
//   S <- decay[h] S + k v^T;  o = S^T q  (the read sees the token's own write).          S: (slots, heads, dim, vdim).
// Long portions are cut into chunks of `chunk` tokens that run side by side (blockIdx.z = sequence * n_chunk_max + chunk), in three
// launches: phase 1 builds every chunk's own contribution from a zero state into ws (no read-out), the carry kernel turns ws into
// the state at every chunk's start (and writes the sequence's final state), phase 3 walks every chunk from there with the read-out.
// Because the decay is a constant, the carry over a chunk of n tokens is decay^n S + (the chunk's own contribution).  phase 0: one
// workgroup walks the whole portion (single tokens, short portions).
// A thread keeps NC value columns: the rows it reads from LDS then serve NC of them.
// With `half` > 0 the pairs (m, m + half) of every staged query and key are rotated by the token's angles (turn), in float32, and keys are
// multiplied by k_mul.
// `tb` tokens are staged at a time: 32 where the key size leaves LDS for them (more than the other recurrences take: an activation
// is applied as they are staged, and fewer, longer stages hide more of the loads), fewer for wide keys.
template <typename A, int PHASE, int NC>
__global__ __launch_bounds__(256) void decay_scan_kernel(const A* __restrict__ x, int64_t x_stride, int q_off, int k_off, int v_off, int act,
                                                        const float* __restrict__ decay, float* __restrict__ S,
                                                        const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                        const int32_t* __restrict__ state_slot, float* __restrict__ out, int heads, int dim,
                                                        int vdim, int p_lanes, int tb, int vec, int chunk, int n_chunk_max, float* __restrict__ ws,
                                                        TurnRows turn, int half, float k_mul) {
    constexpr int phase = PHASE;
    extern __shared__ float sm[];
    const int cb = blockDim.x / p_lanes, rs = p_lanes * KS;
    float* sq = sm;
    float* sk = sq + tb * rs;
    float* sv = sk + tb * rs;
    const int hd = blockIdx.y;
    const int seq = phase ? blockIdx.z / n_chunk_max : blockIdx.z, ck = phase ? blockIdx.z % n_chunk_max : 0;
    SeqSpan sp = seq_span(seq, qo_indptr, pos0, state_slot);
    if (sp.slot < 0 || sp.n <= 0) return;
    if (phase) {                                     // this workgroup's chunk of the portion
        const int64_t first = (int64_t)ck * chunk;
        if (first >= sp.n) return;
        sp.q0 += first;
        sp.n = sp.n - first < chunk ? sp.n - first : chunk;
    }
    const ScanThread th = scan_thread(p_lanes, vdim);
    const int e0 = blockIdx.x * cb * NC + th.col;              // this thread's value columns: e0, e0 + cb, ...
    // where the state comes from and goes to: the pool (phase 0), nothing and ws (1), ws and nothing (3)
    float* Sp = phase ? ws + ((int64_t)blockIdx.z * heads + hd) * dim * vdim : S + ((int64_t)sp.slot * heads + hd) * dim * vdim;
    float s[NC][KR];
    const bool cont = phase == 3 || (phase == 0 && sp.pos0 > 0);
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
#pragma unroll
        for (int n = 0; n < NC; ++n) s[n][r] = (cont && row < dim && e0 + n * cb < vdim) ? Sp[(int64_t)row * vdim + e0 + n * cb] : 0.f;
    }
    zero_rows(sq, 2 * tb * rs);
    const float g = decay[hd];
    for (int64_t t0 = 0; t0 < sp.n; t0 += tb) {
        const int nt = (int)(sp.n - t0 < tb ? sp.n - t0 : tb);
        __syncthreads();
        const A* xr = x + (sp.q0 + t0) * x_stride;
        if (phase != 1) stage_key_rows(sq, rs, xr + q_off + hd * dim, x_stride, nt, dim, vec, act);      // (phase 1 wants the state only)
        stage_key_rows(sk, rs, xr + k_off + hd * dim, x_stride, nt, dim, vec, act, k_mul);
        stage_value_cols(sv, cb * NC, xr + v_off + hd * vdim + blockIdx.x * cb * NC, x_stride, nt, vdim - (int)blockIdx.x * cb * NC, vec, act);
        __syncthreads();
        if (half) {
            for (int i = threadIdx.x; i < nt * half; i += blockDim.x) {
                const int tt = i / half, m = i - tt * half, d0 = lds_row(m), d1 = lds_row(m + half);
                const float* tr = turn.cos + (sp.q0 + t0 + tt) * turn.stride + m;
                const float c = tr[0], sn = tr[turn.sin_off];
                float* kr = sk + tt * rs;
                const float u = kr[d0], v = kr[d1];
                kr[d0] = u * c - v * sn;
                kr[d1] = v * c + u * sn;
                if (phase != 1) {
                    float* qr = sq + tt * rs;
                    const float a = qr[d0], b = qr[d1];
                    qr[d0] = a * c - b * sn;
                    qr[d1] = b * c + a * sn;
                }
            }
            __syncthreads();
        }
        for (int tt = 0; tt < nt; ++tt) {
            float v[NC], o[NC];
#pragma unroll
            for (int n = 0; n < NC; ++n) { v[n] = sv[(tt * NC + n) * cb + th.col]; o[n] = 0.f; }
            const float* kk = sk + tt * rs + th.p * KS;
            const float* qq = sq + tt * rs + th.p * KS;
            if (phase == 1) {
#pragma unroll
                for (int r = 0; r < KR; ++r)
#pragma unroll
                    for (int n = 0; n < NC; ++n) s[n][r] = g * s[n][r] + kk[r] * v[n];
                continue;
            }
#pragma unroll
            for (int r = 0; r < KR; ++r)
#pragma unroll
                for (int n = 0; n < NC; ++n) {
                    s[n][r] = g * s[n][r] + kk[r] * v[n];
                    o[n] += s[n][r] * qq[r];
                }
#pragma unroll
            for (int n = 0; n < NC; ++n) {
                const float sum = lanes_sum(o[n], p_lanes);
                if (th.p == 0 && e0 + n * cb < vdim) out[(sp.q0 + t0 + tt) * (int64_t)heads * vdim + (int64_t)hd * vdim + e0 + n * cb] = sum;
            }
        }
    }
    if (phase == 3) return;
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
#pragma unroll
        for (int n = 0; n < NC; ++n)
            if (row < dim && e0 + n * cb < vdim) Sp[(int64_t)row * vdim + e0 + n * cb] = s[n][r];
    }
}

// The same recurrence for steps of one token per sequence.  A workgroup takes one head of one sequence: the rotated query and key and the
// value wait in LDS, thread (group, column piece) walks every n_groups-th row of the memory V columns at a time (U rows' loads in flight
// together; the memory is read and written once), and the groups' partial read-outs are added through LDS.  The end is that of
// head_norm_gate: the read-out divided by its root mean square, times mul, times the gate (kind 0: none, 1: sigmoid, 2: silu).
template <typename A, int V>
__global__ __launch_bounds__(256) void decay_step_kernel(const A* __restrict__ x, int64_t x_stride, int q_off, int k_off, int v_off, int act,
                                                        const float* __restrict__ decay, float* __restrict__ S, const int64_t* __restrict__ pos0,
                                                        const int32_t* __restrict__ state_slot, int heads, int dim, int vdim, TurnRows turn, int half,
                                                        float k_mul, float eps, int g_off, int kind, float mul, A* __restrict__ out,
                                                        int64_t out_stride) {
    extern __shared__ __align__(16) float sm[];
    float* sq = sm;                        // dim
    float* sk = sq + dim;                  // dim
    float* part = sk + dim;                // n_groups x cols (cols: vdim rounded up to a multiple of V, in pieces)
    __shared__ float red[4];
    typedef float vecf __attribute__((ext_vector_type(V)));
    const int hd = blockIdx.x;
    const int64_t b = blockIdx.y;
    const int slot = state_slot[b];
    const A* xr = x + b * x_stride;
    A* orow = out + b * out_stride + (int64_t)hd * vdim;
    if (slot < 0) {                        // a padding row: its output is read by the products behind it, nothing else
        for (int e = threadIdx.x; e < vdim; e += 256) st_f(orow, e, 0.f);
        return;
    }
    for (int d = threadIdx.x; d < dim; d += 256) {
        float qv = scan_act(ld_f(xr, q_off + hd * dim + d), act), kv = scan_act(ld_f(xr, k_off + hd * dim + d), act);
        if (d < 2 * half) {
            const int o = d < half ? d + half : d - half;
            const float qo = scan_act(ld_f(xr, q_off + hd * dim + o), act), ko = scan_act(ld_f(xr, k_off + hd * dim + o), act);
            const float* tr = turn.cos + b * turn.stride + (d < half ? d : o);
            const float c = tr[0], sn = d < half ? -tr[turn.sin_off] : tr[turn.sin_off];
            qv = qv * c + qo * sn;
            kv = kv * c + ko * sn;
        }
        sq[d] = qv;
        sk[d] = kv * k_mul;
    }
    const int pieces = (vdim + V - 1) / V, n_groups = 256 / pieces;      // (the host keeps pieces <= 256)
    const int grp = threadIdx.x / pieces, e0 = (threadIdx.x % pieces) * V;
    const bool on = grp < n_groups;
    const float g = decay[hd];
    const bool cont = pos0[b] > 0;
    float* Sp = S + ((int64_t)slot * heads + hd) * dim * vdim;
    vecf val, acc;
#pragma unroll
    for (int i = 0; i < V; ++i) { val[i] = on ? scan_act(ld_f(xr, v_off + hd * vdim + e0 + i), act) : 0.f; acc[i] = 0.f; }
    __syncthreads();
    if (on) {
        constexpr int U = 8;
        for (int r0 = grp; r0 < dim; r0 += n_groups * U) {
            vecf s[U];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int r = r0 + u * n_groups;
                if (cont && r < dim) s[u] = *reinterpret_cast<const vecf*>(Sp + (int64_t)r * vdim + e0);
                else {
#pragma unroll
                    for (int i = 0; i < V; ++i) s[u][i] = 0.f;
                }
            }
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int r = r0 + u * n_groups;
                if (r >= dim) continue;
                const float kr = sk[r], qr = sq[r];
#pragma unroll
                for (int i = 0; i < V; ++i) {
                    s[u][i] = g * s[u][i] + kr * val[i];
                    acc[i] += qr * s[u][i];
                }
                *reinterpret_cast<vecf*>(Sp + (int64_t)r * vdim + e0) = s[u];
            }
        }
#pragma unroll
        for (int i = 0; i < V; ++i) part[grp * pieces * V + e0 + i] = acc[i];
    }
    __syncthreads();
    float ss = 0.f;
    for (int e = threadIdx.x; e < vdim; e += 256) {        // (a thread alone reads and writes its columns)
        float o = 0.f;
        for (int k = 0; k < n_groups; ++k) o += part[k * pieces * V + e];
        part[e] = o;
        ss += o * o;
    }
    const float rn = mul / sqrtf(block256_sum(ss, red) / (float)vdim + eps);
    for (int e = threadIdx.x; e < vdim; e += 256) {
        float v = part[e] * rn;
        if (kind) {
            const float z = ld_f(xr, g_off + hd * vdim + e);
            v *= kind == 1 ? sigmoid_f(z) : z * sigmoid_f(z);
        }
        st_f(orow, e, v);
    }
}

// Between the two chunked phases: ws[sequence][chunk] holds every chunk's own contribution and is replaced by the state at the chunk's
// start; the state after the last chunk goes to the pool.  One thread per element of a sequence's state.
__global__ __launch_bounds__(256) void decay_chunk_carry_kernel(const float* __restrict__ decay, float* __restrict__ S, float* __restrict__ ws,
                                                               const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                               const int32_t* __restrict__ state_slot, int heads, int dim, int vdim, int chunk,
                                                               int n_chunk_max) {
    const SeqSpan sp = seq_span(blockIdx.y, qo_indptr, pos0, state_slot);
    if (sp.slot < 0 || sp.n <= 0) return;
    const int64_t per = (int64_t)heads * dim * vdim;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= per) return;
    const float g = decay[i / ((int64_t)dim * vdim)];
    float* Sp = S + (int64_t)sp.slot * per + i;
    float run = sp.pos0 > 0 ? *Sp : 0.f;
    float* w = ws + (int64_t)blockIdx.y * n_chunk_max * per + i;
    const int n_chunks = (int)((sp.n + chunk - 1) / chunk), last = (int)(sp.n - (int64_t)(n_chunks - 1) * chunk);
    float g_chunk = 1.f, g_last = 1.f;               // decay over a chunk: the same products, in the same order, as that many steps of the recurrence
    for (int k = 0; k < chunk; ++k) {
        g_chunk *= g;
        if (k + 1 == last) g_last = g_chunk;
    }
    constexpr int U = 8;                             // chunks whose contributions are asked for together
    for (int c0 = 0; c0 < n_chunks; c0 += U) {
        float own[U];
#pragma unroll
        for (int u = 0; u < U; ++u) own[u] = c0 + u < n_chunks ? w[(c0 + u) * per] : 0.f;
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (c0 + u >= n_chunks) continue;
            w[(c0 + u) * per] = run;
            run = (c0 + u + 1 == n_chunks ? g_last : g_chunk) * run + own[u];
        }
    }
    *Sp = run;
}

// Gated linear attention.  x[t] holds q at q_off, k at k_off (heads * dim each) and v at v_off (heads * vdim); alpha (n_tok, heads * dim)
// float32: the decay of every key channel at every token.
//   S <- diag(alpha) S + k v^T;  o = S^T (q_mul q)  (the read sees the token's own write).          S: (slots, heads, dim, vdim).
// Phases as in decay_scan_kernel; phase 1 also hands out, per key channel, the product of the chunk's decays (ws_keep), which is what the
// carry multiplies the memory in front with.  A thread keeps NC columns: the rows it reads from LDS then serve NC of them.
template <typename A, int PHASE, int NC>
__global__ __launch_bounds__(256) void gla_scan_kernel(const A* __restrict__ x, int64_t x_stride, int q_off, int k_off, int v_off, float q_mul,
                                                      const float* __restrict__ alpha, float* __restrict__ S, const int32_t* __restrict__ qo_indptr,
                                                      const int64_t* __restrict__ pos0, const int32_t* __restrict__ state_slot, float* __restrict__ out,
                                                      int heads, int dim, int vdim, int p_lanes, int tb, int vec, int chunk, int n_chunk_max,
                                                      float* __restrict__ ws, float* __restrict__ ws_keep) {
    extern __shared__ float sm[];
    const int cb = blockDim.x / p_lanes, rs = p_lanes * KS;
    float* sq = sm;
    float* sk = sq + tb * rs;
    float* sa = sk + tb * rs;
    float* sv = sa + tb * rs;
    const int hd = blockIdx.y;
    SeqSpan sp = seq_span(PHASE ? blockIdx.z / n_chunk_max : blockIdx.z, qo_indptr, pos0, state_slot);
    if (sp.slot < 0 || sp.n <= 0) return;
    if (PHASE) {
        const int64_t first = (int64_t)(blockIdx.z % n_chunk_max) * chunk;
        if (first >= sp.n) return;
        sp.q0 += first;
        sp.n = sp.n - first < chunk ? sp.n - first : chunk;
    }
    const ScanThread th = scan_thread(p_lanes, vdim);
    const int e0 = blockIdx.x * cb * NC + th.col;              // this thread's value columns: e0, e0 + cb, ...
    const int64_t at = (int64_t)(PHASE ? (int)blockIdx.z : sp.slot) * heads + hd;
    float* Sp = (PHASE ? ws : S) + at * dim * vdim;
    float s[NC][KR], pr[KR];
    const bool cont = PHASE == 3 || (PHASE == 0 && sp.pos0 > 0);
    const bool keep_here = PHASE == 1 && blockIdx.x == 0 && threadIdx.x < 64;       // the wave that multiplies the decays up
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
#pragma unroll
        for (int n = 0; n < NC; ++n) s[n][r] = (cont && row < dim && e0 + n * cb < vdim) ? Sp[(int64_t)row * vdim + e0 + n * cb] : 0.f;
        pr[r] = 1.f;
    }
    zero_rows(sq, 3 * tb * rs);
    for (int64_t t0 = 0; t0 < sp.n; t0 += tb) {
        const int nt = (int)(sp.n - t0 < tb ? sp.n - t0 : tb);
        __syncthreads();
        const A* xr = x + (sp.q0 + t0) * x_stride;
        if (PHASE != 1) stage_key_rows(sq, rs, xr + q_off + hd * dim, x_stride, nt, dim, vec, 0, q_mul);
        stage_key_rows(sk, rs, xr + k_off + hd * dim, x_stride, nt, dim, vec);
        stage_key_rows(sa, rs, alpha + ((sp.q0 + t0) * heads + hd) * dim, (int64_t)heads * dim, nt, dim, vec);
        stage_value_cols(sv, cb * NC, xr + v_off + hd * vdim + blockIdx.x * cb * NC, x_stride, nt, vdim - (int)blockIdx.x * cb * NC, vec);
        __syncthreads();
        for (int tt = 0; tt < nt; ++tt) {
            float v[NC], o[NC];
#pragma unroll
            for (int n = 0; n < NC; ++n) { v[n] = sv[(tt * NC + n) * cb + th.col]; o[n] = 0.f; }
            const float* kk = sk + tt * rs + th.p * KS;
            const float* qq = sq + tt * rs + th.p * KS;
            const float* aa = sa + tt * rs + th.p * KS;
            if (PHASE == 1) {
#pragma unroll
                for (int r = 0; r < KR; ++r)
#pragma unroll
                    for (int n = 0; n < NC; ++n) s[n][r] = aa[r] * s[n][r] + kk[r] * v[n];
                if (keep_here) {
#pragma unroll
                    for (int r = 0; r < KR; ++r) pr[r] *= aa[r];
                }
                continue;
            }
#pragma unroll
            for (int r = 0; r < KR; ++r)
#pragma unroll
                for (int n = 0; n < NC; ++n) {
                    s[n][r] = aa[r] * s[n][r] + kk[r] * v[n];
                    o[n] += s[n][r] * qq[r];
                }
#pragma unroll
            for (int n = 0; n < NC; ++n) {
                const float sum = lanes_sum(o[n], p_lanes);
                if (th.p == 0 && e0 + n * cb < vdim) out[(sp.q0 + t0 + tt) * (int64_t)heads * vdim + (int64_t)hd * vdim + e0 + n * cb] = sum;
            }
        }
    }
    if (PHASE == 3) return;
#pragma unroll
    for (int r = 0; r < KR; ++r) {
        const int row = th.r0 + r;
#pragma unroll
        for (int n = 0; n < NC; ++n)
            if (row < dim && e0 + n * cb < vdim) Sp[(int64_t)row * vdim + e0 + n * cb] = s[n][r];
        if (keep_here && th.col == 0 && row < dim) ws_keep[at * dim + row] = pr[r];
    }
}

// launch geometry of the recurrences: lanes per column (a power of two), threads per workgroup, value columns per
// workgroup
struct ScanLaunch { int p_lanes, threads, cb; };
static bool scan_launch(int64_t dim, int64_t vdim, ScanLaunch* g) {      // (a thread that keeps several columns: pass vdim over their number)
    int p = 1;
    while ((int64_t)p * KR < dim) p <<= 1;
    if (p > 16) return false;                       // dim <= 512: two staged operands of TB tokens fit the default LDS window
    int64_t threads = ((vdim * p + 63) / 64) * 64;
    if (threads > 256) threads = 256;
    g->p_lanes = p;
    g->threads = (int)threads;
    g->cb = (int)threads / p;
    return true;
}

}  // namespace NVX_NS

using namespace NVX_NS;

#define NVX_LAYOUT_OK(name)                                                                                                         \
    NVX_REQUIRE(fmt >= 0 && fmt <= 2, NVX_EINVAL, name ": fmt must be 0, 1 or 2");                                                  \
    NVX_REQUIRE(n_tok >= 0 && n_seq >= 0 && n_seq <= 65535 && n_tok <= 65535 * 256, NVX_EINVAL, name ": bad token or sequence count"); \
    if (n_tok == 0 || n_seq == 0) return NVX_OK;                                                                                    \
    NVX_REQUIRE(pos0 && state_slot, NVX_EINVAL, name ": null layout");                                                              \
    NVX_REQUIRE(qo_indptr || n_tok == n_seq, NVX_EINVAL, name ": without qo_indptr every sequence has one token")

void nvx_launch_tail_rows(const void* x, int64_t x_stride, int fmt, int taps_n, float* state, const int32_t* qo_indptr, const int64_t* pos0,
                          const int32_t* state_slot, int64_t n_seq, int64_t channels, hipStream_t stream) {
    const unsigned cx = (unsigned)((channels + 255) / 256);
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(tail_rows_kernel<A_>, dim3(cx, (unsigned)n_seq), dim3(256), 0, stream, (const A_*)x, x_stride, taps_n - 1, state,
                                         qo_indptr, pos0, state_slot, (int)channels));
}

extern "C" int nvx_short_conv(const void* x, int64_t x_stride, int fmt, const float* w, const float* bias, int act, int taps_n, float* state,
                              int64_t n_slots, const int32_t* tok_seq, const int32_t* qo_indptr, const int64_t* pos0,
                              const int32_t* state_slot, void* out, int64_t n_tok, int64_t n_seq, int64_t channels, nvx_stream_t stream) {
    NVX_LAYOUT_OK("nvx_short_conv");
    NVX_REQUIRE(channels > 0 && channels < (1 << 30) && x_stride >= channels && taps_n >= 1 && taps_n <= 64 && n_slots >= 0 && n_tok <= 65535 &&
                    (act == 0 || act == 1), NVX_EINVAL, "nvx_short_conv: bad sizes, or an activation other than 0 (none) and 1 (silu)");
    NVX_REQUIRE(x && w && out && (state || taps_n == 1), NVX_EINVAL, "nvx_short_conv: null pointer");
    NVX_REQUIRE((tok_seq != nullptr) == (qo_indptr != nullptr), NVX_EINVAL, "nvx_short_conv: tok_seq and qo_indptr go together");
    const unsigned cx = (unsigned)((channels + 255) / 256);
    NVX_FMT_CALL(fmt, {
        hipLaunchKernelGGL(short_conv_kernel<A_>, dim3(cx, (unsigned)n_tok), dim3(256), 0, (hipStream_t)stream, (const A_*)x, x_stride, w, bias,
                           act, taps_n, (const float*)state, tok_seq, qo_indptr, pos0, state_slot, (A_*)out, (int)channels);
        if (taps_n > 1)
            hipLaunchKernelGGL(tail_rows_kernel<A_>, dim3(cx, (unsigned)n_seq), dim3(256), 0, (hipStream_t)stream, (const A_*)x, x_stride,
                               taps_n - 1, state, qo_indptr, pos0, state_slot, (int)channels);
    });
    return nvx_check_launch("nvx_short_conv");
}

extern "C" int nvx_short_conv_silu(const void* x, int64_t x_stride, int fmt, const float* w, int taps_n, float* state, int64_t n_slots,
                                   const int32_t* tok_seq, const int32_t* qo_indptr, const int64_t* pos0, const int32_t* state_slot,
                                   void* out, int64_t n_tok, int64_t n_seq, int64_t channels, nvx_stream_t stream) {
    return nvx_short_conv(x, x_stride, fmt, w, nullptr, 1, taps_n, state, n_slots, tok_seq, qo_indptr, pos0, state_slot, out, n_tok, n_seq,
                          channels, stream);
}

extern "C" int nvx_token_shift_mix(const void* h, int64_t h_stride, int fmt, const float* mu, int n_mix, float* state, int64_t n_slots,
                                   const int32_t* tok_seq, const int32_t* qo_indptr, const int64_t* pos0, const int32_t* state_slot,
                                   void* out, int64_t n_tok, int64_t n_seq, int64_t width, nvx_stream_t stream) {
    NVX_LAYOUT_OK("nvx_token_shift_mix");
    NVX_REQUIRE(width > 0 && width < (1 << 30) && h_stride >= width && n_mix >= 1 && n_mix <= 64 && n_slots >= 0 && n_tok <= 65535, NVX_EINVAL,
                "nvx_token_shift_mix: bad sizes");
    NVX_REQUIRE(h && mu && out && state, NVX_EINVAL, "nvx_token_shift_mix: null pointer");
    NVX_REQUIRE((tok_seq != nullptr) == (qo_indptr != nullptr), NVX_EINVAL, "nvx_token_shift_mix: tok_seq and qo_indptr go together");
    const unsigned cx = (unsigned)((width + 255) / 256);
    NVX_FMT_CALL(fmt, {
        hipLaunchKernelGGL(token_shift_mix_kernel<A_>, dim3(cx, (unsigned)n_tok), dim3(256), 0, (hipStream_t)stream, (const A_*)h, h_stride, mu,
                           n_mix, (const float*)state, tok_seq, qo_indptr, pos0, state_slot, (A_*)out, n_tok, (int)width);
        hipLaunchKernelGGL(tail_rows_kernel<A_>, dim3(cx, (unsigned)n_seq), dim3(256), 0, (hipStream_t)stream, (const A_*)h, h_stride, 1, state,
                           qo_indptr, pos0, state_slot, (int)width);
    });
    return nvx_check_launch("nvx_token_shift_mix");
}

extern "C" int64_t nvx_scan_column_blocks(int64_t dim, int64_t vdim) {
    ScanLaunch g;
    if (dim <= 0 || vdim <= 0 || !scan_launch(dim, vdim, &g)) return 0;
    return (vdim + g.cb - 1) / g.cb;
}

extern "C" int nvx_mlstm_scan(const void* x, int64_t x_stride, int fmt, int64_t q_off, int64_t k_off, int64_t v_off, const float* gates,
                              const float* gate_bias, float cap, float* S, const float* N_in, const float* M_in, float* N, float* M,
                              int64_t n_slots, const int32_t* qo_indptr,
                              const int64_t* pos0, const int32_t* state_slot, float* out, int64_t n_tok, int64_t n_seq, int64_t heads,
                              int64_t dim, int64_t vdim, int64_t chunk, int64_t n_chunk_max, float* ws, nvx_stream_t stream) {
    NVX_LAYOUT_OK("nvx_mlstm_scan");
    ScanLaunch g;
    NVX_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && vdim > 0 && vdim < (1 << 24) && n_slots >= 0 && cap > 0.f, NVX_EINVAL,
                "nvx_mlstm_scan: bad sizes");
    NVX_REQUIRE(scan_launch(dim, vdim, &g), NVX_EUNSUPPORTED, "nvx_mlstm_scan: key size above 512");
    NVX_REQUIRE(x && gates && gate_bias && S && N && M && N_in && M_in && out, NVX_EINVAL, "nvx_mlstm_scan: null pointer");
    NVX_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && x_stride >= q_off + heads * dim && x_stride >= k_off + heads * dim &&
                    x_stride >= v_off + heads * vdim, NVX_EINVAL, "nvx_mlstm_scan: q, k or v lies outside a row");
    const int tb = g.p_lanes <= 4 ? 32 : (g.p_lanes == 8 ? 16 : TB);
    const size_t lds = (size_t)(2 * tb * g.p_lanes * KS + tb * g.cb + 2 * tb) * sizeof(float);
    NVX_REQUIRE(chunk == 0 || (chunk > 0 && chunk < (1 << 30) && n_chunk_max > 0 && n_seq * n_chunk_max <= 65535 && ws && qo_indptr), NVX_EINVAL,
                "nvx_mlstm_scan: chunks need a ragged step, their workspace, and at most 65535 of them");
    const dim3 grid((unsigned)((vdim + g.cb - 1) / g.cb), (unsigned)heads, (unsigned)(chunk ? n_seq * n_chunk_max : n_seq));
    NVX_REQUIRE(chunk || grid.x == 1 || (N_in != N && M_in != M), NVX_EINVAL,
                "nvx_mlstm_scan: a head with several column blocks reads its normaliser and maximum from copies");
    // the workspace: memories, normalisers, maxima, forget sums / keep factors, put factors of all chunks
    const int64_t n_ws = chunk ? n_seq * n_chunk_max * heads : 0;
    MlstmChunks ck = {ws, ws + n_ws * dim * vdim, ws + n_ws * dim * (vdim + 1), ws + n_ws * (dim * (vdim + 1) + 1), (int)chunk, (int)n_chunk_max};
    float* put = ws + n_ws * (dim * (vdim + 1) + 2);
    const hipStream_t st = (hipStream_t)stream;
#define NVX_MLSTM_SCAN(PHASE)                                                                                                                     \
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL((mlstm_scan_kernel<A_, PHASE>), grid, dim3(g.threads), lds, st, (const A_*)x, x_stride, (int)q_off, (int)k_off, \
                                         (int)v_off, gates, gate_bias, cap, S, N_in, M_in, N, M, qo_indptr, pos0, state_slot, out, (int)heads, (int)dim, \
                                         (int)vdim, g.p_lanes, tb, (int)stage_vec_ok<A_>(x, x_stride, q_off, k_off, v_off, dim, vdim, g.cb), ck))
    if (!chunk) {
        NVX_MLSTM_SCAN(0);
    } else {
        NVX_MLSTM_SCAN(1);
        hipLaunchKernelGGL(mlstm_chunk_scalars_kernel, dim3((unsigned)((n_seq * heads + 63) / 64)), dim3(64), 0, st, M, ck.M, ck.F, put, qo_indptr, pos0,
                           state_slot, (int)heads, (int)chunk, (int)n_chunk_max, (int)n_seq);
        hipLaunchKernelGGL(chunk_carry_kernel, dim3((unsigned)((heads * dim * vdim + 255) / 256), (unsigned)n_seq), dim3(256), 0, st, S, ck.S,
                           (const float*)ck.F, 0, (const float*)put, qo_indptr, pos0, state_slot, (int)heads, (int)dim, (int)vdim, (int)chunk, (int)n_chunk_max);
        hipLaunchKernelGGL(chunk_carry_kernel, dim3((unsigned)((heads * dim + 255) / 256), (unsigned)n_seq), dim3(256), 0, st, N, ck.N,
                           (const float*)ck.F, 0, (const float*)put, qo_indptr, pos0, state_slot, (int)heads, (int)dim, 1, (int)chunk, (int)n_chunk_max);
        NVX_MLSTM_SCAN(3);
    }
#undef NVX_MLSTM_SCAN
    return nvx_check_launch("nvx_mlstm_scan");
}

extern "C" int nvx_delta_scan(const void* x, int64_t x_stride, int fmt, int64_t q_off, int64_t k_off, int64_t v_off, const float* ab,
                              const float* a_log, const float* dt_bias, float* S, int64_t n_slots, const int32_t* qo_indptr,
                              const int64_t* pos0, const int32_t* state_slot, float* out, int64_t n_tok, int64_t n_seq, int64_t heads,
                              int64_t kv_heads, int64_t dim, int64_t vdim, nvx_stream_t stream) {
    NVX_LAYOUT_OK("nvx_delta_scan");
    ScanLaunch g;
    NVX_REQUIRE(heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0 && vdim < (1 << 24) && n_slots >= 0,
                NVX_EINVAL, "nvx_delta_scan: bad sizes");
    NVX_REQUIRE(scan_launch(dim, vdim, &g), NVX_EUNSUPPORTED, "nvx_delta_scan: key size above 512");
    NVX_REQUIRE(x && ab && a_log && dt_bias && S && out, NVX_EINVAL, "nvx_delta_scan: null pointer");
    NVX_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && x_stride >= q_off + kv_heads * dim && x_stride >= k_off + kv_heads * dim &&
                    x_stride >= v_off + heads * vdim, NVX_EINVAL, "nvx_delta_scan: q, k or v lies outside a row");
    const size_t lds = (size_t)(2 * TB * g.p_lanes * KS + TB * g.cb + 2 * TB) * sizeof(float);
    const dim3 grid((unsigned)((vdim + g.cb - 1) / g.cb), (unsigned)heads, (unsigned)n_seq);
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(delta_scan_kernel<A_>, grid, dim3(g.threads), lds, (hipStream_t)stream, (const A_*)x, x_stride, (int)q_off,
                                         (int)k_off, (int)v_off, ab, a_log, dt_bias, S, qo_indptr, pos0, state_slot, out, (int)heads,
                                         (int)kv_heads, (int)dim, (int)vdim, g.p_lanes));
    return nvx_check_launch("nvx_delta_scan");
}

extern "C" int nvx_rwkv_scan(const void* r, const void* k, const void* v, int64_t rkv_stride, int fmt, const float* wlog, const float* w0,
                             const float* bonus, float* S, int64_t n_slots, const int32_t* qo_indptr, const int64_t* pos0,
                             const int32_t* state_slot, float* out, int64_t n_tok, int64_t n_seq, int64_t heads, int64_t dim,
                             nvx_stream_t stream) {
    NVX_LAYOUT_OK("nvx_rwkv_scan");
    ScanLaunch g;
    NVX_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && n_slots >= 0 && rkv_stride >= heads * dim, NVX_EINVAL, "nvx_rwkv_scan: bad sizes");
    NVX_REQUIRE(scan_launch(dim, dim, &g) && g.p_lanes <= 8, NVX_EUNSUPPORTED, "nvx_rwkv_scan: head size above 256");
    NVX_REQUIRE(r && k && v && wlog && w0 && bonus && S && out, NVX_EINVAL, "nvx_rwkv_scan: null pointer");
    const size_t lds = (size_t)(3 * TB * g.p_lanes * KS + TB * g.cb) * sizeof(float);
    const dim3 grid((unsigned)((dim + g.cb - 1) / g.cb), (unsigned)heads, (unsigned)n_seq);
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(rwkv_scan_kernel<A_>, grid, dim3(g.threads), lds, (hipStream_t)stream, (const A_*)r, (const A_*)k,
                                         (const A_*)v, rkv_stride, wlog, w0, bonus, S, qo_indptr, pos0, state_slot, out, (int)heads, (int)dim,
                                         g.p_lanes));
    return nvx_check_launch("nvx_rwkv_scan");
}

extern "C" int nvx_decay_scan(const void* x, int64_t x_stride, int fmt, int64_t q_off, int64_t k_off, int64_t v_off, int act,
                              const float* decay, float* S, int64_t n_slots, const int32_t* qo_indptr, const int64_t* pos0,
                              const int32_t* state_slot, float* out, int64_t n_tok, int64_t n_seq, int64_t heads, int64_t dim, int64_t vdim,
                              int64_t chunk, int64_t n_chunk_max, float* ws, const float* turn, int64_t turn_stride, int64_t turn_sin_off,
                              int rot_dims, float k_mul, nvx_stream_t stream) {
    NVX_LAYOUT_OK("nvx_decay_scan");
    ScanLaunch g;
    NVX_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (rot_dims == 0 || (turn && turn_stride >= turn_sin_off + rot_dims / 2)), NVX_EINVAL,
                "nvx_decay_scan: the rotated part must be even and within a head, and needs its table");
    const TurnRows tr{turn, turn_stride, turn_sin_off};
    NVX_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && vdim > 0 && vdim < (1 << 24) && n_slots >= 0 && (act == 0 || act == 1), NVX_EINVAL,
                "nvx_decay_scan: bad sizes");
    NVX_REQUIRE(scan_launch(dim, vdim, &g), NVX_EUNSUPPORTED, "nvx_decay_scan: key size above 512");
    NVX_REQUIRE(x && decay && S && out, NVX_EINVAL, "nvx_decay_scan: null pointer");
    NVX_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && x_stride >= q_off + heads * dim && x_stride >= k_off + heads * dim &&
                    x_stride >= v_off + heads * vdim, NVX_EINVAL, "nvx_decay_scan: q, k or v lies outside a row");
    const int nc = chunk && vdim > 1 ? 2 : 1;      // value columns per thread: a staged row then serves two of them
    NVX_REQUIRE(scan_launch(dim, (vdim + nc - 1) / nc, &g), NVX_EUNSUPPORTED, "nvx_decay_scan: key size above 512");
    const int tb = g.p_lanes <= 4 ? 32 : (g.p_lanes == 8 ? 16 : TB);
    const size_t lds = (size_t)(2 * tb * g.p_lanes * KS + tb * g.cb * nc) * sizeof(float);
    NVX_REQUIRE(chunk == 0 || (chunk > 0 && chunk < (1 << 30) && n_chunk_max > 0 && n_seq * n_chunk_max <= 65535 && ws && qo_indptr), NVX_EINVAL,
                "nvx_decay_scan: chunks need a ragged step, their workspace, and at most 65535 of them");
    const dim3 grid((unsigned)((vdim + g.cb * nc - 1) / (g.cb * nc)), (unsigned)heads, (unsigned)(chunk ? n_seq * n_chunk_max : n_seq));
#define NVX_DECAY_SCAN(PHASE, NC)                                                                                                                   \
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL((decay_scan_kernel<A_, PHASE, NC>), grid, dim3(g.threads), lds, (hipStream_t)stream, (const A_*)x, x_stride,   \
                                         (int)q_off, (int)k_off, (int)v_off, act, decay, S, qo_indptr, pos0, state_slot, out, (int)heads, (int)dim,  \
                                         (int)vdim, g.p_lanes, tb, (int)stage_vec_ok<A_>(x, x_stride, q_off, k_off, v_off, dim, vdim, g.cb * nc), (int)chunk, (int)n_chunk_max, ws, tr, \
                                         rot_dims / 2, k_mul))
    if (!chunk) {
        NVX_DECAY_SCAN(0, 1);
    } else {
        if (nc == 2) NVX_DECAY_SCAN(1, 2);
        else NVX_DECAY_SCAN(1, 1);
        hipLaunchKernelGGL(decay_chunk_carry_kernel, dim3((unsigned)((heads * dim * vdim + 255) / 256), (unsigned)n_seq), dim3(256), 0,
                           (hipStream_t)stream, decay, S, ws, qo_indptr, pos0, state_slot, (int)heads, (int)dim, (int)vdim, (int)chunk,
                           (int)n_chunk_max);
        if (nc == 2) NVX_DECAY_SCAN(3, 2);
        else NVX_DECAY_SCAN(3, 1);
    }
#undef NVX_DECAY_SCAN
    return nvx_check_launch("nvx_decay_scan");
}

extern "C" int64_t nvx_decay_step_max_vdim() { return 1024; }      // (256 threads of four columns; not a multiple of four: 256)

extern "C" int nvx_decay_step(const void* x, int64_t x_stride, int fmt, int64_t q_off, int64_t k_off, int64_t v_off, int act, const float* decay,
                              float* S, int64_t n_slots, const int64_t* pos0, const int32_t* state_slot, int64_t n_seq, int64_t heads, int64_t dim,
                              int64_t vdim, const float* turn, int64_t turn_stride, int64_t turn_sin_off, int rot_dims, float k_mul, float eps,
                              int64_t g_off, int kind, float mul, void* out, int64_t out_stride, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2, NVX_EINVAL, "nvx_decay_step: fmt must be 0, 1 or 2");
    NVX_REQUIRE(n_seq >= 0 && n_seq <= 65535 && heads > 0 && dim > 0 && dim <= 4096 && vdim > 0 && n_slots >= 0 && (act == 0 || act == 1) && kind >= 0 && kind <= 2,
                NVX_EINVAL, "nvx_decay_step: bad sizes");
    const int v = vdim % 4 == 0 && nvx_aligned16(S) ? 4 : 1;
    NVX_REQUIRE(vdim <= 256 * v, NVX_EUNSUPPORTED, "nvx_decay_step: value size above 1024 (256 where it is not a multiple of four)");
    if (n_seq == 0) return NVX_OK;
    NVX_REQUIRE(x && decay && S && pos0 && state_slot && out && out_stride >= heads * vdim, NVX_EINVAL, "nvx_decay_step: null pointer or row stride");
    NVX_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && g_off >= 0 && x_stride >= q_off + heads * dim && x_stride >= k_off + heads * dim &&
                    x_stride >= v_off + heads * vdim && (kind == 0 || x_stride >= g_off + heads * vdim), NVX_EINVAL,
                "nvx_decay_step: q, k, v or the gate lies outside a row");
    NVX_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (rot_dims == 0 || (turn && turn_stride >= turn_sin_off + rot_dims / 2)), NVX_EINVAL,
                "nvx_decay_step: the rotated part must be even and within a head, and needs its table");
    const TurnRows tr{turn, turn_stride, turn_sin_off};
    const int64_t pieces = (vdim + v - 1) / v;
    const size_t lds = (size_t)(2 * dim + (256 / pieces) * pieces * v) * sizeof(float);
#define NVX_DECAY_STEP(V)                                                                                                                          \
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL((decay_step_kernel<A_, V>), dim3((unsigned)heads, (unsigned)n_seq), dim3(256), lds, (hipStream_t)stream,    \
                                         (const A_*)x, x_stride, (int)q_off, (int)k_off, (int)v_off, act, decay, S, pos0, state_slot, (int)heads, (int)dim, \
                                         (int)vdim, tr, rot_dims / 2, k_mul, eps, (int)g_off, kind, mul, (A_*)out, out_stride))
    if (v == 4) NVX_DECAY_STEP(4);
    else NVX_DECAY_STEP(1);
#undef NVX_DECAY_STEP
    return nvx_check_launch("nvx_decay_step");
}

extern "C" int nvx_gla_scan(const void* x, int64_t x_stride, int fmt, int64_t q_off, int64_t k_off, int64_t v_off, float q_mul, const float* alpha,
                            float* S, int64_t n_slots, const int32_t* qo_indptr, const int64_t* pos0, const int32_t* state_slot, float* out,
                            int64_t n_tok, int64_t n_seq, int64_t heads, int64_t dim, int64_t vdim, int64_t chunk, int64_t n_chunk_max, float* ws,
                            nvx_stream_t stream) {
    NVX_LAYOUT_OK("nvx_gla_scan");
    ScanLaunch g;
    NVX_REQUIRE(heads > 0 && heads <= 65535 && dim > 0 && vdim > 0 && vdim < (1 << 24) && n_slots >= 0, NVX_EINVAL, "nvx_gla_scan: bad sizes");
    NVX_REQUIRE(scan_launch(dim, vdim, &g), NVX_EUNSUPPORTED, "nvx_gla_scan: key size above 512");
    NVX_REQUIRE(x && alpha && S && out, NVX_EINVAL, "nvx_gla_scan: null pointer");
    NVX_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && x_stride >= q_off + heads * dim && x_stride >= k_off + heads * dim &&
                    x_stride >= v_off + heads * vdim, NVX_EINVAL, "nvx_gla_scan: q, k or v lies outside a row");
    const int nc = chunk && vdim > 1 ? 2 : 1;      // value columns per thread: a staged row then serves two of them
    NVX_REQUIRE(scan_launch(dim, (vdim + nc - 1) / nc, &g), NVX_EUNSUPPORTED, "nvx_gla_scan: key size above 512");
    const int tb = g.p_lanes <= 2 && nc == 1 ? 32 : (g.p_lanes <= 4 ? 16 : (g.p_lanes == 8 ? 8 : 4));
    const size_t lds = (size_t)(3 * tb * g.p_lanes * KS + tb * g.cb * nc) * sizeof(float);
    NVX_REQUIRE(chunk == 0 || (chunk > 0 && chunk < (1 << 30) && n_chunk_max > 0 && n_seq * n_chunk_max <= 65535 && ws && qo_indptr), NVX_EINVAL,
                "nvx_gla_scan: chunks need a ragged step, their workspace, and at most 65535 of them");
    const dim3 grid((unsigned)((vdim + g.cb * nc - 1) / (g.cb * nc)), (unsigned)heads, (unsigned)(chunk ? n_seq * n_chunk_max : n_seq));
    float* keep = chunk ? ws + n_seq * n_chunk_max * heads * dim * vdim : nullptr;      // behind the chunks' memories
    const hipStream_t st = (hipStream_t)stream;
#define NVX_GLA_SCAN(PHASE, NC)                                                                                                                        \
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL((gla_scan_kernel<A_, PHASE, NC>), grid, dim3(g.threads), lds, st, (const A_*)x, x_stride, (int)q_off, (int)k_off, \
                                         (int)v_off, q_mul, alpha, S, qo_indptr, pos0, state_slot, out, (int)heads, (int)dim, (int)vdim, g.p_lanes, \
                                         tb, (int)(stage_vec_ok<A_>(x, x_stride, q_off, k_off, v_off, dim, vdim, g.cb * nc) && nvx_aligned16(alpha)), (int)chunk, (int)n_chunk_max, ws, keep))
    if (!chunk) {
        NVX_GLA_SCAN(0, 1);
    } else {
        if (nc == 2) NVX_GLA_SCAN(1, 2);
        else NVX_GLA_SCAN(1, 1);
        hipLaunchKernelGGL(chunk_carry_kernel, dim3((unsigned)((heads * dim * vdim + 255) / 256), (unsigned)n_seq), dim3(256), 0, st, S, ws,
                           (const float*)keep, 1, (const float*)nullptr, qo_indptr, pos0, state_slot, (int)heads, (int)dim, (int)vdim, (int)chunk,
                           (int)n_chunk_max);
        if (nc == 2) NVX_GLA_SCAN(3, 2);
        else NVX_GLA_SCAN(3, 1);
    }
#undef NVX_GLA_SCAN
    return nvx_check_launch("nvx_gla_scan");
}
