// Mixture of small gated feed-forward experts; a choice's weight scales the chosen expert's INPUT (sigmoid routers) or its
// OUTPUT (weight_out: fixed weights from a table).
//   - nvx_moe_route: the `top` largest router logits of every token -> expert ids and sigmoid scores (float32);
//   - nvx_moe_route_softmax: softmax scores, experts in groups of which only the best may be chosen, weights renormalised;
//   - nvx_moe_route_sigmoid: sigmoid scores with a correction that enters the choice only, groups ranked by their two best experts;
//   - nvx_moe_expert_rows: a token's experts evaluated row by row of their weights: the form for steps of few tokens, where
//     every chosen expert's weights have to be streamed once per token anyway;
//   - nvx_moe_order / nvx_moe_scatter_rows / nvx_moe_glu / nvx_moe_gather_rows: the pieces around per-expert matrix products
//     for steps of many tokens (the expert order of the (token, choice) pairs and the experts' counts, scaled inputs gathered
//     into that order, the gated activation, the tokens' results summed back).
// Expert:  g = min(W_gate x, limit), u = clamp(W_up x, -limit, limit), y = g sigmoid(alpha g) (u + shift), out = W_down y
// (limit = infinity, alpha = 1, shift = 0: silu(g) u).  nvx_gelu_glu is the activation of plain gated layers, gelu_tanh(g) u.
#include "fmt_dev.h"

namespace NVX_NS {

__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ logits, int n_exp, int top, int32_t* __restrict__ idx,
                                                       float* __restrict__ wts, int64_t n_tok) {
    const int64_t t = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (t >= n_tok) return;
    const float* z = logits + t * n_exp;
    for (int k = 0; k < top; ++k) {
        int best = -1;
        float bz = -INFINITY;
        for (int e = 0; e < n_exp; ++e) {
            bool taken = false;
            for (int j = 0; j < k; ++j) taken |= idx[t * top + j] == e;
            if (!taken && (best < 0 || z[e] > bz)) { best = e; bz = z[e]; }
        }
        idx[t * top + k] = best;
        wts[t * top + k] = sigmoid_f(bz);
    }
}

// Softmax router with groups: scores = softmax(logits) over all experts; the experts form n_groups equal groups of neighbours, a
// group counts as its best score, and only experts of the keep_groups best groups can be chosen (n_groups <= 1: all of them);
// the `top` largest scores among those are chosen (ties: the lower id) and their scores, divided by their sum + norm_eps, are the
// weights.  One thread per token; everything float32.
__global__ __launch_bounds__(256) void moe_route_softmax_kernel(const float* __restrict__ logits, int64_t logits_stride, int n_exp, int top, int n_groups,
                                                               int keep_groups, float norm_eps, int32_t* __restrict__ idx,
                                                               float* __restrict__ wts, int64_t n_tok) {
    const int64_t t = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (t >= n_tok) return;
    const float* z = logits + t * logits_stride;
    float zmax = -INFINITY;
    for (int e = 0; e < n_exp; ++e) zmax = fmaxf(zmax, z[e]);
    float denom = 0.f;
    for (int e = 0; e < n_exp; ++e) denom += expf(z[e] - zmax);
    // the groups that stay: keep_groups times the best group not yet taken (a group's score is its largest logit: the softmax keeps the order)
    uint64_t kept[4] = {0, 0, 0, 0};                       // n_groups <= 256
    const bool grouped = n_groups > 1 && keep_groups < n_groups;
    const int per = grouped ? n_exp / n_groups : n_exp;
    if (grouped) {
        for (int k = 0; k < keep_groups; ++k) {
            int best = -1;
            float bz = -INFINITY;
            for (int g = 0; g < n_groups; ++g) {
                if ((kept[g >> 6] >> (g & 63)) & 1) continue;
                float gm = -INFINITY;
                for (int e = g * per; e < (g + 1) * per; ++e) gm = fmaxf(gm, z[e]);
                if (best < 0 || gm > bz) { best = g; bz = gm; }
            }
            kept[best >> 6] |= 1ull << (best & 63);
        }
    }
    float sum = 0.f;
    for (int k = 0; k < top; ++k) {
        int best = -1;
        float bz = -INFINITY;
        for (int e = 0; e < n_exp; ++e) {
            if (grouped) { const int g = e / per; if (!((kept[g >> 6] >> (g & 63)) & 1)) continue; }
            bool taken = false;
            for (int j = 0; j < k; ++j) taken |= idx[t * top + j] == e;
            if (!taken && (best < 0 || z[e] > bz)) { best = e; bz = z[e]; }
        }
        idx[t * top + k] = best;
        const float sc = expf(bz - zmax) / denom;
        wts[t * top + k] = sc;
        sum += sc;
    }
    for (int k = 0; k < top; ++k) wts[t * top + k] /= (sum + norm_eps);
}

// Sigmoid router with groups: score = sigmoid(logit); the CHOICE score is score + correction[e] and may be negative.  The experts form
// n_groups equal groups of neighbours, a group counts as the sum of its two largest choice scores (of its one, if it has one), and only
// experts of the keep_groups best groups can be chosen (n_groups <= 1: all).  The `top` largest choice scores are taken (ties: the lower
// id); a chosen expert's weight is its SCORE times w_scale.  A wave per token: its choice scores wait in LDS, a lane looks at every 64th
// group and expert, and the winners are found by lane exchange.
__device__ __forceinline__ void wave_best(float& v, int& i) {       // the largest v of the wave, the lowest i among equals (i < 0: none)
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) {
        const float ov = __shfl_xor(v, m, 64);
        const int oi = __shfl_xor(i, m, 64);
        if (oi >= 0 && (i < 0 || ov > v || (ov == v && oi < i))) { v = ov; i = oi; }
    }
}
// The softmax router without groups, a wave per token (n_exp <= 1024): logits and choices stay in registers and lane exchanges.
__global__ __launch_bounds__(256) void moe_route_softmax_wave_kernel(const float* __restrict__ logits, int64_t logits_stride, int n_exp, int top,
                                                                    float norm_eps, int32_t* __restrict__ idx, float* __restrict__ wts, int64_t n_tok) {
    const int64_t t = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= n_tok) return;                                // (waves share nothing)
    const int lane = threadIdx.x & 63;
    float z[16];
    float zmax = -INFINITY;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
        z[i] = i * 64 + lane < n_exp ? logits[t * logits_stride + i * 64 + lane] : -INFINITY;
        zmax = fmaxf(zmax, z[i]);
    }
    zmax = wave_max(zmax);
    float denom = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i)
        if (i * 64 < n_exp) denom += expf(z[i] - zmax);    // (past the last expert: exp(-inf) = 0)
    denom = wave_sum(denom);
    unsigned taken = 0;                                    // of this lane's experts
    float sum = 0.f, mine = 0.f;
    int mine_e = 0;
    for (int k = 0; k < top; ++k) {
        float v = -INFINITY;
        int e = -1;
#pragma unroll
        for (int i = 0; i < 16; ++i)
            if (i * 64 + lane < n_exp && !((taken >> i) & 1u) && (e < 0 || z[i] > v)) { v = z[i]; e = i * 64 + lane; }
        wave_best(v, e);
        if (e < 0) e = 0;
        if (lane == (e & 63)) taken |= 1u << (e >> 6);
        const float sc = expf(v - zmax) / denom;
        sum += sc;
        if (lane == (k & 63)) { mine = sc; mine_e = e; }   // (top <= 64: choice k is lane k's to write)
    }
    if (lane < top) {
        idx[t * top + lane] = mine_e;
        wts[t * top + lane] = mine / (sum + norm_eps);
    }
}

__global__ __launch_bounds__(256) void moe_route_sigmoid_kernel(const float* __restrict__ logits, const float* __restrict__ correction, int n_exp,
                                                               int top, int n_groups, int keep_groups, float w_scale, int32_t* __restrict__ idx,
                                                               float* __restrict__ wts, int64_t n_tok) {
    extern __shared__ float sm[];                  // per wave: n_exp choice scores, n_groups group scores
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const bool grouped = n_groups > 1 && keep_groups < n_groups;
    const int per = grouped ? n_exp / n_groups : n_exp;
    float* choice = sm + wave * (n_exp + (grouped ? n_groups : 0));
    float* gscore = choice + n_exp;
    const int64_t t = (int64_t)blockIdx.x * 4 + wave;
    const bool on = t < n_tok;
    const float* z = logits + (on ? t : 0) * n_exp;
    for (int e = lane; e < n_exp; e += 64) choice[e] = sigmoid_f(z[e]) + correction[e];
    __syncthreads();
    if (grouped) {
        for (int g = lane; g < n_groups; g += 64) {
            float a = choice[g * per], b = -INFINITY;          // the two largest
            for (int e = 1; e < per; ++e) {
                const float c = choice[g * per + e];
                if (c > a) { b = a; a = c; }
                else if (c > b) b = c;
            }
            gscore[g] = per > 1 ? a + b : a;
        }
        __syncthreads();
        // the groups that stay are marked by an infinite score, the best first
        for (int k = 0; k < keep_groups; ++k) {
            float v = -INFINITY;
            int i = -1;
            for (int g = lane; g < n_groups; g += 64)
                if (gscore[g] < INFINITY && (i < 0 || gscore[g] > v)) { v = gscore[g]; i = g; }
            wave_best(v, i);
            if (lane == 0 && i >= 0) gscore[i] = INFINITY;     // kept
            __syncthreads();
        }
    }
    for (int k = 0; k < top; ++k) {
        float v = -INFINITY;
        int i = -1;
        for (int e = lane; e < n_exp; e += 64) {
            const float c = choice[e];
            if (c == -INFINITY || (grouped && gscore[e / per] != INFINITY)) continue;
            if (i < 0 || c > v) { v = c; i = e; }
        }
        wave_best(v, i);
        if (on && lane == 0) {
            idx[t * top + k] = i < 0 ? 0 : i;
            wts[t * top + k] = i < 0 ? 0.f : sigmoid_f(z[i]) * w_scale;
        }
        if (i >= 0 && lane == (i & 63)) choice[i] = -INFINITY;        // taken (only this lane reads entry i)
    }
}

__device__ __forceinline__ float glu_act(float g, float u, float limit, float alpha, float shift) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * sigmoid_f(alpha * g) * (u + shift);
}

// A token's experts row by row (float32, and sizes that fit no 16-byte loads).  w_gu: (experts, 2 * ff, width) rows [gate | up]; w_d: (experts, width, ff).  Two launches, both
// with a workgroup per 32 weight rows so that a step of a few tokens still fills the chip: the hidden activations of every
// (token, choice) pair into a float32 workspace, then the output rows summed over a token's choices.  A wave takes 8 rows; its
// lanes walk a row 8 elements at a time (16-byte loads) where the format is 16-bit and the rows are 16-byte aligned.
template <typename A, bool VEC>
__device__ __forceinline__ float lane_dot(const A* __restrict__ wrow, const float* __restrict__ xs, int n, int lane) {
    float acc = 0.f;
    if constexpr (VEC) {
        typedef A vec8 __attribute__((ext_vector_type(8)));
        for (int c = lane * 8; c < n; c += 512) {
            const vec8 v = *reinterpret_cast<const vec8*>(wrow + c);
#pragma unroll
            for (int i = 0; i < 8; ++i) acc += (float)v[i] * xs[c + i];
        }
    } else {
        for (int c = lane; c < n; c += 64) acc += ld_f(wrow, c) * xs[c];
    }
    return acc;
}

// Two rows against one LDS vector, with the loads of four 512-element steps of both rows (eight 16-byte loads a lane) issued
// before the first product: a wave alone then keeps 8 KB in flight instead of waiting out one load's latency per step.
template <typename A, bool VEC>
__device__ __forceinline__ void lane_dot2(const A* __restrict__ ra, const A* __restrict__ rb, const float* __restrict__ xs, int n, int lane,
                                          float& out_a, float& out_b) {
    float a = 0.f, b = 0.f;
    if constexpr (VEC) {
        typedef A vec8 __attribute__((ext_vector_type(8)));
        int c = lane * 8;
        for (; c + 1536 < n; c += 2048) {
            vec8 va[4], vb[4];
#pragma unroll
            for (int s = 0; s < 4; ++s) {
                va[s] = *reinterpret_cast<const vec8*>(ra + c + 512 * s);
                vb[s] = *reinterpret_cast<const vec8*>(rb + c + 512 * s);
            }
#pragma unroll
            for (int s = 0; s < 4; ++s) {
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    const float x = xs[c + 512 * s + i];
                    a += (float)va[s][i] * x;
                    b += (float)vb[s][i] * x;
                }
            }
        }
        for (; c < n; c += 512) {
            const vec8 va = *reinterpret_cast<const vec8*>(ra + c);
            const vec8 vb = *reinterpret_cast<const vec8*>(rb + c);
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const float x = xs[c + i];
                a += (float)va[i] * x;
                b += (float)vb[i] * x;
            }
        }
    } else {
        for (int c = lane; c < n; c += 64) {
            const float x = xs[c];
            a += ld_f(ra, c) * x;
            b += ld_f(rb, c) * x;
        }
    }
    out_a = a;
    out_b = b;
}

constexpr int MOE_ROWS = 32;      // weight rows per workgroup (8 per wave)

template <typename A, bool VEC>
__global__ __launch_bounds__(256) void moe_rows_up_kernel(const A* __restrict__ h, int64_t h_stride, const int32_t* __restrict__ idx,
                                                         const float* __restrict__ wts, int top, const A* __restrict__ w_gu, float limit,
                                                         float alpha, float shift, int weight_out, float* __restrict__ y, int width, int ff) {
    extern __shared__ float sm[];      // the scaled input (width)
    const int64_t t = blockIdx.z;
    const int k = blockIdx.y;
    const int e = idx[t * top + k];
    const float wt = weight_out ? 1.0f : wts[t * top + k];
    for (int c = threadIdx.x; c < width; c += 256) sm[c] = (float)(A)(wt * ld_f(h, t * h_stride + c));
    __syncthreads();
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const A* wg = w_gu + (int64_t)e * 2 * ff * width;
    float g[MOE_ROWS / 4], u[MOE_ROWS / 4];
#pragma unroll
    for (int i = 0; i < MOE_ROWS / 4; ++i) {         // all rows' loads in flight before the first reduction
        const int j = blockIdx.x * MOE_ROWS + wave * (MOE_ROWS / 4) + i;
        const int jc = j < ff ? j : ff - 1;
        lane_dot2<A, VEC>(wg + (int64_t)jc * width, wg + (int64_t)(ff + jc) * width, sm, width, lane, g[i], u[i]);
    }
#pragma unroll
    for (int i = 0; i < MOE_ROWS / 4; ++i) {
        const int j = blockIdx.x * MOE_ROWS + wave * (MOE_ROWS / 4) + i;
        const float gs = wave_sum(g[i]), us = wave_sum(u[i]);
        if (lane == 0 && j < ff) y[(t * top + k) * ff + j] = (float)(A)glu_act((float)(A)gs, (float)(A)us, limit, alpha, shift);
    }
}

template <typename A, bool VEC>
__global__ __launch_bounds__(256) void moe_rows_down_kernel(const float* __restrict__ y, const int32_t* __restrict__ idx,
                                                           const float* __restrict__ wts, int top, int weight_out,
                                                           const A* __restrict__ w_d, A* __restrict__ out, int width, int ff) {
    extern __shared__ float sm[];      // one choice's hidden activations (ff)
    const int64_t t = blockIdx.y;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    float o[MOE_ROWS / 4];
#pragma unroll
    for (int i = 0; i < MOE_ROWS / 4; ++i) o[i] = 0.f;
    for (int k = 0; k < top; ++k) {
        __syncthreads();
        for (int j = threadIdx.x; j < ff; j += 256) sm[j] = y[(t * top + k) * ff + j];
        __syncthreads();
        const A* wd = w_d + (int64_t)idx[t * top + k] * width * ff;
        float part[MOE_ROWS / 4];
#pragma unroll
        for (int i = 0; i < MOE_ROWS / 4; i += 2) {
            const int c = blockIdx.x * MOE_ROWS + wave * (MOE_ROWS / 4) + i;
            lane_dot2<A, VEC>(wd + (int64_t)(c < width ? c : width - 1) * ff, wd + (int64_t)(c + 1 < width ? c + 1 : width - 1) * ff, sm, ff, lane,
                              part[i], part[i + 1]);
        }
        const float wo = weight_out ? wts[t * top + k] : 1.0f;
#pragma unroll
        for (int i = 0; i < MOE_ROWS / 4; ++i) o[i] += wo * (float)(A)wave_sum(part[i]);
    }
#pragma unroll
    for (int i = 0; i < MOE_ROWS / 4; ++i) {
        const int c = blockIdx.x * MOE_ROWS + wave * (MOE_ROWS / 4) + i;
        if (c < width && lane == 0) st_f(out, t * (int64_t)width + c, o[i]);
    }
}

// ---- a step of few tokens on the matrix cores (16-bit formats) -------------------------------------------------------------------
// The experts' weights are the bytes that count, and tokens share experts: a workgroup takes 16 weight rows of ONE expert and all (token,
// choice) pairs that chose it, 16 at a time, so a weight is read once for them.  Its four waves share the depth in blocks of 128 (every
// fourth block each): per 32 of them one v_mfma_f32_16x16x32 takes 16 rows (operand A: lane (row, quarter) loads 16 bytes of its row) against
// 16 pairs (operand B: the same of the pair's input), the loads of a block in flight together; the waves' sums meet in LDS in one
// order, so a pair's result does not depend on the batch.  Three launches: hidden activations per pair, output rows per pair, and the sum
// over a token's choices.
typedef __attribute__((ext_vector_type(8))) __bf16 moe_bf16x8;
typedef __attribute__((ext_vector_type(8))) _Float16 moe_f16x8;
template <typename A> __device__ __forceinline__ nvx_f32x4 moe_mfma32(nvx_u32x4 a, nvx_u32x4 b, nvx_f32x4 c) {
    if constexpr (__is_same(A, __bf16))
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(moe_bf16x8, a), __builtin_bit_cast(moe_bf16x8, b), c, 0, 0, 0);
    else
        return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(moe_f16x8, a), __builtin_bit_cast(moe_f16x8, b), c, 0, 0, 0);
}
constexpr int MT_PAD = 17;       // floats per row of a 16 x 16 tile of partial sums in LDS

// the pairs of expert e in their order -> list; returns how many (the same in every thread)
__device__ __forceinline__ int pairs_of_expert(const int32_t* __restrict__ idx, int n_pairs, int e, int* list) {
    __shared__ int wave_n[4];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    int base = 0;
    for (int r0 = 0; r0 < n_pairs; r0 += 256) {
        const int r = r0 + threadIdx.x;
        const bool mine = r < n_pairs && idx[r] == e;
        const unsigned long long mask = __ballot(mine);
        if (lane == 0) wave_n[wave] = __popcll(mask);
        __syncthreads();
        int at = base;
        for (int w = 0; w < wave; ++w) at += wave_n[w];
        if (mine) list[at + __popcll(mask & ((1ull << lane) - 1ull))] = r;
        base += wave_n[0] + wave_n[1] + wave_n[2] + wave_n[3];
        __syncthreads();
    }
    return base;
}

// sums of NM row tiles (rows of `a[m]` at the lane's row) against one tile of inputs at `b`, this wave's blocks of the depth `n`
template <typename A, int NM>
__device__ __forceinline__ void moe_tile_sums(const A* const (&a)[NM], const A* __restrict__ b, float b_mul, bool scaled, int n, int wave, int g, nvx_f32x4 (&acc)[NM]) {
    const nvx_u32x4 none = {0u, 0u, 0u, 0u};
    for (int k0 = wave * 128; k0 < n; k0 += 512) {
        nvx_u32x4 av[NM][4], bv[4];
#pragma unroll
        for (int s = 0; s < 4; ++s) {
            const int k = k0 + 32 * s + 8 * g;
            const bool in = k < n;                     // (n is a multiple of eight)
#pragma unroll
            for (int m = 0; m < NM; ++m) av[m][s] = in ? *reinterpret_cast<const nvx_u32x4*>(a[m] + k) : none;
            bv[s] = in ? *reinterpret_cast<const nvx_u32x4*>(b + k) : none;
        }
        if (scaled) {
            typedef A vec8 __attribute__((ext_vector_type(8)));
#pragma unroll
            for (int s = 0; s < 4; ++s) {
                vec8 v = __builtin_bit_cast(vec8, bv[s]);
#pragma unroll
                for (int i = 0; i < 8; ++i) v[i] = (A)(b_mul * (float)v[i]);
                bv[s] = __builtin_bit_cast(nvx_u32x4, v);
            }
        }
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int m = 0; m < NM; ++m) acc[m] = moe_mfma32<A>(av[m][s], bv[s], acc[m]);
    }
}

template <typename A>
__global__ __launch_bounds__(256) void moe_tile_up_kernel(const A* __restrict__ h, int64_t h_stride, const int32_t* __restrict__ idx,
                                                         const float* __restrict__ wts, int top, int n_pairs, const A* __restrict__ w_gu, float limit,
                                                         float alpha, float shift, int weight_out, A* __restrict__ y, int width, int ff) {
    extern __shared__ int list[];                      // n_pairs
    __shared__ float part[4][2][16 * MT_PAD];
    const int e = blockIdx.y, j0 = blockIdx.x * 16;
    const int count = pairs_of_expert(idx, n_pairs, e, list);
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const int row = j0 + c < ff ? j0 + c : ff - 1;
    const A* const rows[2] = {w_gu + ((int64_t)e * 2 * ff + row) * width, w_gu + ((int64_t)e * 2 * ff + ff + row) * width};
    for (int m0 = 0; m0 < count; m0 += 16) {
        const int pair = list[m0 + c < count ? m0 + c : count - 1];
        nvx_f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
        moe_tile_sums<A, 2>(rows, h + (int64_t)(pair / top) * h_stride, weight_out ? 1.0f : wts[pair], !weight_out, width, wave, g, acc);
#pragma unroll
        for (int m = 0; m < 2; ++m)
#pragma unroll
            for (int r = 0; r < 4; ++r) part[wave][m][(4 * g + r) * MT_PAD + c] = acc[m][r];      // (row 4 g + r, pair c)
        __syncthreads();
        const int rr = threadIdx.x & 15, cc = threadIdx.x >> 4, at = rr * MT_PAD + cc;
        if (m0 + cc < count && j0 + rr < ff) {
            const float gs = part[0][0][at] + part[1][0][at] + part[2][0][at] + part[3][0][at];
            const float us = part[0][1][at] + part[1][1][at] + part[2][1][at] + part[3][1][at];
            y[(int64_t)list[m0 + cc] * ff + j0 + rr] = (A)glu_act((float)(A)gs, (float)(A)us, limit, alpha, shift);
        }
        __syncthreads();
    }
}

template <typename A>
__global__ __launch_bounds__(256) void moe_tile_down_kernel(const A* __restrict__ y, const int32_t* __restrict__ idx, int n_pairs,
                                                           const A* __restrict__ w_d, float* __restrict__ o, int width, int ff) {
    extern __shared__ int list[];                      // n_pairs
    __shared__ float part[4][16 * MT_PAD];
    const int e = blockIdx.y, j0 = blockIdx.x * 16;
    const int count = pairs_of_expert(idx, n_pairs, e, list);
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const int row = j0 + c < width ? j0 + c : width - 1;
    const A* const rows[1] = {w_d + ((int64_t)e * width + row) * ff};
    for (int m0 = 0; m0 < count; m0 += 16) {
        const int pair = list[m0 + c < count ? m0 + c : count - 1];
        nvx_f32x4 acc[1] = {{0.f, 0.f, 0.f, 0.f}};
        moe_tile_sums<A, 1>(rows, y + (int64_t)pair * ff, 1.0f, false, ff, wave, g, acc);
#pragma unroll
        for (int r = 0; r < 4; ++r) part[wave][(4 * g + r) * MT_PAD + c] = acc[0][r];
        __syncthreads();
        const int rr = threadIdx.x & 15, cc = threadIdx.x >> 4, at = rr * MT_PAD + cc;
        if (m0 + cc < count && j0 + rr < width)
            o[(int64_t)list[m0 + cc] * width + j0 + rr] = (float)(A)(part[0][at] + part[1][at] + part[2][at] + part[3][at]);
        __syncthreads();
    }
}

// out[t] = sum over a token's choices of (weight_out ? wts : 1) * o[pair]
template <typename A>
__global__ __launch_bounds__(256) void moe_pair_sum_kernel(const float* __restrict__ o, const float* __restrict__ wts, int top, int weight_out,
                                                          A* __restrict__ out, int width) {
    const int64_t t = blockIdx.y;
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= width) return;
    float v = 0.f;
    for (int k = 0; k < top; ++k) v += (weight_out ? wts[t * top + k] : 1.0f) * o[(t * top + k) * width + c];
    st_f(out, t * (int64_t)width + c, v);
}

// xs[dst[r]] = wts[r] * h[r / top]  for every (token, choice) pair r: the experts' inputs in expert order
template <typename A>
__global__ __launch_bounds__(256) void moe_scatter_rows_kernel(const A* __restrict__ h, int64_t h_stride, const float* __restrict__ wts,
                                                              const int64_t* __restrict__ dst, int top, A* __restrict__ xs, int width) {
    const int64_t r = blockIdx.x;
    const int64_t t = r / top;
    const float wt = wts ? wts[r] : 1.0f;
    A* o = xs + dst[r] * (int64_t)width;
    for (int c = threadIdx.x; c < width; c += 256) st_f(o, c, wt * ld_f(h, t * h_stride + c));
}

// gelu_tanh(g) u
__device__ __forceinline__ float gelu_glu_act(float g, float u) {
    return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g))) * u;
}

// y[r][j] = act(gu[r][j], gu[r][ff + j]) (times sigmoid(row_gate[r]) if given); GELU: gelu_tanh(g) u, the three constants are not read
template <typename A, bool GELU>
__global__ __launch_bounds__(256) void moe_glu_kernel(const A* __restrict__ gu, int64_t gu_stride, A* __restrict__ y, int64_t y_stride, float limit,
                                                     float alpha, float shift, const float* __restrict__ row_gate, int64_t row_gate_stride,
                                                     int64_t rows, int ff) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < rows * ff; i += (int64_t)gridDim.x * 256) {
        const int64_t r = i / ff;
        const int j = (int)(i % ff);
        const float g = ld_f(gu, r * gu_stride + j), u = ld_f(gu, r * gu_stride + ff + j);
        const float v = GELU ? gelu_glu_act(g, u) : glu_act(g, u, limit, alpha, shift);
        st_f(y, r * y_stride + j, row_gate ? v * sigmoid_f(row_gate[r * row_gate_stride]) : v);
    }
}

// The same for 16-bit formats, eight neighbouring entries of a row per thread as one 16-byte load of each half and one store
// (ff8 = ff / 8; rows start on 16-byte borders).
template <typename A, bool GELU>
__global__ __launch_bounds__(256) void moe_glu_vec8_kernel(const A* __restrict__ gu, int64_t gu_stride, A* __restrict__ y, int64_t y_stride,
                                                          float limit, float alpha, float shift, const float* __restrict__ row_gate,
                                                          int64_t row_gate_stride, int64_t rows, int ff8) {
    union Pack { uint4 v; A a[8]; };
    const int64_t n = rows * ff8;
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
        const int64_t r = i / ff8;
        const int64_t j = (i - r * ff8) * 8;
        const A* row = gu + r * gu_stride;
        const float rg = row_gate ? sigmoid_f(row_gate[r * row_gate_stride]) : 1.0f;
        Pack g, u, o;
        g.v = *reinterpret_cast<const uint4*>(row + j);
        u.v = *reinterpret_cast<const uint4*>(row + (int64_t)ff8 * 8 + j);
#pragma unroll
        for (int k = 0; k < 8; ++k)
            o.a[k] = (A)(rg * (GELU ? gelu_glu_act((float)g.a[k], (float)u.a[k]) : glu_act((float)g.a[k], (float)u.a[k], limit, alpha, shift)));
        *reinterpret_cast<uint4*>(y + r * y_stride + j) = o.v;
    }
}

// out[t] = sum_k wts[t * top + k] * ys[dst[t * top + k]]   (wts == null: ones)
template <typename A>
__global__ __launch_bounds__(256) void moe_gather_rows_kernel(const A* __restrict__ ys, const int64_t* __restrict__ dst,
                                                             const float* __restrict__ wts, int top, A* __restrict__ out, int width) {
    const int64_t t = blockIdx.x;
    for (int c = threadIdx.x; c < width; c += 256) {
        float o = 0.f;
        for (int k = 0; k < top; ++k) o += (wts ? wts[t * top + k] : 1.0f) * ld_f(ys, dst[t * top + k] * (int64_t)width + c);
        st_f(out, t * (int64_t)width + c, o);
    }
}


// Expert order of the (token, choice) pairs: dst[r] = position of pair r when the pairs are sorted by expert, pairs of one
// expert keeping their order; counts[e] = pairs of expert e.  One workgroup: a thread takes a contiguous run of pairs, counts
// them per expert into LDS (cnt[e][thread]), the prefix sums over (expert, thread) give every thread its first position per
// expert, and a second walk over the same run hands the positions out.  n_exp * 256 counters must fit LDS.
__global__ __launch_bounds__(256) void moe_order_kernel(const int32_t* __restrict__ idx, int64_t n, int n_exp, int64_t* __restrict__ dst,
                                                       int32_t* __restrict__ counts) {
    extern __shared__ int cnt[];      // n_exp rows of 256, then n_exp bases
    int* base = cnt + n_exp * 256;
    const int tid = threadIdx.x;
    const int64_t per = (n + 255) / 256, lo = tid * per, hi = lo + per < n ? lo + per : n;
    for (int e = 0; e < n_exp; ++e) cnt[e * 256 + tid] = 0;
    for (int64_t r = lo; r < hi; ++r) {
        const int e = idx[r];
        if (e >= 0 && e < n_exp) cnt[e * 256 + tid] += 1;
    }
    __syncthreads();
    for (int e = tid; e < n_exp; e += 256) {       // a thread per expert: exclusive prefix over the threads' counts
        int run = 0;
        for (int j = 0; j < 256; ++j) { const int c = cnt[e * 256 + j]; cnt[e * 256 + j] = run; run += c; }
        base[e] = run;
        counts[e] = run;
    }
    __syncthreads();
    if (tid == 0) {
        int run = 0;
        for (int e = 0; e < n_exp; ++e) { const int c = base[e]; base[e] = run; run += c; }
    }
    __syncthreads();
    for (int64_t r = lo; r < hi; ++r) {
        const int e = idx[r];
        if (e >= 0 && e < n_exp) dst[r] = base[e] + cnt[e * 256 + tid]++;
    }
}

}  // namespace NVX_NS

using namespace NVX_NS;

extern "C" int64_t nvx_moe_order_max_experts(void) { return (64 * 1024 / 4) / 257; }

extern "C" int nvx_moe_order(const int32_t* idx, int64_t n, int64_t n_exp, int64_t* dst, int32_t* counts, nvx_stream_t stream) {
    NVX_REQUIRE(n >= 0 && n < (1ll << 31) && n_exp > 0 && n_exp <= nvx_moe_order_max_experts(), NVX_EINVAL,
                "nvx_moe_order: bad sizes (the experts' counters must fit LDS)");
    NVX_REQUIRE(idx && dst && counts, NVX_EINVAL, "nvx_moe_order: null pointer");
    hipLaunchKernelGGL(moe_order_kernel, dim3(1), dim3(256), (size_t)(n_exp * 257) * sizeof(int), (hipStream_t)stream, idx, n, (int)n_exp, dst,
                       counts);
    return nvx_check_launch("nvx_moe_order");
}

extern "C" int nvx_moe_route(const float* logits, int64_t n_tok, int64_t n_exp, int64_t top, int32_t* idx, float* wts, nvx_stream_t stream) {
    NVX_REQUIRE(n_tok >= 0 && n_exp > 0 && n_exp < (1 << 20) && top > 0 && top <= n_exp, NVX_EINVAL, "nvx_moe_route: bad sizes");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(logits && idx && wts, NVX_EINVAL, "nvx_moe_route: null pointer");
    hipLaunchKernelGGL(moe_route_kernel, dim3((unsigned)((n_tok + 255) / 256)), dim3(256), 0, (hipStream_t)stream, logits, (int)n_exp, (int)top,
                       idx, wts, n_tok);
    return nvx_check_launch("nvx_moe_route");
}

extern "C" int nvx_moe_route_softmax(const float* logits, int64_t logits_stride, int64_t n_tok, int64_t n_exp, int64_t top, int64_t n_groups, int64_t keep_groups,
                                     float norm_eps, int32_t* idx, float* wts, nvx_stream_t stream) {
    NVX_REQUIRE(n_tok >= 0 && n_exp > 0 && n_exp < (1 << 20) && top > 0 && top <= n_exp, NVX_EINVAL, "nvx_moe_route_softmax: bad sizes");
    NVX_REQUIRE(n_groups >= 0 && n_groups <= 256 && (n_groups <= 1 || (n_exp % n_groups == 0 && keep_groups >= 1 && keep_groups <= n_groups &&
                                                                      keep_groups * (n_exp / n_groups) >= top)),
                NVX_EINVAL, "nvx_moe_route_softmax: groups must divide the experts (at most 256 groups) and the kept groups must hold `top` experts");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(logits && idx && wts && logits_stride >= n_exp, NVX_EINVAL, "nvx_moe_route_softmax: null pointer or row stride");
    if ((n_groups <= 1 || keep_groups == n_groups) && n_exp <= 1024 && top <= 64) {
        hipLaunchKernelGGL(moe_route_softmax_wave_kernel, dim3((unsigned)((n_tok + 3) / 4)), dim3(256), 0, (hipStream_t)stream, logits, logits_stride, (int)n_exp,
                           (int)top, norm_eps, idx, wts, n_tok);
        return nvx_check_launch("nvx_moe_route_softmax");
    }
    hipLaunchKernelGGL(moe_route_softmax_kernel, dim3((unsigned)((n_tok + 255) / 256)), dim3(256), 0, (hipStream_t)stream, logits, logits_stride, (int)n_exp,
                       (int)top, (int)n_groups, (int)keep_groups, norm_eps, idx, wts, n_tok);
    return nvx_check_launch("nvx_moe_route_softmax");
}

extern "C" int nvx_moe_route_sigmoid(const float* logits, const float* correction, int64_t n_tok, int64_t n_exp, int64_t top, int64_t n_groups,
                                     int64_t keep_groups, float w_scale, int32_t* idx, float* wts, nvx_stream_t stream) {
    NVX_REQUIRE(n_tok >= 0 && n_exp > 0 && n_exp <= 1024 && top > 0 && top <= n_exp, NVX_EINVAL, "nvx_moe_route_sigmoid: bad sizes (at most 1024 experts)");
    NVX_REQUIRE(n_groups >= 0 && (n_groups <= 1 || (n_exp % n_groups == 0 && keep_groups >= 1 && keep_groups <= n_groups &&
                                                   keep_groups * (n_exp / n_groups) >= top)),
                NVX_EINVAL, "nvx_moe_route_sigmoid: groups must divide the experts and the kept groups must hold `top` experts");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(logits && correction && idx && wts, NVX_EINVAL, "nvx_moe_route_sigmoid: null pointer");
    const size_t lds = 4 * (size_t)(n_exp + (n_groups > 1 ? n_groups : 0)) * sizeof(float);
    hipLaunchKernelGGL(moe_route_sigmoid_kernel, dim3((unsigned)((n_tok + 3) / 4)), dim3(256), lds, (hipStream_t)stream, logits, correction, (int)n_exp,
                       (int)top, (int)n_groups, (int)keep_groups, w_scale, idx, wts, n_tok);
    return nvx_check_launch("nvx_moe_route_sigmoid");
}

extern "C" int64_t nvx_moe_expert_rows_max_width(int64_t ff) {
    return ff > 0 && ff <= 12288 ? 12288 : 0;      // a row of either size waits in LDS as float32
}

template <typename A>
static void launch_moe_rows(const void* h, int64_t h_stride, const int32_t* idx, const float* wts, int top, const void* w_gu, const void* w_d,
                            int n_exp, float limit, float alpha, float shift, int weight_out, float* ws, void* out, int64_t n_tok, int width, int ff,
                            hipStream_t s) {
    const bool vec = sizeof(A) == 2 && width % 8 == 0 && ff % 8 == 0 && nvx_aligned16(w_gu) && nvx_aligned16(w_d);
    if constexpr (sizeof(A) == 2) {
        const int64_t pairs = n_tok * top;
        if (vec && h_stride % 8 == 0 && nvx_aligned16(h) && nvx_aligned16(ws) && pairs <= 8192 && n_exp <= 65535) {
            A* y = reinterpret_cast<A*>(ws);
            float* o = ws + pairs * ff;
            const size_t lds = (size_t)pairs * sizeof(int);
            hipLaunchKernelGGL(moe_tile_up_kernel<A>, dim3((unsigned)((ff + 15) / 16), (unsigned)n_exp), dim3(256), lds, s, (const A*)h, h_stride, idx, wts, top,
                               (int)pairs, (const A*)w_gu, limit, alpha, shift, weight_out, y, width, ff);
            hipLaunchKernelGGL(moe_tile_down_kernel<A>, dim3((unsigned)((width + 15) / 16), (unsigned)n_exp), dim3(256), lds, s, (const A*)y, idx, (int)pairs,
                               (const A*)w_d, o, width, ff);
            hipLaunchKernelGGL(moe_pair_sum_kernel<A>, dim3((unsigned)((width + 255) / 256), (unsigned)n_tok), dim3(256), 0, s, (const float*)o, wts, top, weight_out,
                               (A*)out, width);
            return;
        }
    }
    const dim3 up((unsigned)((ff + MOE_ROWS - 1) / MOE_ROWS), (unsigned)top, (unsigned)n_tok);
    const dim3 down((unsigned)((width + MOE_ROWS - 1) / MOE_ROWS), (unsigned)n_tok);
    if (vec) {
        hipLaunchKernelGGL((moe_rows_up_kernel<A, true>), up, dim3(256), (size_t)width * sizeof(float), s, (const A*)h, h_stride, idx, wts, top,
                           (const A*)w_gu, limit, alpha, shift, weight_out, ws, width, ff);
        hipLaunchKernelGGL((moe_rows_down_kernel<A, true>), down, dim3(256), (size_t)ff * sizeof(float), s, (const float*)ws, idx, wts, top,
                           weight_out, (const A*)w_d, (A*)out, width, ff);
    } else {
        hipLaunchKernelGGL((moe_rows_up_kernel<A, false>), up, dim3(256), (size_t)width * sizeof(float), s, (const A*)h, h_stride, idx, wts, top,
                           (const A*)w_gu, limit, alpha, shift, weight_out, ws, width, ff);
        hipLaunchKernelGGL((moe_rows_down_kernel<A, false>), down, dim3(256), (size_t)ff * sizeof(float), s, (const float*)ws, idx, wts, top,
                           weight_out, (const A*)w_d, (A*)out, width, ff);
    }
}

extern "C" int nvx_moe_expert_rows(const void* h, int64_t h_stride, int fmt, const int32_t* idx, const float* wts, int64_t top,
                                   const void* w_gu, const void* w_d, int64_t n_exp, float limit, float alpha, float shift, int weight_out,
                                   float* ws, void* out, int64_t n_tok, int64_t width, int64_t ff, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2, NVX_EINVAL, "nvx_moe_expert_rows: fmt must be 0, 1 or 2");
    NVX_REQUIRE(n_tok >= 0 && n_tok <= 65535 && top > 0 && top <= 65535 && n_exp > 0 && n_exp < (1 << 20) && width > 0 && ff > 0 && h_stride >= width, NVX_EINVAL,
                "nvx_moe_expert_rows: bad sizes (at most 65535 tokens a step)");
    NVX_REQUIRE(width <= nvx_moe_expert_rows_max_width(ff), NVX_EUNSUPPORTED, "nvx_moe_expert_rows: a row or the hidden size does not fit LDS");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(h && idx && wts && w_gu && w_d && ws && out, NVX_EINVAL, "nvx_moe_expert_rows: null pointer");
    NVX_FMT_CALL(fmt, launch_moe_rows<A_>(h, h_stride, idx, wts, (int)top, w_gu, w_d, (int)n_exp, limit, alpha, shift, weight_out, ws, out, n_tok, (int)width, (int)ff,
                                          (hipStream_t)stream));
    return nvx_check_launch("nvx_moe_expert_rows");
}

extern "C" int nvx_moe_scatter_rows(const void* h, int64_t h_stride, int fmt, const float* wts, const int64_t* dst, int64_t top, void* xs,
                                    int64_t n_tok, int64_t width, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2 && n_tok >= 0 && top > 0 && width > 0 && h_stride >= width && n_tok * top < (1ll << 31), NVX_EINVAL,
                "nvx_moe_scatter_rows: bad arguments");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(h && dst && xs, NVX_EINVAL, "nvx_moe_scatter_rows: null pointer");
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(moe_scatter_rows_kernel<A_>, dim3((unsigned)(n_tok * top)), dim3(256), 0, (hipStream_t)stream,
                                         (const A_*)h, h_stride, wts, dst, (int)top, (A_*)xs, (int)width));
    return nvx_check_launch("nvx_moe_scatter_rows");
}

// gu rows of [gate | up] gu_stride apart, y rows y_stride apart; row_gate: one logit per row, rows row_gate_stride apart (null: no gate)
template <bool GELU>
static int launch_glu(const void* gu, int64_t gu_stride, int fmt, float limit, float alpha, float shift, const float* row_gate, int64_t row_gate_stride,
                      void* y, int64_t y_stride, int64_t rows, int64_t ff, hipStream_t s, const char* name) {
    if (fmt != 2 && ff % 8 == 0 && gu_stride % 8 == 0 && y_stride % 8 == 0 && nvx_aligned16(gu) && nvx_aligned16(y)) {
        int64_t blocks = (rows * (ff / 8) + 255) / 256;
        if (blocks > 256 * 64) blocks = 256 * 64;
        if (fmt == 0)
            hipLaunchKernelGGL((moe_glu_vec8_kernel<__bf16, GELU>), dim3((unsigned)blocks), dim3(256), 0, s, (const __bf16*)gu, gu_stride, (__bf16*)y,
                               y_stride, limit, alpha, shift, row_gate, row_gate_stride, rows, (int)(ff / 8));
        else
            hipLaunchKernelGGL((moe_glu_vec8_kernel<_Float16, GELU>), dim3((unsigned)blocks), dim3(256), 0, s, (const _Float16*)gu, gu_stride,
                               (_Float16*)y, y_stride, limit, alpha, shift, row_gate, row_gate_stride, rows, (int)(ff / 8));
        return nvx_check_launch(name);
    }
    int64_t blocks = (rows * ff + 255) / 256;
    if (blocks > 256 * 64) blocks = 256 * 64;
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL((moe_glu_kernel<A_, GELU>), dim3((unsigned)blocks), dim3(256), 0, s, (const A_*)gu, gu_stride, (A_*)y, y_stride,
                                         limit, alpha, shift, row_gate, row_gate_stride, rows, (int)ff));
    return nvx_check_launch(name);
}

extern "C" int nvx_moe_glu(const void* gu, int64_t gu_stride, int fmt, float limit, float alpha, float shift, const float* row_gate,
                           int64_t row_gate_stride, void* y, int64_t y_stride, int64_t rows, int64_t ff, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2 && rows >= 0 && ff > 0 && gu_stride >= 2 * ff && y_stride >= ff && (!row_gate || row_gate_stride >= 1), NVX_EINVAL,
                "nvx_moe_glu: bad arguments");
    if (rows == 0) return NVX_OK;
    NVX_REQUIRE(gu && y, NVX_EINVAL, "nvx_moe_glu: null pointer");
    return launch_glu<false>(gu, gu_stride, fmt, limit, alpha, shift, row_gate, row_gate_stride, y, y_stride, rows, ff, (hipStream_t)stream, "nvx_moe_glu");
}

extern "C" int nvx_gelu_glu(const void* gu, int fmt, void* y, int64_t rows, int64_t ff, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2 && rows >= 0 && ff > 0, NVX_EINVAL, "nvx_gelu_glu: bad arguments");
    if (rows == 0) return NVX_OK;
    NVX_REQUIRE(gu && y, NVX_EINVAL, "nvx_gelu_glu: null pointer");
    return launch_glu<true>(gu, 2 * ff, fmt, 0.f, 0.f, 0.f, nullptr, 0, y, ff, rows, ff, (hipStream_t)stream, "nvx_gelu_glu");
}

extern "C" int nvx_moe_gather_rows(const void* ys, int fmt, const int64_t* dst, const float* wts, int64_t top, void* out, int64_t n_tok,
                                   int64_t width, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2 && n_tok >= 0 && n_tok < (1ll << 31) && top > 0 && width > 0, NVX_EINVAL, "nvx_moe_gather_rows: bad arguments");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(ys && dst && out, NVX_EINVAL, "nvx_moe_gather_rows: null pointer");
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(moe_gather_rows_kernel<A_>, dim3((unsigned)n_tok), dim3(256), 0, (hipStream_t)stream, (const A_*)ys, dst,
                                         wts, (int)top, (A_*)out, (int)width));
    return nvx_check_launch("nvx_moe_gather_rows");
}
