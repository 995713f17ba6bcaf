// What queries, keys and values of an attention pass between their projection and the cache when a short causal convolution stands there:
//   - nvx_turn_table: cos and sin of every token's rotation angles, once per step for all layers (several rotations share a row);
//   - nvx_conv_attn_prep: convolution over time per channel of q, k and v; rotation of the first part of every query and key head; query and
//     key heads divided by their root mean square; keys and values scattered into the cache.  One launch, the convolved rows stay in
//     registers; the convolution's last inputs are kept per sequence.
// All of it is float32 between the projection's rows and what is stored.  A batch is ragged (see seq_mix.hip).
#include "fmt_dev.h"

namespace NVX_NS {

// out[t] = [cos(positions[t] * freq[m]) (n) | sin (n)]
__global__ __launch_bounds__(256) void turn_table_kernel(const int64_t* __restrict__ positions, const double* __restrict__ freq, int n,
                                                        float* __restrict__ out, int64_t total) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= total) return;
    const int64_t t = i / n;
    const int m = (int)(i - t * n);
    float c, s;
    turn_of((double)positions[t] * freq[m], c, s);
    out[t * 2 * n + m] = c;
    out[t * 2 * n + n + m] = s;
}

// What both forms of the kernel read and write.  A row of x holds q, k and v side by side from column col0 on; channels are counted from
// there, heads * dim + kv_heads * (dim + vdim) of them.  w (taps_n, channels): row j multiplies the input taps_n - 1 - j tokens back.
template <typename A> struct ConvPrep {
    const A* x; int64_t x_stride;
    const float* w; int taps_n;
    float* state;                            // (slots, taps_n - 1, channels)
    const int32_t *tok_seq, *qo_indptr, *state_slot;
    const int64_t* pos0;
    TurnRows turn; int half;
    int norm; float eps;
    const int64_t* slots;
    A *q_out, *k_cache, *v_cache;
    int64_t n_tok;
    int heads, kv_heads, dim, vdim;
    __device__ __forceinline__ int per() const { return heads + 2 * kv_heads; }
    __device__ __forceinline__ int channels() const { return heads * dim + kv_heads * (dim + vdim); }
    // first channel of part `hd` (query heads, then key heads, then value heads)
    __device__ __forceinline__ int first(int hd) const {
        return hd < heads + kv_heads ? hd * dim : (heads + kv_heads) * dim + (hd - heads - kv_heads) * vdim;
    }
    // where token t's part goes (null: nowhere, a padding row's keys and values)
    __device__ __forceinline__ A* target(int64_t t, int64_t slot, int hd) const {
        if (hd < heads) return q_out + (t * heads + hd) * dim;
        if (slot < 0) return nullptr;
        if (hd < heads + kv_heads) return k_cache + (slot * kv_heads + (hd - heads)) * dim;
        return v_cache + (slot * kv_heads + (hd - heads - kv_heads)) * vdim;
    }
};

// Any sizes: a wave per (token, part), the convolved row waits in LDS.
template <typename A>
__global__ __launch_bounds__(256) void conv_attn_prep_kernel(ConvPrep<A> p, int64_t n_items) {
    extern __shared__ float sm[];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int64_t item = (int64_t)blockIdx.x * 4 + wave;
    if (item >= n_items) return;             // (waves share nothing and meet no barrier)
    float* r = sm + wave * (p.dim > p.vdim ? p.dim : p.vdim);
    const int64_t t = item / p.per();
    const int hd = (int)(item % p.per());
    const bool turned = hd < p.heads + p.kv_heads;
    const int n = turned ? p.dim : p.vdim, c0 = p.first(hd), ch = p.channels(), hist_n = p.taps_n - 1;
    const int b = p.tok_seq ? p.tok_seq[t] : (int)t;
    const SeqSpan s = seq_span(b, p.qo_indptr, p.pos0, p.state_slot);
    const int64_t j = t - s.q0;
    const bool has_state = s.pos0 > 0 && s.slot >= 0;
    float ss = 0.f;
    for (int d = lane; d < n; d += 64) {
        float acc = 0.f;
        for (int i = 0; i < p.taps_n; ++i) {
            const int64_t src = j - (hist_n - i);
            float v = 0.f;
            if (src >= 0) v = ld_f(p.x, (s.q0 + src) * p.x_stride + c0 + d);
            else if (has_state) v = p.state[((int64_t)s.slot * hist_n + (hist_n + src)) * ch + c0 + d];
            acc += p.w[(int64_t)i * ch + c0 + d] * v;
        }
        r[d] = acc;
        ss += acc * acc;
    }
    // a rotation keeps the length of every pair, so the root mean square is that of the row before it
    const float rn = turned && p.norm ? 1.0f / sqrtf(wave_sum(ss) / (float)n + p.eps) : 1.0f;
    A* o = p.target(t, p.slots[t], hd);
    if (!o) return;
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
    const float* tr = p.turn.cos + t * p.turn.stride;
    for (int d = lane; d < n; d += 64) {
        float v = r[d];
        if (turned && d < 2 * p.half) {
            if (d < p.half) v = v * tr[d] - r[d + p.half] * tr[p.turn.sin_off + d];
            else v = v * tr[d - p.half] + r[d - p.half] * tr[p.turn.sin_off + d - p.half];
        }
        st_f(o, d, v * rn);
    }
}

// Sizes in multiples of eight, up to four taps: a part of a row per LPR neighbouring lanes of eight channels each.  A lane group walks
// RUN consecutive tokens with the taps and the last inputs in registers, so weights are read once for them and rows little more than once;
// everything of the walk is asked for before the first token is worked on.  Where another sequence begins, the history comes from
// that sequence.  With `own_tail` (one token per sequence) the lane also writes the new history back: no
// other lane touches its channels of that slot.
typedef float f4_any __attribute__((ext_vector_type(4), aligned(4)));       // four floats in one access, on any border of four bytes
__device__ __forceinline__ void load8(const float* __restrict__ src, float (&dst)[8]) {
    const f4_any a = *reinterpret_cast<const f4_any*>(src), b = *reinterpret_cast<const f4_any*>(src + 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) { dst[e] = a[e]; dst[4 + e] = b[e]; }
}
template <typename A, int LPR, int TAPS, int RUN>
__global__ __launch_bounds__(256) void conv_attn_prep_vec_kernel(ConvPrep<A> p, unsigned n_groups, int own_tail) {
    typedef A vec8 __attribute__((ext_vector_type(8)));
    constexpr int HN = TAPS - 1;
    const unsigned item = blockIdx.x * (256 / LPR) + threadIdx.x / LPR;
    const int l = threadIdx.x % LPR;
    const bool item_on = item < n_groups;
    const unsigned run_no = item_on ? item / (unsigned)p.per() : 0u;
    const int64_t t0 = (int64_t)run_no * RUN;
    const int hd = item_on ? (int)(item - run_no * p.per()) : 0;
    const bool turned = hd < p.heads + p.kv_heads;
    const int n = turned ? p.dim : p.vdim, ch = p.channels(), c0 = p.first(hd) + l * 8;
    const bool on = item_on && l * 8 < n;
    const bool rot_here = turned && l * 8 < 2 * p.half, low = l * 8 < p.half;
    const int partner = (threadIdx.x & 63) + (rot_here ? (low ? p.half / 8 : -(p.half / 8)) : 0), m0 = low ? l * 8 : l * 8 - p.half;
    float w[TAPS][8], hist[HN > 0 ? HN : 1][8];
#pragma unroll
    for (int i = 0; i < TAPS; ++i) load8(p.w + (int64_t)i * ch + (on ? c0 : 0), w[i]);      // (a lane without channels keeps channel 0's, unused)
    vec8 rows[RUN];
    int seqs[RUN];
    int64_t slots[RUN];
#pragma unroll
    for (int k = 0; k < RUN; ++k) {
        const int64_t t = t0 + k < p.n_tok ? t0 + k : p.n_tok - 1;
        seqs[k] = p.tok_seq ? p.tok_seq[t] : (int)t;
        slots[k] = p.slots[t];
        rows[k] = *reinterpret_cast<const vec8*>(p.x + t * p.x_stride + (on ? c0 : 0));
    }
    int last_b = -1;
    SeqSpan s{0, 0, 0, -1};
#pragma unroll
    for (int k = 0; k < RUN; ++k) {
        const int64_t t = t0 + k;
        const bool here = on && t < p.n_tok;
        float y[8], cur[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) { y[e] = 0.f; cur[e] = 0.f; }
        if (here) {
            const int b = seqs[k];
            if (b != last_b) {               // the first token of this walk, or of another sequence: its history
                last_b = b;
                s = seq_span(b, p.qo_indptr, p.pos0, p.state_slot);
                const bool has_state = s.pos0 > 0 && s.slot >= 0;
#pragma unroll
                for (int i = 0; i < HN; ++i) {
                    const int64_t src = t - s.q0 - HN + i;
                    if (src >= 0) {
                        const vec8 v = *reinterpret_cast<const vec8*>(p.x + (s.q0 + src) * p.x_stride + c0);
#pragma unroll
                        for (int e = 0; e < 8; ++e) hist[i][e] = (float)v[e];
                    } else if (has_state) {
                        load8(p.state + ((int64_t)s.slot * HN + HN + src) * ch + c0, hist[i]);
                    } else {
#pragma unroll
                        for (int e = 0; e < 8; ++e) hist[i][e] = 0.f;
                    }
                }
            }
            const vec8 v = rows[k];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                cur[e] = (float)v[e];
                float acc = 0.f;
#pragma unroll
                for (int i = 0; i < HN; ++i) acc += w[i][e] * hist[i][e];
                y[e] = acc + w[HN][e] * cur[e];
#pragma unroll
                for (int i = 0; i + 1 < HN; ++i) hist[i][e] = hist[i + 1][e];
                if (HN > 0) hist[HN > 0 ? HN - 1 : 0][e] = cur[e];
            }
            if (own_tail && HN > 0 && s.slot >= 0) {
#pragma unroll
                for (int i = 0; i < HN; ++i) {
                    float* st = p.state + ((int64_t)s.slot * HN + i) * ch + c0;
                    *reinterpret_cast<f4_any*>(st) = f4_any{hist[i][0], hist[i][1], hist[i][2], hist[i][3]};
                    *reinterpret_cast<f4_any*>(st + 4) = f4_any{hist[i][4], hist[i][5], hist[i][6], hist[i][7]};
                }
            }
        }
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += y[e] * y[e];
        const float sum = group_sum<LPR>(ss);          // (every lane of the wave takes part in the exchanges)
        const float rn = turned && p.norm ? 1.0f / sqrtf(sum / (float)n + p.eps) : 1.0f;
        float z[8];
        if (p.half) {
#pragma unroll
            for (int e = 0; e < 8; ++e) z[e] = __shfl(y[e], partner, 64);
        }
        if (!here) continue;
        if (p.half && rot_here) {
            const float* tr = p.turn.cos + t * p.turn.stride + m0;
            float c[8], sn[8];
            load8(tr, c);
            load8(tr + p.turn.sin_off, sn);
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] = low ? y[e] * c[e] - z[e] * sn[e] : y[e] * c[e] + z[e] * sn[e];
        }
        A* o = p.target(t, slots[k], hd);
        if (!o) continue;
        vec8 r;
#pragma unroll
        for (int e = 0; e < 8; ++e) r[e] = (A)(y[e] * rn);
        *reinterpret_cast<vec8*>(o + l * 8) = r;
    }
}

template <typename A> static void launch_conv_prep(const ConvPrep<A>& p, bool vec, int own_tail, hipStream_t st) {
    const int64_t per = p.heads + 2 * p.kv_heads;
    const int longest = p.dim > p.vdim ? p.dim : p.vdim;
    if (!vec) {
        const int64_t items = p.n_tok * per;
        hipLaunchKernelGGL(conv_attn_prep_kernel<A>, dim3((unsigned)((items + 3) / 4)), dim3(256), (size_t)(4 * longest) * sizeof(float), st, p, items);
        return;
    }
    const int lpr = longest <= 64 ? 8 : (longest <= 128 ? 16 : (longest <= 256 ? 32 : 64));
    const int run = p.qo_indptr && p.n_tok * per * lpr >= 256 * 1024 ? 4 : 1;      // (walks of four tokens where they leave workgroups enough)
    const int64_t groups = (p.n_tok + run - 1) / run * per;
    const dim3 grid((unsigned)((groups * lpr + 255) / 256));
#define NVX_CONV_T(LPR, T)                                                                                                                    \
    do {                                                                                                                                      \
        if (run == 4) hipLaunchKernelGGL((conv_attn_prep_vec_kernel<A, LPR, T, 4>), grid, dim3(256), 0, st, p, (unsigned)groups, own_tail);    \
        else hipLaunchKernelGGL((conv_attn_prep_vec_kernel<A, LPR, T, 1>), grid, dim3(256), 0, st, p, (unsigned)groups, own_tail);             \
    } while (0)
#define NVX_CONV(LPR)                                 \
    do {                                              \
        if (p.taps_n == 1) NVX_CONV_T(LPR, 1);        \
        else if (p.taps_n == 2) NVX_CONV_T(LPR, 2);   \
        else if (p.taps_n == 3) NVX_CONV_T(LPR, 3);   \
        else NVX_CONV_T(LPR, 4);                      \
    } while (0)
    if (lpr == 8) NVX_CONV(8);
    else if (lpr == 16) NVX_CONV(16);
    else if (lpr == 32) NVX_CONV(32);
    else NVX_CONV(64);
#undef NVX_CONV
#undef NVX_CONV_T
}

}  // namespace NVX_NS

using namespace NVX_NS;

extern "C" int nvx_turn_table(const int64_t* positions, const double* freq, int64_t n, float* out, int64_t n_tok, nvx_stream_t stream) {
    NVX_REQUIRE(n_tok >= 0 && n > 0 && n < (1 << 20) && n_tok * n < (1ll << 38), NVX_EINVAL, "nvx_turn_table: bad sizes");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(positions && freq && out, NVX_EINVAL, "nvx_turn_table: null pointer");
    const int64_t total = n_tok * n;
    hipLaunchKernelGGL(turn_table_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, (hipStream_t)stream, positions, freq, (int)n, out, total);
    return nvx_check_launch("nvx_turn_table");
}

extern "C" int nvx_conv_attn_prep(const void* x, int64_t x_stride, int fmt, const float* w, int taps_n, float* state, int64_t n_slots,
                                  const int32_t* tok_seq, const int32_t* qo_indptr, const int64_t* pos0, const int32_t* state_slot, const float* turn,
                                  int64_t turn_stride, int64_t turn_sin_off, int rot_dims, int norm, float eps, const int64_t* slots, void* q_out,
                                  void* k_cache, void* v_cache, int64_t n_tok, int64_t n_seq, int64_t heads, int64_t kv_heads, int64_t dim,
                                  int64_t vdim, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2, NVX_EINVAL, "nvx_conv_attn_prep: fmt must be 0, 1 or 2");
    NVX_REQUIRE(n_tok >= 0 && n_seq >= 0 && n_seq <= 65535 && heads > 0 && kv_heads > 0 && dim > 0 && dim <= 4096 && vdim > 0 && vdim <= 4096 &&
                    taps_n >= 1 && taps_n <= 64 && n_slots >= 0, NVX_EINVAL, "nvx_conv_attn_prep: bad sizes (heads of at most 4096, 1 to 64 taps)");
    const int64_t channels = heads * dim + kv_heads * (dim + vdim), per = heads + 2 * kv_heads;
    NVX_REQUIRE(channels < (1 << 30) && x_stride >= channels && n_tok * per < (1ll << 31), NVX_EINVAL, "nvx_conv_attn_prep: row stride, or too many rows");
    NVX_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (rot_dims == 0 || (turn && turn_stride >= turn_sin_off + rot_dims / 2)), NVX_EINVAL,
                "nvx_conv_attn_prep: the rotated part must be even and within a head, and needs its table");
    if (n_tok == 0 || n_seq == 0) return NVX_OK;
    NVX_REQUIRE(x && w && (state || taps_n == 1) && pos0 && state_slot && slots && q_out && k_cache && v_cache, NVX_EINVAL, "nvx_conv_attn_prep: null pointer");
    NVX_REQUIRE((tok_seq != nullptr) == (qo_indptr != nullptr) && (qo_indptr || n_tok == n_seq), NVX_EINVAL,
                "nvx_conv_attn_prep: tok_seq and qo_indptr go together; without them every sequence has one token");
    const hipStream_t st = (hipStream_t)stream;
    const int64_t longest = dim > vdim ? dim : vdim;
    const bool vec = dim % 8 == 0 && vdim % 8 == 0 && longest <= 512 && taps_n <= 4 && x_stride % 8 == 0 && rot_dims % 16 == 0 && nvx_aligned16(x) &&
                     nvx_aligned16(q_out) && nvx_aligned16(k_cache) && nvx_aligned16(v_cache);
    const int own_tail = vec && !qo_indptr;
    NVX_FMT_CALL(fmt, launch_conv_prep((ConvPrep<A_>{(const A_*)x, x_stride, w, taps_n, state, tok_seq, qo_indptr, state_slot, pos0,
                                                     TurnRows{turn, turn_stride, turn_sin_off}, rot_dims / 2, norm, eps, slots, (A_*)q_out, (A_*)k_cache,
                                                     (A_*)v_cache, n_tok, (int)heads, (int)kv_heads, (int)dim, (int)vdim}), vec, own_tail, st));
    if (taps_n > 1 && !own_tail) nvx_launch_tail_rows(x, x_stride, fmt, taps_n, state, qo_indptr, pos0, state_slot, n_seq, channels, st);
    return nvx_check_launch("nvx_conv_attn_prep");
}
