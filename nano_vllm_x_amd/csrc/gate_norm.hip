// Sublayer boundaries of stacks whose residual stream is float32, whose norms work on groups of a row, and whose sublayer
// results pass a learned sigmoid gate before they are added:
//   - gated residual + grouped RMS norm, one launch per boundary (optionally the result is first formed as the mean of two
//     RMS-normed branch outputs);
//   - per-head RMS norm of a recurrence's or attention's read-out, times a weight, times an output gate;
//   - stacks that norm a sublayer's OUTPUT instead of its input: the (weighted sum of one or two) results divided by its root
//     mean square, times a weight (one number or one per channel), added to the stream, which the next sublayer reads as it is;
//   - the two ends of such a stack: scaled embedding rows into the stream, and logits through cap * tanh(. / cap);
//   - plain pre-normed stacks: one or two results (and further float32 terms) added to the stream and the next norm, in one launch,
//     or the stream handed out as a hi + lo pair of 16-bit rows for a matrix product that must see more than 16 bits of it;
//   - the embedding of such a stack: token row + row of a table of token pairs + learned position row, with that first norm.
// Norms, gates and the stream are float32 in every activation format.
#include "fmt_dev.h"

namespace NVX_NS {

// Per token t (one workgroup):
//   r = y[t]                                                   (y2 == null)
//   r = (y[t] / rms(y[t]) * w_y + y2[t] / rms(y2[t]) * w_y2) / 2     (y2 != null; rms over the whole row)
//   r *= sigmoid(gate[t] + gate_bias)                          (gate != null)
//   x[t] += mult * r                                           (y != null)
//   h[t] = x[t], each of `groups` consecutive slices divided by its own root mean square, times w_norm   (w_norm != null)
template <typename A>
__global__ __launch_bounds__(256) void gated_residual_norm_kernel(
    const A* __restrict__ y, int64_t y_stride, const A* __restrict__ y2, int64_t y2_stride, const float* __restrict__ w_y,
    const float* __restrict__ w_y2, const A* __restrict__ gate, int64_t gate_stride, const float* __restrict__ gate_bias, float mult,
    float* __restrict__ x, const float* __restrict__ w_norm, int groups, float eps, A* __restrict__ h_out, int width) {
    __shared__ float red[4];
    const int64_t t = blockIdx.x;
    const int64_t row = t * (int64_t)width;
    const A* yr = y ? y + t * y_stride : nullptr;
    const A* y2r = y2 ? y2 + t * y2_stride : nullptr;
    const A* gr = gate ? gate + t * gate_stride : nullptr;
    float r1 = 1.f, r2 = 1.f;
    if (y2r) {
        float a = 0.f, b = 0.f;
        for (int c = threadIdx.x; c < width; c += 256) {
            const float u = ld_f(yr, c), v = ld_f(y2r, c);
            a += u * u;
            b += v * v;
        }
        r1 = 1.0f / sqrtf(block256_sum(a, red) / (float)width + eps);
        r2 = 1.0f / sqrtf(block256_sum(b, red) / (float)width + eps);
    }
    const int gs = width / groups;
    for (int g = 0; g < groups; ++g) {
        const int lo = g * gs, hi = lo + gs;
        float ss = 0.f;
        for (int c = lo + threadIdx.x; c < hi; c += 256) {
            float xv = x[row + c];
            if (yr) {
                float r = ld_f(yr, c);
                if (y2r) r = 0.5f * (r * r1 * w_y[c] + ld_f(y2r, c) * r2 * w_y2[c]);
                if (gr) r *= sigmoid_f(ld_f(gr, c) + (gate_bias ? gate_bias[c] : 0.f));
                xv += mult * r;
                x[row + c] = xv;
            }
            ss += xv * xv;
        }
        if (!w_norm) continue;
        const float rn = 1.0f / sqrtf(block256_sum(ss, red) / (float)gs + eps);
        for (int c = lo + threadIdx.x; c < hi; c += 256) st_f(h_out, row + c, x[row + c] * rn * w_norm[c]);   // own stores, read back
    }
}

// Per token t (one workgroup):
//   r = a * y[t] (+ b * y2[t]);  x[t] += r / rms(r) * w_post                  (y != null; w_post: one number or `width` of them)
//   h[t] = x[t] / rms(x[t]) * w_next  (w_next != null)   or   h[t] = x[t]     (h_out != null)
template <typename A>
__global__ __launch_bounds__(256) void postnorm_residual_kernel(const A* __restrict__ y, int64_t y_stride, const A* __restrict__ y2,
                                                               int64_t y2_stride, float a, float b, const float* __restrict__ w_post,
                                                               int w_post_n, float* __restrict__ x, const float* __restrict__ w_next,
                                                               int w_next_n, float eps, A* __restrict__ h_out, int width) {
    __shared__ float red[4];
    const int64_t t = blockIdx.x;
    float* xr = x + t * (int64_t)width;
    const A* yr = y ? y + t * y_stride : nullptr;
    const A* y2r = y2 ? y2 + t * y2_stride : nullptr;
    float rn = 0.f;
    if (yr) {
        float ss = 0.f;
        for (int c = threadIdx.x; c < width; c += 256) {
            const float r = a * ld_f(yr, c) + (y2r ? b * ld_f(y2r, c) : 0.f);
            ss += r * r;
        }
        rn = 1.0f / sqrtf(block256_sum(ss, red) / (float)width + eps);
    }
    float sx = 0.f;
    for (int c = threadIdx.x; c < width; c += 256) {
        float xv = xr[c];
        if (yr) {
            const float r = a * ld_f(yr, c) + (y2r ? b * ld_f(y2r, c) : 0.f);
            xv += r * rn * w_post[w_post_n == 1 ? 0 : c];
            xr[c] = xv;
        }
        sx += xv * xv;
    }
    if (!h_out) return;
    A* hr = h_out + t * (int64_t)width;
    if (w_next) {
        const float rx = 1.0f / sqrtf(block256_sum(sx, red) / (float)width + eps);
        for (int c = threadIdx.x; c < width; c += 256) st_f(hr, c, xr[c] * rx * w_next[w_next_n == 1 ? 0 : c]);     // own stores, read back
    } else {
        for (int c = threadIdx.x; c < width; c += 256) st_f(hr, c, xr[c]);
    }
}

// Several residual streams per token (x: (tokens, streams, width) float32) and the sublayer boundary between them.  Per token t:
//   with a result y:   r = y[t] * scale (scale: one number per channel, or none);
//                      every stream at once from the old ones:  x_j' = sum_s mix[s][j] x_s + w_out[j] r      (mix indexed [from][to])
//   without one:       x_j' = x_j  (x_in may be ONE row per token that all streams start from: in_stream_stride 0)
//   then what the next sublayer reads:  u = sum_j w_in[j] x_j'  (w_in null: the plain sum),  h[t] = u / rms(u) * w_norm.
// A thread holds the old values of its columns for all streams before it writes any, so x_in may be x_out.  u waits in LDS for
// the row's mean square.
template <typename A, int MAXS>
__global__ __launch_bounds__(256) void hyper_mix_kernel(const float* x_in, int64_t in_tok_stride, int64_t in_stream_stride,
                                                       const A* __restrict__ y, int64_t y_stride, const float* __restrict__ scale,
                                                       const float* __restrict__ mix, const float* __restrict__ w_out,
                                                       const float* __restrict__ w_in, const float* __restrict__ w_norm, float eps,
                                                       float* x_out, A* __restrict__ h_out, int n_streams, int width) {
    extern __shared__ float su[];                 // width
    __shared__ float s_mix[MAXS * MAXS], s_out[MAXS], s_in[MAXS], red[4];
    const int64_t t = blockIdx.x;
    for (int i = threadIdx.x; i < n_streams * n_streams; i += 256) s_mix[(i / n_streams) * MAXS + (i % n_streams)] = mix ? mix[i] : 0.f;
    for (int i = threadIdx.x; i < n_streams; i += 256) { s_out[i] = w_out ? w_out[i] : 0.f; s_in[i] = w_in ? w_in[i] : 1.0f; }
    __syncthreads();
    const float* xr = x_in + t * in_tok_stride;
    float* xo = x_out + t * (int64_t)n_streams * width;
    const A* yr = y ? y + t * y_stride : nullptr;
    float ss = 0.f;
    for (int c = threadIdx.x; c < width; c += 256) {
        float old[MAXS];
#pragma unroll
        for (int s = 0; s < MAXS; ++s) old[s] = s < n_streams ? xr[s * in_stream_stride + c] : 0.f;
        const float r = yr ? ld_f(yr, c) * (scale ? scale[c] : 1.0f) : 0.f;
        float u = 0.f;
#pragma unroll
        for (int j = 0; j < MAXS; ++j) {
            if (j < n_streams) {
                float v = old[j];
                if (yr) {
                    v = s_out[j] * r;
#pragma unroll
                    for (int s = 0; s < MAXS; ++s) if (s < n_streams) v += s_mix[s * MAXS + j] * old[s];
                }
                if (yr || x_out != x_in || in_stream_stride == 0) xo[(int64_t)j * width + c] = v;
                u += s_in[j] * v;
            }
        }
        su[c] = u;
        ss += u * u;
    }
    if (!h_out) return;
    const float rn = 1.0f / sqrtf(block256_sum(ss, red) / (float)width + eps);
    for (int c = threadIdx.x; c < width; c += 256) st_f(h_out, t * (int64_t)width + c, su[c] * rn * (w_norm ? w_norm[c] : 1.0f));
}

// x[t] = table[ids[t]] * scale (float32), h[t] = the same in the activations' format
template <typename A>
__global__ __launch_bounds__(256) void embed_scale_kernel(const int64_t* __restrict__ ids, const A* __restrict__ table, int64_t vocab, float scale,
                                                         float* __restrict__ x, A* __restrict__ h, int width) {
    const int64_t t = blockIdx.x;
    int64_t id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    for (int c = threadIdx.x; c < width; c += 256) {
        const float v = ld_f(table, id * width + c) * scale;
        x[t * (int64_t)width + c] = v;
        if (h) st_f(h, t * (int64_t)width + c, v);
    }
}

template <typename A>
__global__ __launch_bounds__(256) void tanh_cap_kernel(const A* __restrict__ in, float cap, float* __restrict__ out, int64_t n) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
        const float z = ld_f(in, i);
        out[i] = cap > 0.f ? cap * tanhf(z / cap) : z;
    }
}

// The end of a row that waits in LDS (su, float32, written by this workgroup; a barrier lies in block256_sum, or is placed here):
// nothing (h null), h = su / rms * w, with `b` the layer norm h = (su - mean) / sqrt(variance + eps) * w + b (variance: the mean of the
// squared deviations), or (split) h = [hi | lo], two rows of the activations' format whose sum is su to 16 bits and more.
template <typename A>
__device__ __forceinline__ void row_end(const float* su, float ss, float* red, const float* __restrict__ w, const float* __restrict__ b, float eps,
                                        int split, A* __restrict__ h, int64_t t, int width) {
    if (!h) return;
    if (split) {                                  // (every thread reads back the entries it wrote)
        A* hr = h + t * 2 * (int64_t)width;
        for (int c = threadIdx.x * 4; c < width; c += 1024) {
            for (int i = c; i < c + 4 && i < width; ++i) {
                const float v = su[i];
                const A hi = (A)v;
                hr[i] = hi;
                hr[width + i] = (A)(v - (float)hi);
            }
        }
        return;
    }
    float mean = 0.f;
    if (b) {                                      // (a thread reads entries that the whole workgroup can see, or that it wrote itself)
        auto over_row = [&](auto f) {
            for (int c = threadIdx.x * 4; c < width; c += 1024) {
                if ((width & 3) == 0) {
                    const nvx_f32x4 v = *reinterpret_cast<const nvx_f32x4*>(su + c);
                    f(v[0]); f(v[1]); f(v[2]); f(v[3]);
                } else {
                    for (int i = c; i < c + 4 && i < width; ++i) f(su[i]);
                }
            }
        };
        float s1 = 0.f;
        over_row([&](float v) { s1 += v; });
        mean = block256_sum(s1, red) / (float)width;
        ss = 0.f;
        over_row([&](float v) { const float d = v - mean; ss += d * d; });
    }
    const float rn = 1.0f / sqrtf(block256_sum(ss, red) / (float)width + eps);
    A* hr = h + t * (int64_t)width;
    for (int c = threadIdx.x * 4; c < width; c += 1024) {
        if (c + 4 <= width && (width & 3) == 0) {
            typedef A vec4 __attribute__((ext_vector_type(4)));
            const nvx_f32x4 v = *reinterpret_cast<const nvx_f32x4*>(su + c), g = *reinterpret_cast<const nvx_f32x4*>(w + c);
            nvx_f32x4 add = {0.f, 0.f, 0.f, 0.f};
            if (b) add = *reinterpret_cast<const nvx_f32x4*>(b + c);
            vec4 o;
#pragma unroll
            for (int i = 0; i < 4; ++i) o[i] = (A)((v[i] - mean) * rn * g[i] + add[i]);
            *reinterpret_cast<vec4*>(hr + c) = o;
        } else {
            for (int i = c; i < c + 4 && i < width; ++i) st_f(hr, i, (su[i] - mean) * rn * w[i] + (b ? b[i] : 0.f));
        }
    }
}

// Per token t (one workgroup):  x_out[t] = x_in[t] (+ y[t]) (+ y2[t]) (+ add[t]) (+ bias);  then row_end of it.  V = 4: rows of all operands
// start on borders of four elements and the width is a multiple of four.  x_in may be x_out.
template <typename A, int V>
__global__ __launch_bounds__(256) void residual_norm_kernel(const float* x_in, const A* __restrict__ y, int64_t y_stride, const A* __restrict__ y2,
                                                           int64_t y2_stride, const float* __restrict__ add, const float* __restrict__ bias,
                                                           float* x_out, const float* __restrict__ w, const float* __restrict__ b, float eps,
                                                           int split, A* __restrict__ h, int width) {
    extern __shared__ __align__(16) float row_lds[];      // width
    float* su = row_lds;
    __shared__ float red[4];
    typedef A veca __attribute__((ext_vector_type(V)));
    typedef float vecf __attribute__((ext_vector_type(V)));
    const int64_t t = blockIdx.x;
    const int64_t row = t * (int64_t)width;
    float ss = 0.f;
    for (int c = threadIdx.x * V; c < width; c += 256 * V) {
        vecf v = *reinterpret_cast<const vecf*>(x_in + row + c);
        if (y) { const veca u = *reinterpret_cast<const veca*>(y + t * y_stride + c); for (int i = 0; i < V; ++i) v[i] += (float)u[i]; }
        if (y2) { const veca u = *reinterpret_cast<const veca*>(y2 + t * y2_stride + c); for (int i = 0; i < V; ++i) v[i] += (float)u[i]; }
        if (add) v += *reinterpret_cast<const vecf*>(add + row + c);
        if (bias) v += *reinterpret_cast<const vecf*>(bias + c);
        if (y || add || bias || x_out != x_in) *reinterpret_cast<vecf*>(x_out + row + c) = v;
        *reinterpret_cast<vecf*>(su + c) = v;
        for (int i = 0; i < V; ++i) ss += v[i] * v[i];
    }
    if (V == 1) __syncthreads();                  // (row_end takes four entries a thread)
    row_end<A>(su, ss, red, w, b, eps, split, h, t, width);
}

// Per token t (one workgroup):  x[t] = table[ids[t]] (+ pair[r]) (+ pos_table[position]);  then row_end of it.
//   r = (previous id * mul_prev + id * mul_cur) mod buckets, and the extra row `buckets` for a sequence's first token.  A token's
//   predecessor is the step's own or, for the first token of a portion, the id that the sequence's state slot keeps (its bits in a
//   float32 word).  The workgroup of a portion's first token reads that word before it replaces it by the portion's last id, and no
//   other workgroup touches it.
template <typename A, int V>
__global__ __launch_bounds__(256) void embed_sum_kernel(const int64_t* __restrict__ ids, const A* __restrict__ table, int64_t vocab,
                                                       const A* __restrict__ pair, int64_t buckets, int64_t mul_prev, int64_t mul_cur,
                                                       float* prev_id, const A* __restrict__ pos_table, int64_t n_pos,
                                                       const int64_t* __restrict__ positions, const int32_t* __restrict__ tok_seq,
                                                       const int32_t* __restrict__ qo_indptr, const int64_t* __restrict__ pos0,
                                                       const int32_t* __restrict__ state_slot, float* __restrict__ x, const float* __restrict__ w,
                                                       const float* __restrict__ b, float eps, int split, A* __restrict__ h, int width) {
    extern __shared__ __align__(16) float row_lds[];      // width
    float* su = row_lds;
    __shared__ float red[4];
    __shared__ int64_t pair_row;
    const int64_t t = blockIdx.x;
    int64_t id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    if (pair) {
        if (threadIdx.x == 0) {
            const int b = tok_seq ? tok_seq[t] : (int)t;
            const SeqSpan s = seq_span(b, qo_indptr, pos0, state_slot);
            int64_t prev = -1;                    // no predecessor: a sequence's first token (and a padding row)
            if (t > s.q0) prev = ids[t - 1];
            else if (s.slot >= 0) {
                if (s.pos0 > 0) prev = __float_as_int(prev_id[s.slot]);
                prev_id[s.slot] = __int_as_float((int)ids[s.q0 + s.n - 1]);
            }
            int64_t r = buckets;
            if (prev >= 0) {
                r = (prev * mul_prev + id * mul_cur) % buckets;
                if (r < 0) r += buckets;
            }
            pair_row = r;
        }
        __syncthreads();
    }
    int64_t p = pos_table ? positions[t] : 0;
    p = p < 0 ? 0 : (p >= n_pos ? n_pos - 1 : p);
    const A* er = table + id * width;
    const A* pr = pair ? pair + pair_row * width : nullptr;
    const A* lr = pos_table ? pos_table + p * width : nullptr;
    typedef A veca __attribute__((ext_vector_type(V)));
    typedef float vecf __attribute__((ext_vector_type(V)));
    float ss = 0.f;
    for (int c = threadIdx.x * V; c < width; c += 256 * V) {
        const veca a = *reinterpret_cast<const veca*>(er + c);
        vecf v;
        for (int i = 0; i < V; ++i) v[i] = (float)a[i];
        if (pr) { const veca u = *reinterpret_cast<const veca*>(pr + c); for (int i = 0; i < V; ++i) v[i] += (float)u[i]; }
        if (lr) { const veca u = *reinterpret_cast<const veca*>(lr + c); for (int i = 0; i < V; ++i) v[i] += (float)u[i]; }
        *reinterpret_cast<vecf*>(x + t * (int64_t)width + c) = v;
        *reinterpret_cast<vecf*>(su + c) = v;
        for (int i = 0; i < V; ++i) ss += v[i] * v[i];
    }
    __syncthreads();
    row_end<A>(su, ss, red, w, b, eps, split, h, t, width);
}

// One wave per (token, head): out = mul * o / rms(o) * w * gate, with gate = 1 (kind 0), sigmoid(z) (1) or z * sigmoid(z) (2) of
// the gate pre-activations z (rows of heads * vdim).  w has heads * vdim entries, or vdim shared by the heads, or is null (ones).
template <typename A>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ w, int w_shared,
                                                            const A* __restrict__ gate, int64_t gate_stride, int kind, float eps,
                                                            float mul, A* __restrict__ out, int64_t out_stride, int64_t n_rows, int heads,
                                                            int vdim) {
    const int64_t idx = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (idx >= n_rows) return;
    const int lane = threadIdx.x & 63;
    const int64_t t = idx / heads;
    const int hd = (int)(idx % heads);
    const int64_t base = t * (int64_t)heads * vdim + (int64_t)hd * vdim;
    float ss = 0.f;
    for (int e = lane; e < vdim; e += 64) { const float v = o[base + e]; ss += v * v; }
    const float rn = mul / sqrtf(wave_sum(ss) / (float)vdim + eps);
    for (int e = lane; e < vdim; e += 64) {
        float v = o[base + e] * rn;
        if (w) v *= w[w_shared ? e : hd * vdim + e];
        if (kind) {
            const float z = ld_f(gate, t * gate_stride + (int64_t)hd * vdim + e);
            v *= kind == 1 ? sigmoid_f(z) : z * sigmoid_f(z);
        }
        st_f(out, t * out_stride + (int64_t)hd * vdim + e, v);
    }
}


// Projections onto FEW outputs or from FEW inputs, in float32: gate and router logits (outputs = heads or experts), the two
// halves of a low-rank decay.  out[t][n] = g(sum_k W[n][k] * f(x[t][k]) + bias[n]), f = identity or tanh, g = identity or
// sigmoid(.)^power (formed as exp(power * logsigmoid(.))); W float32 (n_out, k_in), bias float32 or null.  A
// workgroup takes TOK tokens: their inputs wait in LDS as float32, every weight is read once for the TOK of them.  Wide
// inputs: a wave per output, lanes over k.  Narrow inputs (k_in < 256): a thread per output.  No workspace, no atomics: the
// sums have one order, and the launch can be captured.
__device__ __forceinline__ float skinny_end(float z, const float* __restrict__ bias, int n, int out_act, float power) {
    if (bias) z += bias[n];
    return out_act == 1 ? expf(power * logsigmoid_f(z)) : z;
}

template <typename A, int TOK>
__global__ __launch_bounds__(256) void skinny_proj_kernel(const A* __restrict__ x, int64_t x_stride, const float* __restrict__ w,
                                                         int in_act, const float* __restrict__ bias, int out_act, float power,
                                                         float* __restrict__ out, int64_t n_tok, int n_out, int k_in, int out_per_block) {
    extern __shared__ float xs[];      // TOK rows of k_in
    const int64_t t0 = (int64_t)blockIdx.x * TOK;
    const int nt = (int)(n_tok - t0 < TOK ? n_tok - t0 : TOK);
    for (int i = threadIdx.x; i < TOK * k_in; i += 256) {
        const int tt = i / k_in, k = i % k_in;
        float v = tt < nt ? ld_f(x, (t0 + tt) * x_stride + k) : 0.f;
        xs[i] = in_act == 1 ? tanhf(v) : v;
    }
    __syncthreads();
    const int n_lo = blockIdx.y * out_per_block;
    const int n_hi = n_lo + out_per_block < n_out ? n_lo + out_per_block : n_out;
    if (k_in >= 256) {
        const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
        for (int n = n_lo + wave; n < n_hi; n += 4) {
            const float* wr = w + (int64_t)n * k_in;
            float acc[TOK];
#pragma unroll
            for (int tt = 0; tt < TOK; ++tt) acc[tt] = 0.f;
            for (int k = lane; k < k_in; k += 64) {
                const float wv = wr[k];
#pragma unroll
                for (int tt = 0; tt < TOK; ++tt) acc[tt] += wv * xs[tt * k_in + k];
            }
#pragma unroll
            for (int tt = 0; tt < TOK; ++tt) {
                const float sum = wave_sum(acc[tt]);
                if (lane == 0 && tt < nt) out[(t0 + tt) * n_out + n] = skinny_end(sum, bias, n, out_act, power);
            }
        }
    } else {
        for (int n = n_lo + threadIdx.x; n < n_hi; n += 256) {
            const float* wr = w + (int64_t)n * k_in;
            float acc[TOK];
#pragma unroll
            for (int tt = 0; tt < TOK; ++tt) acc[tt] = 0.f;
            for (int k = 0; k < k_in; ++k) {
                const float wv = wr[k];
#pragma unroll
                for (int tt = 0; tt < TOK; ++tt) acc[tt] += wv * xs[tt * k_in + k];
            }
#pragma unroll
            for (int tt = 0; tt < TOK; ++tt)
                if (tt < nt) out[(t0 + tt) * n_out + n] = skinny_end(acc[tt], bias, n, out_act, power);
        }
    }
}

// The same for wide inputs whose rows start on borders of four elements (k_in >= 256 and a multiple of 4).  A workgroup takes SKW_TOK tokens
// and SKW_OUT outputs; its four waves take the inputs 256 at a time, every fourth piece each, a lane four neighbouring inputs: all loads
// of a piece are in flight together, every weight serves SKW_TOK tokens and every input SKW_OUT outputs from registers, and the sums of
// lanes and waves have one order, whatever the batch.
constexpr int SKW_TOK = 4, SKW_OUT = 8;
template <typename A>
__global__ __launch_bounds__(256) void skinny_wide_kernel(const A* __restrict__ x, int64_t x_stride, const float* __restrict__ w, int in_act,
                                                         const float* __restrict__ bias, int out_act, float power, float* __restrict__ out, int64_t n_tok,
                                                         int n_out, int k_in) {
    typedef A veca __attribute__((ext_vector_type(4)));
    __shared__ float part[4][SKW_TOK * SKW_OUT];
    const int64_t t0 = (int64_t)blockIdx.x * SKW_TOK;
    const int n0 = blockIdx.y * SKW_OUT, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    float acc[SKW_TOK][SKW_OUT];
#pragma unroll
    for (int t = 0; t < SKW_TOK; ++t)
#pragma unroll
        for (int n = 0; n < SKW_OUT; ++n) acc[t][n] = 0.f;
    for (int k = wave * 256 + lane * 4; k < k_in; k += 1024) {
        veca xv[SKW_TOK];
        nvx_f32x4 wv[SKW_OUT];
#pragma unroll
        for (int t = 0; t < SKW_TOK; ++t) xv[t] = *reinterpret_cast<const veca*>(x + (t0 + t < n_tok ? t0 + t : n_tok - 1) * x_stride + k);
#pragma unroll
        for (int n = 0; n < SKW_OUT; ++n) wv[n] = *reinterpret_cast<const nvx_f32x4*>(w + (int64_t)(n0 + n < n_out ? n0 + n : n_out - 1) * k_in + k);
#pragma unroll
        for (int t = 0; t < SKW_TOK; ++t) {
            float xf[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) { const float v = (float)xv[t][i]; xf[i] = in_act == 1 ? tanhf(v) : v; }
#pragma unroll
            for (int n = 0; n < SKW_OUT; ++n)
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[t][n] += xf[i] * wv[n][i];
        }
    }
#pragma unroll
    for (int t = 0; t < SKW_TOK; ++t)
#pragma unroll
        for (int n = 0; n < SKW_OUT; ++n) {
            float v = quarter_sum(acc[t][n]);
            v += xor16(v);
            v += xor32(v);
            if (lane == 0) part[wave][t * SKW_OUT + n] = v;
        }
    __syncthreads();
    if (threadIdx.x < SKW_TOK * SKW_OUT) {
        const int t = threadIdx.x / SKW_OUT, n = threadIdx.x % SKW_OUT;
        const float v = part[0][threadIdx.x] + part[1][threadIdx.x] + part[2][threadIdx.x] + part[3][threadIdx.x];
        if (t0 + t < n_tok && n0 + n < n_out) out[(t0 + t) * n_out + n0 + n] = skinny_end(v, bias, n0 + n, out_act, power);
    }
}

}  // namespace NVX_NS

using namespace NVX_NS;

extern "C" int nvx_skinny_proj(const void* x, int64_t x_stride, int fmt, const float* w, int in_act, const float* bias, int out_act,
                               float power, float* out, int64_t n_tok, int64_t n_out, int64_t k_in, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2 && (in_act == 0 || in_act == 1) && (out_act == 0 || out_act == 1), NVX_EINVAL,
                "nvx_skinny_proj: fmt must be 0..2, in_act and out_act 0 or 1");
    NVX_REQUIRE(n_tok >= 0 && n_out > 0 && n_out < (1 << 24) && k_in > 0 && k_in <= 12288 && x_stride >= k_in, NVX_EINVAL,
                "nvx_skinny_proj: bad sizes (at most 12288 inputs)");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(x && w && out, NVX_EINVAL, "nvx_skinny_proj: null pointer");
    // the outputs are split over workgroups too (8 a workgroup for wide inputs, 256 for narrow ones): a step of few tokens would
    // otherwise be a handful of workgroups walking all outputs one after another
    const int opb = k_in >= 256 ? 8 : 256;
    const int64_t chunks = (n_out + opb - 1) / opb;
    NVX_REQUIRE(chunks <= 65535, NVX_EINVAL, "nvx_skinny_proj: too many outputs");
    const uintptr_t x_border = fmt == 2 ? 15u : 7u;
    if (k_in >= 256 && k_in % 4 == 0 && x_stride % 4 == 0 && (reinterpret_cast<uintptr_t>(x) & x_border) == 0 && nvx_aligned16(w)) {
        NVX_REQUIRE((n_tok + SKW_TOK - 1) / SKW_TOK < (1ll << 31), NVX_EINVAL, "nvx_skinny_proj: too many tokens");
        NVX_FMT_CALL(fmt, hipLaunchKernelGGL(skinny_wide_kernel<A_>, dim3((unsigned)((n_tok + SKW_TOK - 1) / SKW_TOK), (unsigned)((n_out + SKW_OUT - 1) / SKW_OUT)),
                                             dim3(256), 0, (hipStream_t)stream, (const A_*)x, x_stride, w, in_act, bias, out_act, power, out, n_tok, (int)n_out,
                                             (int)k_in));
        return nvx_check_launch("nvx_skinny_proj");
    }
    if (k_in <= 3072) {
        const int64_t blocks = (n_tok + 3) / 4;
        NVX_REQUIRE(blocks < (1ll << 31), NVX_EINVAL, "nvx_skinny_proj: too many tokens");
        NVX_FMT_CALL(fmt, hipLaunchKernelGGL((skinny_proj_kernel<A_, 4>), dim3((unsigned)blocks, (unsigned)chunks), dim3(256),
                                             (size_t)(4 * k_in) * sizeof(float), (hipStream_t)stream, (const A_*)x, x_stride, w, in_act, bias, out_act, power, out, n_tok,
                                             (int)n_out, (int)k_in, opb));
    } else {
        NVX_REQUIRE(n_tok < (1ll << 31), NVX_EINVAL, "nvx_skinny_proj: too many tokens");
        NVX_FMT_CALL(fmt, hipLaunchKernelGGL((skinny_proj_kernel<A_, 1>), dim3((unsigned)n_tok, (unsigned)chunks), dim3(256),
                                             (size_t)k_in * sizeof(float), (hipStream_t)stream, (const A_*)x, x_stride, w, in_act, bias, out_act, power, out, n_tok,
                                             (int)n_out, (int)k_in, opb));
    }
    return nvx_check_launch("nvx_skinny_proj");
}

extern "C" int nvx_gated_residual_norm(const void* y, int64_t y_stride, const void* y2, int64_t y2_stride, const float* w_y,
                                       const float* w_y2, const void* gate, int64_t gate_stride, const float* gate_bias, int fmt,
                                       float mult, float* x, const float* w_norm, int groups, float eps, void* h_out, int64_t n_tok,
                                       int64_t width, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2, NVX_EINVAL, "nvx_gated_residual_norm: fmt must be 0, 1 or 2");
    NVX_REQUIRE(n_tok >= 0 && width > 0 && width < (1 << 30) && groups >= 1 && width % groups == 0, NVX_EINVAL,
                "nvx_gated_residual_norm: bad sizes (the width must be a multiple of the groups)");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(x && (y || w_norm), NVX_EINVAL, "nvx_gated_residual_norm: null pointer");
    NVX_REQUIRE(!y || y_stride >= width, NVX_EINVAL, "nvx_gated_residual_norm: row stride of y");
    NVX_REQUIRE(!y2 || (y && w_y && w_y2 && y2_stride >= width), NVX_EINVAL, "nvx_gated_residual_norm: two branches need both weights");
    NVX_REQUIRE(!gate || (y && gate_stride >= width), NVX_EINVAL, "nvx_gated_residual_norm: a gate needs a result to gate");
    NVX_REQUIRE(!w_norm || h_out, NVX_EINVAL, "nvx_gated_residual_norm: the norm needs an output");
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(gated_residual_norm_kernel<A_>, dim3((unsigned)n_tok), dim3(256), 0, (hipStream_t)stream,
                                         (const A_*)y, y_stride, (const A_*)y2, y2_stride, w_y, w_y2, (const A_*)gate, gate_stride,
                                         gate_bias, mult, x, w_norm, groups, eps, (A_*)h_out, (int)width));
    return nvx_check_launch("nvx_gated_residual_norm");
}

extern "C" int nvx_head_norm_gate(const float* o, const float* w, int w_shared, const void* gate, int64_t gate_stride, int kind, int fmt,
                                  float eps, float mul, void* out, int64_t out_stride, int64_t n_tok, int64_t heads, int64_t vdim,
                                  nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2 && kind >= 0 && kind <= 2, NVX_EINVAL, "nvx_head_norm_gate: fmt must be 0..2, kind 0..2");
    NVX_REQUIRE(n_tok >= 0 && heads > 0 && vdim > 0 && heads * vdim < (1 << 30), NVX_EINVAL, "nvx_head_norm_gate: bad sizes");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(o && out && out_stride >= heads * vdim && (kind == 0 || (gate && gate_stride >= heads * vdim)), NVX_EINVAL,
                "nvx_head_norm_gate: null pointer or row stride");
    const int64_t rows = n_tok * heads;
    NVX_REQUIRE((rows + 3) / 4 < (1ll << 31), NVX_EINVAL, "nvx_head_norm_gate: too many rows");
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(head_norm_gate_kernel<A_>, dim3((unsigned)((rows + 3) / 4)), dim3(256), 0, (hipStream_t)stream, o, w,
                                         w_shared, (const A_*)gate, gate_stride, kind, eps, mul, (A_*)out, out_stride, rows, (int)heads, (int)vdim));
    return nvx_check_launch("nvx_head_norm_gate");
}

extern "C" int nvx_postnorm_residual(const void* y, int64_t y_stride, const void* y2, int64_t y2_stride, float a, float b, const float* w_post,
                                     int64_t w_post_n, int fmt, float* x, const float* w_next, int64_t w_next_n, float eps, void* h_out,
                                     int64_t n_tok, int64_t width, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2, NVX_EINVAL, "nvx_postnorm_residual: fmt must be 0, 1 or 2");
    NVX_REQUIRE(n_tok >= 0 && width > 0 && width < (1 << 30), NVX_EINVAL, "nvx_postnorm_residual: bad sizes");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(x && (y || h_out), NVX_EINVAL, "nvx_postnorm_residual: null pointer");
    NVX_REQUIRE(!y || (y_stride >= width && w_post && (w_post_n == 1 || w_post_n == width)), NVX_EINVAL,
                "nvx_postnorm_residual: a result needs its norm weight (one number or one per channel)");
    NVX_REQUIRE(!y2 || (y && y2_stride >= width), NVX_EINVAL, "nvx_postnorm_residual: a second result needs a first");
    NVX_REQUIRE(!w_next || (h_out && (w_next_n == 1 || w_next_n == width)), NVX_EINVAL, "nvx_postnorm_residual: the closing norm needs an output");
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(postnorm_residual_kernel<A_>, dim3((unsigned)n_tok), dim3(256), 0, (hipStream_t)stream, (const A_*)y,
                                         y_stride, (const A_*)y2, y2_stride, a, b, w_post, (int)w_post_n, x, w_next, (int)w_next_n, eps, (A_*)h_out,
                                         (int)width));
    return nvx_check_launch("nvx_postnorm_residual");
}

extern "C" int nvx_hyper_mix(const float* x_in, int64_t in_tok_stride, int64_t in_stream_stride, const void* y, int64_t y_stride, int fmt,
                             const float* scale, const float* mix, const float* w_out, const float* w_in, const float* w_norm, float eps,
                             float* x_out, void* h_out, int64_t n_tok, int64_t n_streams, int64_t width, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2, NVX_EINVAL, "nvx_hyper_mix: fmt must be 0, 1 or 2");
    NVX_REQUIRE(n_tok >= 0 && n_streams >= 1 && n_streams <= 16 && width > 0, NVX_EINVAL, "nvx_hyper_mix: bad sizes (at most 16 streams)");
    NVX_REQUIRE(width <= 15360, NVX_EUNSUPPORTED, "nvx_hyper_mix: a row must fit LDS as float32 (width <= 15360)");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(x_in && x_out, NVX_EINVAL, "nvx_hyper_mix: null pointer");
    NVX_REQUIRE(in_tok_stride >= width && (in_stream_stride == 0 || in_stream_stride >= width), NVX_EINVAL, "nvx_hyper_mix: strides of the streams");
    NVX_REQUIRE(!y || (y_stride >= width && mix && w_out), NVX_EINVAL, "nvx_hyper_mix: a result needs the mixing matrix and its output weights");
    NVX_REQUIRE(x_in != x_out || (in_tok_stride == n_streams * width && in_stream_stride == width), NVX_EINVAL,
                "nvx_hyper_mix: streams updated in place keep their layout");
    const size_t lds = (size_t)width * sizeof(float);
#define NVX_HYPER(MAXS)                                                                                                               \
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL((hyper_mix_kernel<A_, MAXS>), dim3((unsigned)n_tok), dim3(256), lds, (hipStream_t)stream, x_in, \
                                         in_tok_stride, in_stream_stride, (const A_*)y, y_stride, scale, mix, w_out, w_in, w_norm, eps, \
                                         x_out, (A_*)h_out, (int)n_streams, (int)width))
    if (n_streams <= 1) NVX_HYPER(1);
    else if (n_streams <= 2) NVX_HYPER(2);
    else if (n_streams <= 4) NVX_HYPER(4);
    else if (n_streams <= 8) NVX_HYPER(8);
    else NVX_HYPER(16);
#undef NVX_HYPER
    return nvx_check_launch("nvx_hyper_mix");
}

extern "C" int nvx_embed_scale(const int64_t* ids, const void* table, int fmt, int64_t vocab, float scale, float* x, void* h, int64_t n_tok,
                               int64_t width, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2 && n_tok >= 0 && vocab > 0 && width > 0 && width < (1 << 30), NVX_EINVAL, "nvx_embed_scale: bad arguments");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(ids && table && x, NVX_EINVAL, "nvx_embed_scale: null pointer");
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(embed_scale_kernel<A_>, dim3((unsigned)n_tok), dim3(256), 0, (hipStream_t)stream, ids, (const A_*)table, vocab,
                                         scale, x, (A_*)h, (int)width));
    return nvx_check_launch("nvx_embed_scale");
}

#define NVX_ROW_OK(name)                                                                                                               \
    NVX_REQUIRE(fmt >= 0 && fmt <= 2, NVX_EINVAL, name ": fmt must be 0, 1 or 2");                                                     \
    NVX_REQUIRE(n_tok >= 0 && n_tok < (1ll << 31) && width > 0, NVX_EINVAL, name ": bad sizes");                                       \
    NVX_REQUIRE(width <= 15360, NVX_EUNSUPPORTED, name ": a row must fit LDS as float32 (width <= 15360)");                            \
    NVX_REQUIRE(!h || split || w, NVX_EINVAL, name ": the norm needs its weight");                                                     \
    NVX_REQUIRE(!w_bias || (w && !split), NVX_EINVAL, name ": the layer norm's bias goes with its weight")

extern "C" int nvx_residual_norm(const float* x_in, const void* y, int64_t y_stride, const void* y2, int64_t y2_stride, const float* add,
                                 const float* bias, int fmt, float* x_out, const float* w, const float* w_bias, float eps, int split, void* h,
                                 int64_t n_tok, int64_t width, nvx_stream_t stream) {
    NVX_ROW_OK("nvx_residual_norm");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(x_in && x_out && (!y || y_stride >= width) && (!y2 || y2_stride >= width), NVX_EINVAL, "nvx_residual_norm: null pointer or row stride");
    const size_t lds = (size_t)width * sizeof(float);
    const auto ok4 = [&](const void* p, size_t item) { return (reinterpret_cast<uintptr_t>(p) & (4 * item - 1)) == 0; };
    const size_t item = fmt == 2 ? 4 : 2;
    const bool v4 = width % 4 == 0 && ok4(x_in, 4) && ok4(x_out, 4) && ok4(add, 4) && ok4(bias, 4) && ok4(w, 4) && ok4(w_bias, 4) && ok4(y, item) && ok4(y2, item) &&
                    ok4(h, item) && (!y || y_stride % 4 == 0) && (!y2 || y2_stride % 4 == 0);
#define NVX_RESIDUAL_NORM(V)                                                                                                           \
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL((residual_norm_kernel<A_, V>), dim3((unsigned)n_tok), dim3(256), lds, (hipStream_t)stream, x_in, (const A_*)y, \
                                         y_stride, (const A_*)y2, y2_stride, add, bias, x_out, w, w_bias, eps, split, (A_*)h, (int)width))
    if (v4) NVX_RESIDUAL_NORM(4);
    else {
        NVX_REQUIRE(width % 4 != 0, NVX_EINVAL, "nvx_residual_norm: rows of a width that is a multiple of four must start on such borders");
        NVX_RESIDUAL_NORM(1);
    }
#undef NVX_RESIDUAL_NORM
    return nvx_check_launch("nvx_residual_norm");
}

extern "C" int nvx_embed_sum(const int64_t* ids, const void* table, int fmt, int64_t vocab, const void* pair, int64_t buckets, int64_t mul_prev,
                             int64_t mul_cur, float* prev_id, int64_t n_slots, const void* pos_table, int64_t n_pos, const int64_t* positions,
                             const int32_t* tok_seq, const int32_t* qo_indptr, const int64_t* pos0, const int32_t* state_slot, float* x,
                             const float* w, const float* w_bias, float eps, int split, void* h, int64_t n_tok, int64_t n_seq, int64_t width,
                             nvx_stream_t stream) {
    NVX_ROW_OK("nvx_embed_sum");
    if (n_tok == 0) return NVX_OK;
    NVX_REQUIRE(ids && table && vocab > 0 && vocab < (1ll << 31) && x, NVX_EINVAL, "nvx_embed_sum: bad table");
    NVX_REQUIRE(!pair || (buckets > 0 && prev_id && n_slots > 0 && pos0 && state_slot && (tok_seq != nullptr) == (qo_indptr != nullptr) &&
                          (qo_indptr || n_tok == n_seq)), NVX_EINVAL, "nvx_embed_sum: the pair table needs the step's layout and the predecessors' slots");
    NVX_REQUIRE(!pos_table || (positions && n_pos > 0), NVX_EINVAL, "nvx_embed_sum: the position table needs positions");
    NVX_REQUIRE(!h || width % 4 != 0 || (nvx_aligned16(w) && nvx_aligned16(w_bias)), NVX_EINVAL,
                "nvx_embed_sum: the norm's weight and bias must start on a 16-byte border");
#define NVX_EMBED_SUM(V)                                                                                                                       \
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL((embed_sum_kernel<A_, V>), dim3((unsigned)n_tok), dim3(256), (size_t)width * sizeof(float), (hipStream_t)stream, ids, \
                                         (const A_*)table, vocab, (const A_*)pair, buckets, mul_prev, mul_cur, prev_id, (const A_*)pos_table, n_pos,   \
                                         positions, tok_seq, qo_indptr, pos0, state_slot, x, w, w_bias, eps, split, (A_*)h, (int)width))
    if (width % 4 == 0 && nvx_aligned16(table) && nvx_aligned16(pair) && nvx_aligned16(pos_table) && nvx_aligned16(x)) NVX_EMBED_SUM(4);
    else NVX_EMBED_SUM(1);
#undef NVX_EMBED_SUM
    return nvx_check_launch("nvx_embed_sum");
}

extern "C" int nvx_tanh_cap(const void* in, int fmt, float cap, float* out, int64_t n, nvx_stream_t stream) {
    NVX_REQUIRE(fmt >= 0 && fmt <= 2 && n >= 0, NVX_EINVAL, "nvx_tanh_cap: bad arguments");
    if (n == 0) return NVX_OK;
    NVX_REQUIRE(in && out, NVX_EINVAL, "nvx_tanh_cap: null pointer");
    int64_t blocks = (n + 255) / 256;
    if (blocks > 256 * 64) blocks = 256 * 64;
    NVX_FMT_CALL(fmt, hipLaunchKernelGGL(tanh_cap_kernel<A_>, dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, (const A_*)in, cap, out, n));
    return nvx_check_launch("nvx_tanh_cap");
}
