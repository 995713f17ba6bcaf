// Helpers of the kernels that take the activations' format as an argument (`fmt`: 0 bfloat16, 1 float16, 2 float32):
// element loads and stores through float, the dispatch of a launch on the format, and the description of a ragged step.
#pragma once
#include "nvx_dev.h"

namespace NVX_NS {

template <typename A> __device__ __forceinline__ float ld_f(const A* p, int64_t i) { return (float)p[i]; }
template <typename A> __device__ __forceinline__ void st_f(A* p, int64_t i, float v) { p[i] = (A)v; }

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.0f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float logsigmoid_f(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }

// sum over a workgroup of 256 threads; every thread gets the total.  `red` holds 4 floats; safe to call repeatedly.
__device__ __forceinline__ float block256_sum(float v, float* red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return red[0] + red[1] + red[2] + red[3];
}

// Where sequence b's tokens of this step are: first row, count, position of the first, state slot.
struct SeqSpan { int64_t q0; int64_t n; int64_t pos0; int slot; };
__device__ __forceinline__ SeqSpan seq_span(int b, const int32_t* qo_indptr, const int64_t* pos0, const int32_t* state_slot) {
    SeqSpan s;
    s.q0 = qo_indptr ? qo_indptr[b] : b;
    s.n = qo_indptr ? qo_indptr[b + 1] - s.q0 : 1;
    s.pos0 = pos0[b];
    s.slot = state_slot[b];
    return s;
}

// cos and sin of an angle given in double precision (position * frequency, exact to the table's accuracy at any position): the
// angle is brought into [-pi, pi] in double precision, where its float32 value is off by at most 2e-7, and the float32 functions
// take it from there.
__device__ __forceinline__ void turn_of(double a, float& c, float& s) {
    const double two_pi = 6.283185307179586476925286766559;
    const float r = (float)(a - two_pi * rint(a / two_pi));
    sincosf(r, &s, &c);
}

template <int LPR> __device__ __forceinline__ float group_sum(float v) {      // over LPR neighbouring lanes, in the vector ALU
    v += dpp_move<0xB1>(v);                        // lane ^ 1
    v += dpp_move<0x4E>(v);                        // lane ^ 2
    v += dpp_move<0x141>(v);                       // the other quad of eight
    if (LPR >= 16) v += dpp_move<0x140>(v);        // the other eight of sixteen
    if (LPR >= 32) v += xor16(v);
    if (LPR >= 64) v += xor32(v);
    return v;
}

// A step's table of rotations: row t holds cos of token t's angles and, sin_off entries further on, their sin (float32).  `cos` points at
// the first angle of the rotation in question (several rotations share a row).
struct TurnRows { const float* cos; int64_t stride; int64_t sin_off; };

}  // namespace NVX_NS

// state[slot] <- the last taps_n - 1 rows of every sequence (x: the step's rows; older rows of the state move up); defined in state_scan.hip
void nvx_launch_tail_rows(const void* x, int64_t x_stride, int fmt, int taps_n, float* state, const int32_t* qo_indptr, const int64_t* pos0,
                          const int32_t* state_slot, int64_t n_seq, int64_t channels, hipStream_t stream);

#define NVX_FMT_CALL(fmt, CALL)                                             \
    do {                                                                    \
        if ((fmt) == 0) { typedef __bf16 A_; CALL; }                        \
        else if ((fmt) == 1) { typedef _Float16 A_; CALL; }                 \
        else { typedef float A_; CALL; }                                    \
    } while (0)
