// Device helpers shared by the kernels of mixers that carry a matrix state per head: the gates' functions,
// the lanes' share of a column of the state, the causal convolution's inputs in front of a step.
#pragma once
#include "dispatch.h"

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }

__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }
// log(sigmoid(z)) without overflow
__device__ __forceinline__ float logsigmoid_f(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// NT sums over j in [j0, j1) of w2t[j][c] * th[t][j] (th rows `pitch` floats apart), the weight's element
// type known at compile time and eight loads in flight at a time; the additions run in the order of j
template <typename W, int NT>
__device__ __forceinline__ void decay_dots(const W* __restrict__ w2t_c, size_t inner, const float* th, int pitch, int j0,
                                           int j1, float (&acc)[NT]) {
    int j = j0;
    for (; j + 8 <= j1; j += 8) {
        float w[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = to_f(w2t_c[(size_t)(j + e) * inner]);
#pragma unroll
        for (int e = 0; e < 8; ++e)
#pragma unroll
            for (int t = 0; t < NT; ++t) acc[t] = fmaf(w[e], th[t * pitch + j + e], acc[t]);
    }
    for (; j < j1; ++j) {
        const float w = to_f(w2t_c[(size_t)j * inner]);
#pragma unroll
        for (int t = 0; t < NT; ++t) acc[t] = fmaf(w, th[t * pitch + j], acc[t]);
    }
}

// the sum of a value over the L lanes that share a column (L = 4, 8 or 16 neighbouring lanes of a row
// of 16): exchanges inside the row by data-parallel moves; every lane ends with the sum
template <int L>
__device__ __forceinline__ float lanes_sum(float v) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, true));   // quad [1,0,3,2]
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x4E, 0xF, 0xF, true));   // quad [2,3,0,1]
    if constexpr (L >= 8)
        v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x141, 0xF, 0xF, true));  // mirror of 8
    if constexpr (L >= 16)
        v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x140, 0xF, 0xF, true));  // mirror of 16
    return v;
}

// a lane's R rows of its column, between registers and the column's D floats in memory (rows
// sub*R .. sub*R+R-1; rows beyond D are zero and are not stored)
template <int R, bool STORE>
__device__ __forceinline__ void delta_state_io(float (&s)[R], float* column, int sub, int D, bool live) {
    const int i0 = sub * R;
    if ((D & 3) == 0) {
#pragma unroll
        for (int e = 0; e < R; e += 4) {
            const bool ok = live && i0 + e < D;
            float4* p = reinterpret_cast<float4*>(column + (i0 + e < D ? i0 + e : 0));
            if constexpr (STORE) {
                if (ok) *p = float4{s[e], s[e + 1], s[e + 2], s[e + 3]};
            } else {
                const float4 v = *p;                  // always issued (a valid address either way), dropped where it does not count
                s[e] = ok ? v.x : 0.f; s[e + 1] = ok ? v.y : 0.f; s[e + 2] = ok ? v.z : 0.f; s[e + 3] = ok ? v.w : 0.f;
            }
        }
    } else {
#pragma unroll
        for (int e = 0; e < R; ++e) {
            const bool ok = live && i0 + e < D;
            if constexpr (STORE) {
                if (ok) column[i0 + e] = s[e];
            } else {
                const float v = column[i0 + e < D ? i0 + e : 0];
                s[e] = ok ? v : 0.f;
            }
        }
    }
}

// how a head of size D is dealt out: (rows a lane keeps, lanes a column); 0 when D is not served
static inline void delta_scan_shape(int D, int& R, int& L) {
    // few rows a lane and many lanes a column: a token costs the fewest instructions of the one wave a
    // SIMD runs, and a head is spread over the most workgroups
    if (D <= 16) { R = 4; L = 4; }
    else if (D <= 32) { R = 4; L = 8; }
    else if (D <= 64) { R = 4; L = 16; }
    else if (D <= 128) { R = 8; L = 16; }
    else { R = 16; L = 16; }
}

// most taps of a causal convolution over time
#define MS_MAX_TAPS 16

// One input of the causal convolution: row r of the step when the request's rows reach back that far,
// else the request's kept inputs (hist[slot][taps-1][C], the last one the newest).
template <typename T>
__device__ __forceinline__ float conv_input(const T* __restrict__ rows, long ld, const T* __restrict__ hist, int C, int taps,
                                            int first, int r, int c) {
    if (r >= first) return to_f(rows[(size_t)r * ld + c]);
    return to_f(hist[(size_t)(taps - 1 + (r - first)) * C + c]);
}

// The convolution's kept inputs after the step: the last taps-1 inputs of each request, from the step's
// rows and, where the step brought fewer, from what was kept before. Thread (request, channel) reads all
// it needs before it writes, and no other thread touches its channel.
template <typename T>
static __global__ void __launch_bounds__(256)
conv_state_kernel(const T* __restrict__ packed, long ld, int C, int taps, T* __restrict__ conv_state,
                  const int* __restrict__ cu_seqlens, const int* __restrict__ state_slots) {
    const int seq = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    const int first = cu_seqlens[seq], end = cu_seqlens[seq + 1];
    if (end <= first || c >= C) return;
    T* hist = conv_state + (size_t)state_slots[seq] * (taps - 1) * C;
    T keep[MS_MAX_TAPS];
    for (int i = 0; i < taps - 1; ++i) {
        const int r = end - (taps - 1) + i;
        keep[i] = r >= first ? packed[(size_t)r * ld + c] : hist[(size_t)(taps - 1 + (r - first)) * C + c];
    }
    for (int i = 0; i < taps - 1; ++i) hist[(size_t)i * C + c] = keep[i];
}
