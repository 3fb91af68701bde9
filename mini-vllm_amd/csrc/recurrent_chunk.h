// Shared by the kernels that cut a request's tokens of a step into chunks: which rows a workgroup's chunk holds, and float
// products of 64 x 64 tiles in LDS on the MFMA units (v_mfma_f32_16x16x4_f32).
#pragma once
#include "recurrent.h"

typedef float floatx4_t __attribute__((ext_vector_type(4)));

#define CL_TOKENS 64
#define CL_TILE 64                 // channels of a tile
// LDS rows of 68 floats: a lane takes four neighbours of a row for four steps of a product (16 bytes; the four
// steps then sum over k in another order, the same for both operands), and the 16 rows that 16 lanes touch lie in
// different banks
#define CL_PITCH 68
typedef float Tile[CL_TILE][CL_PITCH];

// The chunk `unit` (TOKENS tokens) of the step: which request it belongs to, its first row and its number of rows (0: no such chunk).
// All 256 threads call it; sh holds 8 ints.
template <int TOKENS>
__device__ __forceinline__ void find_chunk(const int* __restrict__ cu, int n_seqs, int unit, int* sh, int& seq, int& row0, int& count) {
    const int tid = threadIdx.x, lane = tid % MV_WAVE, wave = tid / MV_WAVE;
    if (tid == 0) sh[4] = -1;
    int base = 0;
    for (int s0 = 0; s0 < n_seqs; s0 += 256) {
        const int s = s0 + tid;
        const int first = s < n_seqs ? cu[s] : 0, len = s < n_seqs ? cu[s + 1] - first : 0;
        const int mine = (len + TOKENS - 1) / TOKENS;
        int incl = mine;
#pragma unroll
        for (int o = 1; o < MV_WAVE; o <<= 1) {
            const int t = __shfl_up(incl, o, MV_WAVE);
            if (lane >= o) incl += t;
        }
        __syncthreads();
        if (lane == MV_WAVE - 1) sh[wave] = incl;
        __syncthreads();
        int before = base;
        for (int w = 0; w < wave; ++w) before += sh[w];
        incl += before;
        if (unit < incl && unit >= incl - mine) {
            const int c = unit - (incl - mine);
            sh[4] = s;
            sh[5] = first + c * TOKENS;
            sh[6] = len - c * TOKENS < TOKENS ? len - c * TOKENS : TOKENS;
        }
        base += sh[0] + sh[1] + sh[2] + sh[3];
        if (base > unit) break;                        // (the same for every thread)
    }
    __syncthreads();
    seq = sh[4];
    row0 = sh[5];
    count = seq >= 0 ? sh[6] : 0;
}

// acc += A B^T over four k of each lane group: a and b hold a lane's four neighbours of the operands' rows
__device__ __forceinline__ void mfma4(floatx4_t& acc, const float4& a, const float4& b) {
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, acc, 0, 0, 0);
}

__device__ __forceinline__ float4 four(const Tile& t, int row, int k) { return *reinterpret_cast<const float4*>(&t[row][k]); }

// Number of chunks of TOKENS tokens in front of request `seq`'s first one; all 256 threads call it, part holds 4 ints
template <int TOKENS>
__device__ __forceinline__ int chunks_before(const int* __restrict__ cu, int seq, int* part) {
    int before = 0;
    for (int s = threadIdx.x; s < seq; s += 256) before += (cu[s + 1] - cu[s] + TOKENS - 1) / TOKENS;
#pragma unroll
    for (int o = MV_WAVE / 2; o > 0; o >>= 1) before += __shfl_xor(before, o, MV_WAVE);
    if (threadIdx.x % MV_WAVE == 0) part[threadIdx.x / MV_WAVE] = before;
    __syncthreads();
    return part[0] + part[1] + part[2] + part[3];
}
