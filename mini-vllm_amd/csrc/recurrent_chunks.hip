// Linear attention with one constant decay per head, S <- a S + k v^T, o = S^T q, for steps with prompt portions: a
// request's tokens of the step are cut into chunks of CL_TOKENS, and everything that only concerns one chunk is a
// product of small matrices on the MFMA units (float operands: v_mfma_f32_16x16x4_f32), chunks side by side. With i, j
// counted inside a chunk of C tokens and S the state in front of it:
//     o_i  = a^(i+1) S^T q_i + sum_{j <= i} a^(i-j) (q_i . k_j) v_j
//     S'   = a^C S + sum_j a^(C-1-j) k_j v_j^T
// Three launches: each chunk's sum of a^(C-1-j) k_j v_j^T; the walk along a request's chunks that turns these sums into
// the states in front of the chunks (element by element) and leaves the request's new state; the outputs.
// q, k and v are SiLU of the packed rows' columns [q (H*DK) | k (H*DK) | v (H*DV)] from column `off` on. States and
// the chunks' sums are floats [..][H][DV][DK], a head's matrix column by column. Powers of the decay are 2^(n log2 a),
// so 0 < a <= 1.
#include "recurrent_chunk.h"

// silu of up to CL_TOKENS rows x CL_TILE channels into LDS, zero beyond the rows and channels there are: dst[row][channel],
// or TRANSPOSED dst[channel][row], there multiplied by 2^((count - 1 - row) * l2) when WEIGHTED
template <typename T, bool TRANSPOSED, bool WEIGHTED>
__device__ __forceinline__ void load_tile(Tile& dst, const T* __restrict__ src, long ld, int count, int c0, int C, bool vec, float l2) {
    if (vec) {
        for (int x = threadIdx.x; x < CL_TOKENS * (CL_TILE / 8); x += 256) {
            // (transposed: neighbouring lanes take neighbouring rows, so that they write neighbouring words)
            const int r = TRANSPOSED ? x % CL_TOKENS : x / (CL_TILE / 8), c = (TRANSPOSED ? x / CL_TOKENS : x % (CL_TILE / 8)) * 8;
            float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            const bool ok = r < count && c0 + c < C;
            if (ok) Vec8<T>::load(src + (size_t)r * ld + c0 + c, v);
            const float w = WEIGHTED && ok ? exp2f((float)(count - 1 - r) * l2) : 1.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float z = silu_f(v[e]) * w;                              // silu(0) = 0
                if (TRANSPOSED) dst[c + e][r] = z;
                else dst[r][c + e] = z;
            }
        }
        return;
    }
    for (int x = threadIdx.x; x < CL_TOKENS * CL_TILE; x += 256) {
        const int r = TRANSPOSED ? x % CL_TOKENS : x / CL_TILE, c = TRANSPOSED ? x / CL_TOKENS : x % CL_TILE;
        const bool ok = r < count && c0 + c < C;
        const float z = ok ? silu_f(to_f(src[(size_t)r * ld + c0 + c])) * (WEIGHTED ? exp2f((float)(count - 1 - r) * l2) : 1.f) : 0.f;
        if (TRANSPOSED) dst[c][r] = z;
        else dst[r][c] = z;
    }
}

struct ChunkArgs {
    const void* packed; long ld; int off;
    int H, DK, DV;
    int vec;                       // head sizes and rows allow eight columns a load
    const float* decay;
    const int* cu_seqlens; int n_seqs;
    float* sums;                   // [chunks][H][DV][DK]
};

// ---- the chunks' sums: workgroup (chunk, head, tile of DV x tile of DK); a wave owns 16 rows (value channels) of the tile
template <typename T>
__global__ void __launch_bounds__(256)
chunk_sums_kernel(ChunkArgs A) {
    __shared__ __attribute__((aligned(16))) Tile sK, sV;                       // transposed: [channel][token]
    __shared__ int sh[8];
    int seq, row0, count;
    find_chunk<CL_TOKENS>(A.cu_seqlens, A.n_seqs, blockIdx.x, sh, seq, row0, count);
    if (count <= 0) return;
    const int head = blockIdx.y, tk = (A.DK + CL_TILE - 1) / CL_TILE;
    const int k0 = (blockIdx.z % tk) * CL_TILE, v0 = (blockIdx.z / tk) * CL_TILE;
    const float l2 = log2f(A.decay[head]);
    const T* rows = (const T*)A.packed + (size_t)row0 * A.ld + A.off;
    load_tile<T, true, false>(sK, rows + (size_t)(A.H + head) * A.DK, A.ld, count, k0, A.DK, A.vec, l2);
    load_tile<T, true, true>(sV, rows + 2 * (size_t)A.H * A.DK + (size_t)head * A.DV, A.ld, count, v0, A.DV, A.vec, l2);
    __syncthreads();
    const int lane = threadIdx.x % MV_WAVE, wave = threadIdx.x / MV_WAVE, i = lane % 16, g = lane / 16;
    floatx4_t acc[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) acc[t] = floatx4_t{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < (count + 15) / 16; ++s) {
        const float4 a = four(sV, 16 * wave + i, 16 * s + 4 * g);
#pragma unroll
        for (int t = 0; t < 4; ++t) mfma4(acc[t], a, four(sK, 16 * t + i, 16 * s + 4 * g));
    }
    float* out = A.sums + ((size_t)blockIdx.x * A.H + head) * (size_t)A.DV * A.DK;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int dv = v0 + 16 * wave + 4 * g + r, dk = k0 + 16 * t + i;
            if (dv < A.DV && dk < A.DK) out[(size_t)dv * A.DK + dk] = acc[t][r];
        }
}

// ---- the walk: thread per element of a head's matrix; sums[c] becomes the state in front of chunk c, state the one behind
// the last. Eight chunks' sums are asked for at a time.
__global__ void __launch_bounds__(256)
chunk_walk_kernel(ChunkArgs A, float* __restrict__ state, const int* __restrict__ state_slots) {
    __shared__ int part[4];
    const int seq = blockIdx.x, head = blockIdx.y;
    const int len = A.cu_seqlens[seq + 1] - A.cu_seqlens[seq];
    if (len <= 0) return;
    const int c0 = chunks_before<CL_TOKENS>(A.cu_seqlens, seq, part);
    const int chunks = (len + CL_TOKENS - 1) / CL_TOKENS;
    const int size = A.DV * A.DK, e = blockIdx.z * 256 + threadIdx.x;
    if (e >= size) return;
    const float l2 = log2f(A.decay[head]);
    const float full = exp2f((float)CL_TOKENS * l2), tail = exp2f((float)(len - (chunks - 1) * CL_TOKENS) * l2);
    float* st = state + ((size_t)state_slots[seq] * A.H + head) * size + e;
    float* m = A.sums + ((size_t)c0 * A.H + head) * size + e;
    const size_t step = (size_t)A.H * size;
    float s = *st;
    constexpr int AHEAD = 8;
    for (int b = 0; b < chunks; b += AHEAD) {
        float v[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) v[u] = m[(size_t)(b + u < chunks ? b + u : b) * step];
#pragma unroll
        for (int u = 0; u < AHEAD; ++u)
            if (b + u < chunks) {
                m[(size_t)(b + u) * step] = s;
                s = fmaf(b + u == chunks - 1 ? tail : full, s, v[u]);
            }
    }
    *st = s;
}

// ---- the outputs: workgroup (chunk, head, tile of DV); a wave owns 16 tokens (rows). Over the tiles of DK: scores
// P += Q K^T and O += (a^(i+1) Q) S; then P, masked and decayed, goes through LDS into O += P V.
template <typename T>
__global__ void __launch_bounds__(256)
chunk_out_kernel(ChunkArgs A, float* __restrict__ out) {
    // Q (then P), K (then V, transposed: [channel][key]), S (a head's matrix column by column: [value channel][key channel])
    __shared__ __attribute__((aligned(16))) Tile s0, s1, s2;
    __shared__ int sh[8];
    int seq, row0, count;
    find_chunk<CL_TOKENS>(A.cu_seqlens, A.n_seqs, blockIdx.x, sh, seq, row0, count);
    if (count <= 0) return;
    const int head = blockIdx.y, v0 = blockIdx.z * CL_TILE, DK = A.DK, DV = A.DV;
    const T* rows = (const T*)A.packed + (size_t)row0 * A.ld + A.off;
    const float* S = A.sums + ((size_t)blockIdx.x * A.H + head) * (size_t)DV * DK;
    const float l2 = log2f(A.decay[head]);
    const int tid = threadIdx.x, lane = tid % MV_WAVE, wave = tid / MV_WAVE, i = lane % 16, g = lane / 16;
    floatx4_t p[4], o[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) p[t] = o[t] = floatx4_t{0.f, 0.f, 0.f, 0.f};
    const float lead = exp2f((float)(16 * wave + i + 1) * l2);                 // a^(i+1) of the lane's operand row
    for (int k0 = 0; k0 < DK; k0 += CL_TILE) {
        if (k0 > 0) __syncthreads();
        load_tile<T, false, false>(s0, rows + (size_t)head * DK, A.ld, count, k0, DK, A.vec, l2);
        load_tile<T, false, false>(s1, rows + (size_t)(A.H + head) * DK, A.ld, count, k0, DK, A.vec, l2);
        for (int x = tid; x < CL_TILE * CL_TILE; x += 256) {
            const int dv = x / CL_TILE, dk = x % CL_TILE;
            s2[dv][dk] = v0 + dv < DV && k0 + dk < DK ? S[(size_t)(v0 + dv) * DK + k0 + dk] : 0.f;
        }
        __syncthreads();
        const int steps = (min(CL_TILE, DK - k0) + 15) / 16;
        for (int s = 0; s < steps; ++s) {
            const float4 q = four(s0, 16 * wave + i, 16 * s + 4 * g);
            const float4 ql = float4{q.x * lead, q.y * lead, q.z * lead, q.w * lead};
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                if (t <= wave) mfma4(p[t], q, four(s1, 16 * t + i, 16 * s + 4 * g));
                mfma4(o[t], ql, four(s2, 16 * t + i, 16 * s + 4 * g));
            }
        }
    }
    __syncthreads();
    // P: lane holds column j = 16 t + i of rows 16 wave + 4 g + r
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * wave + 4 * g + r, j = 16 * t + i;
            s0[row][j] = j <= row ? p[t][r] * exp2f((float)(row - j) * l2) : 0.f;
        }
    load_tile<T, true, false>(s1, rows + 2 * (size_t)A.H * DK + (size_t)head * DV, A.ld, count, v0, DV, A.vec, l2);
    __syncthreads();
    for (int s = 0; s <= wave; ++s) {                                          // keys up to the wave's last row
        const float4 a = four(s0, 16 * wave + i, 16 * s + 4 * g);
#pragma unroll
        for (int t = 0; t < 4; ++t) mfma4(o[t], a, four(s1, 16 * t + i, 16 * s + 4 * g));
    }
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * wave + 4 * g + r, dv = v0 + 16 * t + i;
            if (row < count && dv < DV) out[((size_t)(row0 + row) * A.H + head) * DV + dv] = o[t][r];
        }
}

extern "C" int mv_constant_chunk_tokens() { return CL_TOKENS; }

// `chunks`: the chunks of the step, or an upper bound (the rest of the grid ends at once); sums: [chunks][H][DV][DK]
extern "C" int mv_constant_chunks(const void* packed, long ld, int off, int n, int H, int DK, int DV, const float* decay,
                                  float* state, const int* cu_seqlens, const int* state_slots, int n_seqs, int chunks, float* sums,
                                  float* out, int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && n_seqs >= 0 && H > 0 && DK > 0 && DV > 0 && off >= 0 && chunks >= 0, "constant_chunks: bad sizes n=%d H=%d DK=%d DV=%d",
               n, H, DK, DV);
    MV_REQUIRE(ld >= off + 2L * H * DK + (long)H * DV && packed && decay && state && cu_seqlens && state_slots && sums && out,
               "constant_chunks: missing operand or rows too short");
    const int tk = (DK + CL_TILE - 1) / CL_TILE, tv = (DV + CL_TILE - 1) / CL_TILE;
    const long walk = ((long)DK * DV + 255) / 256;
    MV_REQUIRE(H <= 65535 && (long)tk * tv <= 65535 && walk <= 65535, "constant_chunks: too many heads or channels");
    if (n == 0 || n_seqs == 0 || chunks == 0) return 0;
    const size_t esz = mv_dtype_size(dtype);
    const int vec = DK % 8 == 0 && DV % 8 == 0 && ((uintptr_t)packed % 16) == 0 && (ld * esz) % 16 == 0 && (off * esz) % 16 == 0;
    const ChunkArgs A{packed, ld, off, H, DK, DV, vec, decay, cu_seqlens, n_seqs, sums};
    MV_DISPATCH_T(dtype, "constant_chunks",
                  hipLaunchKernelGGL(chunk_sums_kernel<T>, dim3(chunks, H, tk * tv), dim3(256), 0, stream, A));
    if (mv_check_launch("chunk_sums")) return 1;
    hipLaunchKernelGGL(chunk_walk_kernel, dim3(n_seqs, H, (unsigned)walk), dim3(256), 0, stream, A, state, state_slots);
    if (mv_check_launch("chunk_walk")) return 1;
    MV_DISPATCH_T(dtype, "constant_chunks",
                  hipLaunchKernelGGL(chunk_out_kernel<T>, dim3(chunks, H, tv), dim3(256), 0, stream, A, out));
    return mv_check_launch("chunk_out");
}
