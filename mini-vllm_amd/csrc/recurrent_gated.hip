// Gated linear attention: per head S [DK key channels][DV] <- diag(alpha) S + k v^T, o = S^T q, with a decay per key channel
// alpha = sigmoid(z)^(1/tau), z = W_a2 (W_a1 h) + bias. Packed rows from column `off` on: [q (H*DK) | k (H*DK) | v (H*DV) |
// g (H*DV)]; q is multiplied by DK^-1/2. States are floats [slots][H][DV][DK], a head's matrix column by column.
//
// Prompt portions: a request's tokens of the step are cut into chunks of CL_TOKENS. With i, j counted inside a chunk, G_i the
// sum of the tokens' log2 alpha up to and with i (a vector over key channels), G the chunk's whole sum, S the state in front:
//     o_i = (q_i * 2^G_i)^T S + sum_{j <= i} (sum_d q_id k_jd 2^(G_id - G_jd)) v_j
//     S'  = diag(2^G) S + sum_j (k_j * 2^(G - G_j)) v_j^T
// Decays are never inverted: between two runs of 16 tokens the ratio goes over the sum R at the end of the run in front of
// the query's, q 2^(G_i - R) and k 2^(R - G_j), both exponents <= 0; inside a run each pair takes its own exponential. All
// products are float (MFMA), whatever the activation type.
#include "qkv_conv.h"
#include "recurrent_chunk.h"

#define GL_MAX_RANK 512
#define GL_MAX_DV 256
#define GL_RUN 16                  // tokens of a run: the rows of one wave

struct GatedChunkArgs {
    const void* packed; long ld; int off;
    int H, DK, DV;
    int vec;                       // head sizes and rows allow eight columns a load
    const float* z; long ldz;      // W_a2 (W_a1 h), [n][H*DK]
    const float* bias;             // [H*DK]
    float to_log2;                 // log2(e) / tau
    const int* cu_seqlens; int n_seqs;
    float* sums;                   // [chunks][H][DV][DK]
    float* decays;                 // [chunks][H][DK]: 2^G
};

// G_i of up to CL_TOKENS rows x CL_TILE channels: dst[row][channel]; rows beyond `count` repeat the last sum
__device__ __forceinline__ void load_decays(Tile& dst, const GatedChunkArgs& A, int row0, int count, int head, int k0) {
    const int ch = threadIdx.x % CL_TILE, run = threadIdx.x / CL_TILE;            // four runs of 16 tokens
    const bool ok = k0 + ch < A.DK;
    const size_t col = (size_t)head * A.DK + (ok ? k0 + ch : 0);
    const float b = A.bias[col];
    float v[GL_RUN];
#pragma unroll
    for (int r = 0; r < GL_RUN; ++r) {
        const int t = run * GL_RUN + r;
        v[r] = A.z[(size_t)(row0 + (t < count ? t : 0)) * A.ldz + col];
    }
    float acc = 0.f;
#pragma unroll
    for (int r = 0; r < GL_RUN; ++r) {
        if (ok && run * GL_RUN + r < count) acc += logsigmoid_f(v[r] + b) * A.to_log2;
        v[r] = acc;
    }
    dst[run * GL_RUN + GL_RUN - 1][ch] = acc;
    __syncthreads();
    float before = 0.f;
    for (int s = 0; s < run; ++s) before += dst[s * GL_RUN + GL_RUN - 1][ch];
    __syncthreads();
#pragma unroll
    for (int r = 0; r < GL_RUN; ++r) dst[run * GL_RUN + r][ch] = v[r] + before;
}

// up to CL_TOKENS rows x CL_TILE channels as floats times `factor`, zero beyond the rows and channels there are: dst[row][channel],
// or TRANSPOSED dst[channel][row]; with WEIGHTED times 2^(G - G_row) of the row and channel (G: row CL_TOKENS - 1 of `decay`)
template <typename T, bool TRANSPOSED, bool WEIGHTED>
__device__ __forceinline__ void load_rows(Tile& dst, const T* __restrict__ src, long ld, int count, int c0, int C, bool vec, float factor,
                                          const Tile* decay) {
    if (vec) {
        for (int x = threadIdx.x; x < CL_TOKENS * (CL_TILE / 8); x += 256) {
            // (transposed: neighbouring lanes take neighbouring rows, so that they write neighbouring words)
            const int r = TRANSPOSED ? x % CL_TOKENS : x / (CL_TILE / 8), c = (TRANSPOSED ? x / CL_TOKENS : x % (CL_TILE / 8)) * 8;
            float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (r < count && c0 + c < C) Vec8<T>::load(src + (size_t)r * ld + c0 + c, v);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                float y = v[e] * factor;
                if (WEIGHTED) y *= exp2f((*decay)[CL_TOKENS - 1][c + e] - (*decay)[r][c + e]);
                if (TRANSPOSED) dst[c + e][r] = y;
                else dst[r][c + e] = y;
            }
        }
        return;
    }
    for (int x = threadIdx.x; x < CL_TOKENS * CL_TILE; x += 256) {
        const int r = TRANSPOSED ? x % CL_TOKENS : x / CL_TILE, c = TRANSPOSED ? x / CL_TOKENS : x % CL_TILE;
        float y = r < count && c0 + c < C ? to_f(src[(size_t)r * ld + c0 + c]) * factor : 0.f;
        if (WEIGHTED) y *= exp2f((*decay)[CL_TOKENS - 1][c] - (*decay)[r][c]);
        if (TRANSPOSED) dst[c][r] = y;
        else dst[r][c] = y;
    }
}

// ---- the chunks' sums: workgroup (chunk, head, tile of DV x tile of DK); a wave owns 16 rows (value channels) of the tile
template <typename T>
__global__ void __launch_bounds__(256)
gated_sums_kernel(GatedChunkArgs A) {
    __shared__ __attribute__((aligned(16))) Tile sK, sV, sG;                   // sK, sV transposed: [channel][token]
    __shared__ int sh[8];
    int seq, row0, count;
    find_chunk<CL_TOKENS>(A.cu_seqlens, A.n_seqs, blockIdx.x, sh, seq, row0, count);
    if (count <= 0) return;
    const int head = blockIdx.y, tk = (A.DK + CL_TILE - 1) / CL_TILE;
    const int k0 = (blockIdx.z % tk) * CL_TILE, v0 = (blockIdx.z / tk) * CL_TILE;
    const T* rows = (const T*)A.packed + (size_t)row0 * A.ld + A.off;
    load_rows<T, true, false>(sV, rows + 2 * (size_t)A.H * A.DK + (size_t)head * A.DV, A.ld, count, v0, A.DV, A.vec, 1.f, nullptr);
    load_decays(sG, A, row0, count, head, k0);
    __syncthreads();
    load_rows<T, true, true>(sK, rows + (size_t)(A.H + head) * A.DK, A.ld, count, k0, A.DK, A.vec, 1.f, &sG);
    if (v0 == 0 && threadIdx.x < CL_TILE && k0 + (int)threadIdx.x < A.DK)
        A.decays[((size_t)blockIdx.x * A.H + head) * A.DK + k0 + threadIdx.x] = exp2f(sG[CL_TOKENS - 1][threadIdx.x]);
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
gated_walk_kernel(GatedChunkArgs A, float* __restrict__ state, const int* __restrict__ state_slots) {
    __shared__ int part[4];
    const int seq = blockIdx.x, head = blockIdx.y;
    const int len = A.cu_seqlens[seq + 1] - A.cu_seqlens[seq];
    if (len <= 0) return;
    const int c0 = chunks_before<CL_TOKENS>(A.cu_seqlens, seq, part);
    const int chunks = (len + CL_TOKENS - 1) / CL_TOKENS;
    const int size = A.DV * A.DK, e = blockIdx.z * 256 + threadIdx.x;
    if (e >= size) return;
    float* st = state + ((size_t)state_slots[seq] * A.H + head) * size + e;
    float* m = A.sums + ((size_t)c0 * A.H + head) * size + e;
    const float* d = A.decays + ((size_t)c0 * A.H + head) * A.DK + e % A.DK;
    const size_t step = (size_t)A.H * size, dstep = (size_t)A.H * A.DK;
    float s = *st;
    constexpr int AHEAD = 8;
    for (int b = 0; b < chunks; b += AHEAD) {
        float v[AHEAD], a[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) {
            const int c = b + u < chunks ? b + u : b;
            v[u] = m[(size_t)c * step];
            a[u] = d[(size_t)c * dstep];
        }
#pragma unroll
        for (int u = 0; u < AHEAD; ++u)
            if (b + u < chunks) {
                m[(size_t)(b + u) * step] = s;
                s = fmaf(a[u], s, v[u]);
            }
    }
    *st = s;
}

__device__ __forceinline__ float4 exp2_4(const float4& a, const float4& b) {
    return float4{exp2f(a.x - b.x), exp2f(a.y - b.y), exp2f(a.z - b.z), exp2f(a.w - b.w)};
}
__device__ __forceinline__ float4 mul4(const float4& a, const float4& b) { return float4{a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w}; }

// ---- the outputs: workgroup (chunk, head, tile of DV); a wave owns a run of 16 tokens (rows). Over the tiles of DK: scores P
// of the wave's queries against the runs in front (products) and against its own run (pair by pair), and O += (2^G Q) S;
// then P goes through LDS into O += P V.
template <typename T>
__global__ void __launch_bounds__(256)
gated_out_kernel(GatedChunkArgs A, float* __restrict__ out) {
    // Q (then P), K (then V, transposed: [channel][key]), the decays' sums, S (a head's matrix column by column)
    __shared__ __attribute__((aligned(16))) Tile sQ, sK, sG, sS;
    __shared__ int sh[8];
    int seq, row0, count;
    find_chunk<CL_TOKENS>(A.cu_seqlens, A.n_seqs, blockIdx.x, sh, seq, row0, count);
    if (count <= 0) return;
    const int head = blockIdx.y, v0 = blockIdx.z * CL_TILE, DK = A.DK, DV = A.DV;
    const T* rows = (const T*)A.packed + (size_t)row0 * A.ld + A.off;
    const float* S = A.sums + ((size_t)blockIdx.x * A.H + head) * (size_t)DV * DK;
    const float unit = 1.f / sqrtf((float)DK);
    const int tid = threadIdx.x, lane = tid % MV_WAVE, wave = tid / MV_WAVE, i = lane % 16, g = lane / 16;
    floatx4_t p[3], o[4];
    float own[4] = {0.f, 0.f, 0.f, 0.f};                                       // scores of rows 16 wave + 4 g + r, key 16 wave + i
#pragma unroll
    for (int t = 0; t < 4; ++t) o[t] = floatx4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < 3; ++t) p[t] = floatx4_t{0.f, 0.f, 0.f, 0.f};
    const float4 zero{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < DK; k0 += CL_TILE) {
        if (k0 > 0) __syncthreads();
        load_rows<T, false, false>(sQ, rows + (size_t)head * DK, A.ld, count, k0, DK, A.vec, unit, nullptr);
        load_rows<T, false, false>(sK, rows + (size_t)(A.H + head) * DK, A.ld, count, k0, DK, A.vec, 1.f, nullptr);
        for (int x = tid; x < CL_TILE * CL_TILE; x += 256) {
            const int dv = x / CL_TILE, dk = x % CL_TILE;
            sS[dv][dk] = v0 + dv < DV && k0 + dk < DK ? S[(size_t)(v0 + dv) * DK + k0 + dk] : 0.f;
        }
        load_decays(sG, A, row0, count, head, k0);
        __syncthreads();
        const int steps = (min(CL_TILE, DK - k0) + 15) / 16;
        for (int s = 0; s < steps; ++s) {
            const int kk = 16 * s + 4 * g;
            const float4 q = four(sQ, 16 * wave + i, kk), gq = four(sG, 16 * wave + i, kk);
            const float4 ql = mul4(q, exp2_4(gq, zero));
#pragma unroll
            for (int t = 0; t < 4; ++t) mfma4(o[t], ql, four(sS, 16 * t + i, kk));
            if (wave > 0) {
                const float4 R = four(sG, 16 * wave - 1, kk);
                const float4 qr = mul4(q, exp2_4(gq, R));
#pragma unroll
                for (int t = 0; t < 3; ++t)
                    if (t < wave) mfma4(p[t], qr, mul4(four(sK, 16 * t + i, kk), exp2_4(R, four(sG, 16 * t + i, kk))));
            }
        }
        // the wave's own run: key i of the run against rows 4 g + r behind it
        const int width = min(CL_TILE, DK - k0);
        for (int d = 0; d < width; d += 4) {
            const float4 k = four(sK, 16 * wave + i, d), gk = four(sG, 16 * wave + i, d);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int row = 16 * wave + 4 * g + r;
                const float4 q = four(sQ, row, d), gq = four(sG, row, d);
                if (4 * g + r >= i) {
                    const float4 w = mul4(mul4(q, k), exp2_4(gq, gk));
                    own[r] += (w.x + w.y) + (w.z + w.w);
                }
            }
        }
    }
    __syncthreads();
    // P: lane holds column j = 16 t + i of rows 16 wave + 4 g + r
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int row = 16 * wave + 4 * g + r;
#pragma unroll
        for (int t = 0; t < 3; ++t)
            if (t < wave) sQ[row][16 * t + i] = p[t][r];
        sQ[row][16 * wave + i] = 4 * g + r >= i ? own[r] : 0.f;
    }
    load_rows<T, true, false>(sK, rows + 2 * (size_t)A.H * DK + (size_t)head * DV, A.ld, count, v0, DV, A.vec, 1.f, nullptr);
    __syncthreads();
    for (int s = 0; s <= wave; ++s) {                                          // keys up to the wave's last row
        const float4 a = four(sQ, 16 * wave + i, 16 * s + 4 * g);
#pragma unroll
        for (int t = 0; t < 4; ++t) mfma4(o[t], a, four(sK, 16 * t + i, 16 * s + 4 * g));
    }
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * wave + 4 * g + r, dv = v0 + 16 * t + i;
            if (row < count && dv < DV) out[((size_t)(row0 + row) * A.H + head) * DV + dv] = o[t][r];
        }
}

extern "C" int mv_gated_linear_chunk_tokens() { return CL_TOKENS; }

// `chunks`: the chunks of the step, or an upper bound (the rest of the grid ends at once); sums [chunks][H][DV][DK] and
// decays [chunks][H][DK] are scratch
extern "C" int mv_gated_linear_chunks(const void* packed, long ld, int off, int n, int H, int DK, int DV, const float* z, long ldz,
                                      const float* bias, float tau, float* state, const int* cu_seqlens, const int* state_slots,
                                      int n_seqs, int chunks, float* sums, float* decays, float* out, int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && n_seqs >= 0 && H > 0 && DK > 0 && DV > 0 && off >= 0 && chunks >= 0 && tau > 0.f,
               "gated_linear_chunks: bad sizes n=%d H=%d DK=%d DV=%d", n, H, DK, DV);
    MV_REQUIRE(ld >= off + 2L * H * DK + (long)H * DV && ldz >= (long)H * DK && packed && z && bias && state && cu_seqlens && state_slots &&
               sums && decays && out, "gated_linear_chunks: missing operand or rows too short");
    const int tk = (DK + CL_TILE - 1) / CL_TILE, tv = (DV + CL_TILE - 1) / CL_TILE;
    const long walk = ((long)DK * DV + 255) / 256;
    MV_REQUIRE(H <= 65535 && (long)tk * tv <= 65535 && walk <= 65535, "gated_linear_chunks: too many heads or channels");
    if (n == 0 || n_seqs == 0 || chunks == 0) return 0;
    const size_t esz = mv_dtype_size(dtype);
    const int vec = DK % 8 == 0 && DV % 8 == 0 && ((uintptr_t)packed % 16) == 0 && (ld * esz) % 16 == 0 && (off * esz) % 16 == 0;
    const GatedChunkArgs A{packed, ld, off, H, DK, DV, vec, z, ldz, bias, 1.4426950408889634f / tau, cu_seqlens, n_seqs, sums, decays};
    MV_DISPATCH_T(dtype, "gated_linear_chunks",
                  hipLaunchKernelGGL(gated_sums_kernel<T>, dim3(chunks, H, tk * tv), dim3(256), 0, stream, A));
    if (mv_check_launch("gated_sums")) return 1;
    hipLaunchKernelGGL(gated_walk_kernel, dim3(n_seqs, H, (unsigned)walk), dim3(256), 0, stream, A, state, state_slots);
    if (mv_check_launch("gated_walk")) return 1;
    MV_DISPATCH_T(dtype, "gated_linear_chunks",
                  hipLaunchKernelGGL(gated_out_kernel<T>, dim3(chunks, H, tv), dim3(256), 0, stream, A, out));
    return mv_check_launch("gated_out");
}

// ---------------------------------------------------------------------------------------
// A step of single tokens: W_a2, the decays, the recurrence, the head's norm and the output gate of one (row, head) in one
// workgroup. Row t is the one new token of request token_seq[t] (a padding row, < 0, gives zeros and touches no state). With
// `conv` given, the first `beside` workgroups of a row run the convolution and cache write of a softmax mixer that reads the
// same packed rows.
// ---------------------------------------------------------------------------------------
struct GatedStepArgs {
    const void* packed; long ld; int off, low_off, ra;
    int H, DK, DV;
    WeightPtr a2t;              // [ra][H*DK]
    const float* bias;          // [H*DK]
    float inv_tau;
    const float* norm_w;        // [DV]
    float eps;
    float* state;
    const int* token_seq; const int* state_slots;
    void* out; long ldo;
};

template <typename T, int R, int L>
__global__ void __launch_bounds__(256)
gated_step_kernel(GatedStepArgs A, ConvStoreArgs conv, int beside) {
    constexpr int DPAD = L * R;
    constexpr int COLS = 256 / L;
    __shared__ float low[GL_MAX_RANK];
    __shared__ float partial[256];
    __shared__ float va[DPAD];
    __shared__ float vals[GL_MAX_DV], outs[GL_MAX_DV];
    __shared__ float red[1];
    const int t = blockIdx.x, tid = threadIdx.x;
    if ((int)blockIdx.y < beside) {
        const int lanes = conv.D / 8;
        conv_store_vec<T>(conv, t, (int)blockIdx.y * (256 / lanes) + tid / lanes, tid % lanes);
        return;
    }
    const int head = (int)blockIdx.y - beside;
    const int H = A.H, DK = A.DK, DV = A.DV, nk = H * DK;
    const int seq = A.token_seq[t];
    T* y = (T*)A.out + (size_t)t * A.ldo + (size_t)head * DV;
    if (seq < 0) {
        for (int d = tid; d < DV; d += 256) y[d] = from_f<T>(0.f);
        return;
    }
    const int sub = tid % L, col = tid / L;
    // the first columns' state is asked for before anything else is computed
    float* S0 = A.state + ((size_t)A.state_slots[seq] * H + head) * (size_t)DV * DK;
    float s[R], s_next[R], q[R], k[R], a[R];
    delta_state_io<R, false>(s, S0 + (size_t)(col < DV ? col : 0) * DK, sub, DK, col < DV);
    const T* row = (const T*)A.packed + (size_t)t * A.ld;
    const T* p = row + A.off;
    for (int j = tid; j < A.ra; j += 256) low[j] = to_f(row[A.low_off + j]);
    const float unit = 1.f / sqrtf((float)DK);
#pragma unroll
    for (int e = 0; e < R; ++e) {
        const int d = sub * R + e, dc = d < DK ? d : 0;
        const float zq = to_f(p[head * DK + dc]), zk = to_f(p[nk + head * DK + dc]);
        q[e] = d < DK ? zq * unit : 0.f;
        k[e] = d < DK ? zk : 0.f;
    }
    for (int d = tid; d < DV; d += 256) vals[d] = to_f(p[2 * nk + head * DV + d]);
    __syncthreads();
    // W_a2 of this head, cut into `parts` runs of the rank
    const int parts = 256 / DK;                               // (DK <= 256)
    if (tid < parts * DK) {
        const int part = tid / DK, d = tid % DK;
        const int per = (A.ra + parts - 1) / parts;
        const int r0 = min(A.ra, part * per), r1 = min(A.ra, r0 + per);
        const size_t c = (size_t)head * DK + d;
        float acc[1] = {0.f};
        if (A.a2t.dtype == MV_F32) decay_dots<float, 1>((const float*)A.a2t.p + c, (size_t)nk, low, 0, r0, r1, acc);
        else decay_dots<bf16, 1>((const bf16*)A.a2t.p + c, (size_t)nk, low, 0, r0, r1, acc);
        partial[tid] = acc[0];
    }
    __syncthreads();
    if (tid < DPAD) {
        float alpha = 0.f;
        if (tid < DK) {
            float z = A.bias[(size_t)head * DK + tid];
            for (int part = 0; part < parts; ++part) z += partial[part * DK + tid];
            alpha = expf(logsigmoid_f(z) * A.inv_tau);
        }
        va[tid] = alpha;
    }
    __syncthreads();
#pragma unroll
    for (int e = 0; e < R; ++e) a[e] = va[sub * R + e];
    for (int j0 = 0; j0 < DV; j0 += COLS) {
        const int j = j0 + col;
        const bool live = j < DV;
        const int jn = j + COLS;
        // the next columns are asked for before these are stored: a load behind a store would wait for it
        if (j0 + COLS < DV) delta_state_io<R, false>(s_next, S0 + (size_t)(jn < DV ? jn : 0) * DK, sub, DK, jn < DV);
        const float v = vals[live ? j : 0];
        float o = 0.f;
#pragma unroll
        for (int e = 0; e < R; ++e) {
            s[e] = fmaf(a[e], s[e], k[e] * v);
            o = fmaf(q[e], s[e], o);
        }
        o = lanes_sum<L>(o);
        delta_state_io<R, true>(s, S0 + (size_t)(live ? j : 0) * DK, sub, DK, live);
        if (live && sub == 0) outs[j] = o;
#pragma unroll
        for (int e = 0; e < R; ++e) s[e] = s_next[e];
    }
    __syncthreads();
    if (tid < MV_WAVE) {
        float ss = 0.f;
        for (int d = tid; d < DV; d += MV_WAVE) ss = fmaf(outs[d], outs[d], ss);
        ss = wave_sum(ss);
        if (tid == 0) red[0] = 1.f / sqrtf(ss / (float)DV + A.eps);
    }
    __syncthreads();
    const float rinv = red[0];
    const T* g = p + 2 * nk + H * DV + head * DV;
    for (int d = tid; d < DV; d += 256) y[d] = from_f<T>(outs[d] * rinv * A.norm_w[d] * silu_f(to_f(g[d])));
}

// `rows` .. describe the softmax mixer whose convolution and cache write ride along (rows null: none). Returns 2 (nothing done)
// for sizes it does not serve, with or without that mixer.
extern "C" int mv_gated_linear_step(const void* packed, long ld, int off, int low_off, int n, int H, int DK, int DV, int ra,
                                    const void* a2t, int a2_dtype, const float* bias, float tau, const float* norm_w, float eps,
                                    float* state, const int* token_seq, const int* state_slots, void* out, long ldo,
                                    const void* rows, long rows_ld, int base, int QH, int QHkv, int QD, int QDv, int taps,
                                    const float* conv_w, void* conv_state, const int* positions, const int* cu_seqlens,
                                    const int* block_table, int bt_width, int page_size, void* k_pages, void* v_pages,
                                    const float* table, int rot, int unit_norm, float conv_eps, void* conv_out, long conv_ldo,
                                    int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && H > 0 && DK > 0 && DV > 0 && off >= 0 && low_off >= 0 && ra > 0 && tau > 0.f && eps > 0.f,
               "gated_linear_step: bad sizes n=%d H=%d DK=%d DV=%d rank=%d", n, H, DK, DV, ra);
    if (DK > 256 || DV > GL_MAX_DV || ra > GL_MAX_RANK) return 2;
    MV_REQUIRE(ld >= off + 2L * H * DK + 2L * H * DV && ld >= (long)low_off + ra && ldo >= (long)H * DV, "gated_linear_step: rows too short");
    MV_REQUIRE(packed && a2t && mv_valid_dtype(a2_dtype) && bias && norm_w && state && token_seq && state_slots && out,
               "gated_linear_step: missing operand");
    ConvStoreArgs conv{};
    int beside = 0;
    if (rows != nullptr) {
        conv = ConvStoreArgs{rows, rows_ld, base, n, QH, QHkv, QD, QDv, taps, conv_w, conv_state, taps > 1, positions, token_seq, cu_seqlens,
                             state_slots, block_table, bt_width, page_size, k_pages, v_pages, table, table ? rot : 0, unit_norm, conv_eps,
                             conv_out, conv_ldo, 1};
        if (int rc = conv_store_check(conv)) return rc;
        if (!conv_store_vec_ok(conv, dtype)) return 2;
        const int per = 256 / (QD / 8);
        beside = (QH + 2 * QHkv + per - 1) / per;
    }
    MV_REQUIRE((long)H + beside <= 65535, "gated_linear_step: too many heads");
    if (n == 0) return 0;
    const GatedStepArgs A{packed, ld, off, low_off, ra, H, DK, DV, WeightPtr{a2t, a2_dtype}, bias, 1.f / tau, norm_w, eps, state,
                          token_seq, state_slots, out, ldo};
    int R = 0, L = 0;
    delta_scan_shape(DK, R, L);
    const dim3 grid(n, H + beside);
#define GS_LAUNCH(RR, LL)                                                                                                   \
    MV_DISPATCH_T(dtype, "gated_linear_step",                                                                               \
                  hipLaunchKernelGGL((gated_step_kernel<T, RR, LL>), grid, dim3(256), 0, stream, A, conv, beside))
    if (R == 4 && L == 4) {
        GS_LAUNCH(4, 4);
    } else if (R == 4 && L == 8) {
        GS_LAUNCH(4, 8);
    } else if (R == 4 && L == 16) {
        GS_LAUNCH(4, 16);
    } else if (R == 8 && L == 16) {
        GS_LAUNCH(8, 16);
    } else {
        GS_LAUNCH(16, 16);
    }
#undef GS_LAUNCH
    return mv_check_launch("gated_linear_step");
}
