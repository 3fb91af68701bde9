// The real-gated linear recurrent unit: one number of state per channel, S <- a S + sqrt(1 - a^2) i u with
//     r = sigmoid(zr + br), i = sigmoid(zi + bi), log a = rate r     (rate = -c softplus(lam), a float per channel)
// u is a causal convolution (with bias) of one half of the packed rows, zr and zi are products of u's parts with square
// matrices, and the output is S * gelu_tanh(y), y the other half. Packed rows: [x (W) | ... y (W) at y_off]. The state is
// float [slots][W]; the convolution's kept inputs [slots][taps-1][W] have the activation type. W channels form B parts of
// P = W / B; gate products are rows [B][2 P], a part's r products in front of its i products.
#include "recurrent_chunk.h"

#define RU_TOKENS 32               // tokens of a chunk of the scan

__device__ __forceinline__ float gelu_tanh_f(float z) {
    // tanh(t) = 1 - 2 / (1 + e^2t): exact at both ends
    const float t = 0.7978845608028654f * (z + 0.044715f * z * z * z);
    return z * (1.f - 1.f / (1.f + expf(2.f * t)));
}

// decay and input of one channel and token
__device__ __forceinline__ void unit_coefficients(float zr, float zi, float u, float rate, float& a, float& x) {
    const float log_a = rate * sigmoid_f(zr);
    a = expf(log_a);
    x = sqrtf(-expm1f(2.f * log_a)) * sigmoid_f(zi) * u;
}

// ---------------------------------------------------------------------------------------
// A causal convolution with bias of C channels from column 0 of the rows: u[t][c] = bias[c] + sum_j w[j][c] x_(t-taps+1+j)
// (w float [taps][C]); eight channels a thread where everything is aligned, one otherwise
// ---------------------------------------------------------------------------------------
struct ShortConvArgs {
    const void* rows; long ld;
    int n, C, taps;
    const float* w; const float* bias;      // bias may be null
    const void* conv_state;
    const int* token_seq; const int* cu_seqlens; const int* state_slots;
    void* out; long ldo;
};

template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
short_conv_kernel(ShortConvArgs A) {
    constexpr int E = VEC ? 8 : 1;
    const int per_row = A.C / E;
    const long gid = (long)blockIdx.x * 256 + threadIdx.x;
    const int t = (int)(gid / per_row), c = (int)(gid % per_row) * E;
    if (t >= A.n) return;
    const int seq = A.token_seq[t];
    T* out = (T*)A.out + (size_t)t * A.ldo + c;
    float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (seq >= 0) {
        const int first = A.cu_seqlens[seq];
        const T* rows = (const T*)A.rows + c;
        const T* hist = (const T*)A.conv_state + (A.taps > 1 ? (size_t)A.state_slots[seq] * (A.taps - 1) * A.C : 0) + c;
        if constexpr (VEC) {
            if (A.bias) Vec8<float>::load(A.bias + c, x);
        } else {
            if (A.bias) x[0] = A.bias[c];
        }
        for (int j = 0; j < A.taps; ++j) {
            const int r = t - (A.taps - 1) + j;
            const T* src = r >= first ? rows + (size_t)r * A.ld : hist + (size_t)(A.taps - 1 + r - first) * A.C;
            if constexpr (VEC) {
                float in[8], w[8];
                Vec8<T>::load(src, in);
                Vec8<float>::load(A.w + (size_t)j * A.C + c, w);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = fmaf(w[e], in[e], x[e]);
            } else {
                x[0] = fmaf(A.w[(size_t)j * A.C + c], to_f(*src), x[0]);
            }
        }
    }
    if constexpr (VEC) Vec8<T>::store(out, x);
    else *out = from_f<T>(x[0]);
}

// out = the convolution of columns 0 .. C-1 of the rows; the kept inputs are moved on afterwards
extern "C" int mv_short_conv(const void* rows, long ld, int n, int n_seqs, int C, int taps, const float* w, const float* bias,
                             void* conv_state, const int* token_seq, const int* cu_seqlens, const int* state_slots, void* out,
                             long ldo, int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && n_seqs >= 0 && C > 0 && ld >= C && ldo >= C, "short_conv: bad sizes n=%d C=%d", n, C);
    MV_REQUIRE(taps >= 1 && taps <= MS_MAX_TAPS, "short_conv: %d taps, 1 to %d are served", taps, MS_MAX_TAPS);
    MV_REQUIRE(rows && w && (conv_state || taps == 1) && token_seq && cu_seqlens && state_slots && out && (C + 255) / 256 <= 65535,
               "short_conv: missing operand");
    if (n == 0) return 0;
    const ShortConvArgs A{rows, ld, n, C, taps, w, bias, conv_state, token_seq, cu_seqlens, state_slots, out, ldo};
    const size_t esz = mv_dtype_size(dtype);
    const bool vec = C % 8 == 0 && ((uintptr_t)rows % 16) == 0 && (ld * esz) % 16 == 0 && ((uintptr_t)w % 16) == 0 &&
                     ((uintptr_t)bias % 16) == 0 && ((uintptr_t)conv_state % 16) == 0 && ((uintptr_t)out % 16) == 0 && (ldo * esz) % 16 == 0;
    const long threads = (long)n * (vec ? C / 8 : C);
    MV_REQUIRE(threads < (1L << 38), "short_conv: too many rows");
    const dim3 grid((unsigned)((threads + 255) / 256));
    MV_DISPATCH_T(dtype, "short_conv",
                  if (vec) hipLaunchKernelGGL((short_conv_kernel<T, true>), grid, dim3(256), 0, stream, A);
                  else hipLaunchKernelGGL((short_conv_kernel<T, false>), grid, dim3(256), 0, stream, A));
    if (mv_check_launch("short_conv")) return 1;
    if (taps > 1 && n_seqs > 0) {
        MV_DISPATCH_T(dtype, "conv_state",
                      hipLaunchKernelGGL(conv_state_kernel<T>, dim3(n_seqs, (unsigned)((C + 255) / 256)), dim3(256), 0, stream,
                                         (const T*)rows, ld, C, taps, (T*)conv_state, cu_seqlens, state_slots));
        return mv_check_launch("conv_state");
    }
    return 0;
}

// ---------------------------------------------------------------------------------------
// The scan over a step's tokens, a request's tokens in chunks of RU_TOKENS side by side: each chunk's decay and its state
// from zero; the walk along a request's chunks, which turns these into the states in front of the chunks and leaves the
// request's new state; the outputs. A thread owns one channel of one chunk.
// ---------------------------------------------------------------------------------------
struct UnitScanArgs {
    const float* z;                         // [n][B][2 P]
    const void* u; long ldu;
    const void* packed; long ld; int y_off;
    int W, P;
    const float* gate_bias;                 // [2][W]
    const float* rate;                      // [W]
    const int* cu_seqlens; int n_seqs;
    float* sums;                            // [chunks][2][W]: decay, state from zero (then: state in front of the chunk)
};

template <typename T, bool OUT>
__global__ void __launch_bounds__(256)
unit_chunk_kernel(UnitScanArgs A, T* __restrict__ out, long ldo) {
    __shared__ int sh[8];
    int seq, row0, count;
    find_chunk<RU_TOKENS>(A.cu_seqlens, A.n_seqs, blockIdx.x, sh, seq, row0, count);
    if (count <= 0) return;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= A.W) return;
    const int part = c / A.P, k = c % A.P;
    const float br = A.gate_bias[c], bi = A.gate_bias[A.W + c], rate = A.rate[c];
    float* sum = A.sums + (size_t)blockIdx.x * 2 * A.W + c;
    const float* z = A.z + (size_t)row0 * 2 * A.W + (size_t)part * 2 * A.P + k;
    const T* u = (const T*)A.u + (size_t)row0 * A.ldu + c;
    const T* y = (const T*)A.packed + (size_t)row0 * A.ld + A.y_off + c;
    float s = OUT ? sum[A.W] : 0.f, decay = 1.f;
    constexpr int AHEAD = 8;
    for (int b = 0; b < count; b += AHEAD) {
        float zr[AHEAD], zi[AHEAD], uu[AHEAD], yy[AHEAD];
#pragma unroll
        for (int e = 0; e < AHEAD; ++e) {
            const size_t r = b + e < count ? b + e : b;
            zr[e] = z[r * 2 * A.W];
            zi[e] = z[r * 2 * A.W + A.P];
            uu[e] = to_f(u[r * A.ldu]);
            if (OUT) yy[e] = to_f(y[r * A.ld]);
        }
#pragma unroll
        for (int e = 0; e < AHEAD; ++e)
            if (b + e < count) {
                float a, x;
                unit_coefficients(zr[e] + br, zi[e] + bi, uu[e], rate, a, x);
                s = fmaf(a, s, x);
                decay *= a;
                if (OUT) out[(size_t)(row0 + b + e) * ldo + c] = from_f<T>(s * gelu_tanh_f(yy[e]));
            }
    }
    if (!OUT) {
        sum[0] = decay;
        sum[A.W] = s;
    }
}

__global__ void __launch_bounds__(256)
unit_walk_kernel(UnitScanArgs A, float* __restrict__ state, const int* __restrict__ state_slots) {
    __shared__ int part[4];
    const int seq = blockIdx.x;
    const int len = A.cu_seqlens[seq + 1] - A.cu_seqlens[seq];
    if (len <= 0) return;
    const int c0 = chunks_before<RU_TOKENS>(A.cu_seqlens, seq, part);
    const int chunks = (len + RU_TOKENS - 1) / RU_TOKENS;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= A.W) return;
    float* st = state + (size_t)state_slots[seq] * A.W + c;
    float* m = A.sums + (size_t)c0 * 2 * A.W + c;
    float s = *st;
    constexpr int AHEAD = 16;
    for (int b = 0; b < chunks; b += AHEAD) {
        float a[AHEAD], v[AHEAD];
#pragma unroll
        for (int e = 0; e < AHEAD; ++e) {
            const size_t k = b + e < chunks ? b + e : b;
            a[e] = m[k * 2 * A.W];
            v[e] = m[k * 2 * A.W + A.W];
        }
#pragma unroll
        for (int e = 0; e < AHEAD; ++e)
            if (b + e < chunks) {
                m[(size_t)(b + e) * 2 * A.W + A.W] = s;
                s = fmaf(a[e], s, v[e]);
            }
    }
    *st = s;
}

extern "C" int mv_unit_chunk_tokens() { return RU_TOKENS; }

// `chunks`: the chunks of the step, or an upper bound (the rest of the grid ends at once); sums [chunks][2][W] is scratch.
// Rows of padding are not written.
extern "C" int mv_unit_scan(const float* z, const void* u, long ldu, const void* packed, long ld, int y_off, int n, int W, int B,
                            const float* gate_bias, const float* rate, float* state, const int* cu_seqlens, const int* state_slots,
                            int n_seqs, int chunks, float* sums, void* out, long ldo, int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && n_seqs >= 0 && W > 0 && B > 0 && W % B == 0 && chunks >= 0 && y_off >= 0, "unit_scan: bad sizes n=%d W=%d B=%d", n, W, B);
    MV_REQUIRE(z && u && ldu >= W && packed && ld >= (long)y_off + W && gate_bias && rate && state && cu_seqlens && state_slots && sums && out
               && ldo >= W && (W + 255) / 256 <= 65535, "unit_scan: missing operand or rows too short");
    if (n == 0 || n_seqs == 0 || chunks == 0) return 0;
    const UnitScanArgs A{z, u, ldu, packed, ld, y_off, W, W / B, gate_bias, rate, cu_seqlens, n_seqs, sums};
    const unsigned tiles = (unsigned)((W + 255) / 256);
    MV_DISPATCH_T(dtype, "unit_scan", hipLaunchKernelGGL((unit_chunk_kernel<T, false>), dim3(chunks, tiles), dim3(256), 0, stream, A,
                                                         (T*)nullptr, 0L));
    if (mv_check_launch("unit_chunk")) return 1;
    hipLaunchKernelGGL(unit_walk_kernel, dim3(n_seqs, tiles), dim3(256), 0, stream, A, state, state_slots);
    if (mv_check_launch("unit_walk")) return 1;
    MV_DISPATCH_T(dtype, "unit_scan", hipLaunchKernelGGL((unit_chunk_kernel<T, true>), dim3(chunks, tiles), dim3(256), 0, stream, A,
                                                         (T*)out, ldo));
    return mv_check_launch("unit_out");
}

// ---------------------------------------------------------------------------------------
// A step of single tokens in one launch: workgroup (ROWS rows, part) makes the part's u (moving the kept inputs on), both
// gate products from the weight with the inputs' rows outside ([B][P inputs][2 P outputs], eight outputs a load, the inputs
// dealt out over the threads and added through LDS), and the recurrence. Row t is the one new token of request token_seq[t]
// (a padding row gives zeros and touches no state).
// ---------------------------------------------------------------------------------------
struct UnitStepArgs {
    const void* packed; long ld; int y_off;
    int n, W, P, taps;
    const float* w; const float* conv_bias;
    void* conv_state;
    WeightPtr gates;
    const float* gate_bias; const float* rate;
    float* state;
    const int* token_seq; const int* state_slots;
    void* out; long ldo;
};

#define RU_MAX_PART 512
#define RU_THREADS 1024

// acc[row][e] += the slice's inputs times the weights of eight neighbouring outputs (w points at the first); four rows of weights
// are asked for at a time
template <typename TW, int ROWS>
__device__ __forceinline__ void unit_dots(const TW* __restrict__ w, int P, int slice, int slices, const float (&su)[ROWS][RU_MAX_PART],
                                          float (&acc)[ROWS][8]) {
    for (int k0 = slice; k0 < P; k0 += 4 * slices) {
        float v[4][8];
#pragma unroll
        for (int q = 0; q < 4; ++q) Vec8<TW>::load(w + (size_t)min(k0 + q * slices, P - 1) * 2 * P, v[q]);
#pragma unroll
        for (int q = 0; q < 4; ++q)
            if (k0 + q * slices < P)
#pragma unroll
                for (int r = 0; r < ROWS; ++r)
#pragma unroll
                    for (int e = 0; e < 8; ++e) acc[r][e] = fmaf(su[r][k0 + q * slices], v[q][e], acc[r][e]);
    }
}

template <typename T, int ROWS>
__global__ void __launch_bounds__(RU_THREADS)
unit_step_kernel(UnitStepArgs A) {
    __shared__ float su[ROWS][RU_MAX_PART];
    __shared__ float partial[ROWS][RU_THREADS * 8];        // [slice][2 P]
    __shared__ float sums[ROWS][2 * RU_MAX_PART];
    const int t0 = blockIdx.x * ROWS, part = blockIdx.y, tid = threadIdx.x;
    const int W = A.W, P = A.P, taps = A.taps;
    for (int e = tid; e < ROWS * P; e += RU_THREADS) {
        const int r = e / P, k = e % P, t = t0 + r, c = part * P + k;
        const int seq = t < A.n ? A.token_seq[t] : -1;
        float acc = 0.f;
        if (seq >= 0) {
            T* hist = (T*)A.conv_state + (taps > 1 ? (size_t)A.state_slots[seq] * (taps - 1) * W : 0) + c;
            const T now = ((const T*)A.packed)[(size_t)t * A.ld + c];
            acc = A.conv_bias[c];
            if (taps == 4) {                                // everything is asked for before anything is used or stored
                const T x0 = hist[0], x1 = hist[(size_t)W], x2 = hist[2 * (size_t)W];
                const float w0 = A.w[c], w1 = A.w[(size_t)W + c], w2 = A.w[2 * (size_t)W + c];
                acc = fmaf(w2, to_f(x2), fmaf(w1, to_f(x1), fmaf(w0, to_f(x0), acc)));
                hist[0] = x1;
                hist[(size_t)W] = x2;
            } else {
                for (int j = 0; j < taps - 1; ++j) {
                    const T x = hist[(size_t)j * W];
                    acc = fmaf(A.w[(size_t)j * W + c], to_f(x), acc);
                    if (j > 0) hist[(size_t)(j - 1) * W] = x;
                }
            }
            acc = fmaf(A.w[(size_t)(taps - 1) * W + c], to_f(now), acc);
            if (taps > 1) hist[(size_t)(taps - 2) * W] = now;
        }
        su[r][k] = to_f(from_f<T>(acc));                    // as the rows of a prompt store it
    }
    __syncthreads();
    const int groups = 2 * P / 8, slices = RU_THREADS / groups;
    const int o = (tid % groups) * 8, slice = tid / groups;
    if (slice < slices) {
        float acc[ROWS][8];
#pragma unroll
        for (int r = 0; r < ROWS; ++r)
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[r][e] = 0.f;
        const size_t w0 = (size_t)part * P * 2 * P + o;
        if (A.gates.dtype == MV_F32) unit_dots<float, ROWS>((const float*)A.gates.p + w0, P, slice, slices, su, acc);
        else unit_dots<bf16, ROWS>((const bf16*)A.gates.p + w0, P, slice, slices, su, acc);
#pragma unroll
        for (int r = 0; r < ROWS; ++r) Vec8<float>::store(&partial[r][slice * 2 * P + o], acc[r]);
    }
    __syncthreads();
    // the slices of an output are added by eight neighbouring lanes (all lanes of a wave take part: 16 P is a multiple of 64)
    for (int e = tid; e < ROWS * 2 * P * 8; e += RU_THREADS) {
        const int r = e / (16 * P), j = e / 8 % (2 * P);
        float v = 0.f;
        for (int s = e % 8; s < slices; s += 8) v += partial[r][s * 2 * P + j];
        v += __shfl_xor(v, 1, MV_WAVE);
        v += __shfl_xor(v, 2, MV_WAVE);
        v += __shfl_xor(v, 4, MV_WAVE);
        if (e % 8 == 0) sums[r][j] = v;
    }
    __syncthreads();
    for (int e = tid; e < ROWS * P; e += RU_THREADS) {
        const int r = e / P, k = e % P, t = t0 + r, c = part * P + k;
        if (t >= A.n) continue;
        T* out = (T*)A.out + (size_t)t * A.ldo + c;
        const int seq = A.token_seq[t];
        if (seq < 0) {
            *out = from_f<T>(0.f);
            continue;
        }
        const float zr = A.gate_bias[c] + sums[r][k], zi = A.gate_bias[W + c] + sums[r][P + k];
        float a, x;
        unit_coefficients(zr, zi, su[r][k], A.rate[c], a, x);
        float* st = A.state + (size_t)A.state_slots[seq] * W + c;
        const float s = fmaf(a, *st, x);
        *st = s;
        *out = from_f<T>(s * gelu_tanh_f(to_f(((const T*)A.packed)[(size_t)t * A.ld + A.y_off + c])));
    }
}

// Returns 2 (nothing done) for sizes it does not serve.
extern "C" int mv_unit_step(const void* packed, long ld, int y_off, int n, int W, int B, int taps, const float* w, const float* conv_bias,
                            void* conv_state, const void* gates, int gates_dtype, const float* gate_bias, const float* rate,
                            float* state, const int* token_seq, const int* state_slots, void* out, long ldo, int dtype,
                            hipStream_t stream) {
    MV_REQUIRE(n >= 0 && W > 0 && B > 0 && W % B == 0 && y_off >= W, "unit_step: bad sizes n=%d W=%d B=%d", n, W, B);
    MV_REQUIRE(taps >= 1 && taps <= MS_MAX_TAPS, "unit_step: %d taps, 1 to %d are served", taps, MS_MAX_TAPS);
    MV_REQUIRE(packed && ld >= (long)y_off + W && w && conv_bias && (conv_state || taps == 1) && gates && mv_valid_dtype(gates_dtype) &&
               gate_bias && rate && state && token_seq && state_slots && out && ldo >= W && B <= 65535, "unit_step: missing operand");
    const int P = W / B;
    if (P % 4 != 0 || P > RU_MAX_PART || ((uintptr_t)gates % 16) != 0) return 2;
    if (n == 0) return 0;
    const UnitStepArgs A{packed, ld, y_off, n, W, P, taps, w, conv_bias, conv_state, WeightPtr{gates, gates_dtype}, gate_bias, rate, state,
                         token_seq, state_slots, out, ldo};
    // (several rows a workgroup share its pass over the weight once the rows fill the chip)
    if ((long)n * B <= 2L * mv_compute_units()) {
        MV_DISPATCH_T(dtype, "unit_step", hipLaunchKernelGGL((unit_step_kernel<T, 1>), dim3(n, B), dim3(RU_THREADS), 0, stream, A));
    } else {
        MV_DISPATCH_T(dtype, "unit_step", hipLaunchKernelGGL((unit_step_kernel<T, 2>), dim3((n + 1) / 2, B), dim3(RU_THREADS), 0, stream, A));
    }
    return mv_check_launch("unit_step");
}
