// The gated delta rule with a decay per head and key channel. Per head, S [key size DK][columns DV]:
//     S <- diag(g) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// q, k and v pass a short causal convolution over time per channel and SiLU, q and k become unit vectors per
// group (q also times DK^-1/2); beta = sigmoid(b); g = exp(-exp(A_log[h]) softplus(z + dt_bias)), z = W_a2 (W_a1 h).
// Packed rows: [q (G*DK) | k (G*DK) | v (H*DV) | ... b (H) at b_off ... | a1 (ra) and g1 (rg) at low_off]. The two
// low-rank products come as floats z[n][ldz] = [decay (H*DK) | output gate (H*DV)] for prompts; a step of single tokens
// makes them itself from the transposed second matrices. States are [slots][H][DV][DK] floats, a head's matrix
// column by column; the convolution's kept inputs [slots][taps-1][C] have the activation type.
#include "recurrent.h"

#define CD_MAX_RANK 512

// ---------------------------------------------------------------------------------------
// Prepare: unit queries and keys qk [n][G][2][DK], values vals [n][H][DV], writing strengths beta [n][H], and the
// decays in place of the decay columns of z. Workgroup (row, unit): units 0..G-1 make a group's q and k, units
// G..G+H-1 a head's values, decays and beta.
// ---------------------------------------------------------------------------------------
struct ChannelRows {
    const void* packed; long ld;
    int H, G, DK, DV, taps;
    int b_off;
    WeightPtr conv_w, a_log, dt_bias;
    float unit_eps;
};

template <typename T>
__global__ void __launch_bounds__(128)
channel_prepare_kernel(ChannelRows A, const T* __restrict__ conv_state, const int* __restrict__ token_seq,
                       const int* __restrict__ cu_seqlens, const int* __restrict__ state_slots, float* __restrict__ qk,
                       float* __restrict__ vals, float* __restrict__ beta, float* __restrict__ z, long ldz) {
    __shared__ float scratch[17];
    const int t = blockIdx.x, unit = blockIdx.y, tid = threadIdx.x;
    const int seq = token_seq[t];
    if (seq < 0) return;                                   // a padding row: nobody reads its vectors
    const int G = A.G, H = A.H, DK = A.DK, DV = A.DV, taps = A.taps;
    const int C = 2 * G * DK + H * DV;
    const int first = cu_seqlens[seq];
    const T* packed = (const T*)A.packed;
    const T* hist = conv_state + (size_t)state_slots[seq] * (taps - 1) * C;
    auto conv = [&](int c) {
        float acc = 0.f;
        for (int j = 0; j < taps; ++j)
            acc = fmaf(A.conv_w.at((size_t)c * taps + j), conv_input(packed, A.ld, hist, C, taps, first, t - (taps - 1) + j, c), acc);
        return silu_f(acc);
    };
    if (unit < G) {
        // a thread keeps its (at most two) channels of both vectors between the sum and the scaling
        float x[2][2], ss[2] = {0.f, 0.f};
#pragma unroll
        for (int which = 0; which < 2; ++which) {
            int u = 0;
#pragma unroll
            for (int d0 = 0; d0 < 256; d0 += 128, ++u) {
                const int d = d0 + tid;
                x[which][u] = d < DK ? conv(which * G * DK + unit * DK + d) : 0.f;
                ss[which] = fmaf(x[which][u], x[which][u], ss[which]);
            }
        }
        const float sq = wave_sum(ss[0]), sk = wave_sum(ss[1]);
        if (tid % MV_WAVE == 0) {
            scratch[tid / MV_WAVE] = sq;
            scratch[2 + tid / MV_WAVE] = sk;
        }
        __syncthreads();
        const float inv[2] = {(1.f / sqrtf((float)DK)) / sqrtf(scratch[0] + scratch[1] + A.unit_eps),
                              1.f / sqrtf(scratch[2] + scratch[3] + A.unit_eps)};
        float* o = qk + ((size_t)t * G + unit) * 2 * DK;
#pragma unroll
        for (int which = 0; which < 2; ++which)
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int d = u * 128 + tid;
                if (d < DK) o[which * DK + d] = x[which][u] * inv[which];
            }
        return;
    }
    const int head = unit - G;
    float* o = vals + ((size_t)t * H + head) * DV;
    for (int d = tid; d < DV; d += 128) o[d] = conv(2 * G * DK + head * DV + d);
    const float rate = -expf(A.a_log.at(head));
    float* zr = z + (size_t)t * ldz + (size_t)head * DK;
    for (int d = tid; d < DK; d += 128) zr[d] = expf(rate * softplus_f(zr[d] + A.dt_bias.at((size_t)head * DK + d)));
    if (tid == 0) beta[(size_t)t * H + head] = sigmoid_f(to_f(packed[(size_t)t * A.ld + A.b_off + head]));
}

// The same for CP_ROWS neighbouring rows a workgroup and 2 to 4 taps: a thread's filter stays in registers, and a row's
// input is read once for all the taps it falls under. The sums are those of the kernel above, term by term.
#define CP_ROWS 8

// silu(convolution) of channel c in rows t0 .. t0 + CP_ROWS - 1 (first[r]: row r's request's first row, -1 for a row
// that does not count; hist[r]: the request's kept inputs)
template <typename T, int TAPS>
__device__ __forceinline__ void conv_rows(float (&x)[CP_ROWS], const ChannelRows& A, const T* __restrict__ conv_state,
                                          const int (&first)[CP_ROWS], const int (&slot)[CP_ROWS], int t0, int n, int C, int c) {
    const T* packed = (const T*)A.packed;
    float w[TAPS], in[CP_ROWS + TAPS - 1];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j] = A.conv_w.at((size_t)c * TAPS + j);
#pragma unroll
    for (int i = 0; i < CP_ROWS + TAPS - 1; ++i) {
        const int r = min(max(t0 - (TAPS - 1) + i, 0), n - 1);
        in[i] = to_f(packed[(size_t)r * A.ld + c]);
    }
#pragma unroll
    for (int r = 0; r < CP_ROWS; ++r) {
        float acc = 0.f;
        if (t0 + r - (TAPS - 1) >= first[r]) {
#pragma unroll
            for (int j = 0; j < TAPS; ++j) acc = fmaf(w[j], in[r + j], acc);
        } else {
            const T* hist = conv_state + (size_t)slot[r] * (TAPS - 1) * C;
#pragma unroll
            for (int j = 0; j < TAPS; ++j)
                acc = fmaf(w[j], conv_input(packed, A.ld, hist, C, TAPS, first[r], t0 + r - (TAPS - 1) + j, c), acc);
        }
        x[r] = silu_f(acc);
    }
}

template <typename T, int TAPS>
__global__ void __launch_bounds__(128)
channel_prepare_rows_kernel(ChannelRows A, const T* __restrict__ conv_state, const int* __restrict__ token_seq,
                            const int* __restrict__ cu_seqlens, const int* __restrict__ state_slots, int n, float* __restrict__ qk,
                            float* __restrict__ vals, float* __restrict__ beta, float* __restrict__ z, long ldz) {
    __shared__ float scratch[CP_ROWS][4];
    const int t0 = blockIdx.x * CP_ROWS, unit = blockIdx.y, tid = threadIdx.x;
    const int G = A.G, H = A.H, DK = A.DK, DV = A.DV;
    const int C = 2 * G * DK + H * DV;
    int first[CP_ROWS], slot[CP_ROWS];
    bool live[CP_ROWS];
#pragma unroll
    for (int r = 0; r < CP_ROWS; ++r) {
        // (a row that does not count is computed as if it were row 0's request's first row and not stored)
        const int seq = t0 + r < n ? token_seq[t0 + r] : -1;
        live[r] = seq >= 0;
        first[r] = live[r] ? cu_seqlens[seq] : -TAPS;
        slot[r] = live[r] ? state_slots[seq] : 0;
    }
    if (unit < G) {
        float x[2][2][CP_ROWS];
#pragma unroll
        for (int which = 0; which < 2; ++which)
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int d = u * 128 + tid;
                if (d < DK) conv_rows<T, TAPS>(x[which][u], A, conv_state, first, slot, t0, n, C, which * G * DK + unit * DK + d);
                else
#pragma unroll
                    for (int r = 0; r < CP_ROWS; ++r) x[which][u][r] = 0.f;
            }
#pragma unroll
        for (int r = 0; r < CP_ROWS; ++r) {
            const float sq = wave_sum(fmaf(x[0][1][r], x[0][1][r], x[0][0][r] * x[0][0][r]));
            const float sk = wave_sum(fmaf(x[1][1][r], x[1][1][r], x[1][0][r] * x[1][0][r]));
            if (tid % MV_WAVE == 0) {
                scratch[r][tid / MV_WAVE] = sq;
                scratch[r][2 + tid / MV_WAVE] = sk;
            }
        }
        __syncthreads();
#pragma unroll
        for (int r = 0; r < CP_ROWS; ++r) {
            if (!live[r]) continue;
            const float inv[2] = {(1.f / sqrtf((float)DK)) / sqrtf(scratch[r][0] + scratch[r][1] + A.unit_eps),
                                  1.f / sqrtf(scratch[r][2] + scratch[r][3] + A.unit_eps)};
            float* o = qk + ((size_t)(t0 + r) * G + unit) * 2 * DK;
#pragma unroll
            for (int which = 0; which < 2; ++which)
#pragma unroll
                for (int u = 0; u < 2; ++u) {
                    const int d = u * 128 + tid;
                    if (d < DK) o[which * DK + d] = x[which][u][r] * inv[which];
                }
        }
        return;
    }
    const int head = unit - G;
    for (int d = tid; d < DV; d += 128) {
        float x[CP_ROWS];
        conv_rows<T, TAPS>(x, A, conv_state, first, slot, t0, n, C, 2 * G * DK + head * DV + d);
#pragma unroll
        for (int r = 0; r < CP_ROWS; ++r)
            if (live[r]) vals[((size_t)(t0 + r) * H + head) * DV + d] = x[r];
    }
    const float rate = -expf(A.a_log.at(head));
    for (int d = tid; d < DK; d += 128) {
        const float bias = A.dt_bias.at((size_t)head * DK + d);
        float x[CP_ROWS];
#pragma unroll
        for (int r = 0; r < CP_ROWS; ++r) x[r] = live[r] ? z[(size_t)(t0 + r) * ldz + (size_t)head * DK + d] : 0.f;
#pragma unroll
        for (int r = 0; r < CP_ROWS; ++r)
            if (live[r]) z[(size_t)(t0 + r) * ldz + (size_t)head * DK + d] = expf(rate * softplus_f(x[r] + bias));
    }
    const int row = t0 + tid;
    if (tid < CP_ROWS && row < n && token_seq[row] >= 0)
        beta[(size_t)row * H + head] = sigmoid_f(to_f(((const T*)A.packed)[(size_t)row * A.ld + A.b_off + head]));
}

static int channel_check(const char* what, const ChannelRows& A, int n, int n_seqs, const void* conv_state) {
    MV_REQUIRE(n >= 0 && n_seqs >= 0 && A.H > 0 && A.G > 0 && A.H % A.G == 0 && A.DK > 0 && A.DV > 0,
               "%s: bad sizes n=%d H=%d G=%d DK=%d DV=%d", what, n, A.H, A.G, A.DK, A.DV);
    MV_REQUIRE(A.DK <= 256, "%s: key size %d exceeds the supported maximum 256", what, A.DK);
    MV_REQUIRE(A.taps >= 1 && A.taps <= MS_MAX_TAPS, "%s: %d taps, 1 to %d are served", what, A.taps, MS_MAX_TAPS);
    const long C = 2L * A.G * A.DK + (long)A.H * A.DV;
    MV_REQUIRE(A.b_off >= C && A.ld >= (long)A.b_off + A.H, "%s: rows of %ld columns are too short", what, A.ld);
    MV_REQUIRE(A.packed && A.conv_w.p && A.a_log.p && A.dt_bias.p && mv_valid_dtype(A.conv_w.dtype) && (conv_state || A.taps == 1),
               "%s: missing operand", what);
    MV_REQUIRE(A.unit_eps > 0.f && A.G + A.H <= 65535 && (C + 255) / 256 <= 65535, "%s: bad constants", what);
    return 0;
}

extern "C" int mv_channel_prepare(const void* packed, long ld, int n, int n_seqs, int H, int G, int DK, int DV, int taps, int b_off,
                                  const void* conv_w, const void* a_log, const void* dt_bias, int weight_dtype, void* conv_state,
                                  float unit_eps, const int* token_seq, const int* cu_seqlens, const int* state_slots, float* qk,
                                  float* vals, float* beta, float* z, long ldz, int dtype, hipStream_t stream) {
    const ChannelRows A{packed, ld, H, G, DK, DV, taps, b_off, WeightPtr{conv_w, weight_dtype}, WeightPtr{a_log, weight_dtype},
                        WeightPtr{dt_bias, weight_dtype}, unit_eps};
    if (int rc = channel_check("channel_prepare", A, n, n_seqs, conv_state)) return rc;
    MV_REQUIRE(token_seq && cu_seqlens && state_slots && qk && vals && beta && z && ldz >= (long)H * DK, "channel_prepare: missing operand");
    if (n == 0) return 0;
#define CHANNEL_ROWS(TAPS)                                                                                                 \
    MV_DISPATCH_T(dtype, "channel_prepare",                                                                               \
                  hipLaunchKernelGGL((channel_prepare_rows_kernel<T, TAPS>), dim3((n + CP_ROWS - 1) / CP_ROWS, G + H), dim3(128), \
                                     0, stream, A, (const T*)conv_state, token_seq, cu_seqlens, state_slots, n, qk, vals, beta, \
                                     z, ldz))
    // (few rows fill the chip only one a workgroup)
    if (taps < 2 || taps > 4 || (long)n * (G + H) < 2L * CP_ROWS * mv_compute_units()) {
        MV_DISPATCH_T(dtype, "channel_prepare",
                      hipLaunchKernelGGL(channel_prepare_kernel<T>, dim3(n, G + H), dim3(128), 0, stream, A, (const T*)conv_state,
                                         token_seq, cu_seqlens, state_slots, qk, vals, beta, z, ldz));
    } else if (taps == 2) {
        CHANNEL_ROWS(2);
    } else if (taps == 3) {
        CHANNEL_ROWS(3);
    } else {
        CHANNEL_ROWS(4);
    }
#undef CHANNEL_ROWS
    if (mv_check_launch("channel_prepare")) return 1;
    if (taps > 1 && n_seqs > 0) {
        const int C = 2 * G * DK + H * DV;
        MV_DISPATCH_T(dtype, "conv_state",
                      hipLaunchKernelGGL(conv_state_kernel<T>, dim3(n_seqs, (unsigned)((C + 255) / 256)), dim3(256), 0, stream,
                                         (const T*)packed, ld, C, taps, (T*)conv_state, cu_seqlens, state_slots));
        return mv_check_launch("conv_state");
    }
    return 0;
}

// ---------------------------------------------------------------------------------------
// The scan: a workgroup of 256 threads owns 256 / L columns of one head of one request, L neighbouring lanes share a
// column and keep R of its DK rows each. The vectors of a run of tokens are staged in LDS in two buffers: the next
// run's loads from memory are in flight while this run is computed, and a token's vectors come from LDS into
// registers while the token before it is computed. The additions of a token depend on nothing but the sizes.
// ---------------------------------------------------------------------------------------
template <int R>
struct ChannelToken {
    float q[R], k[R], g[R], v, b;
};

// one token of one column: the lane's R rows in s; returns the column's output
template <int R, int L>
__device__ __forceinline__ float channel_update(float (&s)[R], const ChannelToken<R>& t) {
    float read = 0.f;
#pragma unroll
    for (int e = 0; e < R; ++e) {
        s[e] *= t.g[e];
        read = fmaf(t.k[e], s[e], read);
    }
    const float u = t.b * (t.v - lanes_sum<L>(read));
    float o = 0.f;
#pragma unroll
    for (int e = 0; e < R; ++e) {
        s[e] = fmaf(t.k[e], u, s[e]);
        o = fmaf(t.q[e], s[e], o);
    }
    return lanes_sum<L>(o);
}

// V4: DK a multiple of four and every vector 16-byte aligned: the staged vectors come in 16 bytes a lane
template <int R, int L, bool V4>
__global__ void __launch_bounds__(256)
channel_scan_kernel(const float* __restrict__ qk, const float* __restrict__ vals, const float* __restrict__ beta,
                    const float* __restrict__ decay, long ldz, float* __restrict__ state, const int* __restrict__ cu_seqlens,
                    const int* __restrict__ state_slots, int H, int G, int DK, int DV, float* __restrict__ out) {
    constexpr int DPAD = L * R;
    constexpr int COLS = 256 / L;
    constexpr int TT = DPAD > 128 ? 4 : (DPAD > 64 ? 8 : 16);          // tokens staged at a time
    constexpr int WORDS = TT * 3 * DPAD;                                // q, k, g of a run
    constexpr int NVEC = V4 ? (WORDS / 4 + 255) / 256 : (WORDS + 255) / 256;
    constexpr int NVAL = (TT * COLS + 255) / 256;
    __shared__ __attribute__((aligned(16))) float sv[2][TT][3][DPAD];
    __shared__ float sx[2][TT][COLS];
    __shared__ float sb[2][TT];
    const int seq = blockIdx.x, head = blockIdx.y, j0 = blockIdx.z * COLS;
    const int begin = cu_seqlens[seq], end = cu_seqlens[seq + 1];
    if (end <= begin) return;
    const int tid = threadIdx.x, sub = tid % L, col = tid / L;
    const int j = j0 + col;
    const bool live = j < DV;
    const int group = head / (H / G);
    float* S = state + (((size_t)state_slots[seq] * H + head) * DV + (live ? j : 0)) * (size_t)DK;
    float s[R];
    delta_state_io<R, false>(s, S, sub, DK, live);
    // where vector `which` (0: q, 1: k, 2: g) of row t starts
    auto vector_of = [&](int t, int which) {
        return which < 2 ? qk + (((size_t)t * G + group) * 2 + which) * DK : decay + (size_t)t * ldz + (size_t)head * DK;
    };
    float gv[V4 ? 1 : NVEC], gx[NVAL], gb = 0.f;
    float4 g4[V4 ? NVEC : 1];
    int fetched = 0;
    // (loads are issued whatever the index, from clamped addresses, and dropped where they do not count)
    auto fetch = [&](int base) {
        const int nt = min(TT, end - base);
        fetched = nt;
#pragma unroll
        for (int x = 0; x < NVEC; ++x) {
            const int w = (tid + x * 256) * (V4 ? 4 : 1);
            const int tt = w / (3 * DPAD), rem = w % (3 * DPAD), which = rem / DPAD, i = rem % DPAD;
            const float* p = vector_of(base + (tt < nt ? tt : 0), which < 3 ? which : 0) + (i < DK ? i : 0);
            if constexpr (V4) g4[x] = *reinterpret_cast<const float4*>(p);
            else gv[x] = *p;
        }
#pragma unroll
        for (int x = 0; x < NVAL; ++x) {
            const int e = tid + x * 256, tt = e / COLS, jj = e % COLS;
            gx[x] = vals[((size_t)(base + (tt < nt ? tt : 0)) * H + head) * DV + (j0 + jj < DV ? j0 + jj : 0)];
        }
        if (tid < TT) gb = beta[(size_t)(base + (tid < nt ? tid : 0)) * H + head];
    };
    auto stash = [&](int buf) {
        float* dst = &sv[buf][0][0][0];
#pragma unroll
        for (int x = 0; x < NVEC; ++x) {
            const int w = (tid + x * 256) * (V4 ? 4 : 1);
            const int tt = w / (3 * DPAD), i = w % DPAD;
            const bool ok = tt < fetched && i < DK;
            if (w < WORDS) {
                if constexpr (V4) *reinterpret_cast<float4*>(dst + w) = ok ? g4[x] : float4{0.f, 0.f, 0.f, 0.f};
                else dst[w] = ok ? gv[x] : 0.f;
            }
        }
#pragma unroll
        for (int x = 0; x < NVAL; ++x) {
            const int e = tid + x * 256;
            if (e < TT * COLS) (&sx[buf][0][0])[e] = gx[x];
        }
        if (tid < TT) sb[buf][tid] = gb;
    };
    auto read_token = [&](ChannelToken<R>& t, int buf, int tt) {
        const float* p = &sv[buf][tt][0][0] + sub * R;
#pragma unroll
        for (int e = 0; e < R; ++e) {
            t.q[e] = p[e];
            t.k[e] = p[DPAD + e];
            t.g[e] = p[2 * DPAD + e];
        }
        t.v = sx[buf][tt][col];
        t.b = sb[buf][tt];
    };
    fetch(begin);
    stash(0);
    __syncthreads();
    int buf = 0;
    for (int base = begin; base < end; base += TT, buf ^= 1) {
        const int nt = min(TT, end - base);
        const bool more = base + TT < end;
        if (more) fetch(base + TT);                        // in flight while this run is computed
        ChannelToken<R> ta, tb;
        read_token(ta, buf, 0);
        for (int tt = 0; tt < nt; tt += 2) {
            if (tt + 1 < nt) read_token(tb, buf, tt + 1);
            const float o0 = channel_update<R, L>(s, ta);
            if (live && sub == 0) out[((size_t)(base + tt) * H + head) * DV + j] = o0;
            if (tt + 1 < nt) {
                if (tt + 2 < nt) read_token(ta, buf, tt + 2);
                const float o1 = channel_update<R, L>(s, tb);
                if (live && sub == 0) out[((size_t)(base + tt + 1) * H + head) * DV + j] = o1;
            }
        }
        if (more) stash(buf ^ 1);                          // nobody reads that buffer: its run was computed before the last barrier
        __syncthreads();
    }
    delta_state_io<R, true>(s, S, sub, DK, live);
}

extern "C" int mv_channel_scan(const float* qk, const float* vals, const float* beta, const float* decay, long ldz, float* state,
                               const int* cu_seqlens, const int* state_slots, int n_seqs, int n, int H, int G, int DK, int DV,
                               float* out, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && n_seqs >= 0 && H > 0 && G > 0 && H % G == 0 && DK > 0 && DV > 0,
               "channel_scan: bad sizes n=%d seqs=%d H=%d G=%d DK=%d DV=%d", n, n_seqs, H, G, DK, DV);
    MV_REQUIRE(DK <= 256, "channel_scan: key size %d exceeds the supported maximum 256", DK);
    MV_REQUIRE(qk && vals && beta && decay && ldz >= (long)H * DK && state && cu_seqlens && state_slots && out, "channel_scan: missing operand");
    int R = 0, L = 0;
    delta_scan_shape(DK, R, L);
    const int cols = 256 / L;
    MV_REQUIRE(H <= 65535 && (DV + cols - 1) / cols <= 65535, "channel_scan: too many heads or columns");
    if (n == 0 || n_seqs == 0) return 0;
    const dim3 grid(n_seqs, H, (DV + cols - 1) / cols);
    const bool v4 = DK % 4 == 0 && ldz % 4 == 0 && ((uintptr_t)qk % 16) == 0 && ((uintptr_t)decay % 16) == 0;
#define CS_LAUNCH(RR, LL)                                                                                                     \
    if (v4)                                                                                                                   \
        hipLaunchKernelGGL((channel_scan_kernel<RR, LL, true>), grid, dim3(256), 0, stream, qk, vals, beta, decay, ldz, state, \
                           cu_seqlens, state_slots, H, G, DK, DV, out);                                                       \
    else                                                                                                                      \
        hipLaunchKernelGGL((channel_scan_kernel<RR, LL, false>), grid, dim3(256), 0, stream, qk, vals, beta, decay, ldz, state, \
                           cu_seqlens, state_slots, H, G, DK, DV, out);
    if (R == 4 && L == 4) {
        CS_LAUNCH(4, 4)
    } else if (R == 4 && L == 8) {
        CS_LAUNCH(4, 8)
    } else if (R == 4 && L == 16) {
        CS_LAUNCH(4, 16)
    } else if (R == 8 && L == 16) {
        CS_LAUNCH(8, 16)
    } else {
        CS_LAUNCH(16, 16)
    }
#undef CS_LAUNCH
    return mv_check_launch("channel_scan");
}

// ---------------------------------------------------------------------------------------
// A step of single tokens: the low-rank products, prepare, the recurrence, the head's norm and the output gate of one
// (row, head) in one workgroup. Row t is the one new token of request token_seq[t] (a padding row, < 0, gives zeros and
// touches no state). `own_conv`: every head has query and key channels of its own (G == H), so the workgroup moves the
// convolution's kept inputs on itself; otherwise conv_state_kernel does it afterwards.
// ---------------------------------------------------------------------------------------
struct ChannelStepArgs {
    ChannelRows rows;
    int low_off, ra, rg;
    WeightPtr a2t, g2t;         // [ra][H*DK], [rg][H*DV]
    WeightPtr norm_w;           // [DV]
    void* conv_state;
    float* state;
    float eps;
    int own_conv;
    const int* token_seq;
    const int* state_slots;
    void* out;
    long ldo;
};

#define CD_MAX_DV 256

template <typename T, int R, int L>
__global__ void __launch_bounds__(256)
channel_step_kernel(ChannelStepArgs A) {
    constexpr int DPAD = L * R;
    constexpr int COLS = 256 / L;
    __shared__ float low[2 * CD_MAX_RANK];
    __shared__ float partial[DPAD + CD_MAX_DV > 256 ? DPAD + CD_MAX_DV : 256];
    __shared__ float vq[DPAD], vk[DPAD], vg[DPAD];
    __shared__ float vals[CD_MAX_DV], gate[CD_MAX_DV], outs[CD_MAX_DV];
    __shared__ float red[8];
    const ChannelRows& P = A.rows;
    const int H = P.H, G = P.G, DK = P.DK, DV = P.DV, taps = P.taps;
    const int t = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
    const int lane = tid % MV_WAVE, wave = tid / MV_WAVE;
    const int seq = A.token_seq[t];
    T* y = (T*)A.out + (size_t)t * A.ldo + (size_t)head * DV;
    if (seq < 0) {
        for (int d = tid; d < DV; d += 256) y[d] = from_f<T>(0.f);
        return;
    }
    const int slot = A.state_slots[seq];
    const T* p = (const T*)P.packed + (size_t)t * P.ld;
    const int C = 2 * G * DK + H * DV, group = head / (H / G);
    const int sub = tid % L, col = tid / L;
    // the first columns' state is asked for before anything else is computed
    float* S0 = A.state + ((size_t)slot * H + head) * (size_t)DV * DK;
    float s[R], s_next[R];
    delta_state_io<R, false>(s, S0 + (size_t)(col < DV ? col : 0) * DK, sub, DK, col < DV);
    for (int j = tid; j < A.ra + A.rg; j += 256) low[j] = to_f(p[A.low_off + j]);
    T* hist = (T*)A.conv_state + (size_t)slot * (taps - 1) * C;
    // the row is its request's only one in the step: every earlier input comes from the kept ones
    auto conv = [&](int c) {
        float acc = 0.f;
        for (int j = 0; j < taps - 1; ++j) {
            const T x = hist[(size_t)j * C + c];
            acc = fmaf(P.conv_w.at((size_t)c * taps + j), to_f(x), acc);
            if (A.own_conv && j > 0) hist[(size_t)(j - 1) * C + c] = x;
        }
        const T now = p[c];
        if (A.own_conv && taps > 1) hist[(size_t)(taps - 2) * C + c] = now;
        acc = fmaf(P.conv_w.at((size_t)c * taps + taps - 1), to_f(now), acc);
        return silu_f(acc);
    };
    // half of the threads take the query's and key's channels, the other half the values'
    float sq = 0.f, sk = 0.f, xq[2] = {0.f, 0.f}, xk[2] = {0.f, 0.f};
    if (tid < 128) {
        int u = 0;
        for (int d = tid; d < DK; d += 128, ++u) {
            xq[u] = conv(group * DK + d);
            xk[u] = conv(G * DK + group * DK + d);
            sq = fmaf(xq[u], xq[u], sq);
            sk = fmaf(xk[u], xk[u], sk);
        }
        sq = wave_sum(sq);
        sk = wave_sum(sk);
        if (lane == 0) {
            red[wave] = sq;
            red[2 + wave] = sk;
        }
    } else {
        for (int d = tid - 128; d < DV; d += 128) vals[d] = conv(2 * G * DK + head * DV + d);
    }
    __syncthreads();
    if (tid < 128) {
        const float iq = (1.f / sqrtf((float)DK)) / sqrtf(red[0] + red[1] + P.unit_eps);
        const float ik = 1.f / sqrtf(red[2] + red[3] + P.unit_eps);
        int u = 0;
        for (int d = tid; d < DPAD; d += 128, ++u) {
            vq[d] = d < DK ? xq[u] * iq : 0.f;
            vk[d] = d < DK ? xk[u] * ik : 0.f;
        }
    }
    // the two low-rank products of this head: DK decays and DV gates, each cut into `parts` runs of the rank
    const int outs_n = DK + DV;
    const int parts = outs_n >= 256 ? 1 : 256 / outs_n;
    for (int x = tid; x < parts * outs_n; x += 256) {
        const int part = x / outs_n, d = x % outs_n;
        const bool dec = d < DK;
        const int rank = dec ? A.ra : A.rg;
        const int per = (rank + parts - 1) / parts;
        const int r0 = min(rank, part * per), r1 = min(rank, r0 + per);
        const size_t inner = dec ? (size_t)H * DK : (size_t)H * DV;
        const size_t c = dec ? (size_t)head * DK + d : (size_t)head * DV + (d - DK);
        const WeightPtr& w = dec ? A.a2t : A.g2t;
        const float* th = low + (dec ? 0 : A.ra);
        float acc[1] = {0.f};
        if (w.dtype == MV_F32) decay_dots<float, 1>((const float*)w.p + c, inner, th, 0, r0, r1, acc);
        else decay_dots<bf16, 1>((const bf16*)w.p + c, inner, th, 0, r0, r1, acc);
        partial[x] = acc[0];
    }
    __syncthreads();
    const float rate = -expf(P.a_log.at(head));
    for (int d = tid; d < DPAD + DV; d += 256) {
        if (d < DPAD) {
            float g = 0.f;
            if (d < DK) {
                float zv = 0.f;
                for (int part = 0; part < parts; ++part) zv += partial[part * outs_n + d];
                g = expf(rate * softplus_f(zv + P.dt_bias.at((size_t)head * DK + d)));
            }
            vg[d] = g;
        } else {
            const int e = d - DPAD;
            float zv = 0.f;
            for (int part = 0; part < parts; ++part) zv += partial[part * outs_n + DK + e];
            gate[e] = sigmoid_f(zv);
        }
    }
    const float beta = sigmoid_f(to_f(p[P.b_off + head]));
    __syncthreads();
    ChannelToken<R> tk;
#pragma unroll
    for (int e = 0; e < R; ++e) {
        tk.q[e] = vq[sub * R + e];
        tk.k[e] = vk[sub * R + e];
        tk.g[e] = vg[sub * R + e];
    }
    tk.b = beta;
    for (int j0 = 0; j0 < DV; j0 += COLS) {
        const int j = j0 + col;
        const bool live = j < DV;
        const int jn = j + COLS;
        // the next columns are asked for before these are stored: a load behind a store would wait for it
        if (j0 + COLS < DV) delta_state_io<R, false>(s_next, S0 + (size_t)(jn < DV ? jn : 0) * DK, sub, DK, jn < DV);
        tk.v = vals[live ? j : 0];
        const float o = channel_update<R, L>(s, tk);
        delta_state_io<R, true>(s, S0 + (size_t)(live ? j : 0) * DK, sub, DK, live);
        if (live && sub == 0) outs[j] = o;
#pragma unroll
        for (int e = 0; e < R; ++e) s[e] = s_next[e];
    }
    __syncthreads();
    if (wave == 0) {
        float ss = 0.f;
        for (int d = lane; d < DV; d += MV_WAVE) ss = fmaf(outs[d], outs[d], ss);
        ss = wave_sum(ss);
        if (lane == 0) red[4] = 1.f / sqrtf(ss / (float)DV + A.eps);
    }
    __syncthreads();
    const float rinv = red[4];
    for (int d = tid; d < DV; d += 256) y[d] = from_f<T>(outs[d] * rinv * A.norm_w.at(d) * gate[d]);
}

// Returns 2 (nothing done) for sizes it does not serve.
extern "C" int mv_channel_step(const void* packed, long ld, int n, int n_seqs, int H, int G, int DK, int DV, int taps, int b_off,
                               int low_off, int ra, int rg, const void* conv_w, const void* a_log, const void* dt_bias,
                               const void* a2t, const void* g2t, const void* norm_w, int weight_dtype, void* conv_state,
                               float* state, float unit_eps, float eps, const int* token_seq, const int* cu_seqlens,
                               const int* state_slots, void* out, long ldo, int dtype, hipStream_t stream) {
    if (DK > 256 || DV > CD_MAX_DV || ra > CD_MAX_RANK || rg > CD_MAX_RANK || taps > MS_MAX_TAPS) return 2;
    ChannelStepArgs A{};
    A.rows = ChannelRows{packed, ld, H, G, DK, DV, taps, b_off, WeightPtr{conv_w, weight_dtype}, WeightPtr{a_log, weight_dtype},
                         WeightPtr{dt_bias, weight_dtype}, unit_eps};
    if (int rc = channel_check("channel_step", A.rows, n, n_seqs, conv_state)) return rc;
    MV_REQUIRE(ra > 0 && rg > 0 && a2t && g2t && norm_w && state && token_seq && cu_seqlens && state_slots && out && eps > 0.f &&
               ld >= (long)low_off + ra + rg && ldo >= (long)H * DV, "channel_step: missing operand or rows too short");
    if (n == 0) return 0;
    A.low_off = low_off; A.ra = ra; A.rg = rg;
    A.a2t = WeightPtr{a2t, weight_dtype}; A.g2t = WeightPtr{g2t, weight_dtype}; A.norm_w = WeightPtr{norm_w, weight_dtype};
    A.conv_state = conv_state; A.state = state; A.eps = eps; A.own_conv = G == H;
    A.token_seq = token_seq; A.state_slots = state_slots; A.out = out; A.ldo = ldo;
    int R = 0, L = 0;
    delta_scan_shape(DK, R, L);
    const dim3 grid(n, H);
#define CP_LAUNCH(RR, LL)                                                                                                   \
    MV_DISPATCH_T(dtype, "channel_step", hipLaunchKernelGGL((channel_step_kernel<T, RR, LL>), grid, dim3(256), 0, stream, A))
    if (R == 4 && L == 4) {
        CP_LAUNCH(4, 4);
    } else if (R == 4 && L == 8) {
        CP_LAUNCH(4, 8);
    } else if (R == 4 && L == 16) {
        CP_LAUNCH(4, 16);
    } else if (R == 8 && L == 16) {
        CP_LAUNCH(8, 16);
    } else {
        CP_LAUNCH(16, 16);
    }
#undef CP_LAUNCH
    if (mv_check_launch("channel_step")) return 1;
    if (!A.own_conv && taps > 1 && n_seqs > 0) {
        const int C = 2 * G * DK + H * DV;
        MV_DISPATCH_T(dtype, "conv_state",
                      hipLaunchKernelGGL(conv_state_kernel<T>, dim3(n_seqs, (unsigned)((C + 255) / 256)), dim3(256), 0, stream,
                                         (const T*)packed, ld, C, taps, (T*)conv_state, cu_seqlens, state_slots));
        return mv_check_launch("conv_state");
    }
    return 0;
}
