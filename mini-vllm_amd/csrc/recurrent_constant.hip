// Linear attention with a matrix state per head and one constant decay per head ("lightning attention"):
//     S <- a_h S + k v^T;   o = S^T q,       q = silu(.), k = silu(.) (DK channels a head), v = silu(.) (DV)
// All heads' outputs of a token together are divided by their root mean square, multiplied by a weight and by the
// logistic function of an output gate. Packed rows, from column `off`: [q (H*DK) | k (H*DK) | v (H*DV) | g (H*DV)].
// States are [slots][H][DV][DK] floats, a head's matrix column by column.
#include "qkv_row_norm.h"
#include "recurrent.h"

// ---------------------------------------------------------------------------------------
// Prepare: the activated vectors as floats, qk [n][H][2][DK] and vals [n][H][DV], and gates [n][H][4] = (a_h, 1, 0, 0),
// the form state_scan_kernel takes. One workgroup per row.
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
constant_prepare_kernel(const T* __restrict__ packed, long ld, int off, int H, int DK, int DV, const float* __restrict__ decay,
                        const int* __restrict__ token_seq, float* __restrict__ qk, float* __restrict__ vals,
                        float* __restrict__ gates) {
    const int t = blockIdx.x, tid = threadIdx.x;
    if (token_seq[t] < 0) return;
    const T* p = packed + (size_t)t * ld + off;
    const int nk = H * DK, nv = H * DV;
    float* o = qk + (size_t)t * 2 * nk;
    for (int c = tid; c < 2 * nk; c += 256) {
        const int which = c / nk, rem = c % nk, head = rem / DK, d = rem % DK;
        o[((size_t)head * 2 + which) * DK + d] = silu_f(to_f(p[c]));
    }
    float* v = vals + (size_t)t * nv;
    for (int c = tid; c < nv; c += 256) v[c] = silu_f(to_f(p[2 * nk + c]));
    for (int h = tid; h < H; h += 256) {
        float* g = gates + ((size_t)t * H + h) * 4;
        g[0] = decay[h];
        g[1] = 1.f;
        g[2] = 0.f;
        g[3] = 0.f;
    }
}

extern "C" int mv_constant_prepare(const void* packed, long ld, int off, int n, int H, int DK, int DV, const float* decay,
                                   const int* token_seq, float* qk, float* vals, float* gates, int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && H > 0 && DK > 0 && DV > 0 && off >= 0, "constant_prepare: bad sizes n=%d H=%d DK=%d DV=%d", n, H, DK, DV);
    MV_REQUIRE(ld >= off + 2L * H * DK + (long)H * DV && packed && decay && token_seq && qk && vals && gates,
               "constant_prepare: missing operand or rows too short");
    if (n == 0) return 0;
    MV_DISPATCH_T(dtype, "constant_prepare",
                  hipLaunchKernelGGL(constant_prepare_kernel<T>, dim3(n), dim3(256), 0, stream, (const T*)packed, ld, off, H, DK, DV,
                                     decay, token_seq, qk, vals, gates));
    return mv_check_launch("constant_prepare");
}

// ---------------------------------------------------------------------------------------
// Finish: out[t][c] = o[t][c] / sqrt(mean over the whole row of o^2 + eps) * weight[c] * sigmoid(g[t][c]), one
// workgroup per row of W columns (g from column g_off of the packed rows).
// ---------------------------------------------------------------------------------------
template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
row_gate_finish_kernel(const float* __restrict__ raw, const T* __restrict__ packed, long ld, int g_off, WeightPtr weight, int W,
                       float eps, const int* __restrict__ token_seq, T* __restrict__ out, long ldo) {
    __shared__ float part[4];
    const int t = blockIdx.x, tid = threadIdx.x;
    T* y = out + (size_t)t * ldo;
    if (token_seq[t] < 0) {
        for (int c = tid; c < W; c += 256) y[c] = from_f<T>(0.f);
        return;
    }
    const float* o = raw + (size_t)t * W;
    float ss = 0.f;
    if constexpr (VEC) {
        for (int c = 8 * tid; c < W; c += 2048) {
            float x[8];
            Vec8<float>::load(o + c, x);
#pragma unroll
            for (int e = 0; e < 8; ++e) ss = fmaf(x[e], x[e], ss);
        }
    } else {
        for (int c = tid; c < W; c += 256) ss = fmaf(o[c], o[c], ss);
    }
    ss = wave_sum(ss);
    if (tid % MV_WAVE == 0) part[tid / MV_WAVE] = ss;
    __syncthreads();
    const float rinv = 1.f / sqrtf((part[0] + part[1] + part[2] + part[3]) / (float)W + eps);
    const T* g = packed + (size_t)t * ld + g_off;
    if constexpr (VEC) {
        for (int c = 8 * tid; c < W; c += 2048) {
            float x[8], w[8], z[8];
            Vec8<float>::load(o + c, x);
            weight.at8(c, w);
            Vec8<T>::load(g + c, z);
#pragma unroll
            for (int e = 0; e < 8; ++e) x[e] = x[e] * rinv * w[e] * sigmoid_f(z[e]);
            Vec8<T>::store(y + c, x);
        }
    } else {
        for (int c = tid; c < W; c += 256) y[c] = from_f<T>(o[c] * rinv * weight.at(c) * sigmoid_f(to_f(g[c])));
    }
}

extern "C" int mv_row_gate_finish(const float* raw, const void* packed, long ld, int g_off, const void* weight, int weight_dtype,
                                  int n, int W, float eps, const int* token_seq, void* out, long ldo, int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && W > 0 && eps > 0.f && g_off >= 0 && ld >= (long)g_off + W && ldo >= W, "row_gate_finish: bad sizes n=%d W=%d", n, W);
    MV_REQUIRE(mv_valid_dtype(weight_dtype) && raw && packed && weight && token_seq && out, "row_gate_finish: missing operand");
    if (n == 0) return 0;
    const WeightPtr w{weight, weight_dtype};
    const size_t esz = mv_dtype_size(dtype);
    const bool vec = W % 8 == 0 && ((uintptr_t)raw % 16) == 0 && ((uintptr_t)packed % 16) == 0 && (ld * esz) % 16 == 0 &&
                     (g_off * esz) % 16 == 0 && ((uintptr_t)weight % 16) == 0 && ((uintptr_t)out % 16) == 0 && (ldo * esz) % 16 == 0;
    MV_DISPATCH_T(dtype, "row_gate_finish",
                  if (vec) hipLaunchKernelGGL((row_gate_finish_kernel<T, true>), dim3(n), dim3(256), 0, stream, raw, (const T*)packed, ld,
                                              g_off, w, W, eps, token_seq, (T*)out, ldo);
                  else hipLaunchKernelGGL((row_gate_finish_kernel<T, false>), dim3(n), dim3(256), 0, stream, raw, (const T*)packed, ld,
                                          g_off, w, W, eps, token_seq, (T*)out, ldo));
    return mv_check_launch("row_gate_finish");
}

// ---------------------------------------------------------------------------------------
// A step of single tokens: one (row, head) per workgroup. The output rows are left weighted and gated but not yet
// divided by the row's root mean square, y = o * weight * sigmoid(g), with the head's sum of o^2 in sums[t][head]
// (the heads of a row run in different workgroups; whoever uses the rows divides). With `norm` given, workgroup
// y = 0 of a row runs the query/key norm and cache write of a softmax mixer that reads the same packed rows.
// ---------------------------------------------------------------------------------------
struct ConstantStepArgs {
    const void* packed; long ld; int off;
    int H, DK, DV;
    const float* decay;
    WeightPtr weight;           // [H * DV]
    float* state;
    const int* token_seq; const int* state_slots;
    void* out; long ldo;
    float* sums;
};

#define CO_MAX_DV 256

template <typename T, int R, int L, bool BESIDE>
__global__ void __launch_bounds__(256)
constant_step_kernel(ConstantStepArgs A, RowNormArgs norm) {
    constexpr int COLS = 256 / L;
    __shared__ float outs[CO_MAX_DV];
    __shared__ float vals[CO_MAX_DV];
    __shared__ float red[8];
    const int t = blockIdx.x, tid = threadIdx.x;
    if constexpr (BESIDE) {
        if (blockIdx.y == 0) {
            row_norm_store<T>(norm, t, red);
            return;
        }
    }
    const int head = (int)blockIdx.y - (BESIDE ? 1 : 0);
    const int H = A.H, DK = A.DK, DV = A.DV;
    const int seq = A.token_seq[t];
    T* y = (T*)A.out + (size_t)t * A.ldo + (size_t)head * DV;
    if (seq < 0) {
        for (int d = tid; d < DV; d += 256) y[d] = from_f<T>(0.f);
        if (tid == 0) A.sums[(size_t)t * H + head] = 0.f;
        return;
    }
    const int sub = tid % L, col = tid / L;
    float* S0 = A.state + ((size_t)A.state_slots[seq] * H + head) * (size_t)DV * DK;
    float s[R], s_next[R], q[R], k[R];
    delta_state_io<R, false>(s, S0 + (size_t)(col < DV ? col : 0) * DK, sub, DK, col < DV);
    const T* p = (const T*)A.packed + (size_t)t * A.ld + A.off;
    const int nk = H * DK;
#pragma unroll
    for (int e = 0; e < R; ++e) {
        const int d = sub * R + e, dc = d < DK ? d : 0;
        const float zq = to_f(p[head * DK + dc]), zk = to_f(p[nk + head * DK + dc]);
        q[e] = d < DK ? silu_f(zq) : 0.f;
        k[e] = d < DK ? silu_f(zk) : 0.f;
    }
    for (int d = tid; d < DV; d += 256) vals[d] = silu_f(to_f(p[2 * nk + head * DV + d]));
    const float a = A.decay[head];
    __syncthreads();
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
            s[e] = fmaf(a, s[e], k[e] * v);
            o = fmaf(q[e], s[e], o);
        }
        o = lanes_sum<L>(o);
        delta_state_io<R, true>(s, S0 + (size_t)(live ? j : 0) * DK, sub, DK, live);
        if (live && sub == 0) outs[j] = o;
#pragma unroll
        for (int e = 0; e < R; ++e) s[e] = s_next[e];
    }
    __syncthreads();
    const T* g = p + 2 * nk + H * DV + head * DV;
    float ss = 0.f;
    for (int d = tid; d < DV; d += 256) {
        const float o = outs[d];
        ss = fmaf(o, o, ss);
        y[d] = from_f<T>(o * A.weight.at((size_t)head * DV + d) * sigmoid_f(to_f(g[d])));
    }
    ss = wave_sum(ss);
    if (tid % MV_WAVE == 0) red[tid / MV_WAVE] = ss;
    __syncthreads();
    if (tid == 0) A.sums[(size_t)t * H + head] = red[0] + red[1] + red[2] + red[3];
}

// `rows` .. `temp_every` describe the softmax mixer whose norm and cache write ride along (rows null: none).
// Returns 2 (nothing done) for sizes it does not serve.
extern "C" int mv_constant_step(const void* packed, long ld, int off, int n, int H, int DK, int DV, const float* decay,
                                const void* weight, int weight_dtype, float* state, const int* token_seq, const int* state_slots,
                                void* out, long ldo, float* sums, void* rows, long stride, int q_off, int k_off, int v_off,
                                const int* positions, const int* block_table, int bt_width, int page_size, void* k_pages,
                                void* v_pages, int NH, int NHkv, int ND, int NDv, const void* q_weight, const void* k_weight,
                                int norm_dtype, float eps, float temp_coef, int temp_every, int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && H > 0 && DK > 0 && DV > 0 && off >= 0, "constant_step: bad sizes n=%d H=%d DK=%d DV=%d", n, H, DK, DV);
    if (DK > 256 || DV > CO_MAX_DV) return 2;
    MV_REQUIRE(ld >= off + 2L * H * DK + 2L * H * DV && ldo >= (long)H * DV && H < 65535, "constant_step: rows too short");
    MV_REQUIRE(packed && decay && weight && mv_valid_dtype(weight_dtype) && state && token_seq && state_slots && out && sums,
               "constant_step: missing operand");
    RowNormArgs rn{};
    if (rows != nullptr) {
        rn = RowNormArgs{rows, stride, q_off, k_off, v_off, positions, token_seq, block_table, bt_width, page_size, k_pages, v_pages,
                         NH, NHkv, ND, NDv, WeightPtr{q_weight, norm_dtype}, WeightPtr{k_weight, norm_dtype}, eps, temp_coef,
                         temp_every, 1, 0};
        if (int rc = row_norm_check(rn, n, dtype)) return rc;
    }
    if (n == 0) return 0;
    const ConstantStepArgs A{packed, ld, off, H, DK, DV, decay, WeightPtr{weight, weight_dtype}, state, token_seq, state_slots, out,
                             ldo, sums};
    int R = 0, L = 0;
    delta_scan_shape(DK, R, L);
    const dim3 grid(n, H + (rows != nullptr ? 1 : 0));
#define CC_LAUNCH(RR, LL)                                                                                                     \
    if (rows != nullptr) {                                                                                                    \
        MV_DISPATCH_T(dtype, "constant_step",                                                                                 \
                      hipLaunchKernelGGL((constant_step_kernel<T, RR, LL, true>), grid, dim3(256), 0, stream, A, rn))          \
    } else {                                                                                                                  \
        MV_DISPATCH_T(dtype, "constant_step",                                                                                 \
                      hipLaunchKernelGGL((constant_step_kernel<T, RR, LL, false>), grid, dim3(256), 0, stream, A, rn))         \
    }
    if (R == 4 && L == 4) {
        CC_LAUNCH(4, 4)
    } else if (R == 4 && L == 8) {
        CC_LAUNCH(4, 8)
    } else if (R == 4 && L == 16) {
        CC_LAUNCH(4, 16)
    } else if (R == 8 && L == 16) {
        CC_LAUNCH(8, 16)
    } else {
        CC_LAUNCH(16, 16)
    }
#undef CC_LAUNCH
    return mv_check_launch("constant_step");
}
