// Query/key norm over whole rows and the cache write, one workgroup of 256 threads per token: the q columns of a
// row together (all heads' at once) are divided by their root mean square and multiplied by a weight as long as
// they are, and so are the k columns; q is further multiplied by the query temperature of its position p,
// 1 + coef * ln(floor((p + 1) / every) + 1) (every <= 0: none). q stays in the rows, k goes to the key page
// K[page][kv_head][slot][D], v (Dv channels a head) to the transposed value page V[page][kv_head][Dv][slot].
#pragma once
#include "dispatch.h"

struct RowNormArgs {
    void* rows;                 // packed rows of the activation type
    long stride;
    int q_off, k_off, v_off;
    const int* positions;
    const int* token_seq;
    const int* block_table;
    int bt_width, page_size;
    void* k_pages;
    void* v_pages;
    int H, Hkv, D, Dv;
    WeightPtr qw, kw;           // [H * D], [Hkv * D]
    float eps;
    float temp_coef;
    int temp_every;
    int store_v;                // 0: another launch takes the values to their pages
    int vec;                    // eight columns a load (sizes and addresses allow it)
};

template <typename T>
__device__ __forceinline__ void row_norm_store(const RowNormArgs& a, int tok, float* sh) {
    const int seq = a.token_seq[tok];
    if (seq < 0) return;
    const int tid = threadIdx.x, lane = tid % MV_WAVE, wave = tid / MV_WAVE;
    const int pos = a.positions[tok];
    T* row = (T*)a.rows + (size_t)tok * a.stride;
    T* q = row + a.q_off;
    const T* k = row + a.k_off;
    const int nq = a.H * a.D, nk = a.Hkv * a.D, nv = a.Hkv * a.Dv;
    const int page = a.block_table[(size_t)seq * a.bt_width + pos / a.page_size];
    const int slot = pos % a.page_size;
    float sq = 0.f, sk = 0.f;
    if (a.vec) {
        for (int c = 8 * tid; c < nq + nk; c += 2048) {
            float x[8];
            const bool is_k = c >= nq;
            Vec8<T>::load(is_k ? k + (c - nq) : q + c, x);
            float s = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) s = fmaf(x[e], x[e], s);
            if (is_k) sk += s; else sq += s;
        }
    } else {
        for (int c = tid; c < nq; c += 256) sq = fmaf(to_f(q[c]), to_f(q[c]), sq);
        for (int c = tid; c < nk; c += 256) sk = fmaf(to_f(k[c]), to_f(k[c]), sk);
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if (lane == 0) {
        sh[wave] = sq;
        sh[4 + wave] = sk;
    }
    __syncthreads();
    const float temp = a.temp_every > 0 ? 1.f + a.temp_coef * logf((float)((pos + 1) / a.temp_every) + 1.f) : 1.f;
    const float rq = temp / sqrtf((sh[0] + sh[1] + sh[2] + sh[3]) / (float)nq + a.eps);
    const float rk = 1.f / sqrtf((sh[4] + sh[5] + sh[6] + sh[7]) / (float)nk + a.eps);
    T* kp = (T*)a.k_pages;
    if (a.vec) {
        for (int c = 8 * tid; c < nq + nk; c += 2048) {
            float x[8], w[8];
            if (c < nq) {
                Vec8<T>::load(q + c, x);
                a.qw.at8(c, w);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = x[e] * rq * w[e];
                Vec8<T>::store(q + c, x);
            } else if (page >= 0) {
                const int kc = c - nq, hh = kc / a.D, d = kc % a.D;
                Vec8<T>::load(k + kc, x);
                a.kw.at8(kc, w);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = x[e] * rk * w[e];
                Vec8<T>::store(kp + (((size_t)page * a.Hkv + hh) * a.page_size + slot) * a.D + d, x);
            }
        }
    } else {
        for (int c = tid; c < nq; c += 256) q[c] = from_f<T>(to_f(q[c]) * rq * a.qw.at(c));
        if (page >= 0)
            for (int c = tid; c < nk; c += 256)
                kp[(((size_t)page * a.Hkv + c / a.D) * a.page_size + slot) * a.D + c % a.D] = from_f<T>(to_f(k[c]) * rk * a.kw.at(c));
    }
    if (a.store_v && page >= 0) {
        const T* v = row + a.v_off;
        T* vp = (T*)a.v_pages + (size_t)page * nv * a.page_size + slot;
        for (int c = tid; c < nv; c += 256) vp[(size_t)c * a.page_size] = v[c];
    }
}

// Checks the operands and fills `vec`; returns 0, or the error of mv_fail.
static inline int row_norm_check(RowNormArgs& a, int n, int dtype) {
    MV_REQUIRE(n >= 0 && a.H > 0 && a.Hkv > 0 && a.H % a.Hkv == 0 && a.D > 0 && a.Dv > 0, "qkv_row_norm_store: bad sizes n=%d H=%d Hkv=%d D=%d Dv=%d",
               n, a.H, a.Hkv, a.D, a.Dv);
    MV_REQUIRE(a.rows && a.positions && a.token_seq && a.block_table && a.k_pages && a.v_pages && a.page_size > 0 && a.bt_width > 0,
               "qkv_row_norm_store: missing operand");
    MV_REQUIRE(a.qw.p && a.kw.p && mv_valid_dtype(a.qw.dtype) && mv_valid_dtype(a.kw.dtype) && a.eps > 0.f,
               "qkv_row_norm_store: norm weights and a positive eps are needed");
    MV_REQUIRE(a.q_off >= 0 && a.k_off >= 0 && a.v_off >= 0 && a.stride >= (long)a.q_off + (long)a.H * a.D &&
               a.stride >= (long)a.k_off + (long)a.Hkv * a.D && a.stride >= (long)a.v_off + (long)a.Hkv * a.Dv,
               "qkv_row_norm_store: rows of %ld columns are too short", a.stride);
    const size_t esz = mv_dtype_size(dtype);
    a.vec = a.D % 8 == 0 && ((uintptr_t)a.rows % 16) == 0 && (a.stride * esz) % 16 == 0 && (a.q_off * esz) % 16 == 0 &&
            (a.k_off * esz) % 16 == 0 && ((uintptr_t)a.k_pages % 16) == 0 && ((uintptr_t)a.qw.p % 16) == 0 && ((uintptr_t)a.kw.p % 16) == 0;
    return 0;
}
