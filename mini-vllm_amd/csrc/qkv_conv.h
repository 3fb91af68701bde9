// Convolution, rotation, unit norm and cache write of softmax attention on the packed rows of a step. The channels
// [q (H*D) | k (Hkv*D) | v (Hkv*Dv)] lie side by side from column `base` on; each passes a causal convolution over time
//     y_t = sum_j w[j] x_(t - taps + 1 + j)        (w float [taps][C], no activation)
// whose inputs in front of the step are the request's kept ones (conv_state [slots][taps-1][C], activation type). Then
//   q, k heads  the first `rot` channels are rotated by the row's position (pairs i, i + rot/2; table[pos] = [cos | sin]),
//               the head is divided by its root mean square (`unit_norm`); q goes to out[token][head*D], k to its key page
//               K[page][kv_head][slot][D]
//   v heads     to the transposed value page V[page][kv_head][Dv][slot], or (store_v 0) to out[token][H*D + head*Dv], from
//               where a tiled launch takes them there
// The rows themselves are only read: neighbouring tokens need each other's raw values. `single`: the step has one row of
// each request, so a channel's thread moves the kept inputs on itself; otherwise conv_state_kernel does it afterwards.
// Rows of padding (token_seq < 0) write nothing; a page that was given back (< 0) is skipped.
#pragma once
#include "recurrent.h"

#define QC_MAX_D 512

struct ConvStoreArgs {
    const void* rows; long ld; int base;
    int n, H, Hkv, D, Dv, taps;
    const float* w;
    void* conv_state;
    int single;
    const int* positions; const int* token_seq; const int* cu_seqlens; const int* state_slots; const int* block_table;
    int bt_width, page_size;
    void* k_pages; void* v_pages;
    const float* table; int rot;
    int unit_norm; float eps;
    void* out; long ldo;
    int store_v;
};

// eight neighbouring channels from c of row tok (first: its request's first row of the step)
template <typename T, int TAPS>
__device__ __forceinline__ void conv8(const ConvStoreArgs& A, int tok, int first, int slot, int c, float (&x)[8]) {
    const int taps = TAPS > 0 ? TAPS : A.taps;
    const int C = A.H * A.D + A.Hkv * (A.D + A.Dv);
    const T* rows = (const T*)A.rows + A.base + c;
    T* hist = (T*)A.conv_state + (size_t)slot * (taps - 1) * C + c;
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = 0.f;
    if constexpr (TAPS > 0) {
        float in[TAPS][8], w[TAPS][8];
#pragma unroll
        for (int j = 0; j < TAPS; ++j) {                     // every load is issued before anything is stored
            const int r = tok - (TAPS - 1) + j;
            Vec8<T>::load(r >= first ? rows + (size_t)r * A.ld : hist + (size_t)(TAPS - 1 + r - first) * C, in[j]);
            Vec8<float>::load(A.w + (size_t)j * C + c, w[j]);
        }
#pragma unroll
        for (int j = 0; j < TAPS; ++j)
#pragma unroll
            for (int e = 0; e < 8; ++e) x[e] = fmaf(w[j][e], in[j][e], x[e]);
        if (A.single) {
#pragma unroll
            for (int j = 1; j < TAPS; ++j) Vec8<T>::store(hist + (size_t)(j - 1) * C, in[j]);
        }
    } else {
        for (int j = 0; j < taps; ++j) {
            const int r = tok - (taps - 1) + j;
            float in[8], w[8];
            Vec8<T>::load(r >= first ? rows + (size_t)r * A.ld : hist + (size_t)(taps - 1 + r - first) * C, in);
            Vec8<float>::load(A.w + (size_t)j * C + c, w);
#pragma unroll
            for (int e = 0; e < 8; ++e) x[e] = fmaf(w[e], in[e], x[e]);
            if (A.single && j > 0) Vec8<T>::store(hist + (size_t)(j - 1) * C, in);      // (row j - 1 was read a turn ago)
        }
    }
}

// Heads of D = Dv = 64, 128 or 256 channels with everything 16-byte aligned: a head is spread over L = D / 8 neighbouring
// lanes. All lanes of a wave call it (shuffles); `tok` < 0 or a head beyond the last one: nothing is written.
template <typename T>
__device__ __forceinline__ void conv_store_vec(const ConvStoreArgs& A, int tok, int head, int j) {
    const int L = A.D / 8, H = A.H, Hkv = A.Hkv, D = A.D;
    const int seq = tok >= 0 && tok < A.n && head < H + 2 * Hkv ? A.token_seq[tok] : -1;
    const bool active = seq >= 0;
    const int kind = head >= H + Hkv ? 2 : (head >= H ? 1 : 0);
    const int hh = kind == 2 ? head - H - Hkv : (kind == 1 ? head - H : head);
    float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    int pos = 0;
    if (active) {
        pos = A.positions[tok];
        const int c = head * D + 8 * j;                       // (k behind q, v behind k, all heads of D channels)
        const int first = A.cu_seqlens[seq], slot = A.taps > 1 ? A.state_slots[seq] : 0;
        if (A.taps == 4) conv8<T, 4>(A, tok, first, slot, c, x);
        else conv8<T, 0>(A, tok, first, slot, c, x);
    }
    if (A.table != nullptr) {
        const int hl = A.rot / 16;                            // lanes that hold the first channel of a pair
        const int lane = threadIdx.x % MV_WAVE;
        const int partner = j < hl ? j + hl : (j < 2 * hl ? j - hl : j);
        const bool turned = active && kind < 2 && j < 2 * hl;
        float c[8], s[8];
        const float* cs = A.table + (size_t)pos * A.rot + 8 * (turned ? j % hl : 0);
        Vec8<float>::load(cs, c);
        Vec8<float>::load(cs + A.rot / 2, s);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float other = __shfl(x[e], (lane - j) + partner, MV_WAVE);
            if (turned) x[e] = j < hl ? x[e] * c[e] - other * s[e] : x[e] * c[e] + other * s[e];
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = fmaf(x[e], x[e], ss);
    for (int o = L / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, MV_WAVE);
    if (!active) return;
    if (kind < 2 && A.unit_norm) {
        const float inv = 1.f / sqrtf(ss / (float)D + A.eps);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] *= inv;
    }
    T* out = (T*)A.out + (size_t)tok * A.ldo;
    if (kind == 0) {
        Vec8<T>::store(out + (size_t)hh * D + 8 * j, x);
        return;
    }
    if (kind == 2 && !A.store_v) {
        Vec8<T>::store(out + (size_t)H * D + (size_t)hh * D + 8 * j, x);
        return;
    }
    const int page = A.block_table[(size_t)seq * A.bt_width + pos / A.page_size];
    if (page < 0) return;
    if (kind == 1) {
        Vec8<T>::store((T*)A.k_pages + (((size_t)page * Hkv + hh) * A.page_size + pos % A.page_size) * D + 8 * j, x);
        return;
    }
    T* dst = (T*)A.v_pages + (((size_t)page * Hkv + hh) * D + 8 * j) * A.page_size + pos % A.page_size;
#pragma unroll
    for (int e = 0; e < 8; ++e) dst[(size_t)e * A.page_size] = from_f<T>(x[e]);
}

// whether conv_store_vec serves these operands
static inline bool conv_store_vec_ok(const ConvStoreArgs& A, int dtype) {
    const size_t esz = mv_dtype_size(dtype);
    return A.D == A.Dv && (A.D == 64 || A.D == 128 || A.D == 256) && (A.table == nullptr || A.rot % 16 == 0) &&
           ((uintptr_t)A.rows % 16) == 0 && (A.ld * esz) % 16 == 0 && (A.base * esz) % 16 == 0 && ((uintptr_t)A.conv_state % 16) == 0 &&
           ((uintptr_t)A.w % 16) == 0 && ((uintptr_t)A.k_pages % 16) == 0 && ((uintptr_t)A.table % 16) == 0 && (A.rot / 2) % 4 == 0 &&
           ((uintptr_t)A.out % 16) == 0 && (A.ldo * esz) % 16 == 0 && (long)A.n * (A.H + 2 * A.Hkv) * (A.D / 8) < (1L << 31);
}

static inline int conv_store_check(const ConvStoreArgs& A) {
    MV_REQUIRE(A.n >= 0 && A.H > 0 && A.Hkv > 0 && A.H % A.Hkv == 0 && A.D > 0 && A.Dv > 0 && A.D <= QC_MAX_D && A.Dv <= QC_MAX_D,
               "qkv_conv_store: bad sizes n=%d H=%d Hkv=%d D=%d Dv=%d (heads of at most %d)", A.n, A.H, A.Hkv, A.D, A.Dv, QC_MAX_D);
    MV_REQUIRE(A.taps >= 1 && A.taps <= MS_MAX_TAPS, "qkv_conv_store: %d taps, 1 to %d are served", A.taps, MS_MAX_TAPS);
    MV_REQUIRE(A.base >= 0 && A.ld >= (long)A.base + (long)A.H * A.D + (long)A.Hkv * (A.D + A.Dv) &&
               A.ldo >= (long)A.H * A.D + (long)A.Hkv * A.Dv, "qkv_conv_store: rows too short");
    MV_REQUIRE(A.rows && A.w && (A.conv_state || A.taps == 1) && A.positions && A.token_seq && A.cu_seqlens && A.state_slots &&
               A.block_table && A.bt_width > 0 && A.page_size > 0 && A.k_pages && A.v_pages && A.out, "qkv_conv_store: missing operand");
    MV_REQUIRE(A.table == nullptr || (A.rot > 0 && A.rot % 2 == 0 && A.rot <= A.D), "qkv_conv_store: %d rotated channels of %d", A.rot, A.D);
    MV_REQUIRE((!A.unit_norm || A.eps > 0.f) && A.H + 2 * A.Hkv <= 4 * 65535, "qkv_conv_store: bad constants");
    return 0;
}
