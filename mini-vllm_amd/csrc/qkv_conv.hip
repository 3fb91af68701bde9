// Launches of qkv_conv.h: a thread group per (token, head), eight channels a lane, or a wave per (token, head) for any sizes.
#include "qkv_conv.h"

template <typename T>
__global__ void __launch_bounds__(256)
qkv_conv_store_vec_kernel(ConvStoreArgs A) {
    const int L = A.D / 8, heads = A.H + 2 * A.Hkv;
    const int gid = blockIdx.x * 256 + threadIdx.x;
    const int hidx = gid / L;
    conv_store_vec<T>(A, hidx / heads, hidx % heads, gid % L);
}

template <typename T>
__global__ void __launch_bounds__(256)
qkv_conv_store_kernel(ConvStoreArgs A) {
    __shared__ float sh[4][QC_MAX_D];
    const int tok = blockIdx.x, wave = threadIdx.x / MV_WAVE, lane = threadIdx.x % MV_WAVE;
    const int head = blockIdx.y * 4 + wave;
    const int H = A.H, Hkv = A.Hkv, D = A.D, Dv = A.Dv, taps = A.taps;
    if (head >= H + 2 * Hkv) return;
    const int seq = A.token_seq[tok];
    if (seq < 0) return;
    const int pos = A.positions[tok], first = A.cu_seqlens[seq];
    const int C = H * D + Hkv * (D + Dv);
    const bool is_v = head >= H + Hkv;
    const int size = is_v ? Dv : D;
    const int c0 = is_v ? (H + Hkv) * D + (head - H - Hkv) * Dv : head * D;
    const T* rows = (const T*)A.rows + A.base;
    T* hist = (T*)A.conv_state + (taps > 1 ? (size_t)A.state_slots[seq] * (taps - 1) * C : 0);
    float* x = sh[wave];
    for (int d = lane; d < size; d += MV_WAVE) {
        const int c = c0 + d;
        float acc = 0.f;
        for (int j = 0; j < taps; ++j) {
            const int r = tok - (taps - 1) + j;
            const T in = r >= first ? rows[(size_t)r * A.ld + c] : hist[(size_t)(taps - 1 + r - first) * C + c];
            acc = fmaf(A.w[(size_t)j * C + c], to_f(in), acc);
            if (A.single && j > 0) hist[(size_t)(j - 1) * C + c] = in;
        }
        x[d] = acc;
    }
    // (a wave's own LDS writes are visible to it in order: no barrier between the phases)
    __builtin_amdgcn_wave_barrier();
    T* out = (T*)A.out + (size_t)tok * A.ldo;
    const int page = A.block_table[(size_t)seq * A.bt_width + pos / A.page_size];
    if (is_v) {
        const int hh = head - H - Hkv;
        if (!A.store_v) {
            for (int d = lane; d < Dv; d += MV_WAVE) out[(size_t)H * D + (size_t)hh * Dv + d] = from_f<T>(x[d]);
        } else if (page >= 0) {
            T* dst = (T*)A.v_pages + ((size_t)page * Hkv + hh) * Dv * A.page_size + pos % A.page_size;
            for (int d = lane; d < Dv; d += MV_WAVE) dst[(size_t)d * A.page_size] = from_f<T>(x[d]);
        }
        return;
    }
    if (A.table != nullptr) {
        const int half = A.rot / 2;
        const float* cs = A.table + (size_t)pos * A.rot;
        for (int p = lane; p < half; p += MV_WAVE) {
            const float c = cs[p], s = cs[half + p], a = x[p], b = x[p + half];
            x[p] = a * c - b * s;
            x[p + half] = b * c + a * s;
        }
        __builtin_amdgcn_wave_barrier();
    }
    float ss = 0.f;
    for (int d = lane; d < D; d += MV_WAVE) ss = fmaf(x[d], x[d], ss);
    ss = wave_sum(ss);
    const float inv = A.unit_norm ? 1.f / sqrtf(ss / (float)D + A.eps) : 1.f;
    if (head < H) {
        for (int d = lane; d < D; d += MV_WAVE) out[(size_t)head * D + d] = from_f<T>(x[d] * inv);
        return;
    }
    if (page < 0) return;
    T* dst = (T*)A.k_pages + (((size_t)page * Hkv + head - H) * A.page_size + pos % A.page_size) * D;
    for (int d = lane; d < D; d += MV_WAVE) dst[d] = from_f<T>(x[d] * inv);
}

extern "C" int mv_store_v_pages(const void* qkv, long row_stride, int v_off, const int* positions, const int* token_seq,
                                const int* block_table, int bt_width, int page_size, void* v_pages, int n, int Hkv, int D,
                                int dtype, hipStream_t stream);

// steps of at least this many tokens write their values tile by tile in a launch of their own
#define QC_TILED_V_TOKENS 64

extern "C" int mv_qkv_conv_store(const void* rows, long ld, int base, int n, int n_seqs, int H, int Hkv, int D, int Dv, int taps,
                                 const float* w, void* conv_state, int single, const int* positions, const int* token_seq,
                                 const int* cu_seqlens, const int* state_slots, const int* block_table, int bt_width, int page_size,
                                 void* k_pages, void* v_pages, const float* table, int rot, int unit_norm, float eps, void* out,
                                 long ldo, int dtype, hipStream_t stream) {
    ConvStoreArgs A{rows, ld, base, n, H, Hkv, D, Dv, taps, w, conv_state, single && taps > 1, positions, token_seq, cu_seqlens,
                    state_slots, block_table, bt_width, page_size, k_pages, v_pages, table, table ? rot : 0, unit_norm, eps, out, ldo,
                    n < QC_TILED_V_TOKENS};
    if (int rc = conv_store_check(A)) return rc;
    if (n == 0) return 0;
    if (conv_store_vec_ok(A, dtype)) {
        const long lanes = (long)n * (H + 2 * Hkv) * (D / 8);
        MV_DISPATCH_T(dtype, "qkv_conv_store", hipLaunchKernelGGL(qkv_conv_store_vec_kernel<T>, dim3((unsigned)((lanes + 255) / 256)),
                                                                   dim3(256), 0, stream, A));
    } else {
        MV_DISPATCH_T(dtype, "qkv_conv_store", hipLaunchKernelGGL(qkv_conv_store_kernel<T>, dim3(n, (H + 2 * Hkv + 3) / 4), dim3(256), 0,
                                                                   stream, A));
    }
    if (mv_check_launch("qkv_conv_store")) return 1;
    if (!A.store_v)
        if (int rc = mv_store_v_pages(out, ldo, H * D, positions, token_seq, block_table, bt_width, page_size, v_pages, n, Hkv, Dv,
                                      dtype, stream)) return rc;
    if (taps > 1 && !A.single && n_seqs > 0) {
        const int C = H * D + Hkv * (D + Dv);
        MV_DISPATCH_T(dtype, "conv_state",
                      hipLaunchKernelGGL(conv_state_kernel<T>, dim3(n_seqs, (unsigned)((C + 255) / 256)), dim3(256), 0, stream,
                                         (const T*)rows + base, ld, C, taps, (T*)conv_state, cu_seqlens, state_slots));
        return mv_check_launch("conv_state");
    }
    return 0;
}
