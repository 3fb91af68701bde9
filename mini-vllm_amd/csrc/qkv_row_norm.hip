// Query/key norm over whole rows with the query temperature, and the cache write (see qkv_row_norm.h).
#include "qkv_row_norm.h"

template <typename T>
__global__ void __launch_bounds__(256)
qkv_row_norm_store_kernel(RowNormArgs a) {
    __shared__ float sh[8];
    row_norm_store<T>(a, blockIdx.x, sh);
}

extern "C" int mv_store_v_pages(const void* qkv, long row_stride, int v_off, const int* positions, const int* token_seq,
                                const int* block_table, int bt_width, int page_size, void* v_pages, int n, int Hkv, int D,
                                int dtype, hipStream_t stream);

// steps of at least this many tokens write their values tile by tile in a launch of their own, so that
// neighbouring tokens write neighbouring slots
#define RN_TILED_V_TOKENS 64

extern "C" int mv_qkv_row_norm_store(void* rows, long stride, int q_off, int k_off, int v_off, const int* positions,
                                     const int* token_seq, const int* block_table, int bt_width, int page_size, void* k_pages,
                                     void* v_pages, int n, int H, int Hkv, int D, int Dv, const void* q_weight,
                                     const void* k_weight, int weight_dtype, float eps, float temp_coef, int temp_every,
                                     int dtype, hipStream_t stream) {
    RowNormArgs a{rows, stride, q_off, k_off, v_off, positions, token_seq, block_table, bt_width, page_size, k_pages, v_pages,
                  H, Hkv, D, Dv, WeightPtr{q_weight, weight_dtype}, WeightPtr{k_weight, weight_dtype}, eps, temp_coef, temp_every,
                  n < RN_TILED_V_TOKENS, 0};
    if (int rc = row_norm_check(a, n, dtype)) return rc;
    if (n == 0) return 0;
    MV_DISPATCH_T(dtype, "qkv_row_norm_store",
                  hipLaunchKernelGGL(qkv_row_norm_store_kernel<T>, dim3(n), dim3(256), 0, stream, a));
    if (int rc = mv_check_launch("qkv_row_norm_store")) return rc;
    if (!a.store_v)
        return mv_store_v_pages(rows, stride, v_off, positions, token_seq, block_table, bt_width, page_size, v_pages, n, Hkv, Dv,
                                dtype, stream);
    return 0;
}
