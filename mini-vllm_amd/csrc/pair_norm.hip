// Two parts that run side by side, joined: a row's delta is half the sum of their two output rows, each divided by
// its root mean square over the row and multiplied by a weight of its own. The delta is added to the float
// residual and the sum normalised for the next part in the same launch, or written out. Also here: what a model
// adds to the residual stream in front of a run of layers (the embedding's row, a vector), with the norm behind it.
#include "dispatch.h"

// One side of the pair. With `sums` the row was left without the division of a root mean square of its own in
// front of the linear map that made it (c = sqrt(sum_p sums[row][p] / inner + inner_eps)): y / c divided by its
// root mean square is y / sqrt(mean(y^2) + eps c^2), so only eps changes.
struct PairSide {
    const void* y;
    long ld;
    WeightPtr w;
    const float* sums;
    int parts;
    int inner;
    float inner_eps;
};

__device__ __forceinline__ float pair_eps(const PairSide& s, int row, float eps) {
    if (s.sums == nullptr) return eps;
    float t = 0.f;
    for (int p = 0; p < s.parts; ++p) t += s.sums[(size_t)row * s.parts + p];
    return eps * (t / (float)s.inner + s.inner_eps);
}

// a sum over the 256 threads of the workgroup for up to two values at once; sh: 8 floats, free before the call
__device__ __forceinline__ void block_sum2(float& a, float& b, float* sh) {
    const int lane = threadIdx.x % MV_WAVE, wave = threadIdx.x / MV_WAVE;
    a = wave_sum(a);
    b = wave_sum(b);
    if (lane == 0) {
        sh[wave] = a;
        sh[4 + wave] = b;
    }
    __syncthreads();
    a = sh[0] + sh[1] + sh[2] + sh[3];
    b = sh[4] + sh[5] + sh[6] + sh[7];
}

// NC chunks of eight columns a thread are kept in registers (NC 0: any number of columns, read again)
template <typename T, int NC>
__global__ void __launch_bounds__(256)
pair_norm_add_norm_kernel(PairSide A, PairSide B, float eps, float* __restrict__ resid, WeightPtr wn, float eps_n, int unit_n,
                          T* __restrict__ out, long ldo, int h) {
    __shared__ float sh[16];
    const int r = blockIdx.x, tid = threadIdx.x;
    const T* ya = (const T*)A.y + (size_t)r * A.ld;
    const T* yb = (const T*)B.y + (size_t)r * B.ld;
    float* x = resid ? resid + (size_t)r * h : nullptr;
    T* o = out ? out + (size_t)r * ldo : nullptr;
    const float ea = pair_eps(A, r, eps), eb = pair_eps(B, r, eps);
    if constexpr (NC > 0) {
        float va[NC][8], vb[NC][8], xr[NC][8], fn[NC][8];
        float sa = 0.f, sb = 0.f;
        const bool normed = x != nullptr && o != nullptr;
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int d = (tid + 256 * c) * 8;
            const bool ok = d < h;
            const int dl = ok ? d : 0;
            Vec8<T>::load(ya + dl, va[c]);
            Vec8<T>::load(yb + dl, vb[c]);
            if (x != nullptr) Vec8<float>::load(x + dl, xr[c]);
            if (normed) wn.at8(dl, fn[c]);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                if (!ok) va[c][e] = vb[c][e] = 0.f;
                sa = fmaf(va[c][e], va[c][e], sa);
                sb = fmaf(vb[c][e], vb[c][e], sb);
            }
        }
        block_sum2(sa, sb, sh);
        const float ra = 0.5f / sqrtf(sa / (float)h + ea), rb = 0.5f / sqrtf(sb / (float)h + eb);
        float ss = 0.f, zero = 0.f;
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int d = (tid + 256 * c) * 8;
            if (d >= h) continue;
            float wa[8], wb[8];
            A.w.at8(d, wa);
            B.w.at8(d, wb);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                va[c][e] = fmaf(va[c][e] * ra, wa[e], vb[c][e] * rb * wb[e]);
                if (x != nullptr) va[c][e] += xr[c][e];
                ss = fmaf(va[c][e], va[c][e], ss);
            }
            if (x != nullptr) Vec8<float>::store(x + d, va[c]);
            else Vec8<T>::store(o + d, va[c]);
        }
        if (!normed) return;
        block_sum2(ss, zero, sh + 8);
        const float rn = 1.f / sqrtf(ss / (float)h + eps_n);
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const int d = (tid + 256 * c) * 8;
            if (d >= h) continue;
            float y[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] = va[c][e] * rn * (fn[c][e] + (unit_n ? 1.f : 0.f));
            Vec8<T>::store(o + d, y);
        }
    } else {
        float sa = 0.f, sb = 0.f;
        for (int d = tid; d < h; d += 256) {
            sa = fmaf(to_f(ya[d]), to_f(ya[d]), sa);
            sb = fmaf(to_f(yb[d]), to_f(yb[d]), sb);
        }
        block_sum2(sa, sb, sh);
        const float ra = 0.5f / sqrtf(sa / (float)h + ea), rb = 0.5f / sqrtf(sb / (float)h + eb);
        float ss = 0.f, zero = 0.f;
        for (int d = tid; d < h; d += 256) {
            float v = fmaf(to_f(ya[d]) * ra, A.w.at(d), to_f(yb[d]) * rb * B.w.at(d));
            if (x != nullptr) {
                v += x[d];
                x[d] = v;
            } else {
                o[d] = from_f<T>(v);
            }
            ss = fmaf(v, v, ss);
        }
        if (x == nullptr || o == nullptr) return;
        block_sum2(ss, zero, sh + 8);
        const float rn = 1.f / sqrtf(ss / (float)h + eps_n);
        // (a thread reads what it wrote itself)
        for (int d = tid; d < h; d += 256) o[d] = from_f<T>(x[d] * rn * (wn.at(d) + (unit_n ? 1.f : 0.f)));
    }
}

static bool pair_side_ok(const PairSide& s, int h) {
    return s.y != nullptr && s.ld >= h && s.w.p != nullptr && mv_valid_dtype(s.w.dtype) && (s.sums == nullptr || (s.parts > 0 && s.inner > 0));
}

// resid[n][h] += delta and, with `out`, out = norm(resid) (weight wn, 1 + wn with unit_n); without `resid`, out = delta.
extern "C" int mv_pair_norm_add_norm(const void* ya, long lda, const void* wa, const float* sums_a, int parts_a, int inner_a,
                                     const void* yb, long ldb, const void* wb, const float* sums_b, int parts_b, int inner_b,
                                     int pair_dtype, float eps, float inner_eps, float* resid, const void* wn, int wn_dtype,
                                     float eps_n, int unit_n, void* out, long ldo, int n, int h, int dtype, hipStream_t stream) {
    const PairSide A{ya, lda, WeightPtr{wa, pair_dtype}, sums_a, parts_a, inner_a, inner_eps};
    const PairSide B{yb, ldb, WeightPtr{wb, pair_dtype}, sums_b, parts_b, inner_b, inner_eps};
    MV_REQUIRE(n >= 0 && h > 0 && eps > 0.f && pair_side_ok(A, h) && pair_side_ok(B, h), "pair_norm: bad sizes or missing operand (n=%d h=%d)", n, h);
    MV_REQUIRE(resid != nullptr || out != nullptr, "pair_norm: nowhere to leave the result");
    MV_REQUIRE(out == nullptr || ldo >= h, "pair_norm: output rows too short");
    const bool normed = resid != nullptr && out != nullptr;
    MV_REQUIRE(!normed || (wn && mv_valid_dtype(wn_dtype) && eps_n > 0.f), "pair_norm: the norm behind lacks its weight");
    if (n == 0) return 0;
    const WeightPtr pn{wn, normed ? wn_dtype : MV_F32};
    const size_t esz = mv_dtype_size(dtype);
    auto al = [](const void* p) { return ((uintptr_t)p % 16) == 0; };
    const bool vec = h % 8 == 0 && h <= 8192 && (lda * esz) % 16 == 0 && (ldb * esz) % 16 == 0 && (ldo * esz) % 16 == 0 && al(ya) && al(yb)
                     && al(wa) && al(wb) && al(wn) && al(resid) && al(out);
#define PN_LAUNCH(NC)                                                                                                          \
    MV_DISPATCH_T(dtype, "pair_norm",                                                                                          \
                  hipLaunchKernelGGL((pair_norm_add_norm_kernel<T, NC>), dim3(n), dim3(256), 0, stream, A, B, eps, resid, pn,   \
                                     eps_n, unit_n, (T*)out, ldo, h))
    if (!vec) {
        PN_LAUNCH(0);
    } else if (h <= 2048) {
        PN_LAUNCH(1);
    } else if (h <= 4096) {
        PN_LAUNCH(2);
    } else {
        PN_LAUNCH(4);
    }
#undef PN_LAUNCH
    return mv_check_launch("pair_norm");
}

// ---------------------------------------------------------------------------------------
// resid[t] += delta[t] (when given) + table[ids[t]] * scale (when ids are given; an id outside the table adds
// nothing) + step (a vector of h, when given); with `out`, out[t] = norm(resid[t]). One workgroup per row.
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
stream_entry_kernel(float* __restrict__ resid, const T* __restrict__ delta, long ldd, const int* __restrict__ ids, WeightPtr table,
                    int vocab, float scale, WeightPtr step, WeightPtr wn, float eps, int unit, T* __restrict__ out, int h) {
    __shared__ float sh[8];
    const int t = blockIdx.x, tid = threadIdx.x;
    float* x = resid + (size_t)t * h;
    const int id = ids ? ids[t] : -1;
    const bool emb = id >= 0 && id < vocab;
    float ss = 0.f, zero = 0.f;
    for (int d = tid; d < h; d += 256) {
        float v = x[d];
        if (delta) v += to_f(delta[(size_t)t * ldd + d]);
        if (emb) v += table.at((size_t)id * h + d) * scale;
        if (step.p) v += step.at(d);
        x[d] = v;
        ss = fmaf(v, v, ss);
    }
    if (out == nullptr) return;
    block_sum2(ss, zero, sh);
    const float rn = 1.f / sqrtf(ss / (float)h + eps);
    for (int d = tid; d < h; d += 256) out[(size_t)t * h + d] = from_f<T>(x[d] * rn * (wn.at(d) + (unit ? 1.f : 0.f)));
}

extern "C" int mv_stream_entry(float* resid, const void* delta, long ldd, const int* ids, const void* table, int table_dtype,
                               int vocab, float scale, const void* step, int step_dtype, const void* wn, int wn_dtype, float eps,
                               int unit, void* out, int n, int h, int dtype, hipStream_t stream) {
    MV_REQUIRE(n >= 0 && h > 0 && resid, "stream_entry: bad sizes n=%d h=%d", n, h);
    MV_REQUIRE(!delta || ldd >= h, "stream_entry: rows too short");
    MV_REQUIRE(!ids || (table && vocab > 0 && mv_valid_dtype(table_dtype)), "stream_entry: token ids without a table");
    MV_REQUIRE(!out || (wn && mv_valid_dtype(wn_dtype) && eps > 0.f), "stream_entry: the norm behind lacks its weight");
    if (n == 0) return 0;
    MV_DISPATCH_T(dtype, "stream_entry",
                  hipLaunchKernelGGL(stream_entry_kernel<T>, dim3(n), dim3(256), 0, stream, resid, (const T*)delta, ldd, ids,
                                     WeightPtr{table, table_dtype}, vocab, scale, WeightPtr{step, step_dtype}, WeightPtr{wn, wn_dtype},
                                     eps, unit, (T*)out, h));
    return mv_check_launch("stream_entry");
}
