// What softmax attention may do to a score beside the scale, in this order (each off by default):
//   cap      s <- cap * tanh(s / cap)
//   slopes   s <- s - slopes[head] * (query position - key position)
// and with `sink` the softmax has one more score, 0, that no value belongs to: its denominator is 1 + sum exp(s).
#pragma once
#include "common.h"

struct ScoreForm {
    float cap;               // <= 0: none
    const float* slopes;     // [query heads] or null
    int sink;
};

// The same on a product q.k that is not scaled yet, in the base-2 domain of the MFMA kernels (the result times
// ln 2 is the score): `lin` multiplies when there is no cap, `in` and `amp` carry scale and cap when there is one.
// tanh(z) = 1 - 2 / (1 + e^(2 z)): exact limits at both ends, an absolute error of 2^-23 of the cap between.
struct ScoreBase2 {
    float lin, in, amp;
    bool capped;
    __device__ __forceinline__ ScoreBase2(const ScoreForm& f, float scale) {
        const float log2e = 1.4426950408889634f;
        capped = f.cap > 0.f;
        lin = scale * log2e;
        in = capped ? 2.f * log2e * scale / f.cap : 0.f;
        amp = f.cap * log2e;
    }
    __device__ __forceinline__ float of(float dot) const {        // (no branch: it stands in unrolled loops)
        const float c = fmaf(-2.f * amp, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(dot * in)), amp);
        return capped ? c : dot * lin;
    }
};
