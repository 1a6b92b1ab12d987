// A decay computed from a pre-activation, a = sigmoid(z)^(1 / tau), by its logarithm: ln a = -softplus(-z) / tau with
// softplus(-z) = max(-z, 0) + ln(1 + e^(-|z|)), which neither overflows nor loses the small a that stand near 1. fp32.
#pragma once

#include "ka_common.h"

// softplus(-z). FAST: on the hardware's exponential and logarithm; ln(1 + e) is then ln(u) e / (u - 1) with u the rounded 1 + e,
// whose rounding error the factor takes back.
template <bool FAST>
__device__ __forceinline__ float ka_softplus_of_minus(float z) {
    if constexpr (FAST) {
        const float e = __expf(-fabsf(z));
        const float u = 1.0f + e;
        const float d = u - 1.0f;
        const float l = d == 0.f ? e : __logf(u) * __fdividef(e, d);
        return fmaxf(-z, 0.f) + l;
    } else {
        return fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)));
    }
}

// log2 of the decay.
template <bool FAST>
__device__ __forceinline__ float ka_log2_decay(float z, float per_tau) {
    return -1.4426950408889634f * per_tau * ka_softplus_of_minus<FAST>(z);
}

template <bool FAST>
__device__ __forceinline__ float ka_decay(float z, float per_tau) {
    if constexpr (FAST) return __builtin_amdgcn_exp2f(ka_log2_decay<true>(z, per_tau));
    else return expf(-per_tau * ka_softplus_of_minus<false>(z));
}
