// Scalar parts of the gated delta rule, shared by the kernels for rows and for one token.
#pragma once
#include "lm_types.hpp"

// e^z by the hardware's power of two: relative error |z| 2^-24 and a few ulp, which the uses below only see where the result no longer counts
__device__ __forceinline__ float delta_exp(float z) { return __builtin_amdgcn_exp2f(z * 1.4426950408889634f); }
// log(1 + e^z) to a few ulp: the logarithm of the rounded sum w = 1 + e, corrected for that rounding by e / (w - 1) (Kahan's method)
__device__ __forceinline__ float delta_softplus(float z) {
    const float e = delta_exp(z), w = 1.0f + e, d = w - 1.0f;
    const float l = d > 0.0f ? __builtin_amdgcn_logf(w) * 0.69314718056f * (e * __builtin_amdgcn_rcpf(d)) : e;
    return z > 20.0f ? z : l; // (there e^-z is below an ulp)
}
// the factor on the state's rows; rate: e^A_log
__device__ __forceinline__ float delta_decay(float rate, float dt) { return delta_exp(-rate * delta_softplus(dt)); }
__device__ __forceinline__ float delta_silu(float z) { return z * __builtin_amdgcn_rcpf(1.0f + delta_exp(-z)); }
