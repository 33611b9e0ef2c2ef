// Scalar parts of the gated delta rule, shared by the kernels for rows and for one token.
#pragma once
#include "lm_types.hpp"

// log(1 + e^z) to a few ulp: the logarithm of the rounded sum w = 1 + e, corrected for that rounding by e / (w - 1) (Kahan's method)
__device__ __forceinline__ float delta_softplus(float z) {
    if (z > 20.0f) return z; // (there e^-z is below an ulp)
    const float e = expf(z), w = 1.0f + e, d = w - 1.0f;
    return d > 0.0f ? __builtin_amdgcn_logf(w) * 0.69314718056f * (e * __builtin_amdgcn_rcpf(d)) : e;
}
// the factor on the state's rows; rate: e^A_log
__device__ __forceinline__ float delta_decay(float rate, float dt) { return expf(-rate * delta_softplus(dt)); }
__device__ __forceinline__ float delta_silu(float z) { return z * __builtin_amdgcn_rcpf(1.0f + expf(-z)); }
