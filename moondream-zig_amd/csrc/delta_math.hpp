// Scalar parts of the gated delta rule, shared by the kernels for rows and for one token.
#pragma once
#include "lm_types.hpp"

__device__ __forceinline__ float delta_softplus(float z) { return z > 20.0f ? z : log1pf(expf(z)); } // (above, exp(-z) is below an ulp)
// the factor on the state's rows
__device__ __forceinline__ float delta_decay(float a_log, float dt) { return expf(-expf(a_log) * delta_softplus(dt)); }
