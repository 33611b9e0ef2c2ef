// Choice of experts for one token by one wavefront, in f32: scores sigmoid(z), the `top` largest of score + correction (the
// lower index wins a tie), weights score / (sum of the chosen scores + EXPERT_WEIGHT_EPS).
#pragma once
#include "layer_list.hpp"
#include "lm_types.hpp"

constexpr int ROUTER_MAX_EXPERTS = 512; // LDS of the kernels that route: 2 floats per expert and wavefront

// scores: 2 * E floats of LDS owned by this wavefront; ids / weight may be global memory or LDS
__device__ __forceinline__ void route_wave(const float *logits, const float *correction, int E, int top, float *scores, int lane, int *ids,
                                           float *weight) {
    float *choice = scores + E;
    for (int e = lane; e < E; e += 64) {
        const float s = lm_sigmoid(logits[e]);
        scores[e] = s;
        choice[e] = s + correction[e];
    }
    float sum = 0.0f;
    for (int k = 0; k < top; k++) { // (a lane only ever looks at the entries it wrote itself)
        float best = -INFINITY;
        int idx = 0x7fffffff;
        for (int e = lane; e < E; e += 64)
            if (choice[e] > best) {
                best = choice[e];
                idx = e;
            }
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) {
            const float ob = __shfl_xor(best, off);
            const int oi = __shfl_xor(idx, off);
            if (ob > best || (ob == best && oi < idx)) {
                best = ob;
                idx = oi;
            }
        }
        if (idx >= E) idx = k; // (scores that are not numbers: stay within the experts)
        const float s = __shfl(lane == (idx & 63) ? scores[idx] : 0.0f, idx & 63);
        if (lane == (idx & 63)) choice[idx] = -INFINITY;
        if (lane == 0) {
            ids[k] = idx;
            weight[k] = s;
        }
        sum += s;
    }
    const float inv = 1.0f / (sum + EXPERT_WEIGHT_EPS);
    if (lane == 0)
        for (int k = 0; k < top; k++) weight[k] *= inv;
}
