// Sums of several values at once over the lanes of a wavefront.
#pragma once
#include "epilogue.hpp"

// Sums of N values over the lanes that differ in the bits of OFF and below down to `stop` (a power of two, the same in every lane).
// At every step a lane hands one half of its values to its partner and keeps the other, so N / 2 + N / 4 + .. exchanges do; done(i, sum)
// is called for the values that end up in this lane (by several lanes where there are fewer values than lanes).
template <int N, int OFF, class Done>
__device__ __forceinline__ void fold_lanes(float (&v)[N], int lane, int stop, int base, Done done) {
    if (OFF < stop) {
#pragma unroll
        for (int i = 0; i < N; i++) done(base + i, v[i]);
        return;
    }
    const bool upper = lane & OFF;
    if constexpr (N > 1) {
        float half[N / 2];
#pragma unroll
        for (int i = 0; i < N / 2; i++) half[i] = (upper ? v[i + N / 2] : v[i]) + __shfl_xor(upper ? v[i] : v[i + N / 2], OFF);
        if constexpr (OFF > 1) fold_lanes<N / 2, OFF / 2>(half, lane, stop, base + (upper ? N / 2 : 0), done);
        else
#pragma unroll
            for (int i = 0; i < N / 2; i++) done(base + (upper ? N / 2 : 0) + i, half[i]);
    } else {
        v[0] += __shfl_xor(v[0], OFF);
        if constexpr (OFF > 1) fold_lanes<1, OFF / 2>(v, lane, stop, base, done);
        else done(base, v[0]);
    }
}
