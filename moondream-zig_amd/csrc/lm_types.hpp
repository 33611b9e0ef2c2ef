// Element types of the layer-list decoders: bf16 storage with f32 arithmetic, or f32 throughout.
#pragma once
#include "epilogue.hpp"

typedef unsigned int lm_u32x4 __attribute__((ext_vector_type(4)));

template <class T> struct Piece; // 16 bytes of T
template <> struct Piece<bf16_t> {
    static constexpr int N = 8;
    static __device__ __forceinline__ void unpack(const lm_u32x4 &v, float (&f)[8]) {
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const unsigned pair = v[i];
            f[2 * i] = __builtin_bit_cast(float, pair << 16);
            f[2 * i + 1] = __builtin_bit_cast(float, pair & 0xffff0000u);
        }
    }
};
template <> struct Piece<float> {
    static constexpr int N = 4;
    static __device__ __forceinline__ void unpack(const lm_u32x4 &v, float (&f)[4]) {
        const float4_t w = __builtin_bit_cast(float4_t, v); // (the whole vector: a bit cast of one element reads element 0)
#pragma unroll
        for (int i = 0; i < 4; i++) f[i] = w[i];
    }
};
template <class T> __device__ __forceinline__ float dot_piece(const lm_u32x4 &w, const lm_u32x4 &x, float acc) {
    float a[Piece<T>::N], b[Piece<T>::N];
    Piece<T>::unpack(w, a);
    Piece<T>::unpack(x, b);
#pragma unroll
    for (int i = 0; i < Piece<T>::N; i++) acc = fmaf(a[i], b[i], acc);
    return acc;
}

// library exponentials: the gates and weights are wanted to f32 accuracy
__device__ __forceinline__ float lm_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float lm_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float lm_softcap(float z, float cap) { return cap * tanhf(z / cap); }
