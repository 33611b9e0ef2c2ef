// One token through a layer of a layer-list decoder, in three launches:
//   decode_proj   h = LayerNorm(x) (or of the embedding row), then the layer's first product: q, k, v, gate, router logits, or a
//                 dense feed-forward's silu(gate) * up.  With only f32 rows it is the LM head.
//   decode_mix    the token's attention over the cache (norm of q and k, value mixing, cache update, sink, output gate), keys split
//                 over workgroups, the one that finishes last merging; beside it, in workgroups of their own, the router's choice and
//                 the chosen experts' silu(gate) * up.
//   decode_out    x += W2 . (heads | dense activation) + the chosen experts' weighted down products.
// All are bound by HBM: weights are read once with 128-bit non-temporal loads.  No workgroup waits for another.
#include "layer_list.hpp"
#include "lm_types.hpp"
#include "norm.hpp"
#include "router.hpp"

#include <algorithm>
#include <type_traits>

namespace {

__device__ __forceinline__ void share(int n, int parts, int i, int &begin, int &end) {
    const int q = n / parts, r = n % parts;
    begin = i * q + min(i, r);
    end = begin + q + (i < r ? 1 : 0);
}

// dots of RG weight rows with a vector in LDS (T, pieces * 16 bytes); every lane returns all of them.  rows[j] null: skipped.
template <class T, int RG, int U>
struct RowDots {
    lm_u32x4 w[RG][U];
    __device__ __forceinline__ void request(const T *const (&rows)[RG], int p0, int pieces, int lane) {
#pragma unroll
        for (int j = 0; j < RG; j++)
#pragma unroll
            for (int u = 0; u < U; u++) {
                const int g = p0 + u * 64 + lane;
                w[j][u] = lm_u32x4{0, 0, 0, 0};
                if (g < pieces && rows[j]) w[j][u] = __builtin_nontemporal_load(reinterpret_cast<const lm_u32x4 *>(rows[j]) + g);
            }
    }
    __device__ __forceinline__ void add(const T *vec, int p0, int pieces, int lane, float (&acc)[RG]) const {
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int g = p0 + u * 64 + lane;
            lm_u32x4 x = {0, 0, 0, 0};
            if (g < pieces) x = *reinterpret_cast<const lm_u32x4 *>(vec + size_t(g) * Piece<T>::N);
#pragma unroll
            for (int j = 0; j < RG; j++) acc[j] = dot_piece<T>(w[j][u], x, acc[j]);
        }
    }
};

// Row of gate/up column pair i (half 0: gate, 1: up) in the interleaved weights
__device__ __forceinline__ int pair_row(int i, int half) { return (i >> 5) * 64 + half * 32 + (i & 31); }

// NV: 16-byte pieces of x, gamma and beta a thread holds (rows of up to 1024 NV elements, a multiple of 4); 0: any row, from memory
template <class T, int U, int NV>
__global__ __launch_bounds__(256) void decode_proj_kernel(DecodeProj p) {
    extern __shared__ __attribute__((aligned(16))) char s_raw[]; // h: T [dp], then (NV = 0) x: float [width]
    T *s_h = reinterpret_cast<T *>(s_raw);
    float *s_x = reinterpret_cast<float *>(s_raw + size_t(p.dp) * sizeof(T));
    __shared__ float s_red[16];
    constexpr int RG = 4;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const T *W = reinterpret_cast<const T *>(p.w1);
    const int pieces = p.dp / Piece<T>::N;
    // The rows in groups of four: the used rows of the 16-bit and the f32 segment (each rounded up to whole groups), then two
    // gate/up pairs per group.
    const int g16 = (p.n16_used + 3) / 4, g32 = g16 + (p.n32_used + 3) / 4, groups = g32 + (p.ff + 1) / 2;
    int g_begin, g_end;
    share(groups, gridDim.x * 4, blockIdx.x * 4 + wave, g_begin, g_end);
    const T *rows[RG];
    auto locate = [&](int g) {
#pragma unroll
        for (int j = 0; j < RG; j++) {
            int row;
            if (g < g16) row = 4 * g + j;
            else if (g < g32) row = p.n16 + 4 * (g - g16) + j;
            else row = p.n32 + pair_row(2 * (g - g32) + (j >> 1), j & 1);
            rows[j] = W + size_t(row) * p.dp; // (segments are padded to whole groups)
        }
    };
    // The norm's inputs are requested first, then the first weights: loads return in order, so the weights stream in while the
    // norm is computed.
    const T *er = p.token ? reinterpret_cast<const T *>(p.embed) + size_t(p.token[0]) * p.dp : nullptr;
    float4_t xv[NV ? NV : 1], gv[NV ? NV : 1], bv[NV ? NV : 1];
    if (NV) {
#pragma unroll
        for (int k = 0; k < NV; k++) {
            const int i = (k * 256 + tid) * 4, j = i < p.width ? i : 0;
            if (er) {
#pragma unroll
                for (int e = 0; e < 4; e++) xv[k][e] = (float)er[j + e];
            } else xv[k] = *reinterpret_cast<const float4_t *>(p.x + j);
            gv[k] = *reinterpret_cast<const float4_t *>(p.gamma + j);
            bv[k] = *reinterpret_cast<const float4_t *>(p.beta + j);
        }
    }
    RowDots<T, RG, U> dots;
    if (g_begin < g_end) {
        locate(g_begin);
        dots.request(rows, 0, pieces, lane);
    }
    float s = 0.0f, m2 = 0.0f;
    if (NV) {
#pragma unroll
        for (int k = 0; k < NV; k++) {
            const int i = (k * 256 + tid) * 4;
            if (er) xv[k] *= p.embed_scale;
            if (i >= p.width) xv[k] = float4_t{0, 0, 0, 0};
            else if (er && blockIdx.x == 0) *reinterpret_cast<float4_t *>(p.x + i) = xv[k];
            s += (xv[k][0] + xv[k][1]) + (xv[k][2] + xv[k][3]);
        }
        const float mean = block_sum(s, s_red) / (float)p.width;
#pragma unroll
        for (int k = 0; k < NV; k++)
            if ((k * 256 + tid) * 4 < p.width) {
                xv[k] -= mean;
#pragma unroll
                for (int e = 0; e < 4; e++) m2 = fmaf(xv[k][e], xv[k][e], m2);
            }
        const float rstd = 1.0f / sqrtf(block_sum(m2, s_red) / (float)p.width + p.eps);
#pragma unroll
        for (int k = 0; k < NV; k++) {
            const int i = (k * 256 + tid) * 4;
            if (i >= p.dp) continue;
            typedef T vec4 __attribute__((ext_vector_type(4)));
            vec4 v;
#pragma unroll
            for (int e = 0; e < 4; e++) v[e] = i < p.width ? (T)(xv[k][e] * rstd * gv[k][e] + bv[k][e]) : (T)0.0f;
            *reinterpret_cast<vec4 *>(s_h + i) = v;
            if (p.h && blockIdx.x == 0) *reinterpret_cast<vec4 *>(reinterpret_cast<T *>(p.h) + i) = v;
        }
    } else {
        for (int i = tid; i < p.width; i += 256) {
            const float v = er ? (float)er[i] * p.embed_scale : p.x[i];
            if (er && blockIdx.x == 0) p.x[i] = v;
            s_x[i] = v;
            s += v;
        }
        const float mean = block_sum(s, s_red) / (float)p.width;
        for (int i = tid; i < p.width; i += 256) {
            const float d = s_x[i] - mean;
            m2 = fmaf(d, d, m2);
        }
        const float rstd = 1.0f / sqrtf(block_sum(m2, s_red) / (float)p.width + p.eps);
        for (int i = tid; i < p.dp; i += 256) {
            const T v = i < p.width ? (T)((s_x[i] - mean) * rstd * p.gamma[i] + p.beta[i]) : (T)0.0f;
            s_h[i] = v;
            if (p.h && blockIdx.x == 0) reinterpret_cast<T *>(p.h)[i] = v;
        }
    }
    lds_barrier();
    for (int g = g_begin; g < g_end; g++) {
        float acc[RG] = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int p0 = 0;;) {
            dots.add(s_h, p0, pieces, lane, acc);
            p0 += 64 * U;
            if (p0 >= pieces) break;
            dots.request(rows, p0, pieces, lane);
        }
        if (g + 1 < g_end) {
            locate(g + 1);
            dots.request(rows, 0, pieces, lane);
        }
#pragma unroll
        for (int j = 0; j < RG; j++) acc[j] = wave_sum(acc[j]);
        if (lane == 0) {
            if (g < g16) *reinterpret_cast<float4 *>(p.proj + 4 * g) = float4{acc[0], acc[1], acc[2], acc[3]};
            else if (g < g32) *reinterpret_cast<float4 *>(p.logits + 4 * (g - g16)) = float4{acc[0], acc[1], acc[2], acc[3]};
            else {
                T *o = reinterpret_cast<T *>(p.glu) + 2 * (g - g32); // (the activation is padded like the weights)
                o[0] = (T)(lm_silu(acc[0]) * acc[1]);
                o[1] = (T)(lm_silu(acc[2]) * acc[3]);
            }
        }
    }
}

constexpr int MIX_HEADS = 8;       // query heads one workgroup serves
constexpr int MIX_KEYS = 1024;     // keys of one split at most
constexpr int MIX_TARGET = 32;     // keys of one split at least
constexpr int MIX_SPLITS = 16;     // splits at most, unless MIX_KEYS asks for more: what the merge requests at once
__host__ __device__ __forceinline__ int mix_head_blocks(int per_group) { return (per_group + MIX_HEADS - 1) / MIX_HEADS; }

__device__ __forceinline__ int next_pow2(int v) { return v <= 1 ? 1 : 1 << (32 - __builtin_clz(v - 1)); }

// LDS of an attention workgroup, in floats: q [NH][dimp], new k [dimp], new v [vdimp], scores [NH][keys], reduction [4][NH][vdimp], misc
__host__ __device__ __forceinline__ size_t mix_lds_floats(int nh, int dimp, int vdimp, int keys) {
    return size_t(nh) * dimp + dimp + vdimp + size_t(nh) * keys + size_t(4) * nh * vdimp + 4 * nh + 8; // (launch_decode_mix: at least nh * S before the misc)
}

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

// Attention of one token: kv head g, query heads h0 .. h0 + nh - 1, split `split` of S.
template <class T, int NH>
__device__ __forceinline__ void mix_attention(const DecodeMix &p, int g, int hb, int split, int S, int keys_max, float *lds) {
    const int per = p.H / p.G, n_hb = mix_head_blocks(per), h0 = g * per + hb * MIX_HEADS, nh = min(MIX_HEADS, per - hb * MIX_HEADS);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int pos = p.pos_dev ? (int)p.pos_dev[0] : (int)p.pos;
    const int lo = p.window ? max(0, pos - p.window + 1) : 0, n_keys = pos - lo + 1, chunk = (n_keys + S - 1) / S;
    const int j0 = lo + split * chunk, j1 = min(j0 + chunk, pos + 1), cnt = max(0, j1 - j0);
    float *s_q = lds, *s_k = s_q + NH * p.dimp, *s_v = s_k + p.dimp, *s_s = s_v + p.vdimp, *s_r = s_s + NH * keys_max, *s_ml = s_r + 4 * NH * p.vdimp;
    T *ck = reinterpret_cast<T *>(p.ck) + size_t(g) * p.cap * p.dimp, *cv = reinterpret_cast<T *>(p.cv) + size_t(g) * p.cap * p.vdimp;
    const bool has_new = cnt > 0 && j1 == pos + 1;
    // K: lpk lanes per key, V: lpv lanes per key (powers of two); a step is the keys the four wavefronts take at once.  The first
    // PF steps' rows are requested before anything else: they do not depend on the new token.
    constexpr int PE = Piece<T>::N, PF = 4;
    const int kp = p.dimp / PE, lpk = min(64, next_pow2(kp)), kpw = 64 / lpk, sub = lane / lpk, c0 = lane % lpk;
    const int vp = p.vdimp / PE, lpv = min(64, next_pow2(vp)), vpw = 64 / lpv, vsub = lane / lpv, vc0 = lane % lpv;
    auto k_piece = [&](int key, int c) { return *reinterpret_cast<const lm_u32x4 *>(ck + size_t(key % p.cap) * p.dimp + c * PE); };
    auto v_piece = [&](int key, int c) { return *reinterpret_cast<const lm_u32x4 *>(cv + size_t(key % p.cap) * p.vdimp + c * PE); };
    lm_u32x4 pk[PF], pv[PF];
#pragma unroll
    for (int i = 0; i < PF; i++) {
        const int key = j0 + (i * 4 + wave) * kpw + sub;
        pk[i] = lm_u32x4{0, 0, 0, 0};
        if (key < j1 && key != pos && c0 < kp) pk[i] = k_piece(key, c0);
    }
#pragma unroll
    for (int i = 0; i < PF; i++) {
        const int key = j0 + (i * 4 + wave) * vpw + vsub;
        pv[i] = lm_u32x4{0, 0, 0, 0};
        if (key < j1 && key != pos && vc0 < vp) pv[i] = v_piece(key, vc0);
    }
    for (int task = wave; task < nh + (has_new ? 2 : 0); task += 4) {
        if (task == nh + 1) { // the new value
            const T *first = p.mixes ? reinterpret_cast<const T *>(p.v_first) + (size_t(g) * p.cap_first + pos % p.cap_first) * p.vdimp : nullptr;
            for (int d = lane; d < p.vdimp; d += 64) {
                float v = (float)(T)p.proj[p.ov + g * p.vdimp + d];
                if (first) v = (1.0f - p.lambda) * v + p.lambda * (float)first[d];
                const T c = (T)v;
                s_v[d] = (float)c;
                if (hb == 0) cv[size_t(pos % p.cap) * p.vdimp + d] = c;
            }
        } else { // a query head or the new key
            const bool is_q = task < nh;
            const float *src = p.proj + (is_q ? (h0 + task) * p.dimp : p.ok + g * p.dimp);
            float ss = 0.0f;
            for (int d = lane; d < p.dimp; d += 64) ss = fmaf(src[d], src[d], ss);
            const float f = p.qk_rms ? 1.0f / sqrtf(wave_sum(ss) / (float)p.dim + p.eps) : 1.0f;
            for (int d = lane; d < p.dimp; d += 64) {
                const T c = (T)(src[d] * f);
                if (is_q) s_q[task * p.dimp + d] = (float)c;
                else {
                    s_k[d] = (float)c;
                    if (hb == 0) ck[size_t(pos % p.cap) * p.dimp + d] = c;
                }
            }
        }
    }
    lds_barrier();
    auto score_step = [&](int key, const lm_u32x4 &first) {
        float acc[NH];
#pragma unroll
        for (int h = 0; h < NH; h++) acc[h] = 0.0f;
        if (key < j1)
            for (int c = c0; c < kp; c += lpk) {
                float kf[PE];
                if (key == pos) {
#pragma unroll
                    for (int e = 0; e < PE; e++) kf[e] = s_k[c * PE + e];
                } else Piece<T>::unpack(c == c0 ? first : k_piece(key, c), kf);
#pragma unroll
                for (int h = 0; h < NH; h++)
                    if (h < nh)
#pragma unroll
                        for (int e = 0; e < PE; e++) acc[h] = fmaf(kf[e], s_q[h * p.dimp + c * PE + e], acc[h]);
            }
#pragma unroll
        for (int h = 0; h < NH; h++) {
            for (int off = lpk >> 1; off >= 1; off >>= 1) acc[h] += __shfl_xor(acc[h], off);
            if (key < j1 && c0 == 0 && h < nh) s_s[h * keys_max + key - j0] = acc[h] * p.scale;
        }
    };
#pragma unroll
    for (int i = 0; i < PF; i++)
        if (j0 + (i * 4 + wave) * kpw < j1) score_step(j0 + (i * 4 + wave) * kpw + sub, pk[i]);
    for (int j = j0 + (PF * 4 + wave) * kpw; j < j1; j += 4 * kpw) {
        const int key = j + sub;
        lm_u32x4 first = {0, 0, 0, 0};
        if (key < j1 && key != pos && c0 < kp) first = k_piece(key, c0);
        score_step(key, first);
    }
    lds_barrier();
    for (int h = wave; h < nh; h += 4) {
        float m = -INFINITY;
        for (int i = lane; i < cnt; i += 64) m = fmaxf(m, s_s[h * keys_max + i]);
        m = wave_max(m);
        float l = 0.0f;
        for (int i = lane; i < cnt; i += 64) {
            const float e = expf(s_s[h * keys_max + i] - m);
            s_s[h * keys_max + i] = e;
            l += e;
        }
        l = wave_sum(l);
        if (lane == 0) {
            s_ml[2 * h] = m;
            s_ml[2 * h + 1] = l;
        }
    }
    lds_barrier();
    for (int c = vc0; c < (vp + lpv - 1) / lpv * lpv; c += lpv) {
        float acc[NH][PE];
#pragma unroll
        for (int h = 0; h < NH; h++)
#pragma unroll
            for (int e = 0; e < PE; e++) acc[h][e] = 0.0f;
        auto value_step = [&](int key, const lm_u32x4 &piece) {
            float vf[PE];
            if (key == pos) {
#pragma unroll
                for (int e = 0; e < PE; e++) vf[e] = s_v[c * PE + e];
            } else Piece<T>::unpack(piece, vf);
#pragma unroll
            for (int h = 0; h < NH; h++)
                if (h < nh) {
                    const float w = s_s[h * keys_max + key - j0];
#pragma unroll
                    for (int e = 0; e < PE; e++) acc[h][e] = fmaf(w, vf[e], acc[h][e]);
                }
        };
        if (c < vp) {
#pragma unroll
            for (int i = 0; i < PF; i++) {
                const int key = j0 + (i * 4 + wave) * vpw + vsub;
                if (key < j1) value_step(key, c == vc0 || key == pos ? pv[i] : v_piece(key, c));
            }
            for (int key = j0 + (PF * 4 + wave) * vpw + vsub; key < j1; key += 4 * vpw) value_step(key, key == pos ? pv[0] : v_piece(key, c));
        }
        float flat[NH * PE];
#pragma unroll
        for (int h = 0; h < NH; h++)
#pragma unroll
            for (int e = 0; e < PE; e++) flat[h * PE + e] = acc[h][e];
        fold_lanes<NH * PE, 32>(flat, lane, lpv, 0, [&](int i, float v) {
            if (c < vp && i / PE < nh) s_r[(wave * NH + i / PE) * p.vdimp + c * PE + i % PE] = v;
        });
    }
    lds_barrier();
    // This split's sums and (m, l) per head to memory; the workgroup that counts in last adds the splits up.
    const int stride = p.vdimp + 2;
    float *part = p.partial + size_t(g * n_hb + hb) * S * MIX_HEADS * stride;
    for (int i = tid; i < nh * p.vdimp; i += 256) {
        const int h = i / p.vdimp, d = i % p.vdimp;
        const float v = (s_r[(0 * NH + h) * p.vdimp + d] + s_r[(1 * NH + h) * p.vdimp + d]) + (s_r[(2 * NH + h) * p.vdimp + d] + s_r[(3 * NH + h) * p.vdimp + d]);
        st_f<true>(part + (size_t(split) * MIX_HEADS + h) * stride + d, v);
    }
    if (tid < 2 * nh) st_f<true>(part + (size_t(split) * MIX_HEADS + (tid >> 1)) * stride + p.vdimp + (tid & 1), s_ml[tid]);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); // stored before the workgroup counts in
    int *s_last = reinterpret_cast<int *>(s_ml + 2 * NH);
    __syncthreads();
    if (tid == 0) {
        uint32_t *counter = p.counter + g * n_hb + hb;
        const uint32_t old = __hip_atomic_fetch_add(counter, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        *s_last = old + 1 == (uint32_t)S;
        if (*s_last) __hip_atomic_store(counter, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); // ready for the next launch
    }
    __syncthreads();
    if (!*s_last) return;
    // Every head's splits: this thread's elements of the first splits and all (m, l) are requested together; the weight of each
    // split (a lane per split) goes through LDS.
    constexpr int AT_ONCE = MIX_SPLITS;
    const size_t pitch = size_t(MIX_HEADS) * stride; // floats between splits
    float *s_w = lds; // [nh][S], over what the phases before have used
    float v[AT_ONCE];
    {
        const int i = min(tid, nh * p.vdimp - 1);
        const float *ph = part + size_t(i / p.vdimp) * stride + i % p.vdimp;
#pragma unroll
        for (int u = 0; u < AT_ONCE; u++) v[u] = ld_f<true>(ph + min(u, S - 1) * pitch);
    }
    for (int h = wave; h < nh; h += 4) {
        const float *ph = part + size_t(h) * stride + p.vdimp, sink = p.sink ? p.sink[h0 + h] : -INFINITY;
        const float m0 = lane < S ? ld_f<true>(ph + lane * pitch) : -INFINITY, l0 = lane < S ? ld_f<true>(ph + lane * pitch + 1) : 0.0f;
        float m = fmaxf(sink, m0), l = 0.0f;
        for (int s = lane + 64; s < S; s += 64) m = fmaxf(m, ld_f<true>(ph + s * pitch));
        m = wave_max(m);
        for (int s = lane; s < S; s += 64) { // (an empty split: m = -inf, weight 0)
            const float w = expf((s == lane ? m0 : ld_f<true>(ph + s * pitch)) - m);
            l = fmaf(s == lane ? l0 : ld_f<true>(ph + s * pitch + 1), w, l);
            s_w[h * S + s] = w;
        }
        l = wave_sum(l) + (p.sink ? expf(sink - m) : 0.0f);
        if (lane == 0) s_ml[h] = 1.0f / l;
    }
    lds_barrier();
    for (int i = tid; i < nh * p.vdimp; i += 256) {
        const int h = i / p.vdimp, d = i % p.vdimp;
        const float *ph = part + size_t(h) * stride + d;
        float o = 0.0f;
        for (int s0 = 0; s0 < S; s0 += AT_ONCE) {
            if (s0 || i != tid)
#pragma unroll
                for (int u = 0; u < AT_ONCE; u++) v[u] = ld_f<true>(ph + min(s0 + u, S - 1) * pitch);
#pragma unroll
            for (int u = 0; u < AT_ONCE; u++)
                if (s0 + u < S) o = fmaf(v[u], s_w[h * S + s0 + u], o);
        }
        o *= s_ml[h];
        if (p.gate) o *= lm_sigmoid(p.proj[p.og + (h0 + h) * p.vdimp + d]);
        reinterpret_cast<T *>(p.out)[(h0 + h) * p.vdimp + d] = (T)o;
    }
}

// The chosen experts' gate and up rows, by the launch's expert workgroups.
template <class T, int U>
__device__ __forceinline__ void mix_experts(const DecodeMix &p, int wg, int n_wgs, char *lds) {
    constexpr int RG = 4;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, pieces = p.dp / Piece<T>::N;
    T *s_h = reinterpret_cast<T *>(lds);
    float *s_scores = reinterpret_cast<float *>(lds + size_t(p.dp) * sizeof(T)); // [2 E]
    float *s_w = s_scores + 2 * p.E;                                              // [top]
    int *s_ids = reinterpret_cast<int *>(s_w + p.top);                            // [top]
    for (int i = tid; i < pieces; i += 256) reinterpret_cast<lm_u32x4 *>(s_h)[i] = reinterpret_cast<const lm_u32x4 *>(p.h)[i];
    if (wave == 0) route_wave(p.logits, p.correction, p.E, p.top, s_scores, lane, s_ids, s_w);
    __syncthreads();
    if (wg == 0)
        for (int k = tid; k < p.top; k += 256) {
            p.ids[k] = s_ids[k];
            p.weight[k] = s_w[k];
        }
    const int per_expert = (p.ff + 1) / 2; // groups of two pairs
    int g_begin, g_end;
    share(p.top * per_expert, n_wgs * 4, wg * 4 + wave, g_begin, g_end);
    RowDots<T, RG, U> dots;
    const T *rows[RG];
    auto locate = [&](int g) {
        const int k = g / per_expert, i = 2 * (g % per_expert);
        const T *W = reinterpret_cast<const T *>(p.wgu) + size_t(s_ids[k]) * 2 * p.ffp * p.dp;
#pragma unroll
        for (int j = 0; j < RG; j++) rows[j] = W + size_t(pair_row(i + (j >> 1), j & 1)) * p.dp;
    };
    if (g_begin < g_end) {
        locate(g_begin);
        dots.request(rows, 0, pieces, lane);
    }
    for (int g = g_begin; g < g_end; g++) {
        float acc[RG] = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int p0 = 0;;) {
            dots.add(s_h, p0, pieces, lane, acc);
            p0 += 64 * U;
            if (p0 >= pieces) break;
            dots.request(rows, p0, pieces, lane);
        }
        if (g + 1 < g_end) {
            locate(g + 1);
            dots.request(rows, 0, pieces, lane);
        }
#pragma unroll
        for (int j = 0; j < RG; j++) acc[j] = wave_sum(acc[j]);
        if (lane == 0) {
            T *o = reinterpret_cast<T *>(p.act) + size_t(g / per_expert) * p.ffp + 2 * (g % per_expert);
            o[0] = (T)(lm_silu(acc[0]) * acc[1]);
            o[1] = (T)(lm_silu(acc[2]) * acc[3]);
        }
    }
}

template <class T, int NH, int U>
__global__ __launch_bounds__(256) void decode_mix_kernel(DecodeMix p, int S, int keys_max, int n_attn, int n_expert) {
    extern __shared__ __attribute__((aligned(16))) char s_mix[];
    // attention first: it is a chain of dependent steps, the experts' part is one long stream
    const int i = blockIdx.x, n_hb = mix_head_blocks(p.H / p.G);
    if (i < n_attn) mix_attention<T, NH>(p, i / S / n_hb, i / S % n_hb, i % S, S, keys_max, reinterpret_cast<float *>(s_mix));
    else mix_experts<T, U>(p, i - n_attn, n_expert, s_mix);
}

// x[n] += sum over the pieces of row n of W2 against a, and of the chosen experts' rows against their activations.  A workgroup
// owns RW rows; its four wavefronts share each row's pieces, so a lane reads its part of the vectors once for all rows.
template <class T, int RW, int U>
__global__ __launch_bounds__(256) void decode_out_kernel(DecodeOut p) {
    __shared__ float s_part[4][RW];
    constexpr int PE = Piece<T>::N;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, row0 = blockIdx.x * RW;
    const int pa = p.k0 / PE, pf = p.top ? p.ffp / PE : 1, total = pa + p.top * pf;
    int begin, end;
    share(total, 4, wave, begin, end);
    float acc[RW];
#pragma unroll
    for (int r = 0; r < RW; r++) acc[r] = 0.0f;
    for (int base = begin; base < end; base += 64 * U) {
        lm_u32x4 w[U][RW], x[U];
        float scale[U];
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int i = base + u * 64 + lane;
            x[u] = lm_u32x4{0, 0, 0, 0};
            scale[u] = 1.0f;
#pragma unroll
            for (int r = 0; r < RW; r++) w[u][r] = lm_u32x4{0, 0, 0, 0};
            if (i < end) {
                const T *m;
                size_t pitch;
                if (i < pa) {
                    x[u] = reinterpret_cast<const lm_u32x4 *>(p.a)[i];
                    m = reinterpret_cast<const T *>(p.w2) + size_t(row0) * p.k0 + size_t(i) * PE;
                    pitch = p.k0;
                } else {
                    const int k = (i - pa) / pf, c = (i - pa) % pf;
                    x[u] = reinterpret_cast<const lm_u32x4 *>(p.act)[size_t(k) * pf + c];
                    scale[u] = p.weight[k];
                    m = reinterpret_cast<const T *>(p.wd) + (size_t(p.ids[k]) * p.dp + row0) * p.ffp + size_t(c) * PE;
                    pitch = p.ffp;
                }
#pragma unroll
                for (int r = 0; r < RW; r++) // (rows are padded to 64)
                    w[u][r] = __builtin_nontemporal_load(reinterpret_cast<const lm_u32x4 *>(m + r * pitch));
            }
        }
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int r = 0; r < RW; r++) acc[r] = fmaf(dot_piece<T>(w[u][r], x[u], 0.0f), scale[u], acc[r]);
    }
#pragma unroll
    for (int r = 0; r < RW; r++) {
        const float s = wave_sum(acc[r]);
        if (lane == 0) s_part[wave][r] = s;
    }
    lds_barrier();
    if (tid < RW && row0 + tid < p.width) p.x[row0 + tid] += (s_part[0][tid] + s_part[1][tid]) + (s_part[2][tid] + s_part[3][tid]);
}

template <class T, int NH> int mix_launch(moon_ctx *ctx, const DecodeMix &p, int S, int keys_max, int n_attn, int n_expert, size_t lds) {
    auto kern = p.dp / Piece<T>::N > 64 ? decode_mix_kernel<T, NH, 4> : decode_mix_kernel<T, NH, 1>;
    if (lds > 64 * 1024) MOON_HIP(ctx, hipFuncSetAttribute(reinterpret_cast<const void *>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(kern, dim3(n_attn + n_expert), dim3(256), lds, ctx->stream, p, S, keys_max, n_attn, n_expert);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

template <class T> int proj_launch(moon_ctx *ctx, const DecodeProj &p) {
    const int cus = ctx->cu_count > 0 ? ctx->cu_count : 256;
    const int groups = (p.n16_used + 3) / 4 + (p.n32_used + 3) / 4 + (p.ff + 1) / 2;
    const dim3 grid((unsigned)std::max(1, std::min(2 * cus, (groups + 3) / 4)));
    const int ch = (p.dp / Piece<T>::N + 63) / 64, nv = p.width % 4 || p.dp > 4096 || (reinterpret_cast<uintptr_t>(p.x) & 15) ? 0 : (p.dp + 1023) / 1024;
    const size_t lds = size_t(p.dp) * sizeof(T) + (nv ? 0 : size_t(p.width) * sizeof(float));
    if (lds > 60 * 1024) return moon_fail(ctx, MOON_EINVAL_DIM, "decode: width %d too large", p.width);
    auto pick = [&](auto u) {
        constexpr int U = decltype(u)::value;
        return nv == 0 ? decode_proj_kernel<T, U, 0> : nv == 1 ? decode_proj_kernel<T, U, 1> : nv == 2 ? decode_proj_kernel<T, U, 2> : decode_proj_kernel<T, U, 4>;
    };
    auto kern = ch == 1 ? pick(std::integral_constant<int, 1>{}) : ch == 2 ? pick(std::integral_constant<int, 2>{}) : ch == 3 ? pick(std::integral_constant<int, 3>{})
                                                                                                                          : pick(std::integral_constant<int, 4>{});
    hipLaunchKernelGGL(kern, grid, dim3(256), lds, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

template <class T> int out_launch(moon_ctx *ctx, const DecodeOut &p) {
    const int cus = ctx->cu_count > 0 ? ctx->cu_count : 256;
    if (p.width >= 4 * 2 * cus) hipLaunchKernelGGL((decode_out_kernel<T, 4, 4>), dim3((p.width + 3) / 4), dim3(256), 0, ctx->stream, p);
    else if (p.width >= 2 * 2 * cus) hipLaunchKernelGGL((decode_out_kernel<T, 2, 6>), dim3((p.width + 1) / 2), dim3(256), 0, ctx->stream, p);
    else hipLaunchKernelGGL((decode_out_kernel<T, 1, 8>), dim3(p.width), dim3(256), 0, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

} // namespace

int launch_decode_proj(moon_ctx *ctx, int dtype, const DecodeProj &p) {
    return dtype == MOON_DTYPE_BF16 ? proj_launch<bf16_t>(ctx, p) : proj_launch<float>(ctx, p);
}

int launch_decode_out(moon_ctx *ctx, int dtype, const DecodeOut &p) {
    return dtype == MOON_DTYPE_BF16 ? out_launch<bf16_t>(ctx, p) : out_launch<float>(ctx, p);
}

size_t decode_mix_counters(size_t heads, size_t kv_heads) { return kv_heads * mix_head_blocks((int)(heads / kv_heads)); }
size_t decode_mix_partial_floats(moon_ctx *ctx, size_t heads, size_t kv_heads, size_t vdimp, size_t max_keys) {
    const size_t cus = ctx->cu_count > 0 ? ctx->cu_count : 256, wgs = decode_mix_counters(heads, kv_heads);
    return std::max(std::max(wgs, cus), wgs * ((max_keys + MIX_KEYS - 1) / MIX_KEYS)) * MIX_HEADS * (vdimp + 2);
}

int launch_decode_mix(moon_ctx *ctx, int dtype, const DecodeMix &p) {
    const int cus = ctx->cu_count > 0 ? ctx->cu_count : 256, per = p.H / p.G, wgs = p.G * mix_head_blocks(per);
    const int n_keys = (int)(p.window ? std::min(p.pos + 1, (size_t)p.window) : p.pos + 1);
    int S = std::min(std::min((n_keys + MIX_TARGET - 1) / MIX_TARGET, MIX_SPLITS), std::max(1, cus / wgs));
    S = std::max(S, (n_keys + MIX_KEYS - 1) / MIX_KEYS);
    if (size_t(wgs) * S * MIX_HEADS * (p.vdimp + 2) > p.partial_floats) return moon_fail(ctx, MOON_ESEQ_TOO_LONG, "decode attention: %d keys", n_keys);
    const int keys_max = (n_keys + S - 1) / S;
    if (p.E && (p.top < 1 || p.top > p.E || p.E > ROUTER_MAX_EXPERTS)) return moon_fail(ctx, MOON_EINVAL_DIM, "router: %d of %d experts", p.top, p.E);
    const int groups = p.E ? p.top * ((p.ff + 1) / 2) : 0;
    const int n_expert = std::min((groups + 3) / 4, std::max(cus, 2 * cus - wgs * S)); // (together two workgroups per CU: more measured slower)
    const int nh = std::min(per, MIX_HEADS), NH = nh <= 1 ? 1 : nh <= 2 ? 2 : nh <= 4 ? 4 : 8;
    const size_t el = dtype == MOON_DTYPE_BF16 ? sizeof(bf16_t) : sizeof(float);
    const size_t lds = std::max(mix_lds_floats(NH, p.dimp, p.vdimp, keys_max) * sizeof(float),
                                p.E ? size_t(p.dp) * el + (size_t(2) * p.E + 2 * p.top) * sizeof(float) : 0);
    if (size_t(NH) * S > mix_lds_floats(NH, p.dimp, p.vdimp, keys_max) - 4 * NH - 8) return moon_fail(ctx, MOON_ESEQ_TOO_LONG, "decode attention: %d splits", S);
    if (lds > 160 * 1024) return moon_fail(ctx, MOON_EINVAL_DIM, "decode attention: heads of %d and %d", p.dimp, p.vdimp);
    auto go = [&](auto tag) -> int {
        using T = decltype(tag);
        switch (NH) {
        case 1: return mix_launch<T, 1>(ctx, p, S, keys_max, wgs * S, n_expert, lds);
        case 2: return mix_launch<T, 2>(ctx, p, S, keys_max, wgs * S, n_expert, lds);
        case 4: return mix_launch<T, 4>(ctx, p, S, keys_max, wgs * S, n_expert, lds);
        default: return mix_launch<T, 8>(ctx, p, S, keys_max, wgs * S, n_expert, lds);
        }
    };
    return dtype == MOON_DTYPE_BF16 ? go(bf16_t{}) : go(float{});
}
