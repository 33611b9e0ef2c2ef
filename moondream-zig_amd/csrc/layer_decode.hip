// One token through a layer of a layer-list decoder, in three launches:
//   decode_proj   h = norm(x) (or of the embedding row; behind a layer of two joined mixers x is completed first), then the layer's
//                 first product: q, k, v, gate, router logits, or a dense feed-forward's silu(gate) * up.  With only f32 rows it is
//                 the LM head.
//   decode_mix    the token's attention over the cache (norm of q and k, rotation, value mixing, cache update, sink, output gate), keys
//                 split over workgroups, the one that finishes last merging; beside it, in workgroups of their own, the router's choice
//                 and the chosen experts' silu(gate) * up, or one token of the gated delta rule, a head per workgroup.
//   decode_out    x += W2 . (heads | dense activation) + the chosen experts' weighted down products, or the parts of W2 . (..) that
//                 the next decode_proj joins.
// All are bound by HBM: weights are read once with 128-bit non-temporal loads.  No workgroup waits for another.
#include "delta_math.hpp"
#include "lane_fold.hpp"
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

// NV: 16-byte pieces of x, gamma and beta a thread holds (rows of up to 1024 NV elements, a multiple of 4); 0: any row, from memory.
// JOIN: x is completed with a joined layer's results first.
template <class T, int U, int NV, bool JOIN>
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
    float4_t jl[JOIN && NV ? NV : 1], jr[JOIN && NV ? NV : 1], wl[JOIN && NV ? NV : 1], wr[JOIN && NV ? NV : 1];
    if (NV) {
#pragma unroll
        for (int k = 0; k < NV; k++) {
            const int i = (k * 256 + tid) * 4, j = i < p.width ? i : 0;
            if (er) {
#pragma unroll
                for (int e = 0; e < 4; e++) xv[k][e] = (float)er[j + e];
            } else xv[k] = *reinterpret_cast<const float4_t *>(p.x + j);
            if (JOIN) {
                jl[k] = *reinterpret_cast<const float4_t *>(p.y + j);
                jr[k] = *reinterpret_cast<const float4_t *>(p.y + p.dp + j);
                xv[k] += *reinterpret_cast<const float4_t *>(p.y + 2 * p.dp + j);
                wl[k] = *reinterpret_cast<const float4_t *>(p.out_l + j);
                wr[k] = *reinterpret_cast<const float4_t *>(p.out_r + j);
            }
            gv[k] = *reinterpret_cast<const float4_t *>(p.gamma + j);
            bv[k] = p.beta ? *reinterpret_cast<const float4_t *>(p.beta + j) : float4_t{0, 0, 0, 0};
        }
    }
    RowDots<T, RG, U> dots;
    if (g_begin < g_end) {
        locate(g_begin);
        dots.request(rows, 0, pieces, lane);
    }
    float s = 0.0f, m2 = 0.0f;
    if (JOIN) {
        float ss[2] = {0.0f, 0.0f}; // of the two results
        if (NV) {
#pragma unroll
            for (int k = 0; k < NV; k++)
                if ((k * 256 + tid) * 4 < p.width)
#pragma unroll
                    for (int e = 0; e < 4; e++) {
                        ss[0] = fmaf(jl[k][e], jl[k][e], ss[0]);
                        ss[1] = fmaf(jr[k][e], jr[k][e], ss[1]);
                    }
        } else
            for (int i = tid; i < p.width; i += 256) {
                ss[0] = fmaf(p.y[i], p.y[i], ss[0]);
                ss[1] = fmaf(p.y[p.dp + i], p.y[p.dp + i], ss[1]);
            }
        ss[0] = wave_sum(ss[0]);
        ss[1] = wave_sum(ss[1]);
        if (lane == 0) {
            s_red[8 + wave] = ss[0];
            s_red[12 + wave] = ss[1];
        }
        lds_barrier();
        const float f_l = 0.5f / sqrtf(((s_red[8] + s_red[9]) + (s_red[10] + s_red[11])) / (float)p.width + p.eps);
        const float f_r = 0.5f / sqrtf(((s_red[12] + s_red[13]) + (s_red[14] + s_red[15])) / (float)p.width + p.eps);
        if (NV) {
#pragma unroll
            for (int k = 0; k < NV; k++) {
                const int i = (k * 256 + tid) * 4;
#pragma unroll
                for (int e = 0; e < 4; e++) xv[k][e] += jl[k][e] * f_l * wl[k][e] + jr[k][e] * f_r * wr[k][e];
                if (i < p.width && blockIdx.x == 0) *reinterpret_cast<float4_t *>(p.x_new + i) = xv[k];
            }
        } else
            for (int i = tid; i < p.width; i += 256) {
                s_x[i] = p.x[i] + p.y[2 * p.dp + i] + (p.y[i] * f_l * p.out_l[i] + p.y[p.dp + i] * f_r * p.out_r[i]);
                if (blockIdx.x == 0) p.x_new[i] = s_x[i];
            }
    }
    if (NV) {
#pragma unroll
        for (int k = 0; k < NV; k++) {
            const int i = (k * 256 + tid) * 4;
            if (er) xv[k] *= p.embed_scale;
            if (i >= p.width) xv[k] = float4_t{0, 0, 0, 0};
            else if (er && blockIdx.x == 0) *reinterpret_cast<float4_t *>(p.x + i) = xv[k];
            s += (xv[k][0] + xv[k][1]) + (xv[k][2] + xv[k][3]);
        }
        const float mean = p.beta ? block_sum(s, s_red) / (float)p.width : 0.0f; // (an RMS norm takes no mean off)
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
            const float v = er ? (float)er[i] * p.embed_scale : JOIN ? s_x[i] : p.x[i];
            if (er && blockIdx.x == 0) p.x[i] = v;
            s_x[i] = v;
            s += v;
        }
        const float mean = p.beta ? block_sum(s, s_red) / (float)p.width : 0.0f;
        for (int i = tid; i < p.width; i += 256) {
            const float d = s_x[i] - mean;
            m2 = fmaf(d, d, m2);
        }
        const float rstd = 1.0f / sqrtf(block_sum(m2, s_red) / (float)p.width + p.eps);
        for (int i = tid; i < p.dp; i += 256) {
            const T v = i < p.width ? (T)((s_x[i] - mean) * rstd * p.gamma[i] + (p.beta ? p.beta[i] : 0.0f)) : (T)0.0f;
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
            else if (g < g32) {
                float4 z = {acc[0], acc[1], acc[2], acc[3]};
                if (p.softcap > 0.0f) z = {lm_softcap(z.x, p.softcap), lm_softcap(z.y, p.softcap), lm_softcap(z.z, p.softcap), lm_softcap(z.w, p.softcap)};
                *reinterpret_cast<float4 *>(p.logits + 4 * (g - g16)) = z;
            }
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

// Attention of one token: kv head g, query heads h0 .. h0 + nh - 1, split `split` of S.  Keys are numbered: the blocks that lie before
// the window, then the window's tokens.  WHOLE: the mechanisms of the last part of DecodeMix.
template <class T, int NH, bool WHOLE>
__device__ __forceinline__ void mix_attention(const DecodeMix &p, int g, int hb, int split, int S, int keys_max, float *lds) {
    const int per = p.H / p.G, n_hb = mix_head_blocks(per), h0 = g * per + hb * MIX_HEADS, nh = min(MIX_HEADS, per - hb * MIX_HEADS);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int pos = p.pos_dev ? (int)p.pos_dev[0] : (int)p.pos;
    const int lo = p.window ? max(0, pos - p.window + 1) : 0, blocks = WHOLE && p.pool ? lo / p.pool : 0, n_keys = blocks + pos - lo + 1;
    const int chunk = (n_keys + S - 1) / S, j0 = split * chunk, j1 = min(j0 + chunk, n_keys), cnt = max(0, j1 - j0);
    const bool own = !(WHOLE && p.borrowed);    // the token's key and value are not in the cache yet
    const int newest = own ? n_keys - 1 : -1;   // their number
    float *s_q = lds, *s_k = s_q + NH * p.dimp, *s_v = s_k + p.dimp, *s_s = s_v + p.vdimp, *s_r = s_s + NH * keys_max, *s_ml = s_r + 4 * NH * p.vdimp;
    T *ck = reinterpret_cast<T *>(p.ck) + size_t(g) * p.cap * p.dimp, *cv = reinterpret_cast<T *>(p.cv) + size_t(g) * p.cap * p.vdimp;
    const T *pk_rows = reinterpret_cast<const T *>(p.pk) + size_t(g) * p.blocks * p.dimp, *pv_rows = reinterpret_cast<const T *>(p.pv) + size_t(g) * p.blocks * p.vdimp;
    const bool has_new = own && cnt > 0 && j1 == n_keys;
    // K: lpk lanes per key, V: lpv lanes per key (powers of two); a step is the keys the four wavefronts take at once.  The first
    // PF steps' rows are requested before anything else: they do not depend on the new token.
    constexpr int PE = Piece<T>::N, PF = 4;
    const int kp = p.dimp / PE, lpk = min(64, next_pow2(kp)), kpw = 64 / lpk, sub = lane / lpk, c0 = lane % lpk;
    const int vp = p.vdimp / PE, lpv = min(64, next_pow2(vp)), vpw = 64 / lpv, vsub = lane / lpv, vc0 = lane % lpv;
    auto k_piece = [&](int key, int c) {
        const T *row = WHOLE && key < blocks ? pk_rows + size_t(key) * p.dimp : ck + size_t((key - blocks + lo) % p.cap) * p.dimp;
        return *reinterpret_cast<const lm_u32x4 *>(row + c * PE);
    };
    auto v_piece = [&](int key, int c) {
        const T *row = WHOLE && key < blocks ? pv_rows + size_t(key) * p.vdimp : cv + size_t((key - blocks + lo) % p.cap) * p.vdimp;
        return *reinterpret_cast<const lm_u32x4 *>(row + c * PE);
    };
    lm_u32x4 pk[PF], pv[PF];
#pragma unroll
    for (int i = 0; i < PF; i++) {
        const int key = j0 + (i * 4 + wave) * kpw + sub;
        pk[i] = lm_u32x4{0, 0, 0, 0};
        if (key < j1 && key != newest && c0 < kp) pk[i] = k_piece(key, c0);
    }
#pragma unroll
    for (int i = 0; i < PF; i++) {
        const int key = j0 + (i * 4 + wave) * vpw + vsub;
        pv[i] = lm_u32x4{0, 0, 0, 0};
        if (key < j1 && key != newest && vc0 < vp) pv[i] = v_piece(key, vc0);
    }
    // element d of a head x, times its weight w, turned by its pair's angle
    auto turned = [&](const float *x, const float *w, int d, const float2 *table, int half) {
        float y = w ? x[d] * w[d] : x[d];
        if (!table || d >= 2 * half) return y;
        const int m = d < half ? d : d - half, other = d < half ? d + half : m;
        const float2 cs = table[size_t(pos) * half + m];
        const float z = w ? x[other] * w[other] : x[other];
        return d < half ? y * cs.x - z * cs.y : y * cs.x + z * cs.y;
    };
    // where the outputs turn back: the angle of this thread's first element, requested early
    const int back = WHOLE && p.rotv ? p.vdim / 2 : 0;
    float2 back_cs = {1.0f, 0.0f};
    if (WHOLE && back && tid % p.vdimp < 2 * back) back_cs = p.rotv[size_t(pos) * back + tid % p.vdimp % back];
    if constexpr (WHOLE) {
        // q and k are normed as a whole: the heads go to LDS turned and weighted, the norms' factors come last
        float ss[2] = {0.0f, 0.0f};
        const int nq = p.H * p.dimp, nk = has_new ? p.G * p.dimp : 0;
        if (p.whole) {
            for (int i = tid * 4; i < nq; i += 1024) {
                const float4_t v = *reinterpret_cast<const float4_t *>(p.proj + i);
                ss[0] += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
            }
            for (int i = tid * 4; i < nk; i += 1024) {
                const float4_t v = *reinterpret_cast<const float4_t *>(p.proj + p.ok + i);
                ss[1] += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
            }
        }
        for (int task = wave; task < nh + (has_new ? 2 : 0); task += 4) {
            const bool is_v = task == nh + 1, is_q = task < nh;
            const float *src = p.proj + (is_v ? p.ov + g * p.vdimp : is_q ? (h0 + task) * p.dimp : p.ok + g * p.dimp);
            const float *w = is_v || !p.whole ? nullptr : is_q ? p.qn + (h0 + task) * p.dimp : p.kn + g * p.dimp;
            for (int d = lane; d < (is_v ? p.vdimp : p.dimp); d += 64)
                (is_v ? s_v : is_q ? s_q + task * p.dimp : s_k)[d] = turned(src, w, d, is_v ? p.rotv : p.rot, (is_v ? p.vdim : p.rot_dims) / 2);
        }
        ss[0] = wave_sum(ss[0]);
        ss[1] = wave_sum(ss[1]);
        if (lane == 0) {
            s_r[2 * wave] = ss[0];
            s_r[2 * wave + 1] = ss[1];
        }
        lds_barrier();
        const float f_q = p.whole ? 1.0f / sqrtf(((s_r[0] + s_r[2]) + (s_r[4] + s_r[6])) / (float)(p.H * p.dim) + p.eps) : 1.0f;
        const float f_k = p.whole ? 1.0f / sqrtf(((s_r[1] + s_r[3]) + (s_r[5] + s_r[7])) / (float)(p.G * p.dim) + p.eps) : 1.0f;
        for (int i = tid; i < nh * p.dimp; i += 256) s_q[i] = (float)(T)(s_q[i] * f_q);
        if (has_new)
            for (int i = tid; i < p.dimp + p.vdimp; i += 256) {
                const bool is_v = i >= p.dimp;
                const int d = is_v ? i - p.dimp : i;
                const T c = (T)(is_v ? s_v[d] : s_k[d] * f_k);
                (is_v ? s_v : s_k)[d] = (float)c;
                if (hb == 0) (is_v ? cv + size_t(pos % p.cap) * p.vdimp : ck + size_t(pos % p.cap) * p.dimp)[d] = c;
            }
    } else
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
    if (WHOLE && p.pool && has_new && hb == 0 && (pos + 1) % p.pool == 0) { // the token completes a block (no window reaches past it yet)
        const int b = pos / p.pool;
        for (int i = tid; i < p.dimp + p.vdimp; i += 256) {
            const bool is_v = i >= p.dimp;
            const int d = is_v ? i - p.dimp : i, size = is_v ? p.vdimp : p.dimp;
            const T *rows = is_v ? cv : ck;
            float sum = 0.0f;
#pragma unroll 4
            for (int j = b * p.pool; j < pos; j++) sum += (float)rows[size_t(j % p.cap) * size + d];
            sum += is_v ? s_v[d] : s_k[d];
            reinterpret_cast<T *>(is_v ? p.pv : p.pk)[(size_t(g) * p.blocks + b) * size + d] = (T)(sum / (float)p.pool);
        }
    }
    float scale[NH];
#pragma unroll
    for (int h = 0; h < NH; h++) scale[h] = WHOLE && p.temp && h < nh ? p.scale * p.temp[h0 + h] : p.scale;
    auto score_step = [&](int key, const lm_u32x4 &first) {
        float acc[NH];
#pragma unroll
        for (int h = 0; h < NH; h++) acc[h] = 0.0f;
        if (key < j1)
            for (int c = c0; c < kp; c += lpk) {
                float kf[PE];
                if (key == newest) {
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
            if (key < j1 && c0 == 0 && h < nh) s_s[h * keys_max + key - j0] = acc[h] * scale[h];
        }
    };
#pragma unroll
    for (int i = 0; i < PF; i++)
        if (j0 + (i * 4 + wave) * kpw < j1) score_step(j0 + (i * 4 + wave) * kpw + sub, pk[i]);
    for (int j = j0 + (PF * 4 + wave) * kpw; j < j1; j += 4 * kpw) {
        const int key = j + sub;
        lm_u32x4 first = {0, 0, 0, 0};
        if (key < j1 && key != newest && c0 < kp) first = k_piece(key, c0);
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
            if (key == newest) {
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
                if (key < j1) value_step(key, c == vc0 || key == newest ? pv[i] : v_piece(key, c));
            }
            for (int key = j0 + (PF * 4 + wave) * vpw + vsub; key < j1; key += 4 * vpw) value_step(key, key == newest ? pv[0] : v_piece(key, c));
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
    float *s_o = s_r; // (free again)
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
        if (WHOLE && p.rotv) {
            s_o[i] = o;
            continue;
        }
        if (p.gate) o *= lm_sigmoid(p.proj[p.og + (h0 + h) * p.vdimp + d]);
        reinterpret_cast<T *>(p.out)[(h0 + h) * p.vdimp + d] = (T)o;
    }
    if (!(WHOLE && p.rotv)) return;
    lds_barrier();
    for (int i = tid; i < nh * p.vdimp; i += 256) { // the outputs turn back
        const int h = i / p.vdimp, d = i % p.vdimp;
        float o = s_o[i];
        if (d < 2 * back) {
            const float2 cs = i == tid ? back_cs : p.rotv[size_t(pos) * back + d % back];
            o = d < back ? o * cs.x + s_o[i + back] * cs.y : o * cs.x - s_o[i - back] * cs.y;
        }
        if (p.gate) o *= lm_sigmoid(p.proj[p.og + (h0 + h) * p.vdimp + d]);
        reinterpret_cast<T *>(p.out)[(h0 + h) * p.vdimp + d] = (T)o;
    }
}

// One token of the gated delta rule (delta_rows.hip has the equations): head h, whole.  A thread holds four columns of every rp-th row of
// the state, up to DELTA_ROWS of them in registers (REG); larger states are read again for the update.
constexpr int DELTA_ROWS = 16;
// LDS in floats: q, k, decay [ddimp], v, gate, u [dvdimp], sums [1024], 8 more, then the two-step projections' inner vectors
__host__ __device__ __forceinline__ size_t delta_lds_floats(int dimp, int vdimp, int kd) { return size_t(3) * dimp + 3 * vdimp + 1024 + 8 + kd; }
template <class T, bool REG>
__device__ __forceinline__ void mix_delta(const DecodeMix &p, int h, float *lds) {
    constexpr int PE = Piece<T>::N;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, dimp = p.ddimp, vdimp = p.dvdimp;
    const int pos = p.pos_dev ? (int)p.pos_dev[0] : (int)p.pos, per = p.dH / p.dG, c = h / per;
    // Behind the end of a generation (the loop's state says so) launches may still come: they must leave the recurrence as it is.
    const bool keep = !(p.pos_dev && p.pos_dev[3]);
    const int vq = vdimp / 4, rp = 256 / vq, col = tid % vq, r0 = tid / vq;
    const bool on = tid < rp * vq;
    float *s_q = lds, *s_k = s_q + dimp, *s_g = s_k + dimp, *s_v = s_g + dimp, *s_gate = s_v + vdimp, *s_u = s_gate + vdimp, *s_sum = s_u + vdimp, *s_misc = s_sum + 1024;
    T *s_in = reinterpret_cast<T *>(s_misc + 8);
    float4_t *state = reinterpret_cast<float4_t *>(p.state + size_t(h) * dimp * vdimp) + col;
    float4_t S[REG ? DELTA_ROWS : 1];
    auto load = [&](int row) { return pos && on && row < dimp ? state[size_t(row) * vq] : float4_t{0, 0, 0, 0}; };
    if (REG)
#pragma unroll
        for (int i = 0; i < DELTA_ROWS; i++) S[i] = load(r0 + i * rp);
    // convolutions
    const T *ring = reinterpret_cast<const T *>(p.ring);
    for (int i = tid; i < 2 * dimp + vdimp; i += 256) {
        const int ch = i < dimp ? c * dimp + i : i < 2 * dimp ? (p.dG + c) * dimp + i - dimp : 2 * p.dG * dimp + h * vdimp + i - 2 * dimp;
        const T now = (T)p.proj[p.oc + ch];
        float acc = 0.0f;
        for (int tap = 0; tap + 1 < p.taps; tap++) {
            const int at = pos - (p.taps - 1) + tap;
            if (at >= 0) acc = fmaf(p.conv[size_t(tap) * p.channels + ch], (float)ring[size_t(at % p.taps) * p.channels + ch], acc);
        }
        acc = delta_silu(fmaf(p.conv[size_t(p.taps - 1) * p.channels + ch], (float)now, acc));
        (i < dimp ? s_q + i : i < 2 * dimp ? s_k + i - dimp : s_v + i - 2 * dimp)[0] = acc;
        if (keep && (i >= 2 * dimp || h % per == 0)) reinterpret_cast<T *>(p.ring)[size_t(pos % p.taps) * p.channels + ch] = now; // (no tap reads this row)
    }
    for (int i = tid; i < p.kd; i += 256) s_in[i] = i < p.rank_a + p.rank_g ? (T)p.proj[p.od + i] : (T)0.0f;
    const float beta = lm_sigmoid(p.beta[h]), rate = expf(p.a_log[h]);
    lds_barrier();
    if (wave < 2) { // unit vectors
        float *x = wave ? s_k : s_q, ss = 0.0f;
        for (int d = lane; d < dimp; d += 64) ss = fmaf(x[d], x[d], ss);
        float f = 1.0f / sqrtf(wave_sum(ss) + DELTA_UNIT_EPS);
        if (!wave) f *= 1.0f / sqrtf((float)p.ddim);
        for (int d = lane; d < dimp; d += 64) x[d] *= f;
    }
    { // second steps of the decay's and the gate's projections, 8 lanes a row
        const int a_end = (p.rank_a + PE - 1) / PE, g_begin = p.rank_a / PE, g_end = (p.rank_a + p.rank_g + PE - 1) / PE, rows = dimp + vdimp;
        constexpr int RU = 4; // rows a lane works on at a time
        for (int base = tid >> 3; base < (rows + 31) / 32 * 32; base += 32 * RU) {
            float acc[RU];
#pragma unroll
            for (int u = 0; u < RU; u++) {
                const int i = base + 32 * u;
                const bool is_a = i < dimp;
                acc[u] = 0.0f;
                if (i >= rows) continue;
                const T *w = reinterpret_cast<const T *>(p.wlr) + size_t(is_a ? p.lr16 + h * dimp + i : h * vdimp + i - dimp) * p.kd;
                const int end = is_a ? a_end : g_end, first = (is_a ? 0 : g_begin) + (tid & 7); // (the other step's columns are zero)
                for (int q = first; q < end; q += 8)
                    acc[u] = dot_piece<T>(reinterpret_cast<const lm_u32x4 *>(w)[q], *reinterpret_cast<const lm_u32x4 *>(s_in + q * PE), acc[u]);
            }
#pragma unroll
            for (int off = 4; off >= 1; off >>= 1)
#pragma unroll
                for (int u = 0; u < RU; u++) acc[u] += __shfl_xor(acc[u], off);
#pragma unroll
            for (int u = 0; u < RU; u++) {
                const int i = base + 32 * u;
                if ((tid & 7) || i >= rows) continue;
                if (i < dimp) s_g[i] = delta_decay(rate, acc[u] + p.dt_bias[h * dimp + i]);
                else s_gate[i - dimp] = lm_sigmoid(acc[u]);
            }
        }
    }
    lds_barrier();
    auto sum_rows = [&](const float4_t &mine, auto done) { // four columns per thread, summed over the row groups
        if (on) *reinterpret_cast<float4_t *>(s_sum + r0 * vdimp + col * 4) = mine;
        lds_barrier();
        for (int d = tid; d < vdimp; d += 256) {
            float t = 0.0f;
            for (int r = 0; r < rp; r++) t += s_sum[r * vdimp + d];
            done(d, t);
        }
        lds_barrier();
    };
    float4_t w = {0, 0, 0, 0}, o = {0, 0, 0, 0};
    if (REG) {
#pragma unroll
        for (int i = 0; i < DELTA_ROWS; i++) {
            const int row = r0 + i * rp;
            if (row >= dimp) continue;
            S[i] *= s_g[row];
            w += S[i] * s_k[row];
        }
    } else
        for (int row = r0; row < dimp; row += rp) w += load(row) * (s_g[row] * s_k[row]);
    sum_rows(w, [&](int d, float t) { s_u[d] = beta * (s_v[d] - t); });
    if (on) {
        const float4_t u = *reinterpret_cast<const float4_t *>(s_u + col * 4);
        auto update = [&](int row, float4_t s) {
            s += u * s_k[row];
            o += s * s_q[row];
            if (keep) state[size_t(row) * vq] = s;
        };
        if (REG) {
#pragma unroll
            for (int i = 0; i < DELTA_ROWS; i++)
                if (r0 + i * rp < dimp) update(r0 + i * rp, S[i]);
        } else
            for (int row = r0; row < dimp; row += rp) update(row, load(row) * s_g[row]);
    }
    sum_rows(o, [&](int d, float t) { s_u[d] = t; });
    float ss = 0.0f;
    for (int d = lane; d < vdimp; d += 64) ss = fmaf(s_u[d], s_u[d], ss); // (every wavefront by itself)
    const float f = 1.0f / sqrtf(wave_sum(ss) / (float)p.dvdim + p.eps);
    for (int d = tid; d < vdimp; d += 256) reinterpret_cast<T *>(p.dout)[h * vdimp + d] = (T)(s_u[d] * f * p.dnorm[d] * s_gate[d]);
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

template <class T, int NH, int U, bool WHOLE>
__global__ __launch_bounds__(256) void decode_mix_kernel(DecodeMix p, int S, int keys_max, int n_attn, int n_expert) {
    extern __shared__ __attribute__((aligned(16))) char s_mix[];
    // attention first: it is a chain of dependent steps, the experts' part is one long stream
    const int i = blockIdx.x, n_hb = mix_head_blocks(p.H / p.G);
    if (WHOLE && i >= n_attn + n_expert) {
        const int h = i - n_attn - n_expert;
        if (p.ddimp <= DELTA_ROWS * (256 / (p.dvdimp / 4))) mix_delta<T, true>(p, h, reinterpret_cast<float *>(s_mix));
        else mix_delta<T, false>(p, h, reinterpret_cast<float *>(s_mix));
    } else if (i < n_attn) mix_attention<T, NH, WHOLE>(p, i / S / n_hb, i / S % n_hb, i % S, S, keys_max, reinterpret_cast<float *>(s_mix));
    else mix_experts<T, U>(p, i - n_attn, n_expert, s_mix);
}

// x[n] += sum over the pieces of row n of W2 against a, and of the chosen experts' rows against their activations.  A workgroup
// owns RW rows; its four wavefronts share each row's pieces, so a lane reads its part of the vectors once for all rows.
// PARTS = 3: the sums over three stretches of the columns are kept apart.
template <class T, int RW, int U, int PARTS>
__global__ __launch_bounds__(256) void decode_out_kernel(DecodeOut p) {
    __shared__ float s_part[4][PARTS][RW];
    constexpr int PE = Piece<T>::N;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, row0 = blockIdx.x * RW;
    const int pa = p.k0 / PE, pf = p.top ? p.ffp / PE : 1, total = pa + p.top * pf;
    int begin, end;
    share(total, 4, wave, begin, end);
    float acc[PARTS][RW];
#pragma unroll
    for (int k = 0; k < PARTS; k++)
#pragma unroll
        for (int r = 0; r < RW; r++) acc[k][r] = 0.0f;
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
            for (int r = 0; r < RW; r++) {
                const float d = dot_piece<T>(w[u][r], x[u], 0.0f);
                const int i = base + u * 64 + lane;
                if (PARTS == 1) acc[0][r] = fmaf(d, scale[u], acc[0][r]);
                else
#pragma unroll
                    for (int k = 0; k < PARTS; k++) acc[k][r] += (i >= p.k1 / PE) + (i >= p.k2 / PE) == k ? d : 0.0f;
            }
    }
#pragma unroll
    for (int k = 0; k < PARTS; k++)
#pragma unroll
        for (int r = 0; r < RW; r++) {
            const float s = wave_sum(acc[k][r]);
            if (lane == 0) s_part[wave][k][r] = s;
        }
    lds_barrier();
    const int k = tid / RW, r = tid % RW;
    if (k >= PARTS || row0 + r >= p.width) return;
    const float s = (s_part[0][k][r] + s_part[1][k][r]) + (s_part[2][k][r] + s_part[3][k][r]);
    if (PARTS == 1) p.x[row0 + r] += s;
    else p.y[k * p.dp + row0 + r] = s;
}

template <class T, int NH, bool WHOLE> int mix_launch_as(moon_ctx *ctx, const DecodeMix &p, int S, int keys_max, int n_attn, int n_expert, size_t lds) {
    auto kern = p.dp / Piece<T>::N > 64 ? decode_mix_kernel<T, NH, 4, WHOLE> : decode_mix_kernel<T, NH, 1, WHOLE>;
    if (lds > 64 * 1024) MOON_HIP(ctx, hipFuncSetAttribute(reinterpret_cast<const void *>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(kern, dim3(n_attn + n_expert + (WHOLE ? p.dH : 0)), dim3(256), lds, ctx->stream, p, S, keys_max, n_attn, n_expert);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}
bool mix_whole(const DecodeMix &p) { return p.whole || p.rot || p.rotv || p.pool || p.temp || p.borrowed || p.dH; }
template <class T, int NH> int mix_launch(moon_ctx *ctx, const DecodeMix &p, int S, int keys_max, int n_attn, int n_expert, size_t lds) {
    return mix_whole(p) ? mix_launch_as<T, NH, true>(ctx, p, S, keys_max, n_attn, n_expert, lds) : mix_launch_as<T, NH, false>(ctx, p, S, keys_max, n_attn, n_expert, lds);
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
        if (p.y) return nv == 0 ? decode_proj_kernel<T, U, 0, true> : nv == 1 ? decode_proj_kernel<T, U, 1, true> : nv == 2 ? decode_proj_kernel<T, U, 2, true> : decode_proj_kernel<T, U, 4, true>;
        return nv == 0 ? decode_proj_kernel<T, U, 0, false> : nv == 1 ? decode_proj_kernel<T, U, 1, false> : nv == 2 ? decode_proj_kernel<T, U, 2, false> : decode_proj_kernel<T, U, 4, false>;
    };
    auto kern = ch == 1 ? pick(std::integral_constant<int, 1>{}) : ch == 2 ? pick(std::integral_constant<int, 2>{}) : ch == 3 ? pick(std::integral_constant<int, 3>{})
                                                                                                                          : pick(std::integral_constant<int, 4>{});
    hipLaunchKernelGGL(kern, grid, dim3(256), lds, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

template <class T> int out_launch(moon_ctx *ctx, const DecodeOut &p) {
    const int cus = ctx->cu_count > 0 ? ctx->cu_count : 256;
    auto go = [&](auto parts) {
        constexpr int N = decltype(parts)::value;
        if (p.width >= 4 * 2 * cus) hipLaunchKernelGGL((decode_out_kernel<T, 4, 4, N>), dim3((p.width + 3) / 4), dim3(256), 0, ctx->stream, p);
        else if (p.width >= 2 * 2 * cus) hipLaunchKernelGGL((decode_out_kernel<T, 2, 6, N>), dim3((p.width + 1) / 2), dim3(256), 0, ctx->stream, p);
        else hipLaunchKernelGGL((decode_out_kernel<T, 1, 8, N>), dim3(p.width), dim3(256), 0, ctx->stream, p);
    };
    if (p.y && (p.top || p.k1 % 64 || p.k2 % 64 || p.k1 > p.k2 || p.k2 > p.k0)) return moon_fail(ctx, MOON_EINVAL, "decode: columns in parts %d %d %d", p.k1, p.k2, p.k0);
    if (p.y) go(std::integral_constant<int, 3>{});
    else go(std::integral_constant<int, 1>{});
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
    const int n_win = (int)(p.window ? std::min(p.pos + 1, (size_t)p.window) : p.pos + 1), n_keys = n_win + (p.pool ? (int)(p.pos + 1 - n_win) / p.pool : 0);
    if (p.pool && ((p.pos + 1) / p.pool > (size_t)p.blocks || (p.pos + 1 >= (size_t)p.pool && p.pool > p.cap))) return moon_fail(ctx, MOON_EINVAL_DIM, "decode attention: %d pooled blocks kept", p.blocks);
    if (mix_whole(p) && (p.qk_rms || p.mixes)) return moon_fail(ctx, MOON_EINVAL, "decode attention: norms per head or mixed values beside rotation, blocks or a norm of all of q");
    if (p.dH && (p.dH % p.dG || p.ddimp % 16 || p.dvdimp % 16 || p.ddimp > (int)DELTA_MAX_DIM || p.dvdimp > (int)DELTA_MAX_DIM || p.oc % 8 || p.kd % 64))
        return moon_fail(ctx, MOON_EINVAL_DIM, "decode: delta rule with head sizes %d and %d", p.ddimp, p.dvdimp);
    int S = std::min(std::min((n_keys + MIX_TARGET - 1) / MIX_TARGET, MIX_SPLITS), std::max(1, cus / wgs));
    S = std::max(S, (n_keys + MIX_KEYS - 1) / MIX_KEYS);
    if (size_t(wgs) * S * MIX_HEADS * (p.vdimp + 2) > p.partial_floats) return moon_fail(ctx, MOON_ESEQ_TOO_LONG, "decode attention: %d keys", n_keys);
    const int keys_max = (n_keys + S - 1) / S;
    if (p.E && (p.top < 1 || p.top > p.E || p.E > ROUTER_MAX_EXPERTS)) return moon_fail(ctx, MOON_EINVAL_DIM, "router: %d of %d experts", p.top, p.E);
    const int groups = p.E ? p.top * ((p.ff + 1) / 2) : 0;
    const int n_expert = std::min((groups + 3) / 4, std::max(cus, 2 * cus - wgs * S)); // (together two workgroups per CU: more measured slower)
    const int nh = std::min(per, MIX_HEADS), NH = nh <= 1 ? 1 : nh <= 2 ? 2 : nh <= 4 ? 4 : 8;
    const size_t el = dtype == MOON_DTYPE_BF16 ? sizeof(bf16_t) : sizeof(float);
    const size_t lds = std::max(std::max(mix_lds_floats(NH, p.dimp, p.vdimp, keys_max) * sizeof(float),
                                         p.E ? size_t(p.dp) * el + (size_t(2) * p.E + 2 * p.top) * sizeof(float) : 0),
                                p.dH ? delta_lds_floats(p.ddimp, p.dvdimp, p.kd) * sizeof(float) : 0);
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
