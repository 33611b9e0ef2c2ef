// Causal attention of several query rows over a KV cache, with a sliding window, grouped key/value heads, a sink in the
// softmax denominator and an output gate; each of them is an argument.  The cache of a layer is [G][cap][head size]; the keys of
// position p lie in row p % cap, so a windowed layer needs no more rows than its window and one call's rows together.
//
// bf16 runs on the matrix cores.  A 256-thread workgroup is four wavefronts of 32 query rows each: HB heads of one key/value
// group times 4 / HB row blocks, HB the largest power of two up to 4 that divides the group.  All four walk the same tiles of 64
// keys, staged in LDS once for the workgroup (the next tile is requested while one is used); a wavefront skips the tiles that
// none of its rows can see.  Per tile, with v_mfma_f32_32x32x16_bf16 and f32 accumulation,
//     S^T[key][q] = K . Q^T     (a lane holds 32 scores of ONE query)
//     O^T[d][q]  += V^T . P^T   (V row-major in LDS, transposed by the LDS load)
// Scores and weights are f32.  A weight enters the second product as two bf16 terms, its rounding and the remainder, so the
// product sees 16 bits of it.
// f32, and head sizes above 256, take one wavefront per (row, head) with plain multiply-adds.
#include "layer_list.hpp"
#include "lm_types.hpp"

#include <algorithm>
#include <atomic>

namespace {

constexpr int WA_KT = 64; // keys per tile
typedef short wa_short4_t __attribute__((ext_vector_type(4)));

template <int P> struct WaCfg { // P: head sizes up to P (a multiple of 32), rows zero padded to it
    static constexpr int KSTEPS = P / 16, DT = P / 32, G = P / 8;
    static constexpr int KS = P + 8; // row strides in elements: 128-bit reads of consecutive K rows and the transposing reads of
    static constexpr int VS = P == 32 ? 32 : P == 64 ? 96 : P + 32 - (P == 96 ? 32 : 0); // 4 consecutive V rows (16 dwords apart mod 64) are conflict free
    static constexpr int LOADS = WA_KT * G / 256; // 16-byte pieces per thread and operand tile
    static constexpr size_t LDS_BYTES = size_t(WA_KT) * (KS + VS) * 2;
    static_assert(WA_KT * G % 256 == 0, "whole pieces");
};

__device__ __forceinline__ wa_short4_t wa_read_tr(const bf16_t *p) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) wa_short4_t *)(p));
}

template <int P>
__global__ __launch_bounds__(256) void window_attn_kernel(WindowAttn p, int HB) {
    using C = WaCfg<P>;
    __shared__ __attribute__((aligned(16))) bf16_t lds[C::LDS_BYTES / 2];
    bf16_t *Ks = lds, *Vs = lds + WA_KT * C::KS;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 31, hf = lane >> 5;
    const int RB = 4 / HB, rows_wg = 32 * RB, n_rb = (p.n + rows_wg - 1) / rows_wg, n_hg = p.H / HB;
    // a key/value group's row blocks stay on one die where the counts divide; late rows see the most keys: they start first
    int item = blockIdx.x;
    const int n_items = n_rb * n_hg;
    if (n_items % 8 == 0) item = (item % 8) * (n_items / 8) + item / 8;
    const int hg = item / n_rb, rb = n_rb - 1 - item % n_rb;
    const int h = hg * HB + wave % HB, g = h / (p.H / p.G);
    const int wg_row0 = rb * rows_wg, row0 = wg_row0 + 32 * (wave / HB);
    const int first_pos = p.pos0 + wg_row0, last_pos = p.pos0 + min(wg_row0 + rows_wg, p.n) - 1;
    const int lo_key = p.window ? max(0, first_pos - p.window + 1) : 0;
    const int t_begin = lo_key / WA_KT, t_end = last_pos / WA_KT + 1; // tiles start at multiples of 64 positions
    const int my_first = p.pos0 + row0, my_last = p.pos0 + min(row0 + 32, p.n) - 1; // (my_last < my_first: no rows)
    const int my_lo = p.window ? max(0, my_first - p.window + 1) : 0;
    const int pos = my_first + col; // this lane's query
    const bf16_t *ck = reinterpret_cast<const bf16_t *>(p.ck) + size_t(g) * p.cap * p.dimp;
    const bf16_t *cv = reinterpret_cast<const bf16_t *>(p.cv) + size_t(g) * p.cap * p.vdimp;
    const int kg = p.dimp / 8, vg = p.vdimp / 8;

    lm_u32x4 rk[C::LOADS], rv[C::LOADS];
    auto load_tile = [&](int t) {
        const int key0 = t * WA_KT, slot0 = key0 % p.cap;
#pragma unroll
        for (int i = 0; i < C::LOADS; i++) {
            const int x = i * 256 + tid, r = x / C::G, c = x % C::G, key = key0 + r;
            int slot = slot0 + r;
            if (slot >= p.cap) slot %= p.cap;
            const bool ok = key >= lo_key && key <= last_pos; // everything else is masked, and may not be there
            rk[i] = rv[i] = lm_u32x4{0, 0, 0, 0};
            if (ok && c < kg) rk[i] = *reinterpret_cast<const lm_u32x4 *>(ck + size_t(slot) * p.dimp + c * 8);
            if (ok && c < vg) rv[i] = *reinterpret_cast<const lm_u32x4 *>(cv + size_t(slot) * p.vdimp + c * 8);
        }
    };
    load_tile(t_begin);

    bf16x8_t qf[C::KSTEPS]; // the MFMA "B" operand: Q[row0 + col][16 s + 8 hf .. + 7]
    {
        const bf16_t *q = reinterpret_cast<const bf16_t *>(p.q) + size_t(min(row0 + col, p.n - 1)) * p.ldq + h * p.dimp;
#pragma unroll
        for (int s = 0; s < C::KSTEPS; s++) {
            lm_u32x4 v = {0, 0, 0, 0};
            if (16 * s + 8 * hf < p.dimp) v = *reinterpret_cast<const lm_u32x4 *>(q + 16 * s + 8 * hf);
            qf[s] = __builtin_bit_cast(bf16x8_t, v);
        }
    }
    int voff[C::DT]; // where this lane points the transposing loads: key 4 hf + (lane % 16) / 4, columns 32 dt + 16 ((lane / 16) % 2) + 4 (lane % 4)
#pragma unroll
    for (int dt = 0; dt < C::DT; dt++) voff[dt] = (4 * hf + ((lane & 15) >> 2)) * C::VS + 32 * dt + 16 * ((lane >> 4) & 1) + 4 * (lane & 3);

    float16_t o[C::DT];
#pragma unroll
    for (int dt = 0; dt < C::DT; dt++)
#pragma unroll
        for (int v = 0; v < 16; v++) o[dt][v] = 0.0f;
    // the sink is one more score that the denominator has seen before the first key (counted once: in the lower half's sum)
    constexpr float LOG2E = 1.4426950408889634f;
    float m_run = p.sink ? p.sink[h] * LOG2E : -INFINITY, l_run = p.sink && hf == 0 ? 1.0f : 0.0f;
    const float c2 = p.scale * LOG2E;

    for (int t = t_begin; t < t_end; t++) {
        const int key0 = t * WA_KT;
        __syncthreads(); // the previous tile has been read
#pragma unroll
        for (int i = 0; i < C::LOADS; i++) {
            const int x = i * 256 + tid, r = x / C::G, c = x % C::G;
            *reinterpret_cast<lm_u32x4 *>(Ks + r * C::KS + c * 8) = rk[i];
            *reinterpret_cast<lm_u32x4 *>(Vs + r * C::VS + c * 8) = rv[i];
        }
        __syncthreads();
        if (t + 1 < t_end) load_tile(t + 1);
        if (key0 > my_last || key0 + WA_KT <= my_lo || my_last < my_first) continue; // (the same for the whole wavefront)

        float16_t s[2];
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int kt = 0; kt < 2; kt++) {
#pragma unroll
            for (int v = 0; v < 16; v++) s[kt][v] = 0.0f;
#pragma unroll
            for (int st = 0; st < C::KSTEPS; st++)
                s[kt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8_t *>(Ks + (32 * kt + col) * C::KS + 16 * st + 8 * hf), qf[st],
                                                                s[kt], 0, 0, 0);
        }
        __builtin_amdgcn_s_setprio(0);
        // s[kt][v]: key key0 + 32 kt + 8 (v / 4) + 4 hf + v % 4 against this lane's query
        const bool edge = key0 + WA_KT - 1 > my_first || (p.window && key0 < my_last - p.window + 1);
        float mx = -INFINITY;
#pragma unroll
        for (int kt = 0; kt < 2; kt++)
#pragma unroll
            for (int v = 0; v < 16; v++) {
                float x = s[kt][v] * c2;
                if (edge) {
                    const int key = key0 + 32 * kt + 8 * (v >> 2) + 4 * hf + (v & 3);
                    if (key > pos || (p.window && pos - key >= p.window)) x = -INFINITY;
                }
                s[kt][v] = x;
                mx = fmaxf(mx, x);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float m_new = fmaxf(m_run, mx), m_use = m_new == -INFINITY ? 0.0f : m_new;
        const float alpha = __builtin_amdgcn_exp2f(m_run - m_use);
        m_run = m_new;
        float psum = 0.0f;
#pragma unroll
        for (int kt = 0; kt < 2; kt++)
#pragma unroll
            for (int v = 0; v < 16; v++) {
                const float e = __builtin_amdgcn_exp2f(s[kt][v] - m_use);
                s[kt][v] = e;
                psum += e;
            }
        l_run = l_run * alpha + psum;
#pragma unroll
        for (int dt = 0; dt < C::DT; dt++)
#pragma unroll
            for (int v = 0; v < 16; v++) o[dt][v] *= alpha;
        // contraction step (kt, sp) uses the keys a lane holds in s[kt][8 sp .. 8 sp + 7]: key0 + 32 kt + 16 sp + {4 hf + 0..3, 8 + 4 hf + 0..3}
#pragma unroll
        for (int kt = 0; kt < 2; kt++)
#pragma unroll
            for (int sp = 0; sp < 2; sp++) {
                bf16x8_t hi, lo;
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const float w = s[kt][8 * sp + e];
                    hi[e] = (bf16_t)w;
                    lo[e] = (bf16_t)(w - (float)hi[e]);
                }
#pragma unroll
                for (int dt = 0; dt < C::DT; dt++) {
                    const bf16_t *vp = Vs + voff[dt] + (32 * kt + 16 * sp) * C::VS;
                    const wa_short4_t a0 = wa_read_tr(vp), a1 = wa_read_tr(vp + 8 * C::VS);
                    const bf16x8_t a = __builtin_bit_cast(bf16x8_t, __builtin_shufflevector(a0, a1, 0, 1, 2, 3, 4, 5, 6, 7));
                    o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, lo, o[dt], 0, 0, 0);
                    o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, hi, o[dt], 0, 0, 0);
                }
            }
    }
    const int row = row0 + col;
    const float inv = 1.0f / (l_run + __shfl_xor(l_run, 32));
    if (row >= p.n) return;
    const bf16_t *gate = p.gate ? reinterpret_cast<const bf16_t *>(p.gate) + size_t(row) * p.ldq + h * p.vdimp : nullptr;
    bf16_t *out = reinterpret_cast<bf16_t *>(p.out) + size_t(row) * p.ldo + h * p.vdimp;
    typedef bf16_t bf16x4_t __attribute__((ext_vector_type(4)));
#pragma unroll
    for (int dt = 0; dt < C::DT; dt++)
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int d = 32 * dt + 8 * j + 4 * hf; // o[dt][4 j .. 4 j + 3] are elements d .. d + 3
            if (d >= p.vdimp) continue;
            bf16x4_t r;
            if (gate) {
                const bf16x4_t gz = *reinterpret_cast<const bf16x4_t *>(gate + d);
#pragma unroll
                for (int e = 0; e < 4; e++) r[e] = (bf16_t)(o[dt][4 * j + e] * inv * lm_sigmoid((float)gz[e]));
            } else
#pragma unroll
                for (int e = 0; e < 4; e++) r[e] = (bf16_t)(o[dt][4 * j + e] * inv);
            *reinterpret_cast<bf16x4_t *>(out + d) = r;
        }
}

// One wavefront per (row, head): 64 keys at a time, one per lane for the scores, one element per lane for the values.
constexpr int ROW_MAX_D = 1024; // elements of a head the values' accumulators cover
template <class T>
__global__ __launch_bounds__(256) void window_attn_rows_kernel(WindowAttn p) {
    __shared__ float s_q[4][ROW_MAX_D], s_w[4][64];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, task = blockIdx.x * 4 + wave;
    if (task >= p.n * p.H) return; // (wavefronts share nothing)
    const int row = task / p.H, h = task % p.H, g = h / (p.H / p.G), pos = p.pos0 + row, lo = p.window ? max(0, pos - p.window + 1) : 0;
    const T *q = reinterpret_cast<const T *>(p.q) + size_t(row) * p.ldq + h * p.dimp;
    const T *ck = reinterpret_cast<const T *>(p.ck) + size_t(g) * p.cap * p.dimp, *cv = reinterpret_cast<const T *>(p.cv) + size_t(g) * p.cap * p.vdimp;
    for (int d = lane; d < p.dimp; d += 64) s_q[wave][d] = (float)q[d];
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    float m = p.sink ? p.sink[h] : -INFINITY, l = p.sink ? 1.0f : 0.0f;
    float o[ROW_MAX_D / 64];
#pragma unroll
    for (int i = 0; i < ROW_MAX_D / 64; i++) o[i] = 0.0f;
    for (int k0 = lo; k0 <= pos; k0 += 64) {
        const int key = k0 + lane, n_keys = min(64, pos - k0 + 1);
        float s = -INFINITY;
        if (key <= pos) {
            const T *kr = ck + size_t(key % p.cap) * p.dimp;
            s = 0.0f;
            for (int d = 0; d < p.dimp; d++) s = fmaf(s_q[wave][d], (float)kr[d], s);
            s *= p.scale;
        }
        const float m_new = fmaxf(m, wave_max(s)), alpha = expf(m - m_new), w = key <= pos ? expf(s - m_new) : 0.0f;
        l = l * alpha + wave_sum(w);
        m = m_new;
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        s_w[wave][lane] = w;
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
        for (int i = 0; i < ROW_MAX_D / 64; i++) {
            const int d = 64 * i + lane;
            if (64 * i >= p.vdimp) continue;
            float acc = o[i] * alpha;
            if (d < p.vdimp)
                for (int j = 0; j < n_keys; j++) acc = fmaf(s_w[wave][j], (float)cv[size_t((k0 + j) % p.cap) * p.vdimp + d], acc);
            o[i] = acc;
        }
    }
#pragma unroll
    for (int i = 0; i < ROW_MAX_D / 64; i++) {
        const int d = 64 * i + lane;
        if (d >= p.vdimp) continue;
        float r = o[i] / l;
        if (p.gate) r *= lm_sigmoid((float)reinterpret_cast<const T *>(p.gate)[size_t(row) * p.ldq + h * p.vdimp + d]);
        reinterpret_cast<T *>(p.out)[size_t(row) * p.ldo + h * p.vdimp + d] = (T)r;
    }
}

template <int P> int launch_mfma(moon_ctx *ctx, const WindowAttn &p) {
    const int per = p.H / p.G, HB = per % 4 == 0 ? 4 : per % 2 == 0 ? 2 : 1, rows_wg = 32 * (4 / HB);
    hipLaunchKernelGGL(window_attn_kernel<P>, dim3((unsigned)((p.n + rows_wg - 1) / rows_wg * (p.H / HB))), dim3(256), 0, ctx->stream, p, HB);
    MOON_HIP(ctx, hipGetLastError());
    MOON_NOTE_KERNEL(ctx, "window_attn_kernel<%d>", P);
    return MOON_OK;
}

} // namespace

int launch_window_attention(moon_ctx *ctx, int dtype, const WindowAttn &p) {
    if (p.n <= 0) return MOON_OK;
    if (p.H % p.G || p.dimp % 8 || p.vdimp % 8 || p.dimp > ROW_MAX_D || p.vdimp > ROW_MAX_D)
        return moon_fail(ctx, MOON_EINVAL_DIM, "window attention: %d heads over %d, head sizes %d and %d", p.H, p.G, p.dimp, p.vdimp);
    if ((p.window ? p.window - 1 + p.n : p.pos0 + p.n) > p.cap && p.pos0 + p.n > p.cap)
        return moon_fail(ctx, MOON_EINVAL_DIM, "window attention: %d rows behind a window of %d do not fit %d cache rows", p.n, p.window, p.cap);
    const int big = std::max(p.dimp, p.vdimp);
    if (dtype == MOON_DTYPE_BF16 && big <= 256) {
        if (big <= 32) return launch_mfma<32>(ctx, p);
        if (big <= 64) return launch_mfma<64>(ctx, p);
        if (big <= 96) return launch_mfma<96>(ctx, p);
        if (big <= 128) return launch_mfma<128>(ctx, p);
        return launch_mfma<256>(ctx, p);
    }
    const dim3 grid((unsigned)((size_t(p.n) * p.H + 3) / 4));
    if (dtype == MOON_DTYPE_BF16) hipLaunchKernelGGL(window_attn_rows_kernel<bf16_t>, grid, dim3(256), 0, ctx->stream, p);
    else hipLaunchKernelGGL(window_attn_rows_kernel<float>, grid, dim3(256), 0, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    MOON_NOTE_KERNEL(ctx, "window_attn_rows_kernel");
    return MOON_OK;
}
