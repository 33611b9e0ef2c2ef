// The gated delta rule over a prompt's rows.  Per head, with a state S [dim][vdim] and a decay g per token and key channel,
//     S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q.
// Tokens are taken in chunks of 16.  With G_t the product of the decays of a chunk's tokens up to t, K_t = k_t G_t, Q_t = q_t G_t and
// R_s = k_s G_15 / G_s, the tokens of a chunk that starts from S0 are
//     (I + A) U = beta (V - K S0),   A[t][s] = beta_t sum_c k_t k_s G_t / G_s  (s < t)
//     O = Q S0 + P U,                P[t][s] = sum_c q_t k_s G_t / G_s          (s <= t)
//     S = G_15 S0 + R^T U
// Three kernels:
//   delta_chunk   one workgroup per chunk and head: convolutions, unit vectors, decays, then A and P, and (I + A)^-1 applied to beta V
//                 and beta K.  Quotients of decays are formed as products of the decays between the tokens, so nothing over- or underflows.
//   delta_scan    one workgroup per head and 16 columns of the state, chunk after chunk: U = V' - K' S0, O, the new S, all with f32
//                 matrix-core products (v_mfma_f32_16x16x4_f32: f32 operands and sums).  Four wavefronts share the key channels; an
//                 accumulator tile is the next product's second operand as it lies in the registers.
//   delta_gate    RMS norm per head, weight, output gate.
#include "delta_math.hpp"
#include "lane_fold.hpp"
#include "layer_list.hpp"

#include <algorithm>
#include <atomic>

namespace {

constexpr int DC = 16;      // tokens of a chunk
constexpr int DC_PITCH = DC + 4;

// One chunk and head in the scratch memory, in floats: K' [16][dimp], Q [16][dimp], R^T [dimp][16], G_15 [dimp], P [16][16], V'^T [vdimp][16]
// (-K' rather than K', so that U is a plain sum)
__host__ __device__ __forceinline__ size_t chunk_floats(int dimp, int vdimp) { return size_t(49) * dimp + 256 + size_t(16) * vdimp; }
__host__ __device__ __forceinline__ size_t chunk_lds_floats(int dimp, int vdimp) {
    return size_t(3) * DC * (dimp + 16) + size_t(DC) * vdimp + 2 * DC * DC_PITCH + DC;
}

// Sixteen threads work on a token (and, for A and P, on a token s) until the columns are distributed.
template <class T>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(6))) void delta_chunk_kernel(DeltaRows p) {
    extern __shared__ __attribute__((aligned(16))) float s_dc[];
    constexpr int PE = Piece<T>::N;
    const int tid = threadIdx.x, lane = tid & 63, tok = tid >> 4, j = tid & 15, chunk = blockIdx.x / p.H, h = blockIdx.x % p.H, c = h / (p.H / p.G);
    const int t0 = chunk * DC, dp = p.dimp + 16; // dp: row pitch
    const bool there = t0 + tok < p.n; // tokens past the end are zero and decay nothing
    float *s_q = s_dc, *s_k = s_q + DC * dp, *s_g = s_k + DC * dp, *s_v = s_g + DC * dp, *s_a = s_v + DC * p.vdimp, *s_p = s_a + DC * DC_PITCH,
          *s_b = s_p + DC * DC_PITCH;
    // the decay's projection is requested before the convolutions' inputs
    const float *dt = p.dt + size_t(t0 + (there ? tok : 0)) * p.lddt + h * p.dimp, *bias = p.dt_bias + h * p.dimp;
    const int d_first = min(j * 4, p.dimp - 4);
    const float4_t dt_first = *reinterpret_cast<const float4_t *>(dt + d_first) + *reinterpret_cast<const float4_t *>(bias + d_first);
    const float rate = expf(p.a_log[h]), b_first = there ? p.beta[size_t(t0 + tok) * p.ldb + h] : 0.0f;
    // convolutions, 16 bytes of channels at a time
    constexpr int TAPS = 4; // inputs requested together
    const int pk = p.dimp / PE, pieces = 2 * pk + p.vdimp / PE;
    const T *rows = reinterpret_cast<const T *>(p.c1) + p.oc, *ring = reinterpret_cast<const T *>(p.ring);
    for (int i = j; i < pieces; i += 16) {
        const int what = (i >= pk) + (i >= 2 * pk), off = (i - what * pk) * PE;
        const int ch = (what == 0 ? c * p.dimp : what == 1 ? (p.G + c) * p.dimp : 2 * p.G * p.dimp + h * p.vdimp) + off;
        float acc[PE];
#pragma unroll
        for (int e = 0; e < PE; e++) acc[e] = 0.0f;
        if (there)
            for (int tap0 = 0; tap0 < p.taps; tap0 += TAPS) {
                lm_u32x4 x[TAPS];
#pragma unroll
                for (int u = 0; u < TAPS; u++) {
                    const int r = t0 + tok - (p.taps - 1) + tap0 + u;
                    x[u] = lm_u32x4{0, 0, 0, 0};
                    if (tap0 + u >= p.taps) continue;
                    if (r >= 0) x[u] = *reinterpret_cast<const lm_u32x4 *>(rows + size_t(r) * p.ld + ch);
                    else if (p.pos0 + r >= 0) x[u] = *reinterpret_cast<const lm_u32x4 *>(ring + size_t((p.pos0 + r) % p.taps) * p.channels + ch);
                }
#pragma unroll
                for (int u = 0; u < TAPS; u++) {
                    if (tap0 + u >= p.taps) continue;
                    float f[PE];
                    Piece<T>::unpack(x[u], f);
                    const float *w = p.conv + size_t(tap0 + u) * p.channels + ch;
#pragma unroll
                    for (int e = 0; e < PE; e++) acc[e] = fmaf(w[e], f[e], acc[e]);
                }
            }
        float *dst = what == 0 ? s_q + tok * dp + off : what == 1 ? s_k + tok * dp + off : s_v + tok * p.vdimp + off;
#pragma unroll
        for (int e = 0; e < PE; e += 4)
            *reinterpret_cast<float4_t *>(dst + e) = float4_t{delta_silu(acc[e]), delta_silu(acc[e + 1]), delta_silu(acc[e + 2]), delta_silu(acc[e + 3])};
    }
    for (int d = j * 4; d < p.dimp; d += 64) {
        const float4_t z = d == j * 4 ? dt_first : *reinterpret_cast<const float4_t *>(dt + d) + *reinterpret_cast<const float4_t *>(bias + d);
        float4_t g = {1.0f, 1.0f, 1.0f, 1.0f};
        if (there)
#pragma unroll
            for (int e = 0; e < 4; e++) g[e] = delta_decay(rate, z[e]);
        *reinterpret_cast<float4_t *>(s_g + tok * dp + d) = g;
    }
    if (j == 0) s_b[tok] = there ? lm_sigmoid(b_first) : 0.0f;
    { // unit vectors (a token's threads are in one wavefront, whose LDS accesses stay in order)
        float *q = s_q + tok * dp, *k = s_k + tok * dp, ss_q = 0.0f, ss_k = 0.0f;
        for (int d = j * 4; d < p.dimp; d += 64) {
            const float4_t a = *reinterpret_cast<const float4_t *>(q + d), b = *reinterpret_cast<const float4_t *>(k + d);
#pragma unroll
            for (int e = 0; e < 4; e++) {
                ss_q = fmaf(a[e], a[e], ss_q);
                ss_k = fmaf(b[e], b[e], ss_k);
            }
        }
#pragma unroll
        for (int off = 8; off >= 1; off >>= 1) {
            ss_q += __shfl_xor(ss_q, off);
            ss_k += __shfl_xor(ss_k, off);
        }
        const float f_q = 1.0f / (sqrtf(ss_q + DELTA_UNIT_EPS) * sqrtf((float)p.dim)), f_k = 1.0f / sqrtf(ss_k + DELTA_UNIT_EPS);
        for (int d = j * 4; d < p.dimp; d += 64) {
            *reinterpret_cast<float4_t *>(q + d) *= f_q;
            *reinterpret_cast<float4_t *>(k + d) *= f_k;
        }
    }
    lds_barrier();
    { // A and P: a thread has token s = tok and four of every 64 channels
        float v[2 * DC];
#pragma unroll
        for (int i = 0; i < 2 * DC; i++) v[i] = 0.0f;
        for (int d = j * 4; d < p.dimp; d += 64) {
            const float4_t ks = *reinterpret_cast<const float4_t *>(s_k + tok * dp + d);
            float4_t w = {0, 0, 0, 0}; // k_s times the decays of the tokens behind s up to t
#pragma unroll
            for (int t = 0; t < DC; t++) {
                const float4_t g = *reinterpret_cast<const float4_t *>(s_g + t * dp + d), k = *reinterpret_cast<const float4_t *>(s_k + t * dp + d),
                               q = *reinterpret_cast<const float4_t *>(s_q + t * dp + d);
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    w[e] = t == tok ? ks[e] : w[e] * g[e];
                    v[t] = fmaf(k[e], w[e], v[t]);
                    v[DC + t] = fmaf(q[e], w[e], v[DC + t]);
                }
            }
        }
        fold_lanes<2 * DC, 8>(v, lane, 1, 0, [&](int i, float x) {
            if (i < DC) s_a[i * DC_PITCH + tok] = i > tok ? s_b[i] * x : 0.0f;
            else s_p[(i - DC) * DC_PITCH + tok] = x;
        });
    }
    lds_barrier();
    float *out = p.scratch + (size_t(h) * ((p.n + DC - 1) / DC) + chunk) * chunk_floats(p.dimp, p.vdimp);
    float *o_k = out, *o_q = o_k + DC * p.dimp, *o_r = o_q + DC * p.dimp, *o_g = o_r + DC * p.dimp, *o_p = o_g + p.dimp, *o_v = o_p + DC * DC;
    for (int i = tid; i < 2 * p.dimp + p.vdimp; i += 256) {
        float x[DC];
        auto store16 = [&](float *dst) {
#pragma unroll
            for (int t = 0; t < DC; t += 4) *reinterpret_cast<float4_t *>(dst + t) = float4_t{x[t], x[t + 1], x[t + 2], x[t + 3]};
        };
        if (i < p.dimp + p.vdimp) { // a column of beta K or beta V, forward substitution
            const bool is_k = i < p.dimp;
            const float *src = is_k ? s_k + i : s_v + i - p.dimp, *g = s_g + i;
            const int pitch = is_k ? dp : p.vdimp;
            float all = 1.0f;
#pragma unroll
            for (int t = 0; t < DC; t++) {
                if (is_k) all *= g[t * dp];
                float y = s_b[t] * src[t * pitch] * all;
#pragma unroll
                for (int s0 = 0; s0 < t; s0 += 4) {
                    const float4_t a = *reinterpret_cast<const float4_t *>(s_a + t * DC_PITCH + s0);
#pragma unroll
                    for (int s = s0; s < t && s < s0 + 4; s++) y = fmaf(-a[s - s0], x[s], y);
                }
                x[t] = y;
            }
            if (is_k) {
#pragma unroll
                for (int t = 0; t < DC; t++) o_k[size_t(t) * p.dimp + i] = -x[t];
            } else store16(o_v + size_t(i - p.dimp) * DC);
        } else { // Q, R and the whole chunk's decay
            const int d = i - p.dimp - p.vdimp;
            float all = 1.0f, rest = 1.0f;
#pragma unroll
            for (int t = 0; t < DC; t++) {
                all *= s_g[t * dp + d];
                o_q[size_t(t) * p.dimp + d] = s_q[t * dp + d] * all;
            }
#pragma unroll
            for (int t = DC - 1; t >= 0; t--) {
                x[t] = s_k[t * dp + d] * rest;
                rest *= s_g[t * dp + d];
            }
            store16(o_r + size_t(d) * DC);
            o_g[d] = all;
        }
    }
    o_p[tid] = s_p[(tid >> 4) * DC_PITCH + (tid & 15)];
}

// Four wavefronts share the key channels, NT tiles of 16 each; the fifth one finishes the outputs, a chunk behind.  AHEAD: chunks whose
// operands are requested before they are needed.
constexpr int SCAN_THREADS = 320;
template <int NT> struct ScanChunk {
    float4_t k[NT], q[NT], r[NT], g[NT], v;
};
__device__ __forceinline__ float4_t scan_load(const float *base, unsigned bytes) { // (a base the wavefront shares and 32-bit offsets)
    return *reinterpret_cast<const float4_t *>(reinterpret_cast<const char *>(base) + bytes);
}
template <class T, int NT, int AHEAD>
__global__ __launch_bounds__(SCAN_THREADS) __attribute__((amdgpu_waves_per_eu(1, 2))) void delta_scan_kernel(DeltaRows p) {
    __shared__ float4_t s_u[2][4][64], s_o[2][4][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15, quad = lane >> 4;
    const int slices = p.vdimp / 16, tiles = p.dimp / 16, chunks = (p.n + DC - 1) / DC;
    // Workgroups are dealt to the eight dies round robin: a head's columns stay on the die whose L2 has its chunks (delta_chunk's mapping).
    int h = blockIdx.x / slices, v0 = blockIdx.x % slices * 16;
    if (p.H % 8 == 0) {
        h = blockIdx.x / 8 / slices * 8 + blockIdx.x % 8;
        v0 = blockIdx.x / 8 % slices * 16;
    }
    const size_t stride = chunk_floats(p.dimp, p.vdimp);
    const float *src = p.scratch + size_t(h) * chunks * stride;
    if (wave == 4) {
        float4_t P[AHEAD], u_before, p_before;
        const unsigned off_p = (49 * p.dimp + col * DC + 4 * quad) * 4;
        auto request = [&](int a, int chunk) { P[a] = scan_load(src + min(chunk, chunks - 1) * stride, off_p); };
        auto finish = [&](int chunk, int half) { // chunk's parts lie in `half`
            float4_t o = (s_o[half][0][lane] + s_o[half][1][lane]) + (s_o[half][2][lane] + s_o[half][3][lane]);
#pragma unroll
            for (int j = 0; j < 4; j++) o = __builtin_amdgcn_mfma_f32_16x16x4f32(p_before[j], u_before[j], o, 0, 0, 0);
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int row = chunk * DC + 4 * quad + e;
                if (row < p.n) p.o[(size_t(row) * p.H + h) * p.vdimp + v0 + col] = o[e];
            }
        };
#pragma unroll
        for (int a = 0; a < AHEAD; a++) request(a, a);
        auto step = [&](int a, int chunk) {
            const int half = chunk & 1;
            lds_barrier();
            const float4_t u = (s_u[half][0][lane] + s_u[half][1][lane]) + (s_u[half][2][lane] + s_u[half][3][lane]);
            if (chunk) finish(chunk - 1, half);
            u_before = u;
            p_before = P[a];
            request(a, chunk + AHEAD);
        };
        int base = 0;
        for (; base + AHEAD <= chunks; base += AHEAD)
#pragma unroll
            for (int a = 0; a < AHEAD; a++) step(a, base + a);
#pragma unroll
        for (int a = 0; a < AHEAD; a++)
            if (base + a < chunks) step(a, base + a);
        lds_barrier();
        finish(chunks - 1, chunks & 1);
        return;
    }
    float *state = p.state + size_t(h) * p.dimp * p.vdimp + v0 + col;
    float4_t S[NT]; // rows 16 tile + 4 quad + e of column v0 + col
#pragma unroll
    for (int i = 0; i < NT; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int tile = wave + 4 * i;
            S[i][e] = p.pos0 && tile < tiles ? state[size_t(16 * tile + 4 * quad + e) * p.vdimp] : 0.0f;
        }
    ScanChunk<NT> ring[AHEAD];
    unsigned off_k[NT], off_r[NT], off_g[NT];
#pragma unroll
    for (int i = 0; i < NT; i++) {
        const int tile = min(wave + 4 * i, tiles - 1);
        off_k[i] = (col * p.dimp + 16 * tile + 4 * quad) * 4;
        off_r[i] = (2 * DC * p.dimp + (16 * tile + col) * DC + 4 * quad) * 4;
        off_g[i] = (3 * DC * p.dimp + 16 * tile + 4 * quad) * 4;
    }
    const unsigned off_v = (49 * p.dimp + (DC + v0 + col) * DC + 4 * quad) * 4;
    auto request = [&](ScanChunk<NT> &b, int chunk) {
        const float *at = src + min(chunk, chunks - 1) * stride;
#pragma unroll
        for (int i = 0; i < NT; i++) {
            b.k[i] = scan_load(at, off_k[i]);
            b.q[i] = scan_load(at + DC * p.dimp, off_k[i]);
            b.r[i] = scan_load(at, off_r[i]);
            b.g[i] = scan_load(at, off_g[i]);
        }
        b.v = scan_load(at, off_v);
    };
#pragma unroll
    for (int a = 0; a < AHEAD; a++) request(ring[a], a);
    float4_t o = {0, 0, 0, 0};
    auto step = [&](ScanChunk<NT> &b, int chunk) {
        const int half = chunk & 1;
        float4_t u = wave == 0 ? b.v : float4_t{0, 0, 0, 0};
#pragma unroll
        for (int i = 0; i < NT; i++) // (a tile past the end is another wavefront's, with a state of zero here)
#pragma unroll
            for (int j = 0; j < 4; j++) u = __builtin_amdgcn_mfma_f32_16x16x4f32(b.k[i][j], S[i][j], u, 0, 0, 0);
        s_u[half][wave][lane] = u;
        s_o[half][wave][lane] = o; // (of the chunk before)
        lds_barrier(); // (one per chunk: what a chunk reads is written again two chunks later)
        const float4_t u0 = s_u[half][0][lane], u1 = s_u[half][1][lane], u2 = s_u[half][2][lane], u3 = s_u[half][3][lane];
        o = float4_t{0, 0, 0, 0};
#pragma unroll
        for (int i = 0; i < NT; i++)
#pragma unroll
            for (int j = 0; j < 4; j++) o = __builtin_amdgcn_mfma_f32_16x16x4f32(b.q[i][j], S[i][j], o, 0, 0, 0);
        u = (u0 + u1) + (u2 + u3);
#pragma unroll
        for (int i = 0; i < NT; i++) {
            S[i] *= b.g[i];
#pragma unroll
            for (int j = 0; j < 4; j++) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(b.r[i][j], u[j], S[i], 0, 0, 0);
            if (wave + 4 * i >= tiles) S[i] = float4_t{0, 0, 0, 0};
        }
        request(b, chunk + AHEAD);
    };
    // (no exit inside the rounds: with one, every wait for a chunk's operands would also wait for the ones requested last)
    int base = 0;
    for (; base + AHEAD <= chunks; base += AHEAD)
#pragma unroll
        for (int a = 0; a < AHEAD; a++) step(ring[a], base + a);
#pragma unroll
    for (int a = 0; a < AHEAD; a++)
        if (base + a < chunks) step(ring[a], base + a);
    s_o[chunks & 1][wave][lane] = o;
    lds_barrier();
#pragma unroll
    for (int i = 0; i < NT; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int tile = wave + 4 * i;
            if (tile < tiles) state[size_t(16 * tile + 4 * quad + e) * p.vdimp] = S[i][e];
        }
    if (v0) return;
    // the convolutions' last inputs (delta_chunk, which reads the older ones, is done)
    const int per = p.H / p.G, c = h / per, n_qk = h % per ? 0 : 2 * p.dimp;
    const T *rows = reinterpret_cast<const T *>(p.c1) + p.oc;
    for (int i = tid; i < n_qk + p.vdimp; i += 256) {
        const int ch = i >= n_qk ? 2 * p.G * p.dimp + h * p.vdimp + i - n_qk : i < p.dimp ? c * p.dimp + i : (p.G + c) * p.dimp + i - p.dimp;
        for (int r = max(0, p.n - (p.taps - 1)); r < p.n; r++)
            reinterpret_cast<T *>(p.ring)[size_t((p.pos0 + r) % p.taps) * p.channels + ch] = rows[size_t(r) * p.ld + ch];
    }
}

// lph lanes (a power of two) per head of a row
template <class T>
__global__ __launch_bounds__(256) void delta_gate_kernel(DeltaRows p, int lph) {
    typedef T vec4 __attribute__((ext_vector_type(4)));
    const int at = (int)(blockIdx.x * 256 + threadIdx.x) / lph, c0 = threadIdx.x % lph, r = at / p.H, h = at % p.H;
    if (r >= p.n) return; // (whole groups of lph lanes)
    const float *o = p.o + (size_t(r) * p.H + h) * p.vdimp;
    const T *z = reinterpret_cast<const T *>(p.gate) + size_t(r) * p.ldg + h * p.vdimp;
    T *out = reinterpret_cast<T *>(p.out) + size_t(r) * p.ldo + h * p.vdimp;
    float ss = 0.0f;
    for (int d = c0 * 4; d < p.vdimp; d += lph * 4) { // (the padding is zero)
        const float4_t v = *reinterpret_cast<const float4_t *>(o + d);
#pragma unroll
        for (int e = 0; e < 4; e++) ss = fmaf(v[e], v[e], ss);
    }
    for (int off = lph >> 1; off >= 1; off >>= 1) ss += __shfl_xor(ss, off);
    const float f = 1.0f / sqrtf(ss / (float)p.vdim + p.eps);
    for (int d = c0 * 4; d < p.vdimp; d += lph * 4) {
        const float4_t v = *reinterpret_cast<const float4_t *>(o + d), w = *reinterpret_cast<const float4_t *>(p.norm + d);
        const vec4 g = *reinterpret_cast<const vec4 *>(z + d);
        vec4 x;
#pragma unroll
        for (int e = 0; e < 4; e++) x[e] = (T)(v[e] * f * w[e] * lm_sigmoid((float)g[e]));
        *reinterpret_cast<vec4 *>(out + d) = x;
    }
}

template <class T> int delta_launch(moon_ctx *ctx, const DeltaRows &p) {
    const int chunks = (p.n + DC - 1) / DC;
    const size_t lds = chunk_lds_floats(p.dimp, p.vdimp) * sizeof(float);
    if (lds > 64 * 1024)
        MOON_HIP(ctx, hipFuncSetAttribute(reinterpret_cast<const void *>(delta_chunk_kernel<T>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(delta_chunk_kernel<T>, dim3((unsigned)chunks * p.H), dim3(256), lds, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    const dim3 grid((unsigned)(p.vdimp / 16) * p.H);
    const int nt = (p.dimp / 16 + 3) / 4;
    if (nt <= 1) hipLaunchKernelGGL((delta_scan_kernel<T, 1, 8>), grid, dim3(SCAN_THREADS), 0, ctx->stream, p);
    else if (nt <= 2) hipLaunchKernelGGL((delta_scan_kernel<T, 2, 4>), grid, dim3(SCAN_THREADS), 0, ctx->stream, p);
    else if (nt <= 4) hipLaunchKernelGGL((delta_scan_kernel<T, 4, 2>), grid, dim3(SCAN_THREADS), 0, ctx->stream, p);
    else hipLaunchKernelGGL((delta_scan_kernel<T, 8, 1>), grid, dim3(SCAN_THREADS), 0, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    int lph = 1;
    while (lph < p.vdimp / 4 && lph < 64) lph *= 2;
    hipLaunchKernelGGL(delta_gate_kernel<T>, dim3((unsigned)((size_t(p.n) * p.H * lph + 255) / 256)), dim3(256), 0, ctx->stream, p, lph);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

} // namespace

size_t delta_scratch_floats(size_t rows, size_t heads, size_t dimp, size_t vdimp) { return (rows + DC - 1) / DC * heads * chunk_floats((int)dimp, (int)vdimp); }

int launch_delta_rows(moon_ctx *ctx, int dtype, const DeltaRows &p) {
    if (p.n <= 0) return MOON_OK;
    if (p.H % p.G || p.dimp % 16 || p.vdimp % 16 || p.dimp > (int)DELTA_MAX_DIM || p.vdimp > (int)DELTA_MAX_DIM || p.taps < 1 || p.oc % 8)
        return moon_fail(ctx, MOON_EINVAL_DIM, "delta rule: %d heads over %d, head sizes %d and %d, %d taps", p.H, p.G, p.dimp, p.vdimp, p.taps);
    return dtype == MOON_DTYPE_BF16 ? delta_launch<bf16_t>(ctx, p) : delta_launch<float>(ctx, p);
}
