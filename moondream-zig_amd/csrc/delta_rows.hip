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
//                 matrix-core products (v_mfma_f32_16x16x4_f32: exact products, f32 sums).  The four wavefronts share the key channels;
//                 an accumulator tile is the next product's second operand as it lies in the registers.
//   delta_gate    RMS norm per head, weight, output gate.
#include "delta_math.hpp"
#include "lane_fold.hpp"
#include "layer_list.hpp"

#include <algorithm>
#include <atomic>

namespace {

constexpr int DC = 16;      // tokens of a chunk
constexpr int DC_PITCH = DC + 4;

// One chunk and head in the scratch memory, in floats: K' [16][dimp], Q [16][dimp], R^T [dimp][16], G_15 [dimp], P [16][16], V' [16][vdimp]
__host__ __device__ __forceinline__ size_t chunk_floats(int dimp, int vdimp) { return size_t(49) * dimp + 256 + size_t(16) * vdimp; }
__host__ __device__ __forceinline__ size_t chunk_lds_floats(int dimp, int vdimp) {
    return size_t(3) * DC * (dimp + 16) + size_t(DC) * vdimp + 2 * DC * DC_PITCH + DC;
}

template <class T>
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaRows p) {
    extern __shared__ __attribute__((aligned(16))) float s_dc[];
    constexpr int PE = Piece<T>::N;
    const int tid = threadIdx.x, lane = tid & 63, chunk = blockIdx.x / p.H, h = blockIdx.x % p.H, c = h / (p.H / p.G);
    const int t0 = chunk * DC, cnt = min(DC, p.n - t0), dp = p.dimp + 16; // dp: row pitch
    float *s_q = s_dc, *s_k = s_q + DC * dp, *s_g = s_k + DC * dp, *s_v = s_g + DC * dp, *s_a = s_v + DC * p.vdimp, *s_p = s_a + DC * DC_PITCH,
          *s_b = s_p + DC * DC_PITCH;
    // convolutions, 16 bytes of channels at a time; tokens past the end are zero
    const int pk = p.dimp / PE, pv = p.vdimp / PE, per_token = 2 * pk + pv;
    const T *rows = reinterpret_cast<const T *>(p.c1) + p.oc, *ring = reinterpret_cast<const T *>(p.ring);
    for (int i = tid; i < DC * per_token; i += 256) {
        const int tok = i / per_token, piece = i % per_token, what = piece < pk ? 0 : piece < 2 * pk ? 1 : 2, off = (piece - what * pk) * PE;
        const int ch = (what == 0 ? c * p.dimp : what == 1 ? (p.G + c) * p.dimp : 2 * p.G * p.dimp + h * p.vdimp) + off;
        float acc[PE];
#pragma unroll
        for (int e = 0; e < PE; e++) acc[e] = 0.0f;
        if (tok < cnt)
            for (int tap = 0; tap < p.taps; tap++) {
                const int r = t0 + tok - (p.taps - 1) + tap, pos = p.pos0 + r;
                if (pos < 0) continue;
                float x[PE];
                Piece<T>::unpack(*reinterpret_cast<const lm_u32x4 *>(r >= 0 ? rows + size_t(r) * p.ld + ch : ring + size_t(pos % p.taps) * p.channels + ch), x);
                const float *w = p.conv + size_t(tap) * p.channels + ch;
#pragma unroll
                for (int e = 0; e < PE; e++) acc[e] = fmaf(w[e], x[e], acc[e]);
            }
        float *dst = what == 0 ? s_q + tok * dp + off : what == 1 ? s_k + tok * dp + off : s_v + tok * p.vdimp + off;
#pragma unroll
        for (int e = 0; e < PE; e++) dst[e] = lm_silu(acc[e]);
    }
    for (int i = tid; i < DC * p.dimp; i += 256) {
        const int tok = i / p.dimp, d = i % p.dimp;
        s_g[tok * dp + d] = tok < cnt ? delta_decay(p.a_log[h], p.dt[size_t(t0 + tok) * p.lddt + h * p.dimp + d] + p.dt_bias[h * p.dimp + d]) : 1.0f;
    }
    if (tid < DC) s_b[tid] = tid < cnt ? lm_sigmoid(p.beta[size_t(t0 + tid) * p.ldb + h]) : 0.0f;
    lds_barrier();
    { // unit vectors: 8 lanes for each of the 32
        float *x = (tid < 128 ? s_q : s_k) + (tid >> 3 & 15) * dp;
        float ss = 0.0f;
        for (int d = tid & 7; d < p.dimp; d += 8) ss = fmaf(x[d], x[d], ss);
#pragma unroll
        for (int off = 4; off >= 1; off >>= 1) ss += __shfl_xor(ss, off);
        float f = 1.0f / sqrtf(ss + DELTA_UNIT_EPS);
        if (tid < 128) f *= 1.0f / sqrtf((float)p.dim);
        for (int d = tid & 7; d < p.dimp; d += 8) x[d] *= f;
    }
    lds_barrier();
    { // A and P: a thread has token s and every 16th channel
        const int s = tid >> 4;
        float v[2 * DC];
#pragma unroll
        for (int i = 0; i < 2 * DC; i++) v[i] = 0.0f;
        for (int d = tid & 15; d < p.dimp; d += 16) {
            float w = s_k[s * dp + d]; // k_s times the decays of the tokens behind s up to t
#pragma unroll
            for (int t = 0; t < DC; t++) {
                if (t > s) w *= s_g[t * dp + d];
                const float on = t >= s ? w : 0.0f;
                v[t] = fmaf(s_k[t * dp + d], on, v[t]);
                v[DC + t] = fmaf(s_q[t * dp + d], on, v[DC + t]);
            }
        }
        fold_lanes<2 * DC, 8>(v, lane, 1, 0, [&](int i, float x) {
            if (i < DC) s_a[i * DC_PITCH + s] = i > s ? s_b[i] * x : 0.0f;
            else s_p[(i - DC) * DC_PITCH + s] = x;
        });
    }
    lds_barrier();
    float *out = p.scratch + (size_t(h) * ((p.n + DC - 1) / DC) + chunk) * chunk_floats(p.dimp, p.vdimp);
    float *o_k = out, *o_q = o_k + DC * p.dimp, *o_r = o_q + DC * p.dimp, *o_g = o_r + DC * p.dimp, *o_p = o_g + p.dimp, *o_v = o_p + DC * DC;
    for (int i = tid; i < 2 * p.dimp + p.vdimp; i += 256) {
        float x[DC];
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
                for (int s = 0; s < t; s++) y = fmaf(-s_a[t * DC_PITCH + s], x[s], y);
                x[t] = y;
            }
            float *dst = is_k ? o_k + i : o_v + i - p.dimp;
            const int ld = is_k ? p.dimp : p.vdimp;
#pragma unroll
            for (int t = 0; t < DC; t++) dst[size_t(t) * ld] = x[t];
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
#pragma unroll
            for (int t = 0; t < DC; t += 4) *reinterpret_cast<float4 *>(o_r + size_t(d) * DC + t) = float4{x[t], x[t + 1], x[t + 2], x[t + 3]};
            o_g[d] = all;
        }
    }
    o_p[tid] = s_p[(tid >> 4) * DC_PITCH + (tid & 15)];
}

// NT: tiles of 16 key channels a wavefront owns; AHEAD: chunks whose operands are requested before they are needed
template <int NT> struct ScanChunk {
    float4_t k[NT], q[NT], r[NT], g[NT], p, v;
};
template <class T, int NT, int AHEAD>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1))) void delta_scan_kernel(DeltaRows p) {
    __shared__ float4_t s_u[2][4][64], s_o[2][4][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15, quad = lane >> 4;
    const int slices = p.vdimp / 16, h = blockIdx.x / slices, v0 = blockIdx.x % slices * 16, tiles = p.dimp / 16, chunks = (p.n + DC - 1) / DC;
    const size_t stride = chunk_floats(p.dimp, p.vdimp);
    const float *src = p.scratch + size_t(h) * chunks * stride;
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
    auto request = [&](ScanChunk<NT> &b, int chunk) {
        const float *at = src + min(chunk, chunks - 1) * stride;
#pragma unroll
        for (int i = 0; i < NT; i++) {
            const int tile = wave + 4 * i;
            if (tile < tiles) {
                b.k[i] = *reinterpret_cast<const float4_t *>(at + col * p.dimp + 16 * tile + 4 * quad);
                b.q[i] = *reinterpret_cast<const float4_t *>(at + (DC + col) * p.dimp + 16 * tile + 4 * quad);
                b.r[i] = *reinterpret_cast<const float4_t *>(at + 2 * DC * p.dimp + (16 * tile + col) * DC + 4 * quad);
                b.g[i] = *reinterpret_cast<const float4_t *>(at + 3 * DC * p.dimp + 16 * tile + 4 * quad);
            } else b.k[i] = b.q[i] = b.r[i] = b.g[i] = float4_t{0, 0, 0, 0};
        }
        const float *ap = at + size_t(49) * p.dimp;
        b.p = *reinterpret_cast<const float4_t *>(ap + col * DC + 4 * quad);
#pragma unroll
        for (int e = 0; e < 4; e++) b.v[e] = ap[DC * DC + (4 * quad + e) * p.vdimp + v0 + col];
    };
#pragma unroll
    for (int a = 0; a < AHEAD; a++) request(ring[a], a);
    for (int base = 0; base < chunks; base += AHEAD) {
#pragma unroll
        for (int a = 0; a < AHEAD; a++) {
            const int chunk = base + a;
            if (chunk >= chunks) break; // (the same in every wavefront)
            ScanChunk<NT> &b = ring[a];
            float4_t u = {0, 0, 0, 0}, o = {0, 0, 0, 0};
#pragma unroll
            for (int i = 0; i < NT; i++)
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    u = __builtin_amdgcn_mfma_f32_16x16x4f32(b.k[i][j], S[i][j], u, 0, 0, 0);
                    o = __builtin_amdgcn_mfma_f32_16x16x4f32(b.q[i][j], S[i][j], o, 0, 0, 0);
                }
            s_u[chunk & 1][wave][lane] = u;
            s_o[chunk & 1][wave][lane] = o;
            lds_barrier(); // (one per chunk: what a chunk reads is written again two chunks later)
            u = b.v - ((s_u[chunk & 1][0][lane] + s_u[chunk & 1][1][lane]) + (s_u[chunk & 1][2][lane] + s_u[chunk & 1][3][lane]));
#pragma unroll
            for (int i = 0; i < NT; i++) {
                S[i] *= b.g[i];
#pragma unroll
                for (int j = 0; j < 4; j++) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(b.r[i][j], u[j], S[i], 0, 0, 0);
            }
            if (wave == (chunk & 3)) {
                o = (s_o[chunk & 1][0][lane] + s_o[chunk & 1][1][lane]) + (s_o[chunk & 1][2][lane] + s_o[chunk & 1][3][lane]);
#pragma unroll
                for (int j = 0; j < 4; j++) o = __builtin_amdgcn_mfma_f32_16x16x4f32(b.p[j], u[j], o, 0, 0, 0);
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    const int row = chunk * DC + 4 * quad + e;
                    if (row < p.n) p.o[(size_t(row) * p.H + h) * p.vdimp + v0 + col] = o[e];
                }
            }
            if (chunk + AHEAD < chunks) request(b, chunk + AHEAD);
        }
    }
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
    if (nt <= 1) hipLaunchKernelGGL((delta_scan_kernel<T, 1, 4>), grid, dim3(256), 0, ctx->stream, p);
    else if (nt <= 2) hipLaunchKernelGGL((delta_scan_kernel<T, 2, 4>), grid, dim3(256), 0, ctx->stream, p);
    else if (nt <= 4) hipLaunchKernelGGL((delta_scan_kernel<T, 4, 2>), grid, dim3(256), 0, ctx->stream, p);
    else hipLaunchKernelGGL((delta_scan_kernel<T, 8, 1>), grid, dim3(256), 0, ctx->stream, p);
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
