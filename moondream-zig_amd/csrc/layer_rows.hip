// Row-wise kernels of the layer-list decoders: embedding, residual sum and LayerNorm; q/k norm, value mixing and the cache
// update of a prompt's rows; the router and the grouping of rows by expert.
#include "layer_list.hpp"
#include "lm_types.hpp"
#include "norm.hpp"
#include "router.hpp"

namespace {

template <class T>
__global__ __launch_bounds__(256) void row_finish_kernel(RowFinish p) {
    extern __shared__ __attribute__((aligned(16))) float s_row[]; // [width]
    __shared__ float sm[16];
    const int r = blockIdx.x, tid = threadIdx.x;
    float *xr = p.x + size_t(p.rows ? p.rows[r] : (uint32_t)r) * p.width;
    const T *er = p.embed ? reinterpret_cast<const T *>(p.embed) + size_t(p.ids[r]) * p.dp : nullptr;
    const bool changes = er || p.splits || p.top;
    float s = 0.0f;
    for (int i = tid; i < p.width; i += 256) {
        float v;
        if (er) v = (float)er[i] * p.embed_scale;
        else {
            float d = 0.0f;
            for (int k = 0; k < p.splits; k++) d += p.partial[(size_t(k) * p.n + r) * p.dp + i];
            for (int k = 0; k < p.top; k++) d = fmaf(p.weight[r * p.top + k], p.expert_out[size_t(p.slot[r * p.top + k]) * p.dp + i], d);
            v = xr[i] + d;
        }
        if (changes) xr[i] = v;
        s_row[i] = v;
        s += v;
    }
    if (!p.h) return;
    const float mean = block_sum(s, sm) / (float)p.width;
    float m2 = 0.0f;
    for (int i = tid; i < p.width; i += 256) { // (each thread reads back what it wrote)
        const float d = s_row[i] - mean;
        m2 = fmaf(d, d, m2);
    }
    const float rstd = 1.0f / sqrtf(block_sum(m2, sm) / (float)p.width + p.eps);
    T *h = reinterpret_cast<T *>(p.h) + size_t(r) * p.dp;
    for (int i = tid; i < p.dp; i += 256) h[i] = i < p.width ? (T)((s_row[i] - mean) * rstd * p.gamma[i] + p.beta[i]) : (T)0.0f;
}

template <class T>
__global__ __launch_bounds__(256) void prep_qkv_kernel(PrepArgs p) {
    const int r = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    T *row = reinterpret_cast<T *>(p.c1) + size_t(r) * p.ld;
    const int pos = p.pos0 + r, slot = pos % p.cap;
    for (int task = blockIdx.y * 4 + wave; task < p.H + 2 * p.G; task += gridDim.y * 4) {
        if (task < p.H + p.G) { // a head of q or k
            const bool is_q = task < p.H;
            const int g = task - p.H;
            T *src = row + (is_q ? p.oq + task * p.dimp : p.ok + g * p.dimp);
            T *dst = is_q ? src : reinterpret_cast<T *>(p.ck) + (size_t(g) * p.cap + slot) * p.dimp;
            if (is_q && !p.qk_rms) continue;
            float ss = 0.0f;
            for (int d = lane; d < p.dimp; d += 64) { // (the padding is zero)
                const float v = (float)src[d];
                ss = fmaf(v, v, ss);
            }
            const float f = p.qk_rms ? 1.0f / sqrtf(wave_sum(ss) / (float)p.dim + p.eps) : 1.0f;
            for (int d = lane; d < p.dimp; d += 64) dst[d] = (T)((float)src[d] * f);
        } else {
            const int g = task - p.H - p.G;
            const T *src = row + p.ov + g * p.vdimp;
            T *dst = reinterpret_cast<T *>(p.cv) + (size_t(g) * p.cap + slot) * p.vdimp;
            const T *first = p.mixes ? reinterpret_cast<const T *>(p.v_first) + (size_t(g) * p.cap_first + pos % p.cap_first) * p.vdimp : nullptr;
            for (int d = lane; d < p.vdimp; d += 64) {
                float v = (float)src[d];
                if (first) v = (1.0f - p.lambda) * v + p.lambda * (float)first[d];
                dst[d] = (T)v;
            }
        }
    }
}

__global__ __launch_bounds__(256) void route_kernel(RouteArgs p) {
    extern __shared__ float s_scores[]; // [4][2][E]
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = blockIdx.x * 4 + wave;
    if (r >= p.n) return; // (nothing below is shared between wavefronts)
    route_wave(p.logits + size_t(r) * p.ld, p.correction, p.E, p.top, s_scores + size_t(wave) * 2 * p.E, lane, p.ids + size_t(r) * p.top,
               p.weight + size_t(r) * p.top);
}

// One workgroup: how many rows every expert gets, where they start, which grouped row each (token, choice) is, the row tiles.
// Rows of an expert keep the order of the tokens.
__global__ __launch_bounds__(1024) void group_kernel(RouteArgs p) {
    extern __shared__ int s_cnt[]; // [E + 1] starts, [E + 1] first tiles, [E] counts, then [16][E] counts per wavefront
    int *start = s_cnt, *tiles = s_cnt + p.E + 1, *count = tiles + p.E + 1, *per_wave = count + p.E;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, total = p.n * p.top;
    const int per = (total + 15) / 16, lo = min(wave * per, total), hi = min(lo + per, total); // a wavefront's run of pairs
    for (int e = tid; e < 16 * p.E; e += 1024) per_wave[e] = 0;
    __syncthreads();
    for (int i = lo + lane; i < hi; i += 64) atomicAdd(&per_wave[wave * p.E + p.ids[i]], 1);
    __syncthreads();
    for (int e = tid; e < p.E; e += 1024) { // rows of expert e
        int c = 0;
        for (int w = 0; w < 16; w++) c += per_wave[w * p.E + e];
        count[e] = c;
    }
    __syncthreads();
    for (int e = tid; e <= p.E; e += 1024) {
        int s = 0, t = 0;
        for (int o = 0; o < e; o++) {
            s += count[o];
            t += (count[o] + p.rows_per_tile - 1) / p.rows_per_tile;
        }
        start[e] = s;
        tiles[e] = t;
        if (e == p.E) p.n_tiles[0] = t;
        else
            for (int w = 0; w < 16; w++) { // counts -> first grouped row of this wavefront's pairs
                const int c = per_wave[w * p.E + e];
                per_wave[w * p.E + e] = s;
                s += c;
            }
    }
    __syncthreads();
    for (int e = tid; e < p.E; e += 1024)
        for (int t = tiles[e]; t < tiles[e + 1]; t++) {
            p.tile_group[t] = e;
            p.tile_row[t] = start[e] + (t - tiles[e]) * p.rows_per_tile;
            p.tile_end[t] = start[e + 1];
        }
    for (int base = lo; base < hi; base += 64) { // 64 pairs at a time, in order
        const int i = base + lane;
        const int e = i < hi ? p.ids[i] : -1;
        int before = 0, same = 0;
        for (int l = 0; l < 64; l++) {
            const int other = __shfl(e, l);
            before += other == e && l < lane ? 1 : 0;
            same += other == e ? 1 : 0;
        }
        if (e >= 0) {
            const int at = per_wave[wave * p.E + e] + before;
            p.slot[i] = at;
            p.rows[at] = (uint32_t)(i / p.top);
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); // every lane has its row before the counters move on
        if (e >= 0 && before == 0) per_wave[wave * p.E + e] += same;
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    }
}

} // namespace

int launch_row_finish(moon_ctx *ctx, int dtype, const RowFinish &p) {
    if (p.n <= 0) return MOON_OK;
    const size_t lds = size_t(p.width) * sizeof(float);
    if (lds > 60 * 1024) return moon_fail(ctx, MOON_EINVAL_DIM, "row kernel: width %d too large", p.width);
    if (dtype == MOON_DTYPE_BF16) hipLaunchKernelGGL(row_finish_kernel<bf16_t>, dim3(p.n), dim3(256), lds, ctx->stream, p);
    else hipLaunchKernelGGL(row_finish_kernel<float>, dim3(p.n), dim3(256), lds, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

int launch_prep_qkv(moon_ctx *ctx, int dtype, const PrepArgs &p) {
    if (p.n <= 0) return MOON_OK;
    if (p.n > p.cap || (p.mixes && p.n > p.cap_first)) return moon_fail(ctx, MOON_EINVAL_DIM, "cache update: %d rows, %d slots", p.n, p.cap);
    const dim3 grid(p.n, p.n < 512 ? (unsigned)((p.H + 2 * p.G + 3) / 4) : 1);
    if (dtype == MOON_DTYPE_BF16) hipLaunchKernelGGL(prep_qkv_kernel<bf16_t>, grid, dim3(256), 0, ctx->stream, p);
    else hipLaunchKernelGGL(prep_qkv_kernel<float>, grid, dim3(256), 0, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

int launch_route(moon_ctx *ctx, const RouteArgs &p) {
    if (p.n <= 0) return MOON_OK;
    if (p.top < 1 || p.top > p.E || p.E > ROUTER_MAX_EXPERTS) return moon_fail(ctx, MOON_EINVAL_DIM, "router: %d of %d experts", p.top, p.E);
    hipLaunchKernelGGL(route_kernel, dim3((p.n + 3) / 4), dim3(256), size_t(8) * p.E * sizeof(float), ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    hipLaunchKernelGGL(group_kernel, dim3(1), dim3(1024), (size_t(19) * p.E + 2) * sizeof(int), ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}
