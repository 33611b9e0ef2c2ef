// Row-wise kernels of the layer-list decoders: embedding, residual sum and norm; q/k norm, rotation, value mixing and the cache
// update of a prompt's rows; the means of blocks of cache rows; the router and the grouping of rows by expert.
#include "layer_list.hpp"
#include "lm_types.hpp"
#include "norm.hpp"
#include "router.hpp"

#include <algorithm>

namespace {

template <class T, int W> struct RowVec; // W consecutive elements
template <class T> struct RowVec<T, 1> {
    static __device__ __forceinline__ void load(const T *p, float (&v)[1]) { v[0] = (float)p[0]; }
    static __device__ __forceinline__ void store(T *p, const float (&v)[1]) { p[0] = (T)v[0]; }
};
template <class T> struct RowVec<T, 4> {
    typedef T vec __attribute__((ext_vector_type(4)));
    static __device__ __forceinline__ void load(const T *p, float (&v)[4]) {
        const vec x = *reinterpret_cast<const vec *>(p);
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] = (float)x[e];
    }
    static __device__ __forceinline__ void store(T *p, const float (&v)[4]) {
        vec x;
#pragma unroll
        for (int e = 0; e < 4; e++) x[e] = (T)v[e];
        *reinterpret_cast<vec *>(p) = x;
    }
};

// W: elements a thread takes at a time (4 where the width allows).  JOIN: the first splits are two outputs that are normed first.
template <class T, int W, bool JOIN>
__global__ __launch_bounds__(256) void row_finish_kernel(RowFinish p) {
    extern __shared__ __attribute__((aligned(16))) float s_row[]; // [width], JOIN: and the two outputs
    __shared__ float sm[16];
    const int r = blockIdx.x, tid = threadIdx.x;
    float *xr = p.x + size_t(p.rows ? p.rows[r] : (uint32_t)r) * p.width;
    const T *er = p.embed ? reinterpret_cast<const T *>(p.embed) + size_t(p.ids[r]) * p.dp : nullptr;
    const T *eo = reinterpret_cast<const T *>(p.expert_out);
    const bool changes = er || p.splits || p.top;
    float s = 0.0f, ss_l = 0.0f, ss_r = 0.0f;
    float *s_l = s_row + p.width, *s_r = s_l + p.width; // (JOIN only)
    for (int i = tid * W; i < p.width; i += 256 * W) {
        float v[W], d[W] = {};
        if (er) {
            RowVec<T, W>::load(er + i, v);
#pragma unroll
            for (int e = 0; e < W; e++) v[e] *= p.embed_scale;
        } else {
            RowVec<float, W>::load(xr + i, v);
            if (JOIN) {
                float l[W] = {}, r2[W] = {};
#pragma unroll 4
                for (int k = 0; k < p.splits_l + p.splits_r; k++) {
                    float t[W];
                    RowVec<float, W>::load(p.partial + (size_t(k) * p.n + r) * p.dp + i, t);
#pragma unroll
                    for (int e = 0; e < W; e++)
                        if (k < p.splits_l) l[e] += t[e];
                        else r2[e] += t[e];
                }
#pragma unroll
                for (int e = 0; e < W; e++) {
                    ss_l = fmaf(l[e], l[e], ss_l);
                    ss_r = fmaf(r2[e], r2[e], ss_r);
                }
                RowVec<float, W>::store(s_l + i, l);
                RowVec<float, W>::store(s_r + i, r2);
            }
#pragma unroll 4
            for (int k = JOIN ? p.splits_l + p.splits_r : 0; k < p.splits; k++) {
                float t[W];
                RowVec<float, W>::load(p.partial + (size_t(k) * p.n + r) * p.dp + i, t);
#pragma unroll
                for (int e = 0; e < W; e++) d[e] += t[e];
            }
#pragma unroll 4
            for (int k = 0; k < p.top; k++) {
                float t[W];
                RowVec<T, W>::load(eo + size_t(p.slot[r * p.top + k]) * p.dp + i, t);
                const float w = p.weight[r * p.top + k];
#pragma unroll
                for (int e = 0; e < W; e++) d[e] = fmaf(w, t[e], d[e]);
            }
#pragma unroll
            for (int e = 0; e < W; e++) v[e] += d[e];
        }
        if (changes && !JOIN) RowVec<float, W>::store(xr + i, v);
        RowVec<float, W>::store(s_row + i, v);
#pragma unroll
        for (int e = 0; e < W; e++) s += v[e];
    }
    if (JOIN) { // (each thread reads back what it wrote)
        const float f_l = 0.5f / sqrtf(block_sum(ss_l, sm) / (float)p.width + p.eps), f_r = 0.5f / sqrtf(block_sum(ss_r, sm) / (float)p.width + p.eps);
        s = 0.0f;
        for (int i = tid * W; i < p.width; i += 256 * W) {
            float v[W], l[W], r2[W], wl[W], wr[W];
            RowVec<float, W>::load(s_row + i, v);
            RowVec<float, W>::load(s_l + i, l);
            RowVec<float, W>::load(s_r + i, r2);
            RowVec<float, W>::load(p.out_l + i, wl);
            RowVec<float, W>::load(p.out_r + i, wr);
#pragma unroll
            for (int e = 0; e < W; e++) {
                v[e] += l[e] * f_l * wl[e] + r2[e] * f_r * wr[e];
                s += v[e];
            }
            RowVec<float, W>::store(xr + i, v);
            RowVec<float, W>::store(s_row + i, v);
        }
    }
    if (!p.h) return;
    const float mean = p.beta ? block_sum(s, sm) / (float)p.width : 0.0f; // (an RMS norm takes no mean off)
    float m2 = 0.0f;
    for (int i = tid * W; i < p.width; i += 256 * W) // (each thread reads back what it wrote)
#pragma unroll
        for (int e = 0; e < W; e++) {
            const float d = s_row[i + e] - mean;
            m2 = fmaf(d, d, m2);
        }
    const float rstd = 1.0f / sqrtf(block_sum(m2, sm) / (float)p.width + p.eps);
    T *h = reinterpret_cast<T *>(p.h) + size_t(r) * p.dp;
    for (int i = tid * W; i < p.dp; i += 256 * W) {
        float v[W] = {}, ga[W], be[W];
        if (i < p.width) {
            RowVec<float, W>::load(p.gamma + i, ga);
            if (p.beta) RowVec<float, W>::load(p.beta + i, be);
#pragma unroll
            for (int e = 0; e < W; e++) v[e] = (s_row[i + e] - mean) * rstd * ga[e] + (p.beta ? be[e] : 0.0f);
        }
        RowVec<T, W>::store(h + i, v);
    }
}

// lph lanes (a power of two) per head of a row; a workgroup's heads follow each other in (row, head) order.
template <class T>
__global__ __launch_bounds__(256) void prep_qkv_kernel(PrepArgs p, int lph) {
    constexpr int PE = Piece<T>::N;
    const int tasks = p.H + 2 * p.G, at = (int)(blockIdx.x * 256 + threadIdx.x) / lph, c0 = threadIdx.x % lph;
    const int r = at / tasks, task = at % tasks;
    if (r >= p.n) return; // (whole groups of lph lanes)
    T *row = reinterpret_cast<T *>(p.c1) + size_t(r) * p.ld;
    const int pos = p.pos0 + r, slot = pos % p.cap;
    if (task < p.H + p.G) { // a head of q or k
        const bool is_q = task < p.H;
        if (is_q && !p.qk_rms) return;
        const int g = task - p.H, pieces = p.dimp / PE;
        T *src = row + (is_q ? p.oq + task * p.dimp : p.ok + g * p.dimp);
        T *dst = is_q ? src : reinterpret_cast<T *>(p.ck) + (size_t(g) * p.cap + slot) * p.dimp;
        float ss = 0.0f, v[PE];
        for (int c = c0; c < pieces; c += lph) { // (the padding is zero)
            Piece<T>::unpack(*reinterpret_cast<const lm_u32x4 *>(src + c * PE), v);
#pragma unroll
            for (int e = 0; e < PE; e++) ss = fmaf(v[e], v[e], ss);
        }
        for (int off = lph >> 1; off >= 1; off >>= 1) ss += __shfl_xor(ss, off);
        const float f = p.qk_rms ? 1.0f / sqrtf(ss / (float)p.dim + p.eps) : 1.0f;
        for (int c = c0; c < pieces; c += lph) {
            Piece<T>::unpack(*reinterpret_cast<const lm_u32x4 *>(src + c * PE), v);
            lm_u32x4 o;
            T *t = reinterpret_cast<T *>(&o);
#pragma unroll
            for (int e = 0; e < PE; e++) t[e] = (T)(v[e] * f);
            *reinterpret_cast<lm_u32x4 *>(dst + c * PE) = o;
        }
    } else {
        const int g = task - p.H - p.G, pieces = p.vdimp / PE;
        const T *src = row + p.ov + g * p.vdimp;
        T *dst = reinterpret_cast<T *>(p.cv) + (size_t(g) * p.cap + slot) * p.vdimp;
        const T *first = p.mixes ? reinterpret_cast<const T *>(p.v_first) + (size_t(g) * p.cap_first + pos % p.cap_first) * p.vdimp : nullptr;
        for (int c = c0; c < pieces; c += lph) {
            float v[PE], f[PE];
            lm_u32x4 o = *reinterpret_cast<const lm_u32x4 *>(src + c * PE);
            if (first) {
                Piece<T>::unpack(o, v);
                Piece<T>::unpack(*reinterpret_cast<const lm_u32x4 *>(first + c * PE), f);
                T *t = reinterpret_cast<T *>(&o);
#pragma unroll
                for (int e = 0; e < PE; e++) t[e] = (T)((1.0f - p.lambda) * v[e] + p.lambda * f[e]);
            }
            *reinterpret_cast<lm_u32x4 *>(dst + c * PE) = o;
        }
    }
}

// One workgroup per row: q and k as a whole through their norms, heads of q, k and v turned, k and v into the cache.
template <class T>
__global__ __launch_bounds__(256) void prep_whole_kernel(PrepWhole p) {
    extern __shared__ __attribute__((aligned(16))) float s_qkv[]; // q, k, v
    __shared__ float sm[16];
    constexpr int PE = Piece<T>::N;
    const int tid = threadIdx.x, r = blockIdx.x, pos = p.pos0 + r, slot = p.G ? pos % p.cap : 0;
    const int nq = p.H * p.dimp, nk = p.G * p.dimp, nv = p.G * p.vdimp;
    T *row = reinterpret_cast<T *>(p.c1) + size_t(r) * p.ld;
    float ss_q = 0.0f, ss_k = 0.0f;
    for (int i = tid * PE; i < nq + nk + nv; i += 256 * PE) {
        float v[PE];
        Piece<T>::unpack(*reinterpret_cast<const lm_u32x4 *>(row + (i < nq ? p.oq + i : i < nq + nk ? p.ok + i - nq : p.ov + i - nq - nk)), v);
        float s = 0.0f;
#pragma unroll
        for (int e = 0; e < PE; e++) {
            s = fmaf(v[e], v[e], s);
            s_qkv[i + e] = v[e];
        }
        if (i < nq) ss_q += s;
        else if (i < nq + nk) ss_k += s;
    }
    ss_q = wave_sum(ss_q);
    ss_k = wave_sum(ss_k);
    if ((tid & 63) == 0) {
        sm[tid >> 6] = ss_q;
        sm[4 + (tid >> 6)] = ss_k;
    }
    lds_barrier(); // (also for the copy in LDS)
    const float f_q = 1.0f / sqrtf(((sm[0] + sm[1]) + (sm[2] + sm[3])) / (float)(p.H * p.dim) + p.eps);
    const float f_k = p.G ? 1.0f / sqrtf(((sm[4] + sm[5]) + (sm[6] + sm[7])) / (float)(p.G * p.dim) + p.eps) : 0.0f;
    for (int i = tid * PE; i < nq + nk + nv; i += 256 * PE) {
        const bool is_v = i >= nq + nk, is_q = i < nq;
        const int at = is_q ? i : is_v ? i - nq - nk : i - nq, size = is_v ? p.vdimp : p.dimp, head = at / size, d0 = at % size;
        const float *x = s_qkv + i - d0, *w = is_v ? nullptr : (is_q ? p.qn : p.kn) + at - d0; // this head's elements and weights
        const float f = is_v ? 1.0f : is_q ? f_q : f_k;
        const float2 *table = is_v ? p.rotv : p.rot;
        const int half = !table ? 0 : (is_v ? p.vdim : p.rot_dims) / 2;
        lm_u32x4 o;
        T *t = reinterpret_cast<T *>(&o);
        auto weighted = [&](int d, float (&y)[PE]) { // PE elements from d on
            RowVec<float, 4>::load(x + d, reinterpret_cast<float (&)[4]>(y[0]));
            if (PE > 4) RowVec<float, 4>::load(x + d + 4, reinterpret_cast<float (&)[4]>(y[PE - 4]));
#pragma unroll
            for (int e = 0; e < PE; e++) y[e] *= f;
            if (!w) return;
            float a[PE];
            RowVec<float, 4>::load(w + d, reinterpret_cast<float (&)[4]>(a[0]));
            if (PE > 4) RowVec<float, 4>::load(w + d + 4, reinterpret_cast<float (&)[4]>(a[PE - 4]));
#pragma unroll
            for (int e = 0; e < PE; e++) y[e] *= a[e];
        };
        if (d0 >= 2 * half) {
            float y[PE];
            weighted(d0, y);
#pragma unroll
            for (int e = 0; e < PE; e++) t[e] = (T)y[e];
        } else if (half % PE == 0) { // the other halves of the pairs lie side by side, too
            const bool first = d0 < half;
            float y[PE], z[PE];
            weighted(d0, y);
            weighted(first ? d0 + half : d0 - half, z);
            const float4_t *cs = reinterpret_cast<const float4_t *>(table + size_t(pos) * half + (first ? d0 : d0 - half)); // two pairs each
#pragma unroll
            for (int e = 0; e < PE; e += 2) {
                const float4_t c = cs[e / 2];
                t[e] = (T)(first ? y[e] * c[0] - z[e] * c[1] : y[e] * c[0] + z[e] * c[1]);
                t[e + 1] = (T)(first ? y[e + 1] * c[2] - z[e + 1] * c[3] : y[e + 1] * c[2] + z[e + 1] * c[3]);
            }
        } else
#pragma unroll
        for (int e = 0; e < PE; e++) {
            const int d = d0 + e;
            float y = w ? x[d] * f * w[d] : x[d];
            if (d < 2 * half) {
                const int m = d < half ? d : d - half, other = d < half ? d + half : m;
                const float2 cs = table[size_t(pos) * half + m];
                const float z = w ? x[other] * f * w[other] : x[other];
                y = d < half ? y * cs.x - z * cs.y : y * cs.x + z * cs.y;
            }
            t[e] = (T)y;
        }
        T *dst = is_q ? row + p.oq + i : is_v ? reinterpret_cast<T *>(p.cv) + (size_t(head) * p.cap + slot) * p.vdimp + d0
                                              : reinterpret_cast<T *>(p.ck) + (size_t(head) * p.cap + slot) * p.dimp + d0;
        *reinterpret_cast<lm_u32x4 *>(dst) = o;
    }
}

// 16 bytes of a block's row per thread
template <class T>
__global__ __launch_bounds__(256) void pool_kernel(PoolArgs p, int first, int tasks) {
    constexpr int PE = Piece<T>::N;
    const int i = blockIdx.x * 256 + threadIdx.x, pk = p.dimp / PE, per_head = pk + p.vdimp / PE;
    if (i >= tasks) return;
    const int piece = i % per_head, g = i / per_head % p.G, b = first + i / per_head / p.G;
    const bool is_v = piece >= pk;
    const int size = is_v ? p.vdimp : p.dimp, d = (is_v ? piece - pk : piece) * PE;
    const T *src = reinterpret_cast<const T *>(is_v ? p.cv : p.ck) + size_t(g) * p.cap * size + d;
    float acc[PE];
#pragma unroll
    for (int e = 0; e < PE; e++) acc[e] = 0.0f;
#pragma unroll 4
    for (int j = 0; j < p.pool; j++) {
        float v[PE];
        Piece<T>::unpack(*reinterpret_cast<const lm_u32x4 *>(src + size_t((b * p.pool + j) % p.cap) * size), v);
#pragma unroll
        for (int e = 0; e < PE; e++) acc[e] += v[e];
    }
    lm_u32x4 o;
    T *t = reinterpret_cast<T *>(&o);
#pragma unroll
    for (int e = 0; e < PE; e++) t[e] = (T)(acc[e] / (float)p.pool);
    *reinterpret_cast<lm_u32x4 *>(reinterpret_cast<T *>(is_v ? p.pv : p.pk) + (size_t(g) * p.blocks + b) * size + d) = o;
}

__global__ __launch_bounds__(256) void rotation_table_kernel(float2 *table, size_t n, int half, double base, double factor) {
    const size_t i = size_t(blockIdx.x) * 256 + threadIdx.x;
    if (i >= n) return;
    double s, c;
    sincos(double(i / half) * (pow(base, -double(i % half) / half) / factor), &s, &c);
    table[i] = float2{(float)c, (float)s};
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
    constexpr int AHEAD = 8; // ids requested together
    for (int base = lo; base < hi; base += 64 * AHEAD) {
        int e[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; u++) e[u] = base + u * 64 + lane < hi ? p.ids[base + u * 64 + lane] : -1;
#pragma unroll
        for (int u = 0; u < AHEAD; u++)
            if (e[u] >= 0) atomicAdd(&per_wave[wave * p.E + e[u]], 1);
    }
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
    int next = lo + lane < hi ? p.ids[lo + lane] : -1;
    for (int base = lo; base < hi; base += 64) { // 64 pairs at a time, in order
        const int i = base + lane, e = next;
        next = i + 64 < hi ? p.ids[i + 64] : -1;
        unsigned long long match = ~0ull; // the lanes with this lane's expert
        for (int bit = 1; bit < 2 * p.E; bit <<= 1) { // (lanes past the end count as expert E)
            const unsigned long long ones = __ballot(((e < 0 ? p.E : e) & bit) != 0);
            match &= (e < 0 ? p.E : e) & bit ? ones : ~ones;
        }
        const int before = __popcll(match & ((1ull << lane) - 1)), same = __popcll(match);
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

template <class T> static int row_finish_launch(moon_ctx *ctx, const RowFinish &p) {
    const bool join = p.out_l != nullptr;
    const size_t lds = size_t(p.width) * sizeof(float) * (join ? 3 : 1);
    if (lds > 156 * 1024) return moon_fail(ctx, MOON_EINVAL_DIM, "row kernel: width %d too large", p.width);
    auto kern = join ? (p.width % 4 ? row_finish_kernel<T, 1, true> : row_finish_kernel<T, 4, true>)
                     : (p.width % 4 ? row_finish_kernel<T, 1, false> : row_finish_kernel<T, 4, false>);
    if (lds > 60 * 1024) MOON_HIP(ctx, hipFuncSetAttribute(reinterpret_cast<const void *>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(kern, dim3(p.n), dim3(256), lds, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}
int launch_row_finish(moon_ctx *ctx, int dtype, const RowFinish &p) {
    if (p.n <= 0) return MOON_OK;
    if (p.out_l && (p.splits_l < 1 || p.splits_r < 1 || p.splits_l + p.splits_r > p.splits || p.embed))
        return moon_fail(ctx, MOON_EINVAL, "row kernel: %d and %d of %d splits are joined", p.splits_l, p.splits_r, p.splits);
    return dtype == MOON_DTYPE_BF16 ? row_finish_launch<bf16_t>(ctx, p) : row_finish_launch<float>(ctx, p);
}

int launch_prep_whole(moon_ctx *ctx, int dtype, const PrepWhole &p) {
    if (p.n <= 0) return MOON_OK;
    if (p.G && p.n > p.cap) return moon_fail(ctx, MOON_EINVAL_DIM, "cache update: %d rows, %d slots", p.n, p.cap);
    if (p.dimp % 8 || p.vdimp % 8 || p.rot_dims % 2 || p.rot_dims > p.dim || (p.rotv && p.vdim % 2))
        return moon_fail(ctx, MOON_EINVAL_DIM, "cache update: head sizes %d and %d, %d dimensions turn", p.dim, p.vdim, p.rot_dims);
    const size_t lds = (size_t(p.H + p.G) * p.dimp + size_t(p.G) * p.vdimp) * sizeof(float);
    if (lds > 156 * 1024) return moon_fail(ctx, MOON_EINVAL_DIM, "cache update: %d heads too wide for one workgroup", p.H);
    auto kern = dtype == MOON_DTYPE_BF16 ? prep_whole_kernel<bf16_t> : prep_whole_kernel<float>;
    if (lds > 60 * 1024) MOON_HIP(ctx, hipFuncSetAttribute(reinterpret_cast<const void *>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    hipLaunchKernelGGL(kern, dim3(p.n), dim3(256), lds, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

int launch_pool(moon_ctx *ctx, int dtype, const PoolArgs &p) {
    const int first = p.pos0 / p.pool, blocks = (p.pos0 + p.n) / p.pool - first;
    if (p.n <= 0 || blocks <= 0) return MOON_OK;
    if (first + blocks > p.blocks || (p.pool - 1 + p.n > p.cap && p.pos0 + p.n > p.cap))
        return moon_fail(ctx, MOON_EINVAL_DIM, "pooled blocks: %d of %d blocks, %d rows behind %d positions", first + blocks, p.blocks, p.n, p.pool);
    const int tasks = blocks * p.G * (p.dimp + p.vdimp) / (dtype == MOON_DTYPE_BF16 ? Piece<bf16_t>::N : Piece<float>::N);
    auto kern = dtype == MOON_DTYPE_BF16 ? pool_kernel<bf16_t> : pool_kernel<float>;
    hipLaunchKernelGGL(kern, dim3((unsigned)(tasks + 255) / 256), dim3(256), 0, ctx->stream, p, first, tasks);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

int launch_rotation_table(moon_ctx *ctx, float2 *table, size_t positions, size_t dims, double base, double factor) {
    const size_t n = positions * (dims / 2);
    if (!n) return MOON_OK;
    hipLaunchKernelGGL(rotation_table_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, ctx->stream, table, n, (int)(dims / 2), base, factor);
    MOON_HIP(ctx, hipGetLastError());
    return MOON_OK;
}

int launch_prep_qkv(moon_ctx *ctx, int dtype, const PrepArgs &p) {
    if (p.n <= 0) return MOON_OK;
    if (p.n > p.cap || (p.mixes && p.n > p.cap_first)) return moon_fail(ctx, MOON_EINVAL_DIM, "cache update: %d rows, %d slots", p.n, p.cap);
    const int pieces = std::max(p.dimp, p.vdimp) / (dtype == MOON_DTYPE_BF16 ? Piece<bf16_t>::N : Piece<float>::N);
    int lph = 1;
    while (lph < pieces && lph < 64) lph *= 2;
    const dim3 grid((unsigned)((size_t(p.n) * (p.H + 2 * p.G) * lph + 255) / 256));
    if (dtype == MOON_DTYPE_BF16) hipLaunchKernelGGL(prep_qkv_kernel<bf16_t>, grid, dim3(256), 0, ctx->stream, p, lph);
    else hipLaunchKernelGGL(prep_qkv_kernel<float>, grid, dim3(256), 0, ctx->stream, p, lph);
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
