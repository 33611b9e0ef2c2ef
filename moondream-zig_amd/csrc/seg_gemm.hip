// Products of the layer-list decoders: C[M, N] = A . W^T with the columns in segments (16-bit, f32, gated pairs), rows gathered
// and grouped where a router asks for it.  bf16 runs on the matrix cores through the wavefront-specialised tile product of
// gemm_dma.hpp; f32 is computed with f32 multiply-adds (no reduced-precision mode).
#include "gemm_dma.hpp"
#include "layer_list.hpp"
#include "lm_types.hpp"

#include <algorithm>
#include <atomic>

namespace {

struct TilePos {
    int m0, m_end, n0, group, split;
};
// Tile of this workgroup: consecutive workgroups land on different XCDs, so each XCD gets a contiguous run of tiles, walked m
// first (tiles that share weight columns meet in one L2).  false: nothing to do.
__device__ __forceinline__ bool seg_tile(const SegGemm &p, int tile_m, int tile_n, TilePos &t) {
    const int tiles_n = (p.N + tile_n - 1) / tile_n;
    const int tiles_m = p.tile_group ? p.max_tiles : (p.M + tile_m - 1) / tile_m;
    const int tiles = tiles_m * tiles_n, total = tiles * p.splits, per_xcd = (total + 7) / 8;
    int wg = (blockIdx.x % 8) * per_xcd + blockIdx.x / 8;
    if (p.last_first) { // each XCD: its run of tiles of the last range, then of the one before, ..
        const int run = (tiles + 7) / 8, j = blockIdx.x / 8, tile = (blockIdx.x % 8) * run + j % run;
        if (j >= run * p.splits || tile >= tiles) return false;
        wg = (p.splits - 1 - j / run) * tiles + tile;
    } else if ((int)(blockIdx.x / 8) >= per_xcd || wg >= total) return false;
    t.split = wg / tiles;
    const int tile = wg % tiles, tn = tile / tiles_m, tm = tile % tiles_m;
    t.n0 = tn * tile_n;
    if (p.tile_group) {
        if (tm >= p.n_tiles[0]) return false;
        t.group = p.tile_group[tm];
        t.m0 = p.tile_row[tm];
        t.m_end = min(t.m0 + tile_m, p.tile_end[tm]);
    } else {
        t.group = 0;
        t.m0 = tm * tile_m;
        t.m_end = min(t.m0 + tile_m, p.M);
    }
    return true;
}

// A wavefront's 64 x 64 accumulators -> its segment, through LDS so that the stores are whole lines.  scratch: 64 * 68 halfs.
constexpr int SEG_PITCH16 = 72, SEG_PITCHG = 40, SEG_PITCH32 = 68;
constexpr int SEG_SCRATCH_BYTES = 64 * SEG_PITCH16 * 2; // >= 64 * SEG_PITCHG * 2 and 32 * SEG_PITCH32 * 4
static_assert(SEG_SCRATCH_BYTES >= 32 * SEG_PITCH32 * 4, "scratch");
typedef bf16_t bf16x4_t __attribute__((ext_vector_type(4)));
__device__ __forceinline__ void seg_store(const SegGemm &p, const float16_t (&acc)[2][2], const TilePos &t, int wm, int wn, int lane, void *scratch) {
    const int n = t.n0 + wn * 64, col = lane & 31, g = lane >> 5;
    if (n >= p.N) return;
    if (n < p.n16) {
        bf16_t *s = reinterpret_cast<bf16_t *>(scratch);
#pragma unroll
        for (int ni = 0; ni < 2; ni++)
#pragma unroll
            for (int mi = 0; mi < 2; mi++)
#pragma unroll
                for (int q = 0; q < 4; q++) {
                    bf16x4_t o;
#pragma unroll
                    for (int e = 0; e < 4; e++) o[e] = (bf16_t)acc[ni][mi][4 * q + e];
                    *reinterpret_cast<bf16x4_t *>(s + (mi * 32 + col) * SEG_PITCH16 + ni * 32 + 8 * q + 4 * g) = o;
                }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); // the wavefront reads back what its own lanes wrote
#pragma unroll
        for (int r = 0; r < 8; r++) {
            const int ml = r * 8 + (lane >> 3), m = t.m0 + wm * 64 + ml;
            if (m >= t.m_end) continue;
            *reinterpret_cast<lm_u32x4 *>(reinterpret_cast<bf16_t *>(p.c16) + size_t(m) * p.ld16 + n + (lane & 7) * 8) =
                *reinterpret_cast<const lm_u32x4 *>(s + ml * SEG_PITCH16 + (lane & 7) * 8);
        }
    } else if (n < p.n32) {
        float *s = reinterpret_cast<float *>(scratch);
        float *dst = p.c32 + size_t(t.split) * p.M * p.ld32;
#pragma unroll
        for (int mi = 0; mi < 2; mi++) {
#pragma unroll
            for (int ni = 0; ni < 2; ni++)
#pragma unroll
                for (int q = 0; q < 4; q++) {
                    float4 o = {acc[ni][mi][4 * q], acc[ni][mi][4 * q + 1], acc[ni][mi][4 * q + 2], acc[ni][mi][4 * q + 3]};
                    if (p.softcap > 0.0f) o = {lm_softcap(o.x, p.softcap), lm_softcap(o.y, p.softcap), lm_softcap(o.z, p.softcap), lm_softcap(o.w, p.softcap)};
                    *reinterpret_cast<float4 *>(s + col * SEG_PITCH32 + ni * 32 + 8 * q + 4 * g) = o;
                }
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
            for (int r = 0; r < 8; r++) {
                const int ml = r * 4 + (lane >> 4), m = t.m0 + wm * 64 + mi * 32 + ml;
                if (m >= t.m_end) continue;
                *reinterpret_cast<float4 *>(dst + size_t(m) * p.ld32 + (n - p.n16) + (lane & 15) * 4) =
                    *reinterpret_cast<const float4 *>(s + ml * SEG_PITCH32 + (lane & 15) * 4);
            }
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); // the reads are done before the other half overwrites the rows
        }
    } else {
        bf16_t *s = reinterpret_cast<bf16_t *>(scratch);
#pragma unroll
        for (int mi = 0; mi < 2; mi++)
#pragma unroll
            for (int q = 0; q < 4; q++) {
                bf16x4_t o;
#pragma unroll
                for (int e = 0; e < 4; e++) o[e] = (bf16_t)(lm_silu(acc[0][mi][4 * q + e]) * acc[1][mi][4 * q + e]);
                *reinterpret_cast<bf16x4_t *>(s + (mi * 32 + col) * SEG_PITCHG + 8 * q + 4 * g) = o;
            }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int ml = r * 16 + (lane >> 2), m = t.m0 + wm * 64 + ml;
            if (m >= t.m_end) continue;
            *reinterpret_cast<lm_u32x4 *>(reinterpret_cast<bf16_t *>(p.glu) + size_t(m) * p.ldg + (n - p.n32) / 2 + (lane & 3) * 8) =
                *reinterpret_cast<const lm_u32x4 *>(s + ml * SEG_PITCHG + (lane & 3) * 8);
        }
    }
}

__global__ __launch_bounds__(DMA_THREADS) void seg_gemm_bf16_kernel(SegGemm p) {
    extern __shared__ __attribute__((aligned(16))) half_t lds_dma[]; // (the tile product addresses LDS from 0: nothing static beside it)
    TilePos t;
    if (!seg_tile(p, BM, BN, t)) return;
    const int k_begin = p.kb[t.split], k_end = p.kb[t.split + 1], n_ktiles = (k_end - k_begin + BK - 1) / BK;
    if (n_ktiles <= 0) return;
    const int lane = threadIdx.x & 63, role_wave = (threadIdx.x >> 6) & 3;
    if (threadIdx.x >= 256) {
        DmaSource s;
        s.a = p.A;
        s.w = reinterpret_cast<const bf16_t *>(p.W) + size_t(t.group) * p.w_group;
        s.a_bytes = p.a_rows * p.lda * 2; // (the launcher has checked that both fit)
        s.w_bytes = p.N * p.K * 2;
        s.w_k_bytes = 2;
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int r = dma_row(role_wave, j, lane), g8 = swz(r, lane & 7) * 8;
            const int m = min(t.m0 + r, t.m_end - 1);
            s.off_a[j] = ((p.rows ? (int)p.rows[m] : m) * p.lda + g8) * 2;
            s.off_w[j] = (min(t.n0 + r, p.N - 1) * p.K + g8) * 2;
        }
        dma_load_tiles(s, lds_dma, k_begin, n_ktiles, role_wave);
        return;
    }
    const int wm = role_wave & 1, wn = role_wave >> 1;
    float16_t acc[2][2];
    dma_multiply_tiles<MfmaBf16, false>(acc, k_begin, k_end, n_ktiles, wm, wn, lane);
    seg_store(p, acc, t, wm, wn, lane, reinterpret_cast<char *>(dma_free_stages(lds_dma, n_ktiles)) + size_t(role_wave) * SEG_SCRATCH_BYTES);
}

// f32: 64 x 64 tile, a thread owns rows ty, ty + 16, .. and columns tx, tx + 16, tx + 32, tx + 48 (so a gate column and its up
// column are in one thread).  Tile lists are 128 rows high: two passes over m.
constexpr int F32_K = 16;
__global__ __launch_bounds__(256) void seg_gemm_f32_kernel(SegGemm p) {
    __shared__ float sa[F32_K][64 + 4], sw[F32_K][64 + 4];
    TilePos t;
    if (!seg_tile(p, SEG_TILE_ROWS, 64, t)) return;
    const int k_begin = p.kb[t.split], k_end = p.kb[t.split + 1];
    const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4, lr = tid >> 2, lk = (tid & 3) * 4;
    const float *A = reinterpret_cast<const float *>(p.A), *W = reinterpret_cast<const float *>(p.W) + size_t(t.group) * p.w_group;
    for (int mb = t.m0; mb < t.m_end; mb += 64) {
        float acc[4][4] = {};
        const int m_src = min(mb + lr, t.m_end - 1);
        const float *arow = A + size_t(p.rows ? (int)p.rows[m_src] : m_src) * p.lda, *wrow = W + size_t(t.n0 + lr) * p.K;
        for (int k = k_begin; k < k_end; k += F32_K) {
            const float4 a = *reinterpret_cast<const float4 *>(arow + k + lk), w = *reinterpret_cast<const float4 *>(wrow + k + lk);
            __syncthreads();
            sa[lk][lr] = a.x; sa[lk + 1][lr] = a.y; sa[lk + 2][lr] = a.z; sa[lk + 3][lr] = a.w;
            sw[lk][lr] = w.x; sw[lk + 1][lr] = w.y; sw[lk + 2][lr] = w.z; sw[lk + 3][lr] = w.w;
            __syncthreads();
#pragma unroll
            for (int kk = 0; kk < F32_K; kk++)
#pragma unroll
                for (int i = 0; i < 4; i++)
#pragma unroll
                    for (int j = 0; j < 4; j++) acc[i][j] = fmaf(sa[kk][ty + 16 * i], sw[kk][tx + 16 * j], acc[i][j]);
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int m = mb + ty + 16 * i;
            if (m >= t.m_end) continue;
            if (t.n0 < p.n16)
                for (int j = 0; j < 4; j++) reinterpret_cast<float *>(p.c16)[size_t(m) * p.ld16 + t.n0 + tx + 16 * j] = acc[i][j];
            else if (t.n0 < p.n32)
                for (int j = 0; j < 4; j++) p.c32[(size_t(t.split) * p.M + m) * p.ld32 + t.n0 - p.n16 + tx + 16 * j] = p.softcap > 0.0f ? lm_softcap(acc[i][j], p.softcap) : acc[i][j];
            else
                for (int j = 0; j < 2; j++)
                    reinterpret_cast<float *>(p.glu)[size_t(m) * p.ldg + (t.n0 - p.n32) / 2 + tx + 16 * j] = lm_silu(acc[i][j]) * acc[i][j + 2];
        }
        __syncthreads();
    }
}

} // namespace

int seg_gemm_splits(moon_ctx *ctx, size_t M, size_t N, size_t K) {
    const size_t cus = ctx->cu_count > 0 ? ctx->cu_count : 256, tiles = (M + BM - 1) / BM * ((N + BN - 1) / BN);
    size_t s = std::min<size_t>(std::min<size_t>(cus / std::max<size_t>(tiles, 1), K / 512), 8);
    return (int)std::max<size_t>(s, 1);
}

int launch_seg_gemm(moon_ctx *ctx, int dtype, SegGemm p) {
    if (p.M <= 0 || p.N <= 0) return MOON_OK;
    if (p.N % 64 || p.K % 64 || p.K <= 0 || p.n16 % 64 || p.n32 % 64 || p.n16 > p.n32 || p.n32 > p.N || p.lda < p.K)
        return moon_fail(ctx, MOON_EINVAL_DIM, "segmented product: sizes must be padded to 64 (N %d, K %d, segments %d %d)", p.N, p.K, p.n16, p.n32);
    if (p.splits < 1) p.splits = 1;
    if (p.splits > 1 && (p.n16 || p.n32 != p.N || p.tile_group)) return moon_fail(ctx, MOON_EINVAL, "segmented product: only a plain f32 result splits k");
    if (p.splits > SEG_MAX_SPLITS) return moon_fail(ctx, MOON_EINVAL, "segmented product: %d k splits", p.splits);
    if (!p.kb[p.splits])
        for (int s = 0, per = (int)pad_to((p.K + p.splits - 1) / p.splits, BK); s <= p.splits; s++) p.kb[s] = std::min(p.K, s * per);
    for (int s = 0; s < p.splits; s++)
        if (p.kb[0] || p.kb[s] >= p.kb[s + 1] || p.kb[s + 1] % BK || p.kb[p.splits] != p.K)
            return moon_fail(ctx, MOON_EINVAL, "segmented product: %d k splits leave one empty", p.splits);
    const int tile_n = dtype == MOON_DTYPE_BF16 ? BN : 64;
    const size_t tiles = size_t(p.tile_group ? p.max_tiles : (p.M + SEG_TILE_ROWS - 1) / SEG_TILE_ROWS) * ((p.N + tile_n - 1) / tile_n) * p.splits;
    const dim3 grid((unsigned)(p.last_first ? (tiles / p.splits + 7) / 8 * 8 * p.splits : (tiles + 7) / 8 * 8));
    if (dtype == MOON_DTYPE_BF16) {
        const size_t lim = (size_t(1) << 31) - 4096;
        if (size_t(p.a_rows) * p.lda * 2 >= lim || size_t(p.N) * p.K * 2 >= lim)
            return moon_fail(ctx, MOON_EINVAL_DIM, "segmented product: an operand of 2 GiB or more");
        static std::atomic<bool> attr_set[64];
        const int dev = ctx->device >= 0 && ctx->device < 64 ? ctx->device : -1;
        if (dev < 0 || !attr_set[dev].load()) {
            MOON_HIP(ctx, hipFuncSetAttribute(reinterpret_cast<const void *>(seg_gemm_bf16_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)DMA_LDS_BYTES));
            if (dev >= 0) attr_set[dev].store(true);
        }
        hipLaunchKernelGGL(seg_gemm_bf16_kernel, grid, dim3(DMA_THREADS), DMA_LDS_BYTES, ctx->stream, p);
    } else
        hipLaunchKernelGGL(seg_gemm_f32_kernel, grid, dim3(256), 0, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    MOON_NOTE_KERNEL(ctx, "%s %d workgroups, k split %d", dtype == MOON_DTYPE_BF16 ? "seg_gemm_bf16_kernel" : "seg_gemm_f32_kernel", (int)tiles, p.splits);
    return MOON_OK;
}
