// Causal attention of several query rows over a KV cache, with a sliding window, pooled blocks before it, grouped key/value heads, a
// sink in the softmax denominator, a factor per head on the scale, outputs that turn back by their position's angles (where the values
// were turned by theirs) and an output gate; each of them is an argument.  The cache of a layer is [G][cap][head size]; the keys of
// position p lie in row p % cap, so a windowed layer needs no more rows than its window and one call's rows together.
//
// bf16 runs on the matrix cores, arranged like the kernel of attn_prefill.hip: a 256-thread workgroup owns 32 query rows of one
// head, its four wavefronts take every fourth tile of 64 keys of the range the rows can see, each with an online softmax of its
// own over private LDS staging, and the four results are merged at the end.  Per tile, with v_mfma_f32_32x32x16_bf16 and f32
// accumulation,
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

// Blocks that lie wholly before the window of position pos: block b ends at b pool + pool - 1 <= pos - window
__device__ __forceinline__ int blocks_seen(int pos, int window, int pool) { return max(0, pos - window + 1) / pool; }

constexpr int WA_KT = 64, WA_Q = 32, WA_WAVES = 4; // keys per tile, query rows and wavefronts per workgroup
typedef short wa_short4_t __attribute__((ext_vector_type(4)));
typedef bf16_t bf16x2_t __attribute__((ext_vector_type(2)));
typedef float float2_t __attribute__((ext_vector_type(2)));

template <int P> struct WaCfg { // P: head sizes up to P (a multiple of 32), rows zero padded to it
    static constexpr int KSTEPS = P / 16, DT = P / 32, G = P / 8;
    static constexpr int KS = P + 8; // K row stride: 128-bit reads of consecutive rows are conflict free
    // V rows are unpadded.  The transposing reads take 16 dwords of each of 4 consecutive rows: rows of 16 or 48 dwords lie apart
    // mod 64 by themselves, in the others granule c of row r sits at c ^ SWZ * (r % 4).
    static constexpr int VS = P, SWZ = P == 64 ? 2 : P >= 128 ? 4 : 0;
    static constexpr int WAVE_ELEMS = WA_KT * KS; // K is only read before the scores, V only after: they share the area
    static constexpr int LOADS = G;  // 16-byte pieces per lane and operand tile
    static constexpr bool AHEAD = P <= 128; // the next tile's pieces wait in registers (above, there are too many)
    static constexpr int SD = P + 4; // merge: O as [wave][q][SD] floats, (m, l) [wave][q] behind them
    static constexpr size_t TILE_BYTES = size_t(WA_WAVES) * WAVE_ELEMS * 2, MERGE_BYTES = size_t(WA_WAVES) * WA_Q * SD * 4;
    static constexpr size_t ML_OFFSET = TILE_BYTES > MERGE_BYTES ? TILE_BYTES : MERGE_BYTES;
    static constexpr size_t LDS_BYTES = ML_OFFSET + 2 * WA_WAVES * WA_Q * 4;
};

__device__ __forceinline__ wa_short4_t wa_read_tr(const bf16_t *p) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) wa_short4_t *)(p));
}

// POOL: the tiles of the blocks' keys come first, in the same softmax
template <int P, bool POOL>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(P <= 64 ? 2 : 1))) void window_attn_kernel(WindowAttn p) {
    using C = WaCfg<P>;
    extern __shared__ __attribute__((aligned(16))) bf16_t wa_lds[];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 31, hf = lane >> 5;
    const int n_qb = (p.n + WA_Q - 1) / WA_Q;
    // Workgroups are dealt to the eight dies round robin: where the count divides, a die takes whole stretches of the (head, block)
    // list, so heads that share keys and values meet in one L2.  Late blocks see the most keys: they start first.
    int item = blockIdx.x;
    const int n_items = n_qb * p.H;
    if (n_items % 8 == 0) item = (item % 8) * (n_items / 8) + item / 8;
    int h = item / n_qb, qb = item % n_qb;
    if (n_items % 8 == 0 && (n_items / 8) % n_qb == 0) { // whole heads per die: their blocks walk together
        const int per_die = n_items / 8, heads = per_die / n_qb, j = item % per_die;
        h = item / per_die * heads + j % heads;
        qb = j / heads;
    }
    qb = n_qb - 1 - qb;
    const int g = h / (p.H / p.G), row0 = qb * WA_Q;
    const int first_pos = p.pos0 + row0, last_pos = p.pos0 + min(row0 + WA_Q, p.n) - 1, pos = first_pos + col; // pos: this lane's query
    const int lo_key = p.window ? max(0, first_pos - p.window + 1) : 0;
    // tiles start at multiples of 64 positions; POOL: tile numbers below t_window stand for blocks (of the first one, from 0 on)
    const int seen = POOL ? blocks_seen(last_pos, p.window, p.pool) : 0, t_blocks = (seen + WA_KT - 1) / WA_KT;
    const int t_begin = POOL ? lo_key / WA_KT - t_blocks : lo_key / WA_KT, t_end = last_pos / WA_KT + 1;
    const int t_window = POOL ? lo_key / WA_KT : 0;
    // the head's cache rows as buffers: a 32-bit offset per piece, and what must not be read is an offset past the end (zeros)
    const int k_bytes = p.cap * p.dimp * 2, v_bytes = p.cap * p.vdimp * 2;
    const __amdgpu_buffer_rsrc_t kr = __builtin_amdgcn_make_buffer_rsrc(const_cast<bf16_t *>(reinterpret_cast<const bf16_t *>(p.ck) + size_t(g) * p.cap * p.dimp), 0, k_bytes, 0x00020000);
    const __amdgpu_buffer_rsrc_t vr = __builtin_amdgcn_make_buffer_rsrc(const_cast<bf16_t *>(reinterpret_cast<const bf16_t *>(p.cv) + size_t(g) * p.cap * p.vdimp), 0, v_bytes, 0x00020000);
    const __amdgpu_buffer_rsrc_t pkr = __builtin_amdgcn_make_buffer_rsrc(const_cast<bf16_t *>(reinterpret_cast<const bf16_t *>(p.pk) + size_t(g) * p.blocks * p.dimp), 0, POOL ? p.blocks * p.dimp * 2 : 0, 0x00020000);
    const __amdgpu_buffer_rsrc_t pvr = __builtin_amdgcn_make_buffer_rsrc(const_cast<bf16_t *>(reinterpret_cast<const bf16_t *>(p.pv) + size_t(g) * p.blocks * p.vdimp), 0, POOL ? p.blocks * p.vdimp * 2 : 0, 0x00020000);
    bf16_t *Ks = wa_lds + wave * C::WAVE_ELEMS, *Vs = Ks;

    constexpr int NOWHERE = 0x7fffffff; // past the end of either buffer
    lm_u32x4 rk[C::LOADS], rv[C::LOADS];
    int k_off[C::LOADS], v_off[C::LOADS]; // this lane's pieces of a tile whose first row is row 0
#pragma unroll
    for (int i = 0; i < C::LOADS; i++) {
        const int x = i * 64 + lane, row = x / C::G, c = x % C::G;
        k_off[i] = c * 8 < p.dimp ? (row * p.dimp + c * 8) * 2 : NOWHERE;
        v_off[i] = c * 8 < p.vdimp ? (row * p.vdimp + c * 8) * 2 : NOWHERE;
    }
    auto load = [&](lm_u32x4 (&r)[C::LOADS], const __amdgpu_buffer_rsrc_t rs, const __amdgpu_buffer_rsrc_t blocks, const int (&offs)[C::LOADS], int d, int t) {
        if (POOL && t < t_window) {
            const int b0 = __builtin_amdgcn_readfirstlane((t - t_begin) * WA_KT);
#pragma unroll
            for (int i = 0; i < C::LOADS; i++) {
                const int off = offs[i] == NOWHERE || b0 + (i * 64 + lane) / C::G >= seen ? NOWHERE : offs[i] + b0 * d * 2;
                r[i] = __builtin_bit_cast(lm_u32x4, __builtin_amdgcn_raw_buffer_load_b128(blocks, off, 0, 0));
            }
            return;
        }
        const int key0 = __builtin_amdgcn_readfirstlane(t * WA_KT), slot0 = key0 < p.cap ? key0 : key0 % p.cap, row_bytes = d * 2;
        if (key0 >= lo_key && key0 + WA_KT - 1 <= last_pos && slot0 + WA_KT <= p.cap) { // the whole tile, in one piece
#pragma unroll
            for (int i = 0; i < C::LOADS; i++) r[i] = __builtin_bit_cast(lm_u32x4, __builtin_amdgcn_raw_buffer_load_b128(rs, offs[i], slot0 * row_bytes, 0));
        } else {
#pragma unroll
            for (int i = 0; i < C::LOADS; i++) {
                const int row = (i * 64 + lane) / C::G, key = key0 + row;
                int off = (offs[i] == NOWHERE ? 0 : offs[i]) + slot0 * row_bytes;
                if (slot0 + row >= p.cap) off -= p.cap * row_bytes; // (a cache that wraps has more rows than a tile)
                if (offs[i] == NOWHERE || key < lo_key || key > last_pos) off = NOWHERE;
                r[i] = __builtin_bit_cast(lm_u32x4, __builtin_amdgcn_raw_buffer_load_b128(rs, off, 0, 0));
            }
        }
    };
    auto store = [&](const lm_u32x4 (&r)[C::LOADS], bf16_t *dst, int stride, int swz) {
#pragma unroll
        for (int i = 0; i < C::LOADS; i++) {
            const int x = i * 64 + lane, row = x / C::G;
            *reinterpret_cast<lm_u32x4 *>(dst + row * stride + (x % C::G ^ swz * (row & 3)) * 8) = r[i];
        }
    };
    int t = t_begin + wave;
    if (C::AHEAD && t < t_end) load(rk, kr, pkr, k_off, p.dimp, t);
    const float scale = p.temp ? p.scale * p.temp[h] : p.scale;
    bf16x8_t qf[C::KSTEPS]; // the MFMA "B" operand: Q[row0 + col][16 s + 8 hf .. + 7]
    {
        const bf16_t *q = reinterpret_cast<const bf16_t *>(p.q) + size_t(min(row0 + col, p.n - 1)) * p.ldq + h * p.dimp;
#pragma unroll
        for (int s = 0; s < C::KSTEPS; s++) {
            lm_u32x4 v = {0, 0, 0, 0};
            if (16 * s + 8 * hf < p.dimp) v = *reinterpret_cast<const lm_u32x4 *>(q + 16 * s + 8 * hf);
            if (scale < 0.0f) v ^= 0x80008000u; // scores are kept unscaled and the scale enters as its magnitude: the sign goes here
            qf[s] = __builtin_bit_cast(bf16x8_t, v);
        }
    }
    if (C::AHEAD && t < t_end) load(rv, vr, pvr, v_off, p.vdimp, t);
    int voff[C::DT]; // where this lane points the transposing loads: key 4 hf + (lane % 16) / 4, columns 32 dt + 16 ((lane / 16) % 2) + 4 (lane % 4)
#pragma unroll
    for (int dt = 0; dt < C::DT; dt++) {
        const int rq = (lane & 15) >> 2, d = 32 * dt + 16 * ((lane >> 4) & 1) + 4 * (lane & 3);
        voff[dt] = (4 * hf + rq) * C::VS + ((d >> 3 ^ C::SWZ * rq) << 3 | (d & 7));
    }

    float16_t o[C::DT];
#pragma unroll
    for (int dt = 0; dt < C::DT; dt++)
#pragma unroll
        for (int v = 0; v < 16; v++) o[dt][v] = 0.0f;
    constexpr float LOG2E = 1.4426950408889634f;
    const float c2 = fmaxf(fabsf(scale) * LOG2E, 1e-37f); // > 0: the maximum of the scaled scores is the scaled maximum, -inf stays -inf
    const float sink = p.sink ? p.sink[h] * LOG2E : -INFINITY;
    float m_run = -INFINITY, l_run = 0.0f; // m_run: scaled, in base-2 units; l_run: this lane's half of the row's sum

    for (; t < t_end; t += WA_WAVES) {
        const int key0 = t * WA_KT;
        if (!C::AHEAD) load(rk, kr, pkr, k_off, p.dimp, t);
        asm volatile("" ::: "memory"); // the V tile of the round before has been read: the K tile takes its place
        store(rk, Ks, C::KS, 0);
        if (C::AHEAD && t + WA_WAVES < t_end) load(rk, kr, pkr, k_off, p.dimp, t + WA_WAVES);
        if (!C::AHEAD) load(rv, vr, pvr, v_off, p.vdimp, t);
        float16_t s[2];
#pragma unroll
        for (int kt = 0; kt < 2; kt++) {
#pragma unroll
            for (int v = 0; v < 16; v++) s[kt][v] = 0.0f;
#pragma unroll
            for (int st = 0; st < C::KSTEPS; st++)
                s[kt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8_t *>(Ks + (32 * kt + col) * C::KS + 16 * st + 8 * hf), qf[st],
                                                                s[kt], 0, 0, 0);
        }
        // s[kt][v]: key key0 + 32 kt + 8 (v / 4) + 4 hf + v % 4 against this lane's query
        float mx = -INFINITY;
        if (POOL && t < t_window) {
            const int mine = blocks_seen(pos, p.window, p.pool) - (t - t_begin) * WA_KT - 4 * hf;
#pragma unroll
            for (int kt = 0; kt < 2; kt++)
#pragma unroll
                for (int v = 0; v < 16; v++) {
                    const float x = 32 * kt + 8 * (v >> 2) + (v & 3) < mine ? s[kt][v] : -INFINITY;
                    s[kt][v] = x;
                    mx = fmaxf(mx, x);
                }
        } else if (key0 + WA_KT - 1 > first_pos || (p.window && key0 < last_pos - p.window + 1)) { // some row does not see the whole tile
            const int age0 = pos - key0 - 4 * hf; // how far back this lane's first key is
            const unsigned ages = p.window ? (unsigned)p.window : 0x7fffffffu;
#pragma unroll
            for (int kt = 0; kt < 2; kt++)
#pragma unroll
                for (int v = 0; v < 16; v++) { // (a key ahead of the query wraps to a large age)
                    const float x = (unsigned)(age0 - (32 * kt + 8 * (v >> 2) + (v & 3))) < ages ? s[kt][v] : -INFINITY;
                    s[kt][v] = x;
                    mx = fmaxf(mx, x);
                }
        } else {
#pragma unroll
            for (int kt = 0; kt < 2; kt++)
#pragma unroll
                for (int v = 0; v < 16; v++) mx = fmaxf(mx, s[kt][v]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float m_new = fmaxf(m_run, mx * c2), m_use = m_new == -INFINITY ? 0.0f : m_new;
        const float alpha = __builtin_amdgcn_exp2f(m_run - m_use);
        const bool rescale = __any(m_new != m_run);
        m_run = m_new;
        float psum = 0.0f;
#pragma unroll
        for (int kt = 0; kt < 2; kt++)
#pragma unroll
            for (int v = 0; v < 16; v++) {
                const float e = __builtin_amdgcn_exp2f(__builtin_fmaf(s[kt][v], c2, -m_use));
                s[kt][v] = e;
                psum += e;
            }
        l_run = l_run * alpha + psum;
        if (rescale)
#pragma unroll
            for (int dt = 0; dt < C::DT; dt++)
#pragma unroll
                for (int v = 0; v < 16; v++) o[dt][v] *= alpha;
        asm volatile("" ::: "memory"); // the K tile has been read (LDS serves a wavefront in order): V takes its place
        store(rv, Vs, C::VS, C::SWZ);
        if (C::AHEAD && t + WA_WAVES < t_end) load(rv, vr, pvr, v_off, p.vdimp, t + WA_WAVES);
        // contraction step (kt, sp) uses the keys a lane holds in s[kt][8 sp .. 8 sp + 7]: key0 + 32 kt + 16 sp + {4 hf + 0..3, 8 + 4 hf + 0..3}
#pragma unroll
        for (int kt = 0; kt < 2; kt++)
#pragma unroll
            for (int sp = 0; sp < 2; sp++) {
                lm_u32x4 hi_bits, lo_bits; // two at a time: a packed conversion, its two halves back as f32, the remainders
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    const float2_t w = {s[kt][8 * sp + 2 * e], s[kt][8 * sp + 2 * e + 1]};
                    hi_bits[e] = __builtin_bit_cast(unsigned, __builtin_convertvector(w, bf16x2_t));
                    const unsigned pair = hi_bits[e];
                    const float2_t rest = {w[0] - __builtin_bit_cast(float, pair << 16), w[1] - __builtin_bit_cast(float, pair & 0xffff0000u)};
                    lo_bits[e] = __builtin_bit_cast(unsigned, __builtin_convertvector(rest, bf16x2_t));
                }
                const bf16x8_t hi = __builtin_bit_cast(bf16x8_t, hi_bits), lo = __builtin_bit_cast(bf16x8_t, lo_bits);
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

    // this thread's gate values for the merged result, requested before the merge
    const int q = tid & 31, row = row0 + q, d0 = (tid >> 5) * 8;
    const bf16_t *gate = p.gate ? reinterpret_cast<const bf16_t *>(p.gate) + size_t(min(row, p.n - 1)) * p.ldq + h * p.vdimp : nullptr;
    bf16x8_t gz = {};
    if (gate && d0 < p.vdimp) gz = *reinterpret_cast<const bf16x8_t *>(gate + d0);
    // merge the wavefronts' results; the sink is one more term of the denominator
    const float l_wave = l_run + __shfl_xor(l_run, 32);
    float *so = reinterpret_cast<float *>(wa_lds), *sm = reinterpret_cast<float *>(reinterpret_cast<char *>(wa_lds) + C::ML_OFFSET), *sl = sm + WA_WAVES * WA_Q;
    if (hf == 0) {
        sm[wave * WA_Q + col] = m_run;
        sl[wave * WA_Q + col] = l_wave;
    }
    __syncthreads(); // every wavefront is done with its staging area
    float m_all = sink;
#pragma unroll
    for (int w = 0; w < WA_WAVES; w++) m_all = fmaxf(m_all, sm[w * WA_Q + col]);
    const float f = m_run == -INFINITY ? 0.0f : __builtin_amdgcn_exp2f(m_run - m_all);
#pragma unroll
    for (int dt = 0; dt < C::DT; dt++)
#pragma unroll
        for (int j = 0; j < 4; j++) { // o[dt][4 j .. 4 j + 3] are elements 32 dt + 8 j + 4 hf .. + 3
            const float4 r = {o[dt][4 * j] * f, o[dt][4 * j + 1] * f, o[dt][4 * j + 2] * f, o[dt][4 * j + 3] * f};
            *reinterpret_cast<float4 *>(so + (wave * WA_Q + col) * C::SD + 32 * dt + 8 * j + 4 * hf) = r;
        }
    __syncthreads();
    if (row >= p.n) return;
    float l_all = p.sink ? __builtin_amdgcn_exp2f(sink - m_all) : 0.0f;
#pragma unroll
    for (int w = 0; w < WA_WAVES; w++) {
        const float mw = sm[w * WA_Q + q];
        if (mw != -INFINITY) l_all += __builtin_amdgcn_exp2f(mw - m_all) * sl[w * WA_Q + q];
    }
    const float inv = 1.0f / l_all;
    bf16_t *out = reinterpret_cast<bf16_t *>(p.out) + size_t(row) * p.ldo + h * p.vdimp;
    for (int d = d0; d < p.vdimp; d += 64) {
        float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < WA_WAVES; w++)
#pragma unroll
            for (int e = 0; e < 8; e++) acc[e] += so[(w * WA_Q + q) * C::SD + d + e];
#pragma unroll
        for (int e = 0; e < 8; e++) acc[e] *= inv;
        if (p.rotv) { // each element with the other one of its pair
            const int half = p.vdim / 2;
#pragma unroll
            for (int e = 0; e < 8; e++)
                if (d + e < 2 * half) {
                    const bool second = d + e >= half;
                    const int m = second ? d + e - half : d + e, other = second ? m : m + half;
                    const float2 cs = p.rotv[size_t(p.pos0 + row) * half + m];
                    float z = 0.0f;
#pragma unroll
                    for (int w = 0; w < WA_WAVES; w++) z += so[(w * WA_Q + q) * C::SD + other];
                    z *= inv;
                    acc[e] = second ? acc[e] * cs.x - z * cs.y : acc[e] * cs.x + z * cs.y;
                }
        }
        bf16x8_t r;
        if (gate && d != d0) gz = *reinterpret_cast<const bf16x8_t *>(gate + d);
#pragma unroll
        for (int e = 0; e < 8; e++) r[e] = (bf16_t)(acc[e] * (gate ? lm_sigmoid((float)gz[e]) : 1.0f));
        *reinterpret_cast<bf16x8_t *>(out + d) = r;
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
    const float scale = p.temp ? p.scale * p.temp[h] : p.scale;
    const int seen = p.pool ? blocks_seen(pos, p.window, p.pool) : 0; // the blocks come first, then the tokens from lo on
    const T *pk = reinterpret_cast<const T *>(p.pk) + size_t(g) * p.blocks * p.dimp, *pv = reinterpret_cast<const T *>(p.pv) + size_t(g) * p.blocks * p.vdimp;
    float m = p.sink ? p.sink[h] : -INFINITY, l = p.sink ? 1.0f : 0.0f;
    float o[ROW_MAX_D / 64];
#pragma unroll
    for (int i = 0; i < ROW_MAX_D / 64; i++) o[i] = 0.0f;
    const int total = seen + pos - lo + 1;
    for (int k0 = 0; k0 < total; k0 += 64) {
        const int key = k0 + lane, n_keys = min(64, total - k0);
        float s = -INFINITY;
        if (key < total) {
            const T *kr = key < seen ? pk + size_t(key) * p.dimp : ck + size_t((key - seen + lo) % p.cap) * p.dimp;
            s = 0.0f;
            for (int d = 0; d < p.dimp; d++) s = fmaf(s_q[wave][d], (float)kr[d], s);
            s *= scale;
        }
        const float m_new = fmaxf(m, wave_max(s)), alpha = expf(m - m_new), w = key < total ? expf(s - m_new) : 0.0f;
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
                for (int j = 0; j < n_keys; j++) {
                    const int at = k0 + j;
                    acc = fmaf(s_w[wave][j], (float)(at < seen ? pv + size_t(at) * p.vdimp : cv + size_t((at - seen + lo) % p.cap) * p.vdimp)[d], acc);
                }
            o[i] = acc;
        }
    }
#pragma unroll
    for (int i = 0; i < ROW_MAX_D / 64; i++)
        if (64 * i + lane < p.vdimp) s_q[wave][64 * i + lane] = o[i] / l; // (the query is not needed any more)
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    const int half = p.rotv ? p.vdim / 2 : 0;
    for (int d = lane; d < p.vdimp; d += 64) {
        float r = s_q[wave][d];
        if (d < 2 * half) {
            const int m = d < half ? d : d - half;
            const float2 cs = p.rotv[size_t(pos) * half + m];
            r = d < half ? r * cs.x + s_q[wave][d + half] * cs.y : r * cs.x - s_q[wave][m] * cs.y;
        }
        if (p.gate) r *= lm_sigmoid((float)reinterpret_cast<const T *>(p.gate)[size_t(row) * p.ldq + h * p.vdimp + d]);
        reinterpret_cast<T *>(p.out)[size_t(row) * p.ldo + h * p.vdimp + d] = (T)r;
    }
}

template <int P, bool POOL> int launch_mfma_as(moon_ctx *ctx, const WindowAttn &p) {
    using C = WaCfg<P>;
    static std::atomic<bool> attr_set[64]; // the opt-in to this much dynamic LDS is per device (and per instantiation)
    const int dev = ctx->device >= 0 && ctx->device < 64 ? ctx->device : -1;
    if (dev < 0 || !attr_set[dev].load()) {
        MOON_HIP(ctx, hipFuncSetAttribute(reinterpret_cast<const void *>(window_attn_kernel<P, POOL>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)C::LDS_BYTES));
        if (dev >= 0) attr_set[dev].store(true);
    }
    hipLaunchKernelGGL((window_attn_kernel<P, POOL>), dim3((unsigned)((p.n + WA_Q - 1) / WA_Q * p.H)), dim3(256), C::LDS_BYTES, ctx->stream, p);
    MOON_HIP(ctx, hipGetLastError());
    MOON_NOTE_KERNEL(ctx, "window_attn_kernel<%d>", P);
    return MOON_OK;
}
template <int P> int launch_mfma(moon_ctx *ctx, const WindowAttn &p) { return p.pool ? launch_mfma_as<P, true>(ctx, p) : launch_mfma_as<P, false>(ctx, p); }

} // namespace

int launch_window_attention(moon_ctx *ctx, int dtype, const WindowAttn &p) {
    if (p.n <= 0) return MOON_OK;
    if (p.H % p.G || p.dimp % 8 || p.vdimp % 8 || p.dimp > ROW_MAX_D || p.vdimp > ROW_MAX_D)
        return moon_fail(ctx, MOON_EINVAL_DIM, "window attention: %d heads over %d, head sizes %d and %d", p.H, p.G, p.dimp, p.vdimp);
    if ((p.window ? p.window - 1 + p.n : p.pos0 + p.n) > p.cap && p.pos0 + p.n > p.cap)
        return moon_fail(ctx, MOON_EINVAL_DIM, "window attention: %d rows behind a window of %d do not fit %d cache rows", p.n, p.window, p.cap);
    if (p.pool && (!p.window || (p.pos0 + p.n - p.window) / p.pool > p.blocks)) // (no block is seen before it is whole)
        return moon_fail(ctx, MOON_EINVAL_DIM, "window attention: blocks of %d before a window of %d, %d of them kept", p.pool, p.window, p.blocks);
    const int big = std::max(p.dimp, p.vdimp);
    if (dtype == MOON_DTYPE_BF16 && big <= 256 && size_t(std::max(p.cap, p.blocks)) * big * 2 < (size_t(1) << 30)) { // (32-bit offsets within a head's rows)
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
