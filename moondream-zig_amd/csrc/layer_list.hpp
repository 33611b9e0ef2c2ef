// Decoders that are described as a list of layers (a mixer and a feed-forward each) instead of one fixed block: the
// description, what one layer looks like on the device, and the launchers of the kernels the layers are made of.
// Every size below that a kernel walks is padded when the weights are packed: widths, projections and feed-forward sizes to
// multiples of 64, head sizes to multiples of 8, with zero weights, so no kernel has a tail in n or k.
#pragma once
#include <string>
#include <vector>

#include "moon_internal.hpp"

// ---- description (host)
struct MixerSpec { // softmax attention over a KV cache; the mechanisms are independent of each other
    size_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    size_t window = 0;      // position i sees j with i - j < window; 0: every j <= i
    float scale = 1.0f;     // on q . k
    bool qk_rms = false;    // q and k divided by their root mean square per head
    bool sink = false;      // a learned number per head in the softmax denominator
    bool gate = false;      // heads multiplied by sigmoid(W_g h)
    bool v_mix = false;     // v <- (1 - lambda) v + lambda v_first
    bool qk_whole_norm = false; // RMS norm with weights over all of q (of k) before the heads are split
    size_t rot_dims = 0;    // the first dimensions of each head of q and k turn with the position, pair (m, m + rot_dims / 2) ..
    double rot_base = 0.0, rot_factor = 1.0; // .. by position * base^(-2 m / rot_dims) / factor
    bool rot_values = false; // values turn too, over all vdim dimensions and without the factor, and each head's output turns back
    bool temp = false;      // a learned factor per head on the scale
    size_t pool = 0;        // before the window: one key and value per whole block of `pool` positions, their means
    int kv_from = -1;       // keys and values are those of this earlier layer's cache
};
// Gated delta rule: a state S [dim][vdim] per head, S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, with a decay g per key
// channel, q and k unit vectors, short convolutions over q, k and v, and an RMS norm and a gate on o.  heads = 0: none.
struct DeltaSpec {
    size_t heads = 0, kv_heads = 0, dim = 0, vdim = 0, conv = 0;
    size_t rank_a = 0, rank_g = 0; // inner sizes of the two-step projections of the decay and of the gate (the tensors' own)
};
struct FeedForwardSpec {
    enum Kind { NONE, DENSE, EXPERTS } kind = NONE;
    size_t ff = 0;               // of the dense layer or of one expert; gated: down(silu(gate h) * (up h))
    size_t experts = 0, top = 0; // sigmoid router: chosen by score + correction, weighted by the scores over their sum
};
struct LayerSpec {
    MixerSpec mixer;
    DeltaSpec delta; // beside the mixer: the result is half the sum of the two outputs, each RMS-normed over the width
    FeedForwardSpec ff;
};
struct LayerListSpec {
    std::string design; // registry name
    size_t vocab = 0, width = 0;
    float embed_scale = 1.0f, eps = 0.0f;
    bool rms_norm = false;         // RMS norms with a weight, otherwise LayerNorms with weight and bias
    float softcap = 0.0f;          // logits <- softcap tanh(logits / softcap); 0: none
    std::vector<LayerSpec> layers; // parallel layers: x += mixer(norm(x)) + ff(norm(x))
};

inline size_t pad_to(size_t n, size_t m) { return (n + m - 1) / m * m; }
constexpr float DELTA_UNIT_EPS = 1e-6f;     // added to the squared length of the delta rule's q and k
constexpr float EXPERT_WEIGHT_EPS = 1e-20f; // added to the sum of the chosen experts' scores

// ---- one layer on the device.  T is bf16_t or float; void pointers hold T.
struct LayerDev {
    LayerSpec spec;
    int dimp, vdimp;                 // padded head sizes
    int oq, ok, ov, og;              // columns of q, k, v and the gate in the first product (heads dimp / vdimp apart)
    int n16, n32, nall;              // segment ends of the first product: [q k v g) as T, [router logits) as f32, [gate/up pairs)
    int ffp, ka, k0;                 // padded ff; columns of the heads and of heads + dense activation in the second product
    void *w1 = nullptr;              // [nall][dp]
    void *w2 = nullptr;              // [dp][k0]: W_o beside a dense layer's W_down
    void *wgu = nullptr, *wd = nullptr; // experts: [E][2 ffp][dp] gate/up pairs, [E][dp][ffp]
    float *correction = nullptr, *gamma = nullptr, *beta = nullptr, *sink = nullptr;
    float lambda = 0.0f;
    bool mixes = false;              // takes v_first from the first mixing layer
    int cap = 0;                     // cache rows per head: position p lives in row p % cap
    void *ck = nullptr, *cv = nullptr; // [G][cap][dimp], [G][cap][vdimp]
    int blocks = 0;                  // rows of the pooled caches
    void *pk = nullptr, *pv = nullptr; // [G][blocks][dimp], [G][blocks][vdimp]
    float *qn = nullptr, *kn = nullptr; // weights of the norms over all of q and of k, laid out like q and k
    float *temp = nullptr;
    const float2 *rot = nullptr, *rotv = nullptr; // cosine and sine per position and pair: [max_seq][rot_dims / 2], [max_seq][vdim / 2]
    // gated delta rule.  Second product's columns: [heads ka | its heads kr | dense activation]
    int ddimp = 0, dvdimp = 0;       // padded to 16
    int oc = 0, channels = 0;        // its q, k, v columns in the first product start at oc: the channels of the convolutions
    int od = 0, kd = 0;              // columns of the two-step projections' inner vectors [a | g), padded to kd
    int lr16 = 0, lrn = 0;           // segment ends of their second product: [gate) as T, [decay) as f32
    int kr = 0;
    void *wlr = nullptr;             // [lrn][kd]
    float *conv = nullptr;           // [taps][channels]
    float *a_log = nullptr, *dt_bias = nullptr, *dnorm = nullptr; // [heads], [heads][ddimp], [dvdimp]
    float *out_l = nullptr, *out_r = nullptr; // [width]: norms of the two outputs
    float *state = nullptr;          // [heads][ddimp][dvdimp]; means nothing at position 0
    void *ring = nullptr;            // T [taps][channels]: the convolutions' inputs of position p lie in row p % taps
};

constexpr int SEG_MAX_SPLITS = 8;
// ---- products (seg_gemm.hip)
// C[M, N] = A[M, K] . W[N, K]^T, N a multiple of 64, K of 64.  The columns fall into up to three segments, each a multiple of 64
// wide: [0, n16) rounded to T into c16; [n16, n32) as f32 into c32; [n32, N) gate/up pairs (32 gate columns, then the 32 up
// columns that belong to them, and so on) as silu(gate) * up in T into glu, half as wide.
// Grouped (tile_group set): rows are runs of one group each, group g uses the weights at W + g * w_group; a row tile covers rows
// [tile_row[i], min(tile_row[i] + tile height, tile_end[i])) with the weights of group tile_group[i], n_tiles[0] tiles in all
// (at most max_tiles).
// rows: row m of A is rows[m] (otherwise m).
struct SegGemm {
    const void *A;
    int lda, a_rows;          // row pitch in elements, rows in the buffer
    const uint32_t *rows;
    const void *W;
    size_t w_group;           // elements between groups
    int M, N, K;
    int n16, n32;
    void *c16;
    float *c32;
    void *glu;
    int ld16, ld32, ldg;
    const int *tile_group, *tile_row, *tile_end, *n_tiles;
    int max_tiles;
    int splits;               // splits > 1: n16 = 0, n32 = N, slab s of c32 (M x ld32 apart) gets k-range s
    int kb[SEG_MAX_SPLITS + 1]; // k-range s is [kb[s], kb[s + 1]), multiples of 64; all zero: even ranges
    int last_first;           // the last k-range's tiles start first, on every die (where the last ranges are the long ones)
    float softcap;            // > 0: on the f32 segment
};
constexpr int SEG_TILE_ROWS = 128; // rows of a tile (both element types walk tile lists of this height)
int launch_seg_gemm(moon_ctx *ctx, int dtype, SegGemm p);
// k splits worth taking for an all-f32 product of this shape
int seg_gemm_splits(moon_ctx *ctx, size_t M, size_t N, size_t K);

// ---- row kernels (layer_rows.hip)
// x[n] = embed[ids[n]] * scale (embed != null), or x += the k splits of a product + the chosen experts' weighted rows; then the
// LayerNorm of x into h (T, dp wide, if h != null).  One workgroup per row.
struct RowFinish {
    float *x;                 // [n][width]
    const void *embed;        // T [vocab][dp]
    const uint32_t *ids;
    float embed_scale;
    const float *partial;     // [splits][n][dp]
    int splits;
    const void *expert_out;   // T [n * top][dp], rows in the order of `slot`
    const int *slot;          // [n][top]
    const float *weight;      // [n][top]
    int top;
    const float *gamma, *beta; // beta null: RMS norm
    float eps;
    void *h;
    int n, width, dp;
    const uint32_t *rows;     // rows != null: read x row rows[i], write h row i, x itself stays as it is
    const float *out_l, *out_r; // set: the first splits_l splits are one output, the next splits_r another, and half the sum of the two,
    int splits_l, splits_r;   // each RMS-normed with its weights, enters x beside the other splits
};
int launch_row_finish(moon_ctx *ctx, int dtype, const RowFinish &p);

// q and k normalised, v mixed, k and v into the cache rows of positions pos0 .. pos0 + n - 1; q stays in c1.
struct PrepArgs {
    void *c1;                 // T [n][n16]
    int ld, n, pos0;
    int H, G, dim, vdim, dimp, vdimp, oq, ok, ov;
    int qk_rms, mixes, cap, cap_first;
    float eps, lambda;
    void *ck, *cv;
    const void *v_first;      // the first mixing layer's value cache
};
int launch_prep_qkv(moon_ctx *ctx, int dtype, const PrepArgs &p);

// The same for a mixer whose q and k are normed as a whole: norm, rotation, cache rows.  One workgroup per row.
struct PrepWhole {
    void *c1;                 // T [n][ld]
    int ld, n, pos0;
    int H, G, dim, vdim, dimp, vdimp, oq, ok, ov; // G = 0: only q
    int cap, rot_dims;
    float eps;
    const float *qn, *kn;
    const float2 *rot, *rotv; // null: none
    void *ck, *cv;
};
int launch_prep_whole(moon_ctx *ctx, int dtype, const PrepWhole &p);

// Means of the cache rows of every block of `pool` positions that ends in [pos0, pos0 + n).
struct PoolArgs {
    const void *ck, *cv;
    void *pk, *pv;
    int G, dimp, vdimp, cap, blocks, pool, pos0, n;
};
int launch_pool(moon_ctx *ctx, int dtype, const PoolArgs &p);

// cos and sin of position * base^(-2 m / dims) / factor -> table [positions][dims / 2]
int launch_rotation_table(moon_ctx *ctx, float2 *table, size_t positions, size_t dims, double base, double factor);

// ---- gated delta rule over several rows (delta_rows.hip)
struct DeltaRows {
    const void *c1;           // T [n][ld]: the first product; the channels start at column oc
    int ld, oc, channels, taps;
    const float *beta;        // [n][ldb], before the sigmoid
    int ldb;
    const float *dt;          // [n][lddt]: the decay's projection, (row, head, channel) at head * dimp + channel
    int lddt;
    const void *gate;         // T [n][ldg]
    int ldg;
    int n, pos0, H, G, dim, vdim, dimp, vdimp;
    const float *conv, *a_log, *dt_bias, *norm;
    float eps;
    float *scratch;           // delta_scratch_floats
    float *o;                 // [n][H * vdimp]
    float *state;
    void *ring;
    void *out;                // T, (row, head, d) at row * ldo + head * vdimp + d
    int ldo;
};
size_t delta_scratch_floats(size_t rows, size_t heads, size_t dimp, size_t vdimp);
int launch_delta_rows(moon_ctx *ctx, int dtype, const DeltaRows &p);
constexpr size_t DELTA_MAX_DIM = 512; // head sizes

// Router logits -> chosen experts and weights per row, then the rows of every expert side by side.
struct RouteArgs {
    const float *logits;      // [n][ld]
    const float *correction;
    int n, ld, E, top, rows_per_tile;
    int *ids;                 // [n][top]
    float *weight;            // [n][top]
    int *slot;                // [n][top]: row of the pair (token, choice) in the grouped order
    uint32_t *rows;           // [n * top]: token of a grouped row
    int *tile_group, *tile_row, *tile_end, *n_tiles; // row tiles of the grouped products
};
int launch_route(moon_ctx *ctx, const RouteArgs &p);

// ---- attention over several query rows (attn_window.hip): causal, windowed, grouped heads, sink, output gate
struct WindowAttn {
    const void *q;            // T, element (row, head, d) at row * ldq + head * dimp + d
    const void *gate;         // T, (row, head, d) at row * ldq + head * vdimp + d; may be null
    int ldq;
    const void *ck, *cv;
    int cap;
    void *out;                // T, (row, head, d) at row * ldo + head * vdimp + d
    int ldo;
    int n, pos0, H, G, dimp, vdimp, window;
    float scale;
    const float *sink;        // [H] or null
    const float *temp;        // [H] or null: factors on the scale
    int pool, blocks;         // pool > 0: beside the window, blocks of `pool` positions wholly before it
    const void *pk, *pv;
    const float2 *rotv;       // set: the outputs turn back, over the first vdim dimensions
    int vdim;
};
int launch_window_attention(moon_ctx *ctx, int dtype, const WindowAttn &p);

// ---- one token (layer_decode.hip): three launches per layer
struct DecodeProj {           // h = LayerNorm(x); the first product
    float *x;
    const uint32_t *token;    // set: x = embed[token] * scale, also written to x
    const void *embed;
    float embed_scale;
    const float *gamma, *beta; // beta null: RMS norm
    float eps;
    int width, dp;
    // set: x is first brought up to date with a joined layer's results y (DecodeOut), as in RowFinish, and written to x_new
    const float *y, *out_l, *out_r;
    float *x_new;
    float softcap;            // > 0: on the f32 segment
    const void *w1;
    int n16, n32, nall, ff;   // segments as in SegGemm; ff: gate/up pairs that are not padding
    int n16_used, n32_used;   // rows of the first two segments that are not padding (n32_used counts from n16)
    float *proj;              // [n16]
    float *logits;            // [n32 - n16]
    void *glu;                // T [ff]
    void *h;                  // T [dp] or null
};
int launch_decode_proj(moon_ctx *ctx, int dtype, const DecodeProj &p);

struct DecodeMix {            // attention of the token (and its cache update) beside the chosen experts' first product
    const float *proj;
    int H, G, dim, vdim, dimp, vdimp, ok, ov, og;
    int qk_rms, gate, mixes, window, cap, cap_first;
    float eps, lambda, scale;
    const float *sink;
    void *ck, *cv;
    const void *v_first;
    size_t pos;
    const uint32_t *pos_dev;
    float *partial;           // decode_mix_partial_floats
    size_t partial_floats;
    uint32_t *counter;        // [G * head blocks], zero between launches
    void *out;                // T [H][vdimp]
    // experts (E = 0: none)
    const float *logits, *correction;
    int E, top, ff, ffp, dp;
    const void *h, *wgu;
    void *act;                // T [top][ffp]
    int *ids;
    float *weight;            // [top]
    // norm over all of q and k, rotation, pooled blocks, borrowed keys and values
    int whole, rot_dims, pool, blocks, borrowed;
    const float *qn, *kn, *temp;
    const float2 *rot, *rotv;
    void *pk, *pv;
    // a gated delta rule beside the attention (dH = 0: none)
    int dH, dG, ddim, dvdim, ddimp, dvdimp, taps, oc, channels, od, rank_a, rank_g, kd, lr16;
    const float *beta;        // [dH], before the sigmoid
    const float *conv, *a_log, *dt_bias, *dnorm;
    const void *wlr;
    float *state;
    void *ring;
    void *dout;               // T [dH][dvdimp]
};
size_t decode_mix_partial_floats(moon_ctx *ctx, size_t heads, size_t kv_heads, size_t vdimp, size_t max_keys);
size_t decode_mix_counters(size_t heads, size_t kv_heads);
int launch_decode_mix(moon_ctx *ctx, int dtype, const DecodeMix &p);

struct DecodeOut {            // x += W2 . a + the chosen experts' weighted second product
    float *x;
    float *y;                 // set: x stays as it is, and the products over a's columns [0, k1), [k1, k2), [k2, k0) go to y [3][dp]
    int k1, k2;
    int width, dp, k0;
    const void *w2, *a;
    int top, ffp;
    const void *wd, *act;
    const int *ids;
    const float *weight;
};
int launch_decode_out(moon_ctx *ctx, int dtype, const DecodeOut &p);

// ---- the engine (layer_list.hip): weights, caches and buffers of one sequence's session, prompt rows and single tokens
struct LayerList;
struct Design;
struct SafeTensors;
constexpr size_t LIST_MAX_ROWS = 2048; // rows of one call of layer_list_forward
constexpr size_t LIST_LOGIT_ROWS = 256; // rows of one call of layer_list_logits
// weights from a file under the design's tensor names, or (file null) random: matrices ~N(0, std), norms 1 and 0, sinks,
// corrections 0, lambda 1/2; random weights need every size to be a multiple of 64 (head sizes: of 8)
int layer_list_create(moon_ctx *ctx, const LayerListSpec &spec, const Design *design, const SafeTensors *file, uint64_t seed, float std_dev, int dtype,
                      size_t max_seq, LayerList **out);
void layer_list_destroy(LayerList *l);
size_t layer_list_rows(const LayerList *l); // rows one forward call takes
// n rows at positions pos .. pos + n - 1 (the cache holds everything before); x is left in rows 0 .. n - 1
int layer_list_forward(LayerList *l, const uint32_t *ids_dev, size_t n, size_t pos);
// one token with the decode kernels; pos_dev: the position is read on the device, pos is the largest it can be
int layer_list_step(LayerList *l, const uint32_t *token_dev, size_t pos, const uint32_t *pos_dev);
// logits of the given rows of x (host list of n <= LIST_LOGIT_ROWS) -> *logits, [n][*ld] f32 on the device
int layer_list_logits(LayerList *l, const uint32_t *rows, size_t n, const float **logits, size_t *ld);
const float *layer_list_hidden(const LayerList *l); // [rows][width] on the device
size_t layer_list_weight_bytes(const LayerList *l); // read per decoded token
