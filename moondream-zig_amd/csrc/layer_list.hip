// Engine of the layer-list decoders: packs a model's weights for the kernels, owns the caches (a ring of rows per layer as long as
// its window and one call's rows together, or the whole sequence), the pooled blocks, the recurrent states and the activations, and
// runs prompts and single tokens.
#include "layer_list.hpp"

#include <algorithm>
#include <cstring>
#include <vector>

#include "model_folder.hpp"

struct LayerList {
    moon_ctx *ctx = nullptr;
    LayerListSpec spec;
    int dtype = MOON_DTYPE_BF16;
    size_t el = 2, max_rows = 0, max_seq = 0, dp = 0, vp = 0;
    std::vector<LayerDev> layers;
    int first_mix = -1;
    void *embed = nullptr, *head = nullptr;
    float *fgamma = nullptr, *fbeta = nullptr;
    float *x = nullptr, *router = nullptr, *partial = nullptr, *proj = nullptr, *logits = nullptr, *mix_partial = nullptr, *weight = nullptr;
    void *h = nullptr, *c1 = nullptr, *a2 = nullptr, *act = nullptr, *y = nullptr;
    int *ids = nullptr, *slot = nullptr, *tile_group = nullptr, *tile_row = nullptr, *tile_end = nullptr, *n_tiles = nullptr;
    uint32_t *grouped_rows = nullptr, *counter = nullptr, *want = nullptr;
    uint32_t *want_pinned = nullptr;
    size_t mix_partial_floats = 0;
    float *x1 = nullptr, *y3 = nullptr;                    // one token: the other copy of x, the parts of a joined layer's second product
    float *dt = nullptr, *delta_o = nullptr, *scratch = nullptr; // delta rule's rows: decays, outputs, chunks
    void *dgate = nullptr;
    struct Table {
        size_t dims;
        double base, factor;
        float2 *at;
    };
    std::vector<Table> tables;
    std::vector<void *> allocs;
};

namespace {

int alloc_bytes(LayerList *l, size_t bytes, void **p) {
    bytes = pad_to(bytes ? bytes : 16, 16);
    MOON_HIP(l->ctx, hipMalloc(p, bytes));
    l->allocs.push_back(*p);
    return launch_fill_uniform_u32(l->ctx, (uint32_t *)*p, bytes / 4, 0, 0, 1); // zeros: padding is multiplied by zero weights, so it must be finite
}
template <class P> int alloc_n(LayerList *l, size_t n, P **p) { return alloc_bytes(l, n * sizeof(P), (void **)p); }
int alloc_t(LayerList *l, size_t n, void **p) { return alloc_bytes(l, n * l->el, p); }

float read_element(const StTensor &t, size_t i) {
    uint32_t bits;
    if (t.dtype == "BF16") {
        uint16_t b;
        memcpy(&b, t.data + 2 * i, 2);
        bits = (uint32_t)b << 16;
    } else memcpy(&bits, t.data + 4 * i, 4);
    float f;
    memcpy(&f, &bits, 4);
    return f;
}
uint16_t to_bf16(float f) {
    uint32_t u;
    memcpy(&u, &f, 4);
    if ((u & 0x7fffffff) > 0x7f800000) return (uint16_t)(u >> 16 | 0x40);
    return (uint16_t)((u + 0x7fff + (u >> 16 & 1)) >> 16);
}

// Packs and uploads the weights of one model.
struct Loader {
    LayerList *l;
    const Design *design;
    const SafeTensors *file;
    uint64_t seed, stream = 0;
    float std_dev;
    std::vector<unsigned char> host; // the matrix being packed

    // (read_model_folder has checked every tensor of the description)
    int get(const std::string &name, size_t elements, const StTensor **t) {
        *t = file->find(name);
        if (!*t || (*t)->bytes != elements * ((*t)->dtype == "BF16" ? 2 : 4)) return moon_fail(l->ctx, MOON_EFORMAT, "tensor '%s'", name.c_str());
        return MOON_OK;
    }
    void begin(size_t rows, size_t cols) {
        if (file) host.assign(rows * cols * l->el, 0);
    }
    // tensor `name` [rows][cols]: row r goes to row place(r) of the matrix being packed, columns in blocks of `block` (0: all) that
    // lie `pitch` apart from column col0 on
    template <class Place>
    int put(const std::string &name, size_t rows, size_t cols, size_t ld, Place place, size_t col0 = 0, size_t block = 0, size_t pitch = 0) {
        if (!file) return MOON_OK;
        const StTensor *t;
        MOON_TRY(get(name, rows * cols, &t));
        if (!block) block = cols;
        for (size_t r = 0; r < rows; r++)
            for (size_t b = 0; b < cols; b += block) {
                const size_t src = r * cols + b, dst = place(r) * ld + col0 + b / block * pitch, n = std::min(block, cols - b);
                if (l->dtype == MOON_DTYPE_BF16 && t->dtype == "BF16") memcpy(host.data() + 2 * dst, t->data + 2 * src, 2 * n);
                else
                    for (size_t i = 0; i < n; i++) {
                        const float f = read_element(*t, src + i);
                        if (l->dtype == MOON_DTYPE_F32) memcpy(host.data() + 4 * (dst + i), &f, 4);
                        else {
                            const uint16_t v = to_bf16(f);
                            memcpy(host.data() + 2 * (dst + i), &v, 2);
                        }
                    }
            }
        return MOON_OK;
    }
    // the packed matrix -> dst (or random values)
    int end(void *dst, size_t n) {
        if (!file) return launch_fill_normal_t(l->ctx, l->dtype, dst, n, seed, stream++, std_dev);
        MOON_HIP(l->ctx, hipMemcpyAsync(dst, host.data(), n * l->el, hipMemcpyHostToDevice, l->ctx->stream));
        MOON_HIP(l->ctx, hipStreamSynchronize(l->ctx->stream)); // the staging vector is used again
        return MOON_OK;
    }
    // a vector kept in f32
    int vec(const std::string &name, size_t n, float fallback, float **dst) {
        return vec_at(name, n, fallback, n, [](size_t i) { return i; }, dst);
    }
    // the same with element i at place(i) of `padded` elements, the others zero
    template <class Place> int vec_at(const std::string &name, size_t n, float fallback, size_t padded, Place place, float **dst) {
        std::vector<float> v(padded, 0.0f);
        const StTensor *t = nullptr;
        if (file) MOON_TRY(get(name, n, &t));
        for (size_t i = 0; i < n; i++) v[place(i)] = t ? read_element(*t, i) : fallback;
        MOON_TRY(alloc_n(l, padded, dst));
        MOON_HIP(l->ctx, hipMemcpyAsync(*dst, v.data(), padded * sizeof(float), hipMemcpyHostToDevice, l->ctx->stream));
        MOON_HIP(l->ctx, hipStreamSynchronize(l->ctx->stream));
        return MOON_OK;
    }
    int scalar(const std::string &name, float *dst) {
        *dst = 0.5f;
        if (!file) return MOON_OK;
        const StTensor *t;
        MOON_TRY(get(name, 1, &t));
        *dst = read_element(*t, 0);
        return MOON_OK;
    }
};

int rotation_table(LayerList *l, size_t dims, double base, double factor, const float2 **table) {
    for (const LayerList::Table &t : l->tables)
        if (t.dims == dims && t.base == base && t.factor == factor) {
            *table = t.at;
            return MOON_OK;
        }
    LayerList::Table t{dims, base, factor, nullptr};
    MOON_TRY(alloc_n(l, l->max_seq * (dims / 2), &t.at));
    MOON_TRY(launch_rotation_table(l->ctx, t.at, l->max_seq, dims, base, factor));
    l->tables.push_back(t);
    *table = t.at;
    return MOON_OK;
}

size_t pair_row_host(size_t i, size_t half) { return i / 32 * 64 + half * 32 + i % 32; } // gate/up pairs: 32 gate rows, their 32 up rows, ...

int load_layer(Loader &ld, size_t i) {
    LayerList *l = ld.l;
    LayerDev &d = l->layers[i];
    const MixerSpec &mx = d.spec.mixer;
    const FeedForwardSpec &ff = d.spec.ff;
    const size_t w = l->spec.width, dp = l->dp, H = mx.heads, G = mx.kv_heads;
    const DeltaSpec &de = d.spec.delta;
    auto mix = [&](const std::string &what) { return ld.file ? ld.design->names.mixer(i, ((de.heads ? ld.design->names.attention_part : "") + what).c_str()) : what; };
    auto del = [&](const std::string &what) { return ld.file ? ld.design->names.mixer(i, (ld.design->names.delta_part + what).c_str()) : what; };
    auto mlp = [&](const char *what) { return ld.file ? ld.design->names.ff(i, what) : std::string(); };
    auto heads = [](size_t base, size_t n, size_t padded) { return [=](size_t r) { return base + r / n * padded + r % n; }; };
    const std::string norm = ld.file ? ld.design->names.norm(i) : std::string();
    MOON_TRY(ld.vec(norm, w, 1.0f, &d.gamma));
    if (!l->spec.rms_norm) MOON_TRY(ld.vec(ld.file ? norm + ld.design->names.bias_suffix : norm, w, 0.0f, &d.beta));
    const bool own = mx.kv_from < 0;
    if (mx.qk_whole_norm) {
        MOON_TRY(ld.vec_at(mix("q.norm"), H * mx.dim, 1.0f, H * d.dimp, heads(0, mx.dim, d.dimp), &d.qn));
        if (own) MOON_TRY(ld.vec_at(mix("k.norm"), G * mx.dim, 1.0f, G * d.dimp, heads(0, mx.dim, d.dimp), &d.kn));
    }
    if (mx.temp) MOON_TRY(ld.vec(mix("temp"), H, 1.0f, &d.temp));
    if (mx.rot_dims) MOON_TRY(rotation_table(l, mx.rot_dims, mx.rot_base, mx.rot_factor, &d.rot));
    if (mx.rot_values) MOON_TRY(rotation_table(l, mx.vdim, mx.rot_base, 1.0, &d.rotv));
    if (mx.sink) MOON_TRY(ld.vec(mix("sink"), H, 0.0f, &d.sink));
    if (d.mixes) MOON_TRY(ld.scalar(mix("vmix"), &d.lambda));

    MOON_TRY(alloc_t(l, size_t(d.nall) * dp, &d.w1));
    ld.begin(d.nall, dp);
    MOON_TRY(ld.put(mix("q"), H * mx.dim, w, dp, heads(d.oq, mx.dim, d.dimp)));
    if (own) {
        MOON_TRY(ld.put(mix("k"), G * mx.dim, w, dp, heads(d.ok, mx.dim, d.dimp)));
        MOON_TRY(ld.put(mix("v"), G * mx.vdim, w, dp, heads(d.ov, mx.vdim, d.vdimp)));
    }
    if (mx.gate) MOON_TRY(ld.put(mix("g"), H * mx.vdim, w, dp, heads(d.og, mx.vdim, d.vdimp)));
    const size_t dq = de.kv_heads * de.dim, dv = de.heads * de.vdim, first_k = de.kv_heads * d.ddimp, first_v = 2 * first_k;
    if (de.heads) {
        MOON_TRY(ld.put(del("q"), dq, w, dp, heads(d.oc, de.dim, d.ddimp)));
        MOON_TRY(ld.put(del("k"), dq, w, dp, heads(d.oc + first_k, de.dim, d.ddimp)));
        MOON_TRY(ld.put(del("v"), dv, w, dp, heads(d.oc + first_v, de.vdim, d.dvdimp)));
        MOON_TRY(ld.put(del("a1"), de.rank_a, w, dp, [&](size_t r) { return d.od + r; }));
        MOON_TRY(ld.put(del("g1"), de.rank_g, w, dp, [&](size_t r) { return d.od + de.rank_a + r; }));
        MOON_TRY(ld.put(del("b"), de.heads, w, dp, [&](size_t r) { return d.n16 + r; }));
    }
    if (ff.kind == FeedForwardSpec::EXPERTS) MOON_TRY(ld.put(mlp("router"), ff.experts, w, dp, [&](size_t r) { return d.n16 + r; }));
    if (ff.kind == FeedForwardSpec::DENSE) {
        MOON_TRY(ld.put(mlp("gate"), ff.ff, w, dp, [&](size_t r) { return d.n32 + pair_row_host(r, 0); }));
        MOON_TRY(ld.put(mlp("up"), ff.ff, w, dp, [&](size_t r) { return d.n32 + pair_row_host(r, 1); }));
    }
    MOON_TRY(ld.end(d.w1, size_t(d.nall) * dp));

    MOON_TRY(alloc_t(l, dp * d.k0, &d.w2));
    ld.begin(dp, d.k0);
    auto same = [](size_t r) { return r; };
    MOON_TRY(ld.put(mix("o"), w, H * mx.vdim, d.k0, same, 0, mx.vdim, d.vdimp));
    if (ff.kind == FeedForwardSpec::DENSE) MOON_TRY(ld.put(mlp("down"), w, ff.ff, d.k0, same, d.ka + d.kr));
    if (de.heads) MOON_TRY(ld.put(del("o"), w, dv, d.k0, same, d.ka, de.vdim, d.dvdimp));
    MOON_TRY(ld.end(d.w2, dp * d.k0));

    if (de.heads) {
        const size_t taps = de.conv, n_lr = size_t(d.lrn) * d.kd;
        MOON_TRY(alloc_t(l, n_lr, &d.wlr));
        ld.begin(d.lrn, d.kd);
        MOON_TRY(ld.put(del("g2"), dv, de.rank_g, d.kd, heads(0, de.vdim, d.dvdimp), de.rank_a));
        MOON_TRY(ld.put(del("a2"), de.heads * de.dim, de.rank_a, d.kd, heads(d.lr16, de.dim, d.ddimp)));
        if (!ld.file) { // random, but each step's rows have the other one's columns zero
            MOON_TRY(ld.end(d.wlr, n_lr));
            ld.host.resize(n_lr * l->el);
            MOON_HIP(l->ctx, hipMemcpyAsync(ld.host.data(), d.wlr, n_lr * l->el, hipMemcpyDeviceToHost, l->ctx->stream));
            MOON_HIP(l->ctx, hipStreamSynchronize(l->ctx->stream));
            for (size_t r = 0; r < size_t(d.lrn); r++)
                for (size_t k = 0; k < size_t(d.kd); k++)
                    if ((k < de.rank_a) != (r >= size_t(d.lr16)) || k >= de.rank_a + de.rank_g) memset(ld.host.data() + (r * d.kd + k) * l->el, 0, l->el);
            MOON_HIP(l->ctx, hipMemcpyAsync(d.wlr, ld.host.data(), n_lr * l->el, hipMemcpyHostToDevice, l->ctx->stream));
            MOON_HIP(l->ctx, hipStreamSynchronize(l->ctx->stream));
        } else MOON_TRY(ld.end(d.wlr, n_lr));
        std::vector<float> conv(taps * d.channels, 0.0f);
        auto taps_of = [&](const char *what, size_t rows, size_t first, size_t size, size_t padded) -> int {
            const StTensor *t = nullptr;
            if (ld.file) MOON_TRY(ld.get(del(what), rows * taps, &t));
            for (size_t r = 0; r < rows; r++)
                for (size_t k = 0; k < taps; k++) conv[k * d.channels + first + r / size * padded + r % size] = t ? read_element(*t, r * taps + k) : 0.5f;
            return MOON_OK;
        };
        MOON_TRY(taps_of("q.conv", dq, 0, de.dim, d.ddimp));
        MOON_TRY(taps_of("k.conv", dq, first_k, de.dim, d.ddimp));
        MOON_TRY(taps_of("v.conv", dv, first_v, de.vdim, d.dvdimp));
        MOON_TRY(alloc_n(l, conv.size(), &d.conv));
        MOON_HIP(l->ctx, hipMemcpyAsync(d.conv, conv.data(), conv.size() * sizeof(float), hipMemcpyHostToDevice, l->ctx->stream));
        MOON_HIP(l->ctx, hipStreamSynchronize(l->ctx->stream));
        MOON_TRY(ld.vec(del("A_log"), de.heads, 0.0f, &d.a_log));
        MOON_TRY(ld.vec_at(del("dt_bias"), de.heads * de.dim, -2.0f, de.heads * d.ddimp, heads(0, de.dim, d.ddimp), &d.dt_bias));
        MOON_TRY(ld.vec_at(del("norm"), de.vdim, 1.0f, d.dvdimp, same, &d.dnorm));
        MOON_TRY(ld.vec(mix("out"), w, 1.0f, &d.out_l));
        MOON_TRY(ld.vec(del("out"), w, 1.0f, &d.out_r));
        MOON_TRY(alloc_n(l, de.heads * d.ddimp * d.dvdimp, &d.state));
        MOON_TRY(alloc_t(l, taps * d.channels, &d.ring));
    }

    if (ff.kind == FeedForwardSpec::EXPERTS) {
        MOON_TRY(ld.vec(mlp("correction"), ff.experts, 0.0f, &d.correction));
        const size_t gu = size_t(2) * d.ffp * dp, dn = dp * d.ffp;
        MOON_TRY(alloc_t(l, ff.experts * gu, &d.wgu));
        MOON_TRY(alloc_t(l, ff.experts * dn, &d.wd));
        for (size_t e = 0; e < ff.experts; e++) {
            auto ex = [&](const char *what) { return ld.file ? ld.design->names.expert(i, e, what) : std::string(); };
            ld.begin(2 * d.ffp, dp);
            MOON_TRY(ld.put(ex("gate"), ff.ff, w, dp, [&](size_t r) { return pair_row_host(r, 0); }));
            MOON_TRY(ld.put(ex("up"), ff.ff, w, dp, [&](size_t r) { return pair_row_host(r, 1); }));
            MOON_TRY(ld.end((char *)d.wgu + e * gu * l->el, gu));
            ld.begin(dp, d.ffp);
            MOON_TRY(ld.put(ex("down"), w, ff.ff, d.ffp, same));
            MOON_TRY(ld.end((char *)d.wd + e * dn * l->el, dn));
        }
    }
    if (!own) { // (the layer it borrows from keeps rows enough for both windows)
        const LayerDev &src = l->layers[mx.kv_from];
        d.cap = src.cap;
        d.ck = src.ck;
        d.cv = src.cv;
        d.blocks = src.blocks;
        d.pk = src.pk;
        d.pv = src.pv;
        return MOON_OK;
    }
    MOON_TRY(alloc_t(l, G * size_t(d.cap) * d.dimp, &d.ck));
    MOON_TRY(alloc_t(l, G * size_t(d.cap) * d.vdimp, &d.cv));
    if (!mx.pool) return MOON_OK;
    MOON_TRY(alloc_t(l, G * size_t(d.blocks) * d.dimp, &d.pk));
    return alloc_t(l, G * size_t(d.blocks) * d.vdimp, &d.pv);
}

int create(LayerList *l, const Design *design, const SafeTensors *file, uint64_t seed, float std_dev) {
    moon_ctx *ctx = l->ctx;
    const size_t cus = ctx->cu_count > 0 ? ctx->cu_count : 256;
    l->dp = pad_to(l->spec.width, 64);
    l->vp = pad_to(l->spec.vocab, 64);
    l->max_rows = std::min(l->max_seq, LIST_MAX_ROWS);
    size_t n16 = 64, nr = 64, k0 = 64, act = 16, y = 16, pairs = 16, tiles = 16, counters = 1;
    size_t dgate = 0, dt = 0, delta_o = 0, scratch = 0, parts = 1;
    std::vector<size_t> reach; // rows before a call's first one that a layer's cache keeps: its own window's or block's, or a borrower's
    for (size_t i = 0; i < l->spec.layers.size(); i++) {
        const MixerSpec &mx = l->spec.layers[i].mixer;
        const size_t r = mx.window ? std::max(mx.window, mx.pool) - 1 : l->max_seq;
        reach.push_back(r);
        if (mx.kv_from >= 0) reach[mx.kv_from] = std::max(reach[mx.kv_from], r);
    }
    for (size_t i = 0; i < l->spec.layers.size(); i++) {
        LayerDev d;
        d.spec = l->spec.layers[i];
        const MixerSpec &mx = d.spec.mixer;
        const FeedForwardSpec &ff = d.spec.ff;
        DeltaSpec &de = d.spec.delta;
        if (!file) {
            if (de.heads && !de.rank_a) de.rank_a = de.rank_g = de.vdim;
            if (l->spec.width % 64 || mx.dim % 8 || mx.vdim % 8 ||
                (mx.heads * mx.dim + (mx.kv_from < 0 ? mx.kv_heads * (mx.dim + mx.vdim) : 0) + (mx.gate ? mx.heads * mx.vdim : 0)) % 64 ||
                (mx.heads * mx.vdim) % 64 || ff.ff % 64 || ff.experts % 64 || de.dim % 16 || de.vdim % 16 ||
                (2 * de.kv_heads * de.dim + de.heads * de.vdim) % 64 || (de.heads * de.vdim) % 64 || (de.rank_a + de.rank_g) % 64)
                return moon_fail(ctx, MOON_EINVAL_DIM, "random weights: layer %zu has a size that would be padded", i);
        }
        if (mx.dim > 1024 || mx.vdim > 1024 || mx.heads > 4096) return moon_fail(ctx, MOON_EINVAL_DIM, "layer %zu: head size above 1024", i);
        d.dimp = (int)pad_to(mx.dim, 8);
        d.vdimp = (int)pad_to(mx.vdim, 8);
        if (de.heads && (de.dim > DELTA_MAX_DIM || de.vdim > DELTA_MAX_DIM || de.heads > 4096 || de.conv > 4096))
            return moon_fail(ctx, MOON_EINVAL_DIM, "layer %zu: delta rule with head sizes above %zu", i, DELTA_MAX_DIM);
        if (de.heads && ff.kind == FeedForwardSpec::EXPERTS) return moon_fail(ctx, MOON_EINVAL_DIM, "layer %zu: experts beside a delta rule", i);
        const size_t own = mx.kv_from < 0 ? mx.kv_heads : 0; // heads whose keys and values are this layer's own
        const size_t q = mx.heads * d.dimp, k = own * d.dimp, v = own * d.vdimp, o = mx.heads * d.vdimp;
        d.oq = 0;
        d.ok = (int)q;
        d.ov = (int)(q + k);
        d.og = (int)(q + k + v);
        d.n16 = (int)pad_to(q + k + v + (mx.gate ? o : 0), 64);
        if (de.heads) {
            d.ddimp = (int)pad_to(de.dim, 16);
            d.dvdimp = (int)pad_to(de.vdim, 16);
            d.oc = d.n16;
            d.channels = (int)(2 * de.kv_heads * d.ddimp + de.heads * d.dvdimp);
            d.od = (int)pad_to(d.oc + d.channels, 64);
            d.kd = (int)pad_to(de.rank_a + de.rank_g, 64);
            d.n16 = d.od + d.kd;
            d.kr = (int)pad_to(de.heads * d.dvdimp, 64);
            d.lr16 = d.kr;
            d.lrn = d.lr16 + (int)pad_to(de.heads * d.ddimp, 64);
            dgate = std::max(dgate, l->max_rows * d.lr16);
            dt = std::max(dt, l->max_rows * (d.lrn - d.lr16));
            delta_o = std::max(delta_o, l->max_rows * de.heads * d.dvdimp);
            scratch = std::max(scratch, delta_scratch_floats(l->max_rows, de.heads, d.ddimp, d.dvdimp));
            parts = 3;
        }
        d.n32 = d.n16 + (int)pad_to(de.heads ? de.heads : ff.experts, 64);
        d.ffp = (int)pad_to(ff.ff, 64);
        const bool dense = ff.kind == FeedForwardSpec::DENSE;
        d.nall = d.n32 + (dense ? 2 * d.ffp : 0);
        d.ka = (int)pad_to(o, 64);
        d.k0 = d.ka + d.kr + (dense ? d.ffp : 0);
        // (before any row of a call is attended all of them are in the cache: behind the first row's window there must be room for the rest)
        d.cap = (int)std::min(l->max_seq, reach[i] + l->max_rows);
        d.blocks = mx.pool ? (int)(l->max_seq / mx.pool) : 0;
        if (mx.v_mix) {
            if (l->first_mix < 0) l->first_mix = (int)i;
            else {
                const MixerSpec &f = l->spec.layers[l->first_mix].mixer;
                if (f.kv_heads != mx.kv_heads || f.vdim != mx.vdim) return moon_fail(ctx, MOON_ESHAPE, "layer %zu mixes values of another shape", i);
                d.mixes = true;
            }
        }
        n16 = std::max<size_t>(n16, d.n16);
        nr = std::max<size_t>(nr, d.n32 - d.n16);
        k0 = std::max<size_t>(k0, d.k0);
        counters = std::max(counters, decode_mix_counters(mx.heads, mx.kv_heads));
        l->mix_partial_floats = std::max(l->mix_partial_floats, decode_mix_partial_floats(ctx, mx.heads, mx.kv_heads, d.vdimp, (mx.window ? std::min(mx.window, l->max_seq) : l->max_seq) + d.blocks));
        if (ff.kind == FeedForwardSpec::EXPERTS) {
            const size_t np = l->max_rows * ff.top;
            pairs = std::max(pairs, np);
            act = std::max(act, np * d.ffp);
            y = std::max(y, np * l->dp);
            tiles = std::max(tiles, np / SEG_TILE_ROWS + ff.experts);
        }
        l->layers.push_back(d);
    }
    Loader ld{l, design, file, seed};
    ld.std_dev = std_dev;
    MOON_TRY(alloc_t(l, l->spec.vocab * l->dp, &l->embed));
    ld.begin(l->spec.vocab, l->dp);
    auto same = [](size_t r) { return r; };
    MOON_TRY(ld.put(file ? design->names.embed() : std::string(), l->spec.vocab, l->spec.width, l->dp, same));
    MOON_TRY(ld.end(l->embed, l->spec.vocab * l->dp));
    for (size_t i = 0; i < l->layers.size(); i++) MOON_TRY(load_layer(ld, i));
    const std::string fin = file ? design->names.final_norm() : std::string();
    MOON_TRY(ld.vec(fin, l->spec.width, 1.0f, &l->fgamma));
    if (!l->spec.rms_norm) MOON_TRY(ld.vec(file ? fin + design->names.bias_suffix : fin, l->spec.width, 0.0f, &l->fbeta));
    MOON_TRY(alloc_t(l, l->vp * l->dp, &l->head));
    ld.begin(l->vp, l->dp);
    MOON_TRY(ld.put(file ? design->names.head() : std::string(), l->spec.vocab, l->spec.width, l->dp, same));
    MOON_TRY(ld.end(l->head, l->vp * l->dp));

    const size_t R = l->max_rows, hr = std::max(R, LIST_LOGIT_ROWS), tiles_n = (l->dp + 127) / 128;
    MOON_TRY(alloc_n(l, R * l->spec.width, &l->x));
    MOON_TRY(alloc_t(l, hr * l->dp, &l->h));
    MOON_TRY(alloc_t(l, R * n16, &l->c1));
    MOON_TRY(alloc_n(l, R * nr, &l->router));
    MOON_TRY(alloc_t(l, R * k0, &l->a2));
    MOON_TRY(alloc_n(l, n16, &l->proj));
    MOON_TRY(alloc_n(l, std::max(parts * R, std::min(SEG_MAX_SPLITS * R, 128 * cus / tiles_n)) * l->dp, &l->partial)); // (see seg_gemm_splits, joined_splits)
    if (parts > 1) {
        MOON_TRY(alloc_n(l, l->dp, &l->x1));
        MOON_TRY(alloc_n(l, 3 * l->dp, &l->y3));
        MOON_TRY(alloc_t(l, dgate, &l->dgate));
        MOON_TRY(alloc_n(l, dt, &l->dt));
        MOON_TRY(alloc_n(l, delta_o, &l->delta_o));
        MOON_TRY(alloc_n(l, scratch, &l->scratch));
    }
    MOON_TRY(alloc_t(l, act, &l->act));
    MOON_TRY(alloc_t(l, y, &l->y));
    MOON_TRY(alloc_n(l, pairs, &l->ids));
    MOON_TRY(alloc_n(l, pairs, &l->slot));
    MOON_TRY(alloc_n(l, pairs, &l->weight));
    MOON_TRY(alloc_n(l, pairs, &l->grouped_rows));
    MOON_TRY(alloc_n(l, tiles, &l->tile_group));
    MOON_TRY(alloc_n(l, tiles, &l->tile_row));
    MOON_TRY(alloc_n(l, tiles, &l->tile_end));
    MOON_TRY(alloc_n(l, 1, &l->n_tiles));
    MOON_TRY(alloc_n(l, LIST_LOGIT_ROWS * l->vp, &l->logits));
    MOON_TRY(alloc_n(l, LIST_LOGIT_ROWS, &l->want));
    MOON_TRY(alloc_n(l, counters, &l->counter));
    MOON_TRY(alloc_n(l, l->mix_partial_floats, &l->mix_partial));
    MOON_HIP(ctx, hipHostMalloc((void **)&l->want_pinned, LIST_LOGIT_ROWS * sizeof(uint32_t), hipHostMallocDefault));
    MOON_HIP(ctx, hipStreamSynchronize(ctx->stream));
    return MOON_OK;
}

} // namespace

int layer_list_create(moon_ctx *ctx, const LayerListSpec &spec, const Design *design, const SafeTensors *file, uint64_t seed, float std_dev, int dtype,
                      size_t max_seq, LayerList **out) {
    LayerList *l = new LayerList();
    l->ctx = ctx;
    l->spec = spec;
    l->dtype = dtype;
    l->el = dtype == MOON_DTYPE_BF16 ? 2 : 4;
    l->max_seq = max_seq;
    const int rc = create(l, design, file, seed, std_dev);
    if (rc != MOON_OK) {
        layer_list_destroy(l);
        return rc;
    }
    *out = l;
    return MOON_OK;
}

void layer_list_destroy(LayerList *l) {
    if (!l) return;
    (void)hipStreamSynchronize(l->ctx->stream);
    for (void *p : l->allocs) (void)hipFree(p);
    if (l->want_pinned) (void)hipHostFree(l->want_pinned);
    delete l;
}

size_t layer_list_rows(const LayerList *l) { return l->max_rows; }
const float *layer_list_hidden(const LayerList *l) { return l->x; }

static const void *first_values(const LayerList *l, const LayerDev &d, int *cap) {
    *cap = d.mixes ? l->layers[l->first_mix].cap : 1;
    return d.mixes ? l->layers[l->first_mix].cv : nullptr;
}

// k ranges of a joined layer's second product: each of its parts by itself, and more of them where there are CUs for more tiles
static int joined_splits(moon_ctx *ctx, const LayerDev &d, int n, int dp, SegGemm *g, int *left, int *right) {
    const int cus = ctx->cu_count > 0 ? ctx->cu_count : 256, tiles = (n + 127) / 128 * ((dp + 127) / 128);
    const int ends[4] = {0, d.ka, d.ka + d.kr, d.k0}, n_parts = d.k0 > ends[2] ? 3 : 2;
    int of[3] = {1, 1, n_parts - 2}; // ranges of each part
    for (int total = n_parts; total < std::min(SEG_MAX_SPLITS, cus / tiles); total++) {
        int widest = 0;
        for (int p = 1; p < n_parts; p++)
            if ((ends[p + 1] - ends[p]) * of[widest] > (ends[widest + 1] - ends[widest]) * of[p]) widest = p;
        if ((ends[widest + 1] - ends[widest]) / (of[widest] + 1) < 512) break;
        of[widest]++;
    }
    int s = 0;
    for (int p = 0; p < n_parts; p++)
        for (int r = 0; r < of[p]; r++) g->kb[s++] = ends[p] + (int)((ends[p + 1] - ends[p]) / 64 * (size_t)r / of[p]) * 64;
    g->kb[s] = d.k0;
    g->last_first = 1;
    *left = of[0];
    *right = of[1];
    return s;
}

int layer_list_forward(LayerList *l, const uint32_t *ids_dev, size_t n_rows, size_t pos) {
    moon_ctx *ctx = l->ctx;
    if (n_rows > l->max_rows || pos + n_rows > l->max_seq) return moon_fail(ctx, MOON_ESEQ_TOO_LONG, "layer list: %zu rows at position %zu", n_rows, pos);
    const int n = (int)n_rows, dt = l->dtype, dp = (int)l->dp;
    RowFinish f{};
    f.x = l->x;
    f.embed = l->embed;
    f.ids = ids_dev;
    f.embed_scale = l->spec.embed_scale;
    f.eps = l->spec.eps;
    f.gamma = l->layers[0].gamma;
    f.beta = l->layers[0].beta;
    f.h = l->h;
    f.n = n;
    f.width = (int)l->spec.width;
    f.dp = dp;
    MOON_TRY(launch_row_finish(ctx, dt, f));
    f.embed = nullptr;
    for (size_t i = 0; i < l->layers.size(); i++) {
        const LayerDev &d = l->layers[i];
        const MixerSpec &mx = d.spec.mixer;
        const FeedForwardSpec &ff = d.spec.ff;
        SegGemm g{};
        g.A = l->h;
        g.lda = dp;
        g.a_rows = n;
        g.W = d.w1;
        g.M = n;
        g.N = d.nall;
        g.K = dp;
        g.n16 = d.n16;
        g.n32 = d.n32;
        g.c16 = l->c1;
        g.ld16 = d.n16;
        g.c32 = l->router;
        g.ld32 = d.n32 - d.n16;
        g.glu = (char *)l->a2 + size_t(d.ka + d.kr) * l->el;
        g.ldg = d.k0;
        MOON_TRY(launch_seg_gemm(ctx, dt, g));
        const DeltaSpec &de = d.spec.delta;
        if (mx.qk_whole_norm) {
            PrepWhole pr{};
            pr.c1 = l->c1;
            pr.ld = d.n16;
            pr.n = n;
            pr.pos0 = (int)pos;
            pr.H = (int)mx.heads;
            pr.G = mx.kv_from < 0 ? (int)mx.kv_heads : 0;
            pr.dim = (int)mx.dim;
            pr.vdim = (int)mx.vdim;
            pr.dimp = d.dimp;
            pr.vdimp = d.vdimp;
            pr.oq = d.oq;
            pr.ok = d.ok;
            pr.ov = d.ov;
            pr.cap = d.cap;
            pr.rot_dims = (int)mx.rot_dims;
            pr.eps = l->spec.eps;
            pr.qn = d.qn;
            pr.kn = d.kn;
            pr.rot = d.rot;
            pr.rotv = d.rotv;
            pr.ck = d.ck;
            pr.cv = d.cv;
            MOON_TRY(launch_prep_whole(ctx, dt, pr));
        } else {
            PrepArgs pr{};
            pr.c1 = l->c1;
            pr.ld = d.n16;
            pr.n = n;
            pr.pos0 = (int)pos;
            pr.H = (int)mx.heads;
            pr.G = (int)mx.kv_heads;
            pr.dim = (int)mx.dim;
            pr.vdim = (int)mx.vdim;
            pr.dimp = d.dimp;
            pr.vdimp = d.vdimp;
            pr.oq = d.oq;
            pr.ok = d.ok;
            pr.ov = d.ov;
            pr.qk_rms = mx.qk_rms;
            pr.mixes = d.mixes;
            pr.cap = d.cap;
            pr.eps = l->spec.eps;
            pr.lambda = d.lambda;
            pr.ck = d.ck;
            pr.cv = d.cv;
            pr.v_first = first_values(l, d, &pr.cap_first);
            MOON_TRY(launch_prep_qkv(ctx, dt, pr));
        }
        if (mx.pool && mx.kv_from < 0) {
            PoolArgs po{};
            po.ck = d.ck;
            po.cv = d.cv;
            po.pk = d.pk;
            po.pv = d.pv;
            po.G = (int)mx.kv_heads;
            po.dimp = d.dimp;
            po.vdimp = d.vdimp;
            po.cap = d.cap;
            po.blocks = d.blocks;
            po.pool = (int)mx.pool;
            po.pos0 = (int)pos;
            po.n = n;
            MOON_TRY(launch_pool(ctx, dt, po));
        }
        if (de.heads) {
            SegGemm lr{}; // second steps of the gate's and the decay's projections
            lr.A = (const char *)l->c1 + size_t(d.od) * l->el;
            lr.lda = d.n16;
            lr.a_rows = n;
            lr.W = d.wlr;
            lr.M = n;
            lr.N = lr.n32 = d.lrn;
            lr.K = d.kd;
            lr.n16 = d.lr16;
            lr.c16 = l->dgate;
            lr.ld16 = d.lr16;
            lr.c32 = l->dt;
            lr.ld32 = d.lrn - d.lr16;
            MOON_TRY(launch_seg_gemm(ctx, dt, lr));
            DeltaRows r{};
            r.c1 = l->c1;
            r.ld = d.n16;
            r.oc = d.oc;
            r.channels = d.channels;
            r.taps = (int)de.conv;
            r.beta = l->router;
            r.ldb = d.n32 - d.n16;
            r.dt = l->dt;
            r.lddt = d.lrn - d.lr16;
            r.gate = l->dgate;
            r.ldg = d.lr16;
            r.n = n;
            r.pos0 = (int)pos;
            r.H = (int)de.heads;
            r.G = (int)de.kv_heads;
            r.dim = (int)de.dim;
            r.vdim = (int)de.vdim;
            r.dimp = d.ddimp;
            r.vdimp = d.dvdimp;
            r.conv = d.conv;
            r.a_log = d.a_log;
            r.dt_bias = d.dt_bias;
            r.norm = d.dnorm;
            r.eps = l->spec.eps;
            r.scratch = l->scratch;
            r.o = l->delta_o;
            r.state = d.state;
            r.ring = d.ring;
            r.out = (char *)l->a2 + size_t(d.ka) * l->el;
            r.ldo = d.k0;
            MOON_TRY(launch_delta_rows(ctx, dt, r));
        }
        WindowAttn at{};
        at.q = l->c1;
        at.gate = mx.gate ? (const char *)l->c1 + size_t(d.og) * l->el : nullptr;
        at.ldq = d.n16;
        at.ck = d.ck;
        at.cv = d.cv;
        at.cap = d.cap;
        at.out = l->a2;
        at.ldo = d.k0;
        at.n = n;
        at.pos0 = (int)pos;
        at.H = (int)mx.heads;
        at.G = (int)mx.kv_heads;
        at.dimp = d.dimp;
        at.vdimp = d.vdimp;
        at.window = (int)mx.window;
        at.scale = mx.scale;
        at.sink = d.sink;
        at.temp = d.temp;
        at.pool = (int)mx.pool;
        at.blocks = d.blocks;
        at.pk = d.pk;
        at.pv = d.pv;
        at.rotv = d.rotv;
        at.vdim = (int)mx.vdim;
        MOON_TRY(launch_window_attention(ctx, dt, at));
        f.top = 0;
        if (ff.kind == FeedForwardSpec::EXPERTS) {
            RouteArgs r{};
            r.logits = l->router;
            r.correction = d.correction;
            r.n = n;
            r.ld = d.n32 - d.n16;
            r.E = (int)ff.experts;
            r.top = (int)ff.top;
            r.rows_per_tile = SEG_TILE_ROWS;
            r.ids = l->ids;
            r.weight = l->weight;
            r.slot = l->slot;
            r.rows = l->grouped_rows;
            r.tile_group = l->tile_group;
            r.tile_row = l->tile_row;
            r.tile_end = l->tile_end;
            r.n_tiles = l->n_tiles;
            MOON_TRY(launch_route(ctx, r));
            SegGemm e{};
            e.A = l->h;
            e.lda = dp;
            e.a_rows = n;
            e.rows = l->grouped_rows;
            e.W = d.wgu;
            e.w_group = size_t(2) * d.ffp * dp;
            e.M = n * r.top;
            e.N = 2 * d.ffp;
            e.K = dp;
            e.glu = l->act;
            e.ldg = d.ffp;
            e.tile_group = l->tile_group;
            e.tile_row = l->tile_row;
            e.tile_end = l->tile_end;
            e.n_tiles = l->n_tiles;
            e.max_tiles = e.M / SEG_TILE_ROWS + std::min(r.E, e.M);
            MOON_TRY(launch_seg_gemm(ctx, dt, e));
            e.A = l->act;
            e.lda = d.ffp;
            e.a_rows = e.M;
            e.rows = nullptr;
            e.W = d.wd;
            e.w_group = size_t(dp) * d.ffp;
            e.N = e.n16 = e.n32 = dp;
            e.K = d.ffp;
            e.glu = nullptr;
            e.c16 = l->y;
            e.ld16 = dp;
            MOON_TRY(launch_seg_gemm(ctx, dt, e));
            f.expert_out = l->y;
            f.slot = l->slot;
            f.weight = l->weight;
            f.top = r.top;
        }
        SegGemm o{};
        o.A = l->a2;
        o.lda = d.k0;
        o.a_rows = n;
        o.W = d.w2;
        o.M = n;
        o.N = o.n32 = dp;
        o.K = d.k0;
        o.c32 = l->partial;
        o.ld32 = dp;
        f.out_l = d.out_l;
        f.out_r = d.out_r;
        o.splits = d.out_l ? joined_splits(ctx, d, n, dp, &o, &f.splits_l, &f.splits_r) : seg_gemm_splits(ctx, n, dp, d.k0);
        MOON_TRY(launch_seg_gemm(ctx, dt, o));
        f.partial = l->partial;
        f.splits = o.splits;
        const bool last = i + 1 == l->layers.size();
        f.gamma = last ? nullptr : l->layers[i + 1].gamma;
        f.beta = last ? nullptr : l->layers[i + 1].beta;
        f.h = last ? nullptr : l->h;
        MOON_TRY(launch_row_finish(ctx, dt, f));
    }
    return MOON_OK;
}

int layer_list_step(LayerList *l, const uint32_t *token_dev, size_t pos, const uint32_t *pos_dev) {
    moon_ctx *ctx = l->ctx;
    if (pos >= l->max_seq) return moon_fail(ctx, MOON_ESEQ_TOO_LONG, "layer list: position %zu", pos);
    const int dt = l->dtype, dp = (int)l->dp;
    // Behind a joined layer the next first product completes x and moves it to the other copy; it ends up in l->x.
    const LayerDev *joined = nullptr; // the layer before, if x waits for its parts
    float *x_now = l->x, *x_next = l->x1;
    for (size_t i = 0; i + 1 < l->layers.size(); i++)
        if (l->layers[i].out_l) std::swap(x_now, x_next);
    for (size_t i = 0; i < l->layers.size(); i++) {
        const LayerDev &d = l->layers[i];
        const MixerSpec &mx = d.spec.mixer;
        const FeedForwardSpec &ff = d.spec.ff;
        const DeltaSpec &de = d.spec.delta;
        const bool experts = ff.kind == FeedForwardSpec::EXPERTS;
        DecodeProj p{};
        p.x = x_now;
        if (joined) {
            p.y = l->y3;
            p.out_l = joined->out_l;
            p.out_r = joined->out_r;
            p.x_new = x_next;
            std::swap(x_now, x_next);
        }
        joined = d.out_l ? &d : nullptr;
        p.token = i == 0 ? token_dev : nullptr;
        p.embed = l->embed;
        p.embed_scale = l->spec.embed_scale;
        p.gamma = d.gamma;
        p.beta = d.beta;
        p.eps = l->spec.eps;
        p.width = (int)l->spec.width;
        p.dp = dp;
        p.w1 = d.w1;
        p.n16 = d.n16;
        p.n32 = d.n32;
        p.nall = d.nall;
        p.n16_used = de.heads ? d.od + (int)(de.rank_a + de.rank_g) : d.og + (mx.gate ? (int)mx.heads * d.vdimp : 0);
        p.n32_used = (int)(de.heads ? de.heads : ff.experts);
        p.ff = ff.kind == FeedForwardSpec::DENSE ? (int)ff.ff : 0;
        p.proj = l->proj;
        p.logits = l->router;
        p.glu = (char *)l->a2 + size_t(d.ka + d.kr) * l->el;
        p.h = experts ? l->h : nullptr;
        MOON_TRY(launch_decode_proj(ctx, dt, p));
        DecodeMix x{};
        x.proj = l->proj;
        x.H = (int)mx.heads;
        x.G = (int)mx.kv_heads;
        x.dim = (int)mx.dim;
        x.vdim = (int)mx.vdim;
        x.dimp = d.dimp;
        x.vdimp = d.vdimp;
        x.ok = d.ok;
        x.ov = d.ov;
        x.og = d.og;
        x.qk_rms = mx.qk_rms;
        x.gate = mx.gate;
        x.mixes = d.mixes;
        x.window = (int)mx.window;
        x.cap = d.cap;
        x.eps = l->spec.eps;
        x.lambda = d.lambda;
        x.scale = mx.scale;
        x.sink = d.sink;
        x.ck = d.ck;
        x.cv = d.cv;
        x.v_first = first_values(l, d, &x.cap_first);
        x.pos = pos;
        x.pos_dev = pos_dev;
        x.partial = l->mix_partial;
        x.partial_floats = l->mix_partial_floats;
        x.counter = l->counter;
        x.out = l->a2;
        x.whole = mx.qk_whole_norm;
        x.rot_dims = (int)mx.rot_dims;
        x.pool = (int)mx.pool;
        x.blocks = d.blocks;
        x.borrowed = mx.kv_from >= 0;
        x.qn = d.qn;
        x.kn = d.kn;
        x.temp = d.temp;
        x.rot = d.rot;
        x.rotv = d.rotv;
        x.pk = d.pk;
        x.pv = d.pv;
        if (de.heads) {
            x.dH = (int)de.heads;
            x.dG = (int)de.kv_heads;
            x.ddim = (int)de.dim;
            x.dvdim = (int)de.vdim;
            x.ddimp = d.ddimp;
            x.dvdimp = d.dvdimp;
            x.taps = (int)de.conv;
            x.oc = d.oc;
            x.channels = d.channels;
            x.od = d.od;
            x.rank_a = (int)de.rank_a;
            x.rank_g = (int)de.rank_g;
            x.kd = d.kd;
            x.lr16 = d.lr16;
            x.beta = l->router;
            x.conv = d.conv;
            x.a_log = d.a_log;
            x.dt_bias = d.dt_bias;
            x.dnorm = d.dnorm;
            x.wlr = d.wlr;
            x.state = d.state;
            x.ring = d.ring;
            x.dout = (char *)l->a2 + size_t(d.ka) * l->el;
        }
        DecodeOut o{};
        if (experts) {
            x.logits = l->router;
            x.correction = d.correction;
            x.E = (int)ff.experts;
            x.top = (int)ff.top;
            x.ff = (int)ff.ff;
            x.ffp = d.ffp;
            x.h = l->h;
            x.wgu = d.wgu;
            x.act = l->act;
            x.ids = l->ids;
            x.weight = l->weight;
            o.top = x.top;
            o.ffp = d.ffp;
            o.wd = d.wd;
            o.act = l->act;
            o.ids = l->ids;
            o.weight = l->weight;
        }
        x.dp = dp;
        MOON_TRY(launch_decode_mix(ctx, dt, x));
        o.x = x_now;
        o.y = joined ? l->y3 : nullptr;
        o.k1 = d.ka;
        o.k2 = d.ka + d.kr;
        o.width = (int)l->spec.width;
        o.dp = dp;
        o.k0 = d.k0;
        o.w2 = d.w2;
        o.a = l->a2;
        MOON_TRY(launch_decode_out(ctx, dt, o));
    }
    if (!joined) return MOON_OK;
    RowFinish f{};
    f.x = l->x;
    f.partial = l->y3;
    f.splits = 3;
    f.splits_l = f.splits_r = 1;
    f.out_l = joined->out_l;
    f.out_r = joined->out_r;
    f.eps = l->spec.eps;
    f.n = 1;
    f.width = (int)l->spec.width;
    f.dp = dp;
    return launch_row_finish(ctx, dt, f);
}

int layer_list_logits(LayerList *l, const uint32_t *rows, size_t n, const float **logits, size_t *ld) {
    moon_ctx *ctx = l->ctx;
    const int dp = (int)l->dp;
    *logits = l->logits;
    *ld = l->vp;
    if (n > LIST_LOGIT_ROWS) return moon_fail(ctx, MOON_EINVAL_DIM, "layer list: logits of %zu rows at once", n);
    for (size_t i = 0; i < n; i++)
        if (rows[i] >= l->max_rows) return moon_fail(ctx, MOON_EINVAL_DIM, "layer list: row %u", rows[i]);
    if (n == 1) {
        DecodeProj p{};
        p.x = l->x + size_t(rows[0]) * l->spec.width;
        p.gamma = l->fgamma;
        p.beta = l->fbeta;
        p.eps = l->spec.eps;
        p.width = (int)l->spec.width;
        p.dp = dp;
        p.w1 = l->head;
        p.n32 = p.nall = (int)l->vp;
        p.n32_used = (int)l->spec.vocab;
        p.logits = l->logits;
        p.softcap = l->spec.softcap;
        return launch_decode_proj(ctx, l->dtype, p);
    }
    memcpy(l->want_pinned, rows, n * sizeof(uint32_t)); // (the callers drain the stream before they come back)
    MOON_HIP(ctx, hipMemcpyAsync(l->want, l->want_pinned, n * sizeof(uint32_t), hipMemcpyHostToDevice, ctx->stream));
    RowFinish f{};
    f.x = l->x;
    f.rows = l->want;
    f.gamma = l->fgamma;
    f.beta = l->fbeta;
    f.eps = l->spec.eps;
    f.h = l->h;
    f.n = (int)n;
    f.width = (int)l->spec.width;
    f.dp = dp;
    MOON_TRY(launch_row_finish(ctx, l->dtype, f));
    SegGemm g{};
    g.A = l->h;
    g.lda = dp;
    g.a_rows = (int)n;
    g.W = l->head;
    g.M = (int)n;
    g.N = g.n32 = (int)l->vp;
    g.K = dp;
    g.c32 = l->logits;
    g.ld32 = (int)l->vp;
    g.softcap = l->spec.softcap;
    return launch_seg_gemm(ctx, l->dtype, g);
}

size_t layer_list_weight_bytes(const LayerList *l) {
    size_t n = l->spec.vocab * l->spec.width, vecs = 2 * l->spec.width;
    for (const LayerDev &d : l->layers) {
        const MixerSpec &m = d.spec.mixer;
        const FeedForwardSpec &f = d.spec.ff;
        const size_t w = l->spec.width;
        const DeltaSpec &e = d.spec.delta;
        n += w * (m.heads * m.dim + (m.kv_from < 0 ? m.kv_heads * (m.dim + m.vdim) : 0) + m.heads * m.vdim * (m.gate ? 2 : 1));
        n += w * (2 * e.kv_heads * e.dim + 2 * e.heads * e.vdim + e.heads + e.rank_a + e.rank_g) + e.heads * (e.dim * e.rank_a + e.vdim * e.rank_g);
        n += f.kind == FeedForwardSpec::DENSE ? 3 * w * f.ff : f.kind == FeedForwardSpec::EXPERTS ? w * f.experts + f.top * 3 * w * f.ff : 0;
        vecs += 2 * w;
    }
    return n * l->el + vecs * sizeof(float);
}
