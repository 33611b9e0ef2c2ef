// Model folders (config.json + model.safetensors) and the registry of designs that are described as a list of layers.
#include "model_folder.hpp"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cerrno>

// ------------------------------------------------------------------ safetensors
SafeTensors::~SafeTensors() {
    if (map) munmap(map, size);
}

int SafeTensors::open(const std::string &path, std::string *err) {
    const int fd = ::open(path.c_str(), O_RDONLY);
    struct stat st;
    if (fd < 0 || fstat(fd, &st) != 0) {
        *err = path + ": " + strerror(errno);
        if (fd >= 0) close(fd);
        return MOON_EINVAL;
    }
    size = (size_t)st.st_size;
    map = size >= 8 ? mmap(nullptr, size, PROT_READ, MAP_PRIVATE, fd, 0) : MAP_FAILED;
    close(fd);
    if (map == MAP_FAILED) {
        map = nullptr;
        *err = path + ": not a safetensors file";
        return MOON_EFORMAT;
    }
    const unsigned char *p = (const unsigned char *)map;
    uint64_t header = 0;
    for (int i = 7; i >= 0; i--) header = header << 8 | p[i];
    Json j;
    if (header > size - 8 || !Json::parse((const char *)p + 8, (size_t)header, &j, err) || j.type != Json::OBJECT) {
        *err = path + ": bad header " + *err;
        return MOON_EFORMAT;
    }
    const size_t base = 8 + (size_t)header;
    for (const auto &m : j.members) {
        if (m.first == "__metadata__") continue;
        const Json *dt = m.second.find("dtype"), *sh = m.second.find("shape"), *off = m.second.find("data_offsets");
        StTensor t;
        bool ok = dt && dt->type == Json::STRING && sh && sh->type == Json::ARRAY && off && off->type == Json::ARRAY && off->items.size() == 2 &&
                  off->items[0].is_size() && off->items[1].is_size();
        if (ok) {
            t.dtype = dt->str;
            const size_t el = t.dtype == "BF16" || t.dtype == "F16" ? 2 : t.dtype == "F32" || t.dtype == "I32" ? 4 : 0;
            unsigned __int128 n = 1;
            for (const Json &d : sh->items) {
                ok = ok && d.is_size();
                t.shape.push_back(ok ? (size_t)d.num : 0);
                n *= t.shape.back();
                ok = ok && n < ((unsigned __int128)1 << 62);
            }
            const size_t a = (size_t)off->items[0].num, b = (size_t)off->items[1].num;
            ok = ok && el && a <= b && b <= size - base && n * el == b - a;
            t.data = p + base + a;
            t.bytes = b - a;
        }
        if (!ok) {
            *err = path + ": tensor '" + m.first + "' does not fit its header entry";
            return MOON_EFORMAT;
        }
        tensors[m.first] = t;
    }
    return MOON_OK;
}

const StTensor *SafeTensors::find(const std::string &name) const {
    const auto it = tensors.find(name);
    return it == tensors.end() ? nullptr : &it->second;
}

// ------------------------------------------------------------------ config.json
namespace {

struct Fields { // typed access to a config's members; the first failure is kept
    std::string *err;
    bool ok = true;
    bool fail(const std::string &what) {
        if (ok) *err = "config.json: " + what;
        return ok = false;
    }
    const Json *object(const Json &j, const char *key, const std::string &where) {
        const Json *v = j.find(key);
        if (!v || v->type != Json::OBJECT) fail(where + key + " is missing or no object");
        return v && v->type == Json::OBJECT ? v : nullptr;
    }
    size_t size(const Json *j, const char *key, const std::string &where) {
        const Json *v = j ? j->find(key) : nullptr;
        if (!v || !v->is_size() || v->num < 1 || v->num > 1e9) {
            fail(where + key + " is missing or no positive integer");
            return 1;
        }
        return (size_t)v->num;
    }
    double real(const Json *j, const char *key, const std::string &where) {
        const Json *v = j ? j->find(key) : nullptr;
        if (!v || v->type != Json::NUMBER) {
            fail(where + key + " is missing or no number");
            return 1.0;
        }
        return v->num;
    }
    float number(const Json *j, const char *key, const std::string &where) { return (float)real(j, key, where); }
};

std::string indexed(const char *prefix, size_t i, const std::string &rest) { return prefix + std::to_string(i) + rest; }

// Rikanex: parallel layers of windowed attention without positions (unit-RMS q and k, sink, output gate, values mixed with the
// first layer's) and a gated feed-forward, dense or of routed experts.
bool parse_rikanex(const Json &c, LayerListSpec *s, std::string *err) {
    Fields f{err};
    s->vocab = f.size(&c, "vocab", "");
    s->width = f.size(&c, "width", "");
    s->embed_scale = f.number(f.object(c, "embedding", ""), "scale", "embedding.");
    s->eps = f.number(f.object(c, "norm", ""), "eps", "norm.");
    if (!(s->eps > 0.0f)) f.fail("norm.eps must be positive");
    const Json *layers = c.find("layers");
    if (!layers || layers->type != Json::ARRAY || layers->items.empty()) return f.fail("layers is missing or empty");
    for (size_t i = 0; i < layers->items.size() && f.ok; i++) {
        const Json &l = layers->items[i];
        const std::string at = "layers[" + std::to_string(i) + "].";
        LayerSpec spec;
        const Json *type = l.find("type");
        if (!type || type->str != "attention") return f.fail(at + "type is not 'attention'");
        const Json *m = f.object(l, "mixer", at);
        MixerSpec &mx = spec.mixer;
        mx.heads = f.size(m, "heads", at + "mixer.");
        mx.kv_heads = f.size(m, "kv_heads", at + "mixer.");
        mx.dim = f.size(m, "dim", at + "mixer.");
        mx.vdim = f.size(m, "vdim", at + "mixer.");
        mx.scale = f.number(m, "scale", at + "mixer.");
        if (mx.heads % mx.kv_heads) f.fail(at + "mixer.kv_heads does not divide heads");
        const Json *mask = m ? m->find("mask") : nullptr, *mix = m ? m->find("v_mix") : nullptr;
        if (mask && mask->type != Json::NIL) mx.window = f.size(mask, "size", at + "mixer.mask.");
        mx.v_mix = mix && mix->type == Json::BOOL && mix->b;
        mx.qk_rms = mx.sink = mx.gate = true;
        const Json *mlp = l.find("mlp");
        if (mlp && mlp->type != Json::NIL) {
            const Json *kind = mlp->find("kind");
            if (kind && kind->str == "dense") {
                spec.ff.kind = FeedForwardSpec::DENSE;
                spec.ff.ff = f.size(mlp, "ff", at + "mlp.");
            } else if (kind && kind->str == "moe") {
                spec.ff.kind = FeedForwardSpec::EXPERTS;
                spec.ff.ff = f.size(f.object(*mlp, "expert", at + "mlp."), "ff", at + "mlp.expert.");
                const Json *router = f.object(*mlp, "router", at + "mlp.");
                spec.ff.experts = f.size(router, "experts", at + "mlp.router.");
                spec.ff.top = f.size(router, "top", at + "mlp.router.");
                if (spec.ff.top > spec.ff.experts) f.fail(at + "mlp.router.top exceeds experts");
            } else f.fail(at + "mlp.kind is neither 'dense' nor 'moe'");
        }
        s->layers.push_back(spec);
    }
    return f.ok;
}

// Generax: parallel layers with RMS norms.  The mixer is windowed attention with rotated queries, keys and values, or windowed attention
// without positions over tokens and pooled blocks beside a gated delta rule; the feed-forward is gated and dense.
struct GeneraxReader {
    Fields f;
    const LayerListSpec *s;

    void heads(const Json *m, const std::string &at, size_t *h, size_t *g, size_t *dim, size_t *vdim) {
        *h = f.size(m, "heads", at);
        *g = f.size(m, "kv_heads", at);
        *dim = f.size(m, "dim", at);
        *vdim = f.size(m, "vdim", at);
        if (*h % *g) f.fail(at + "kv_heads does not divide heads");
    }
    // index of layer i, for kv_from
    void attention(const Json *m, const std::string &at, size_t i, MixerSpec *x) {
        heads(m, at, &x->heads, &x->kv_heads, &x->dim, &x->vdim);
        x->scale = f.number(m, "scale", at);
        x->qk_whole_norm = true;
        const Json *mask = m ? m->find("mask") : nullptr;
        if (mask && mask->type != Json::NIL) {
            x->window = f.size(mask, "size", at + "mask.");
            if (const Json *pool = mask->find("pool"); pool && pool->type != Json::NIL) x->pool = f.size(mask, "pool", at + "mask.");
        }
        const Json *rot = m ? m->find("rot") : nullptr;
        if (rot && rot->type != Json::NIL) {
            x->rot_dims = f.size(rot, "dims", at + "rot.");
            x->rot_base = f.real(rot, "base", at + "rot.");
            const Json *scaling = rot->find("scaling");
            if (scaling && scaling->type != Json::NIL) x->rot_factor = f.real(scaling, "factor", at + "rot.scaling.");
            x->rot_values = true;
            if (x->rot_dims % 2 || x->rot_dims > x->dim) f.fail(at + "rot.dims is odd or exceeds dim");
            if (x->vdim % 2) f.fail(at + "vdim is odd");
            if (!(x->rot_base > 0.0) || !(x->rot_factor > 0.0)) f.fail(at + "rot.base and rot.scaling.factor must be positive");
        }
        const Json *from = m ? m->find("kv_from") : nullptr;
        if (!from || from->type == Json::NIL) return;
        if (!from->is_size() || from->num >= (double)i) {
            f.fail(at + "kv_from is no earlier layer");
            return;
        }
        x->kv_from = (int)from->num;
        const LayerSpec &src = s->layers[x->kv_from];
        const MixerSpec &y = src.mixer;
        if (src.delta.heads || y.kv_from >= 0 || y.kv_heads != x->kv_heads || y.dim != x->dim || y.vdim != x->vdim || y.rot_dims != x->rot_dims ||
            y.rot_base != x->rot_base || y.rot_factor != x->rot_factor || (x->pool && x->pool != y.pool))
            f.fail(at + "kv_from names a layer without keys and values of its own, or of other heads or rotation");
    }
};
bool parse_generax(const Json &c, LayerListSpec *s, std::string *err) {
    GeneraxReader r{{err}, s};
    Fields &f = r.f;
    s->vocab = f.size(&c, "vocab", "");
    s->width = f.size(&c, "width", "");
    s->eps = f.number(f.object(c, "norm", ""), "eps", "norm.");
    if (!(s->eps > 0.0f)) f.fail("norm.eps must be positive");
    s->rms_norm = true;
    if (const Json *cap = c.find("logit_softcap"); cap && cap->type != Json::NIL) {
        s->softcap = f.number(&c, "logit_softcap", "");
        if (!(s->softcap > 0.0f)) f.fail("logit_softcap must be positive");
    }
    const Json *layers = c.find("layers");
    if (!layers || layers->type != Json::ARRAY || layers->items.empty()) return f.fail("layers is missing or empty");
    for (size_t i = 0; i < layers->items.size() && f.ok; i++) {
        const Json &l = layers->items[i];
        const std::string at = "layers[" + std::to_string(i) + "].";
        LayerSpec spec;
        const Json *type = l.find("type"), *m = f.object(l, "mixer", at);
        if (type && type->str == "attention") {
            r.attention(m, at + "mixer.", i, &spec.mixer);
            spec.mixer.temp = true;
        } else if (type && type->str == "parallel") {
            r.attention(m ? f.object(*m, "left", at + "mixer.") : nullptr, at + "mixer.left.", 0, &spec.mixer);
            const std::string right = at + "mixer.right.";
            const Json *d = m ? f.object(*m, "right", at + "mixer.") : nullptr;
            r.heads(d, right, &spec.delta.heads, &spec.delta.kv_heads, &spec.delta.dim, &spec.delta.vdim);
            spec.delta.conv = f.size(d, "conv", right);
        } else return f.fail(at + "type is neither 'attention' nor 'parallel'");
        const Json *mlp = l.find("mlp");
        if (mlp && mlp->type != Json::NIL) {
            const Json *kind = mlp->find("kind");
            if (!kind || kind->str != "dense") return f.fail(at + "mlp.kind is not 'dense'");
            spec.ff.kind = FeedForwardSpec::DENSE;
            spec.ff.ff = f.size(mlp, "ff", at + "mlp.");
        }
        s->layers.push_back(spec);
    }
    return f.ok;
}

const TensorNames RIKANEX_NAMES = {
    [] { return std::string("embed"); },
    [] { return std::string("head"); },
    [] { return std::string("final.norm"); },
    [](size_t i) { return indexed("l", i, ".norm1"); },
    [](size_t i, const char *what) { return indexed("l", i, std::string(".mix.") + what); },
    [](size_t i, const char *what) { return indexed("l", i, std::string(".mlp.") + what); },
    [](size_t i, size_t e, const char *what) { return indexed("l", i, indexed(".mlp.e", e, std::string(".") + what)); },
    ".b",
};
const TensorNames GENERAX_NAMES = {
    RIKANEX_NAMES.embed, RIKANEX_NAMES.head, RIKANEX_NAMES.final_norm, RIKANEX_NAMES.norm, RIKANEX_NAMES.mixer, RIKANEX_NAMES.ff,
    RIKANEX_NAMES.expert, nullptr, "left.", "right.",
};

const Design DESIGNS[] = {
    {"Rikanex", parse_rikanex, RIKANEX_NAMES},
    {"Generax", parse_generax, GENERAX_NAMES},
};

} // namespace

const Design *find_design(const std::string &architecture) {
    for (const Design &d : DESIGNS)
        if (architecture == d.name) return &d;
    return nullptr;
}

std::string known_designs() {
    std::string s;
    for (const Design &d : DESIGNS) s += std::string(s.empty() ? "" : ", ") + d.name;
    return s;
}

int parse_model_config(const char *text, size_t len, const Design **design, LayerListSpec *spec, std::string *err) {
    Json c;
    if (!Json::parse(text, len, &c, err)) return MOON_EFORMAT;
    const Json *a = c.find("architecture");
    *design = a && a->type == Json::STRING ? find_design(a->str) : nullptr;
    if (!*design) {
        *err = "config.json: architecture '" + (a ? a->str : std::string()) + "' is not one of: " + known_designs();
        return MOON_EFORMAT;
    }
    spec->design = (*design)->name;
    return (*design)->parse(c, spec, err) ? MOON_OK : MOON_EFORMAT;
}

namespace {

int check_tensor(const SafeTensors &file, const std::string &name, std::initializer_list<size_t> shape, std::string *err) {
    const StTensor *t = file.find(name);
    if (!t) {
        *err = "model.safetensors has no tensor '" + name + "'";
        return MOON_EFORMAT;
    }
    if (t->dtype != "BF16" && t->dtype != "F32") {
        *err = "tensor '" + name + "' is " + t->dtype + ", not BF16 or F32";
        return MOON_EFORMAT;
    }
    if (t->shape != std::vector<size_t>(shape)) {
        *err = "tensor '" + name + "' does not have the configuration's shape";
        return MOON_ESHAPE;
    }
    return MOON_OK;
}

} // namespace

// Every tensor of the description, with its shape.  Sizes that only the tensors have (the ranks of two-step projections) are taken
// from them.
static int check_tensors(const Design &design, LayerListSpec &s, const SafeTensors &file, std::string *err) {
    const TensorNames &n = design.names;
    const size_t w = s.width;
    int rc = MOON_OK;
    auto need = [&](const std::string &name, std::initializer_list<size_t> shape) {
        if (rc == MOON_OK) rc = check_tensor(file, name, shape, err);
    };
    auto norm = [&](const std::string &name) {
        need(name, {w});
        if (n.bias_suffix) need(name + n.bias_suffix, {w});
    };
    need(n.embed(), {s.vocab, w});
    need(n.head(), {s.vocab, w});
    norm(n.final_norm());
    bool mixing = false;
    for (size_t i = 0; i < s.layers.size() && rc == MOON_OK; i++) {
        const MixerSpec &m = s.layers[i].mixer;
        DeltaSpec &d = s.layers[i].delta;
        const FeedForwardSpec &f = s.layers[i].ff;
        norm(n.norm(i));
        auto mix = [&](const std::string &what) { return n.mixer(i, ((d.heads ? n.attention_part : "") + what).c_str()); };
        need(mix("q"), {m.heads * m.dim, w});
        if (m.kv_from < 0) {
            need(mix("k"), {m.kv_heads * m.dim, w});
            need(mix("v"), {m.kv_heads * m.vdim, w});
        }
        need(mix("o"), {w, m.heads * m.vdim});
        if (m.qk_whole_norm) {
            need(mix("q.norm"), {m.heads * m.dim});
            if (m.kv_from < 0) need(mix("k.norm"), {m.kv_heads * m.dim});
        }
        if (m.temp) need(mix("temp"), {m.heads});
        if (m.gate) need(mix("g"), {m.heads * m.vdim, w});
        if (m.sink) need(mix("sink"), {m.heads});
        if (m.v_mix && mixing) need(mix("vmix"), {});
        mixing = mixing || m.v_mix;
        if (d.heads) {
            auto delta = [&](const std::string &what) { return n.mixer(i, (n.delta_part + what).c_str()); };
            auto rank = [&](const std::string &name, size_t *r) {
                const StTensor *t = file.find(name);
                if (t && t->shape.size() == 2) *r = t->shape[0];
                if (rc == MOON_OK && t && (!*r || *r > 1 << 20)) {
                    *err = "tensor '" + name + "' has no rows";
                    rc = MOON_ESHAPE;
                }
                need(name, {*r, w});
            };
            const size_t q = d.kv_heads * d.dim, v = d.heads * d.vdim;
            for (const char *what : {"q", "k", "v"}) {
                const size_t rows = *what == 'v' ? v : q;
                need(delta(what), {rows, w});
                need(delta(what + std::string(".conv")), {rows, d.conv});
            }
            rank(delta("a1"), &d.rank_a);
            rank(delta("g1"), &d.rank_g);
            need(delta("a2"), {d.heads * d.dim, d.rank_a});
            need(delta("g2"), {v, d.rank_g});
            need(delta("b"), {d.heads, w});
            need(delta("A_log"), {d.heads});
            need(delta("dt_bias"), {d.heads * d.dim});
            need(delta("norm"), {d.vdim});
            need(delta("o"), {w, v});
            need(mix("out"), {w});
            need(delta("out"), {w});
        }
        if (f.kind == FeedForwardSpec::DENSE) {
            need(n.ff(i, "gate"), {f.ff, w});
            need(n.ff(i, "up"), {f.ff, w});
            need(n.ff(i, "down"), {w, f.ff});
        } else if (f.kind == FeedForwardSpec::EXPERTS) {
            need(n.ff(i, "router"), {f.experts, w});
            need(n.ff(i, "correction"), {f.experts});
            for (size_t e = 0; e < f.experts && rc == MOON_OK; e++) {
                need(n.expert(i, e, "gate"), {f.ff, w});
                need(n.expert(i, e, "up"), {f.ff, w});
                need(n.expert(i, e, "down"), {w, f.ff});
            }
        }
    }
    return rc;
}

int read_model_folder(const std::string &dir, const Design **design, LayerListSpec *spec, SafeTensors *file, std::string *err) {
    const std::string config = dir + "/config.json";
    FILE *f = fopen(config.c_str(), "rb");
    if (!f) {
        *err = "cannot read " + config;
        return MOON_EINVAL;
    }
    std::string text;
    char buf[4096];
    for (size_t n; (n = fread(buf, 1, sizeof buf, f)) > 0;) text.append(buf, n);
    fclose(f);
    if (int rc = parse_model_config(text.data(), text.size(), design, spec, err); rc != MOON_OK) return rc;
    if (int rc = file->open(dir + "/model.safetensors", err); rc != MOON_OK) return rc;
    return check_tensors(**design, *spec, *file, err);
}

extern "C" int moon_text_folder_check(const char *dir, const char **design, size_t *n_layers, char *err, size_t err_len) {
    const Design *d = nullptr;
    LayerListSpec spec;
    SafeTensors file;
    std::string text = "null folder";
    const int rc = dir ? read_model_folder(dir, &d, &spec, &file, &text) : MOON_EINVAL;
    if (rc != MOON_OK) {
        if (err && err_len) snprintf(err, err_len, "%s", text.c_str());
        return rc;
    }
    if (design) *design = d->name;
    if (n_layers) *n_layers = spec.layers.size();
    return MOON_OK;
}

extern "C" const char *moon_text_designs(void) {
    static const std::string names = known_designs();
    return names.c_str();
}
