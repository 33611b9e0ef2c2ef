"""Small Generax models for the tests: configurations and random bf16 weights."""
import generax_oracle as G
import numpy as np
from rikanex_oracle import bf16_round


def softmax_mixer(heads, kv_heads, dim, vdim, window, scale, pool=None):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window, **(dict(pool=pool) if pool else {})), scale=scale)


def rotation(dims, base, factor=None):
    return dict(dims=dims, base=base, **(dict(scaling=dict(factor=factor)) if factor else {}))


def attention(heads, kv_heads, dim, vdim, window, scale, rot, kv_from=None):
    return dict(softmax_mixer(heads, kv_heads, dim, vdim, window, scale), rot=rot, **({} if kv_from is None else dict(kv_from=kv_from)))


def delta(heads, kv_heads, dim, vdim, conv):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)


def plain(mixer, ff=None):
    return dict(type="attention", mixer=mixer, mlp=dict(kind="dense", ff=ff) if ff else None)


def parallel(left, right, ff=None):
    return dict(type="parallel", mixer=dict(left=left, right=right), mlp=dict(kind="dense", ff=ff) if ff else None)


def config(vocab, width, layers, eps=1e-5, softcap=9.0):
    return dict(architecture="Generax", vocab=vocab, width=width, norm=dict(eps=eps), logit_softcap=softcap, layers=layers)


# Sizes that are padded in every way; blocks longer and shorter than the window; keys borrowed by a longer window and by more heads
ODD = config(101, 90, [
    plain(attention(6, 2, 24, 10, 11, 0.2, rotation(16, 500.0, 2.5)), 70),
    parallel(softmax_mixer(5, 5, 12, 20, 9, 0.31, 4), delta(3, 1, 20, 12, 4), 33),
    plain(attention(4, 2, 24, 10, 30, 0.3, rotation(16, 500.0, 2.5), kv_from=0)),
    parallel(softmax_mixer(4, 1, 17, 9, 5, 0.4, 7), delta(4, 2, 33, 40, 1)),
    plain(attention(2, 1, 33, 14, 1, 0.4, rotation(2, 30.0)), 8),
    parallel(softmax_mixer(3, 3, 8, 8, 1, 0.5, 1), delta(2, 2, 8, 8, 7), 65),
], eps=1e-3, softcap=2.0)
# More than eight query heads on one key/value head, head sizes 128 and 96, products long enough to split k
WIDE = config(700, 512, [
    parallel(softmax_mixer(12, 1, 128, 64, 100, 0.05, 3), delta(4, 2, 128, 96, 4), 1024),
    parallel(softmax_mixer(6, 3, 64, 96, 64, 0.1, 64), delta(6, 3, 64, 64, 2)),
    plain(attention(12, 1, 64, 128, 65, 0.1, rotation(32, 1e4, 8.0)), 192),
    plain(attention(12, 1, 64, 128, 20, 0.1, rotation(32, 1e4, 8.0), kv_from=2), 512),
], softcap=30.0)
# Heads above the matrix-core kernels' sizes, a state too large for one workgroup's registers
TALL = config(64, 64, [
    parallel(softmax_mixer(2, 1, 264, 16, 20, 0.02, 5), delta(2, 1, 272, 260, 3), 64),
    plain(attention(3, 1, 96, 260, 40, 0.05, rotation(96, 100.0))),
    parallel(softmax_mixer(2, 2, 40, 250, 40, 0.05, 10), delta(1, 1, 130, 24, 2), 8),
], softcap=5.0)
MODELS = {"odd": ODD, "wide": WIDE, "tall": TALL}


def weights(cfg, seed=0, rank_a=5, rank_g=7):
    """Random weights at bf16 precision, of a size that keeps every mechanism visible in the logits."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in G.tensor_shapes(cfg, rank_a, rank_g).items():
        part = name.split(".")[-1]
        if part == "conv":
            a = rng.normal(size=shape) * shape[1] ** -0.5 * 1.5
        elif len(shape) == 2:
            a = rng.normal(size=shape) * (1.0 if name == "embed" else shape[1] ** -0.5 * (2.0 if part in ("down", "o") else 1.2))
        elif part == "A_log":
            a = rng.uniform(-3.0, 1.0, size=shape)
        elif part == "dt_bias":
            a = rng.normal(size=shape) - 1.0
        else:
            a = rng.uniform(0.6, 1.4, size=shape)
        out[name] = bf16_round(a).reshape(shape)
    return out


def beacon_weights(cfg, seed=0):
    """weights() in which the last token id asks for the last but one: queries and keys of the attention are the same projection of the
    first half of the width, its values one of the second half, and the two tokens agree in the first half only.  So in the first layer
    the strongest scores of a query vocab - 1 are those of itself and of a visible key vocab - 2, whose value is another."""
    w = weights(cfg, seed)
    half = cfg["width"] // 2
    w["embed"][-1, :half] = w["embed"][-2, :half]
    for i, l in enumerate(cfg["layers"]):
        m, p = (l["mixer"]["left"], f"l{i}.mix.left") if l["type"] == "parallel" else (l["mixer"], f"l{i}.mix")
        w[p + ".k"][:, half:] = 0.0
        w[p + ".v"][:, :half] = 0.0
        q = w[p + ".k"].reshape(m["kv_heads"], m["dim"], -1)
        w[p + ".q"] = np.repeat(q, m["heads"] // m["kv_heads"], axis=0).reshape(m["heads"] * m["dim"], -1)
        w[p + ".q.norm"] = np.ones_like(w[p + ".q.norm"])
        w[p + ".k.norm"] = np.ones_like(w[p + ".k.norm"])
        w[f"l{i}.norm1"] = np.ones(cfg["width"], np.float32)
    return w
