"""Small Rikanex models for the tests: configurations, random bf16 weights, the safetensors writer."""
import json
import os
import struct

import numpy as np
import rikanex_oracle as R


def attention(heads, kv_heads, dim, vdim, window, scale, v_mix=False):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window), scale=scale, v_mix=v_mix)


def layer(mixer, mlp=None):
    return dict(type="attention", mixer=mixer, mlp=mlp)


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff):
    return dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))


def config(vocab, width, layers, embed_scale=1.0, eps=1e-5):
    return dict(architecture="Rikanex", vocab=vocab, width=width, embedding=dict(scale=embed_scale), norm=dict(eps=eps), layers=layers)


# Sizes that are padded in every way, layers of different heads, windows and feed-forwards, values mixed in some layers only
ODD = config(101, 90, [
    layer(attention(5, 5, 12, 20, 9, 0.31), moe(5, 3, 20)),
    layer(attention(6, 2, 24, 40, 7, 0.2, True), dense(70)),
    layer(attention(4, 1, 17, 9, 33, 0.4), None),
    layer(attention(2, 2, 33, 40, 130, 0.15, True), moe(70, 5, 33)),
    layer(attention(6, 2, 8, 40, 1, 0.5, True), moe(1, 1, 64)),
], embed_scale=3.5, eps=1e-3)
# More than eight query heads on one key/value head, head sizes 128 and 64, products long enough to split k
WIDE = config(700, 512, [
    layer(attention(12, 1, 128, 64, 100, 0.05, True), dense(1024)),
    layer(attention(8, 4, 64, 128, 64, 0.1), moe(3, 2, 192)),
    layer(attention(12, 1, 64, 64, 65, 0.1, True), moe(8, 1, 128)),
], embed_scale=0.5)
# Heads above the matrix-core kernel's sizes, and its largest
TALL = config(64, 64, [
    layer(attention(2, 1, 264, 16, 20, 0.02), dense(64)),
    layer(attention(2, 2, 250, 256, 40, 0.02), None),
    layer(attention(3, 1, 96, 72, 40, 0.05, True), dense(8)),
], embed_scale=2.0)
MODELS = {"odd": ODD, "wide": WIDE, "tall": TALL}


def weights(cfg, seed=0):
    """Random weights at bf16 precision, of a size that keeps every mechanism visible in the logits."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in R.tensor_shapes(cfg).items():
        part = name.split(".")[-1]
        if len(shape) == 2:
            a = rng.normal(size=shape) * (1.0 if name == "embed" else shape[1] ** -0.5 * (2.0 if part in ("down", "o") else 1.2))
        elif part == "vmix":
            a = np.array(rng.uniform(0.2, 0.8))
        elif part == "sink":
            a = rng.normal(size=shape) + 1.0
        elif part == "b":
            a = rng.normal(size=shape) * 0.2
        elif part == "correction":
            a = rng.normal(size=shape) * 0.5
        else:
            a = rng.uniform(0.6, 1.4, size=shape)
        out[name] = R.bf16_round(a).reshape(shape)
    return out


def write_folder(path, cfg, w):
    """config.json and model.safetensors (bf16)."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {"__metadata__": {"format": "pt"}}, [], 0
    for name, a in w.items():
        b = R.bf16_bits(a).tobytes()
        header[name] = dict(dtype="BF16", shape=list(np.shape(a)), data_offsets=[at, at + len(b)])
        blobs.append(b)
        at += len(b)
    head = json.dumps(header).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + b"".join(blobs))
    return str(path)


def tokens(n, vocab, seed=1):
    return np.random.default_rng(seed).integers(0, vocab, size=n).astype(np.uint32)


def beacon_weights(cfg, seed=0):
    """weights() in which the last token id asks for the last but one: queries and keys are the same projection of the first half
    of the width, values one of the second half, and the two tokens agree in the first half only.  So in the first layer the
    strongest scores of a query vocab - 1 are those of itself and of a visible key vocab - 2, whose value is another."""
    w = weights(cfg, seed)
    half = cfg["width"] // 2
    w["embed"][-1, :half] = w["embed"][-2, :half]
    for i, l in enumerate(cfg["layers"]):
        m = l["mixer"]
        w[f"l{i}.mix.k"][:, half:] = 0.0
        w[f"l{i}.mix.v"][:, :half] = 0.0
        q = w[f"l{i}.mix.k"].reshape(m["kv_heads"], m["dim"], -1)
        w[f"l{i}.mix.q"] = np.repeat(q, m["heads"] // m["kv_heads"], axis=0).reshape(m["heads"] * m["dim"], -1)
        w[f"l{i}.mix.sink"] = np.full(m["heads"], -2.0, np.float32)
        w[f"l{i}.norm1"] = np.ones(cfg["width"], np.float32)
        w[f"l{i}.norm1.b"] = np.zeros(cfg["width"], np.float32)
    return w
