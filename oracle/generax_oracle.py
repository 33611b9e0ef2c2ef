"""Plain, slow CPU statement of the Generax decoder (test infrastructure only; shares nothing with the product path).

One function per mechanism, numpy float64 throughout.  A sequence is always evaluated whole: no cache, no chunks, the recurrence
token by token.  Model = (config dict as in config.json, {tensor name: array}).
"""
from __future__ import annotations

import numpy as np
from rikanex_oracle import gated_ff, linear, sigmoid, silu


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def softplus(z):
    return np.logaddexp(0.0, z)


# ---- rotation: pair m of the first `dims` dimensions is (m, m + dims / 2)
def frequencies(dims, base, factor):
    return base ** (-2.0 * np.arange(dims // 2) / dims) / factor


def turn(x, angle):
    """x [..., dims] turned pair by pair by angle [..., dims / 2]."""
    half = x.shape[-1] // 2
    u, v = x[..., :half], x[..., half:]
    c, s = np.cos(angle), np.sin(angle)
    return np.concatenate([u * c - v * s, v * c + u * s], -1)


def rotate_heads(x, dims, base, factor):
    """x [T, heads, size]: the first `dims` dimensions of each head turn with the position, the others stay."""
    a = np.arange(x.shape[0])[:, None, None] * frequencies(dims, base, factor)
    return np.concatenate([turn(x[..., :dims], a), x[..., dims:]], -1)


def rotate_values(v, base):
    return rotate_heads(v, v.shape[-1], base, 1.0)


def rotate_back(o, base):
    return turn(o, -np.arange(o.shape[0])[:, None, None] * frequencies(o.shape[-1], base, 1.0))


# ---- attention
def whole_norm(x, w, eps):
    """All rows of a projection at once, before they are heads."""
    return rms_norm(x, w, eps)


def visible(i, j, window):
    return j <= i and (window is None or i - j < window)


def block_visible(i, b, window, pool):
    """Is block b (positions b pool .. b pool + pool - 1) wholly before the window of position i?"""
    return b * pool + pool - 1 <= i - window


def pooled(x, pool):
    """Means of the whole blocks, [T // pool, heads, size]."""
    n = x.shape[0] // pool
    return x[:n * pool].reshape(n, pool, *x.shape[1:]).mean(1)


def softmax(s):
    e = np.exp(s - s.max())
    return e / e.sum()


def attention(q, k, v, scale, window, pool=None):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim]; scale [H].  Tokens in the window and, with pool, the blocks before it share
    one softmax."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    kb, vb = (pooled(k, pool), pooled(v, pool)) if pool else (k[:0], v[:0])
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        lo = 0 if window is None else next(j for j in range(max(0, i - window - 1), i + 1) if visible(i, j, window))
        n = next(b for b in range(max(0, (i - (window or 0)) // pool - 2), len(kb) + 1) if b == len(kb) or not block_visible(i, b, window, pool)) if pool else 0
        keys, values = np.concatenate([kb[:n], k[lo:i + 1]]), np.concatenate([vb[:n], v[lo:i + 1]])
        for h in range(H):
            out[i, h] = softmax(keys[:, h // per] @ q[i, h] * scale[h]) @ values[:, h // per]
    return out


def heads_of(x, n):
    return x.reshape(x.shape[0], n, -1)


def keys_values(mc, w, p, h, eps):
    """The keys and values a layer's cache holds: normed and rotated."""
    G = mc["kv_heads"]
    k = heads_of(whole_norm(linear(w[p + ".k"], h), w[p + ".k.norm"], eps), G)
    v = heads_of(linear(w[p + ".v"], h), G)
    if mc.get("rot"):
        r = mc["rot"]
        k = rotate_heads(k, r["dims"], r["base"], r.get("scaling", {}).get("factor", 1.0))
        v = rotate_values(v, r["base"])
    return k, v


def softmax_mixer(mc, w, p, h, eps, kv):
    """-> (output before the output projection [T, H vdim], the keys and values used)"""
    H, rot = mc["heads"], mc.get("rot")
    q = heads_of(whole_norm(linear(w[p + ".q"], h), w[p + ".q.norm"], eps), H)
    if rot:
        q = rotate_heads(q, rot["dims"], rot["base"], rot.get("scaling", {}).get("factor", 1.0))
    k, v = kv if kv is not None else keys_values(mc, w, p, h, eps)
    scale = mc["scale"] * w.get(p + ".temp", np.ones(H))
    mask = mc.get("mask") or {}
    o = attention(q, k, v, scale, mask.get("size"), mask.get("pool"))
    if rot:
        o = rotate_back(o, rot["base"])
    return linear(w[p + ".o"], o.reshape(len(h), -1)), (k, v)


# ---- gated delta rule
def short_conv(x, w):
    """Causal convolution per channel: x [T, C], w [C, taps], the last column is the current token's."""
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(padded[t:t + len(x)] * w[:, t] for t in range(taps))


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def decay(a_log, dt):
    """dt [..., heads, dim] (before the softplus), a_log [heads] -> the factor on the state's rows."""
    return np.exp(-np.exp(a_log)[:, None] * softplus(dt))


def delta_step(S, q, k, v, g, beta):
    """One token of one head: S [dim, vdim] -> (new S, output)."""
    S = g[:, None] * S
    u = beta * (v - S.T @ k)
    S = S + np.outer(k, u)
    return S, S.T @ q


def delta_mixer(mc, w, p, h, eps):
    T, H, G, dim, vdim = len(h), mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    q, k, v = (silu(short_conv(linear(w[f"{p}.{n}"], h), w[f"{p}.{n}.conv"])) for n in "qkv")
    q, k, v = unit(heads_of(q, G)) * dim**-0.5, unit(heads_of(k, G)), heads_of(v, H)
    beta = sigmoid(linear(w[p + ".b"], h))
    g = decay(w[p + ".A_log"], heads_of(linear(w[p + ".a2"], linear(w[p + ".a1"], h)) + w[p + ".dt_bias"], H))
    gate = sigmoid(heads_of(linear(w[p + ".g2"], linear(w[p + ".g1"], h)), H))
    o = np.zeros((T, H, vdim))
    for n in range(H):
        S = np.zeros((dim, vdim))
        c = n // (H // G)
        for t in range(T):
            S, o[t, n] = delta_step(S, q[t, c], k[t, c], v[t, n], g[t, n], beta[t, n])
    o = rms_norm(o, w[p + ".norm"], eps) * gate
    return linear(w[p + ".o"], o.reshape(T, -1))


def join(left, right, w_left, w_right, eps):
    return 0.5 * (rms_norm(left, w_left, eps) + rms_norm(right, w_right, eps))


# ---- the model
def mixer(cfg, i, w, h, kv):
    layer, p, eps = cfg["layers"][i], f"l{i}.mix", cfg["norm"]["eps"]
    mc = layer["mixer"]
    if layer["type"] == "parallel":
        left, _ = softmax_mixer(mc["left"], w, p + ".left", h, eps, None)
        right = delta_mixer(mc["right"], w, p + ".right", h, eps)
        return join(left, right, w[p + ".left.out"], w[p + ".right.out"], eps)
    out, kv[i] = softmax_mixer(mc, w, p, h, eps, kv[mc["kv_from"]] if "kv_from" in mc else None)
    return out


def softcap(z, cap):
    return cap * np.tanh(z / cap)


def forward(cfg, weights, ids):
    """-> (logits [T, vocab], residual stream after every layer [L, T, width])"""
    w = {k: np.asarray(a, dtype=np.float64) for k, a in weights.items()}
    eps, x, taps, kv = cfg["norm"]["eps"], w["embed"][np.asarray(ids)], [], {}
    for i, layer in enumerate(cfg["layers"]):
        h = rms_norm(x, w[f"l{i}.norm1"], eps)
        out = mixer(cfg, i, w, h, kv)
        if layer.get("mlp"):
            out = out + gated_ff(h, *(w[f"l{i}.mlp.{n}"] for n in ("gate", "up", "down")))
        x = x + out
        taps.append(x)
    z = linear(w["head"], rms_norm(x, w["final.norm"], eps))
    return softcap(z, cfg["logit_softcap"]) if cfg.get("logit_softcap") else z, np.array(taps)


def tensor_shapes(cfg, rank_a=5, rank_g=7):
    """Name -> shape of every tensor of a model with this configuration; the ranks of the two-step projections are free."""
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}

    def softmax_shapes(p, m):
        H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.update({p + ".q": (H * dim, d), p + ".q.norm": (H * dim,), p + ".o": (d, H * vdim)})
        if "kv_from" not in m:
            out.update({p + ".k": (G * dim, d), p + ".k.norm": (G * dim,), p + ".v": (G * vdim, d)})

    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        out[p + "norm1"] = (d,)
        if layer["type"] == "parallel":
            softmax_shapes(p + "mix.left", m["left"])
            r, n = p + "mix.right", m["right"]
            H, G, dim, vdim, taps = n["heads"], n["kv_heads"], n["dim"], n["vdim"], n["conv"]
            for what, rows in (("q", G * dim), ("k", G * dim), ("v", H * vdim)):
                out[f"{r}.{what}"], out[f"{r}.{what}.conv"] = (rows, d), (rows, taps)
            out.update({r + ".b": (H, d), r + ".A_log": (H,), r + ".norm": (vdim,), r + ".a1": (rank_a, d), r + ".a2": (H * dim, rank_a),
                        r + ".dt_bias": (H * dim,), r + ".g1": (rank_g, d), r + ".g2": (H * vdim, rank_g), r + ".o": (d, H * vdim),
                        p + "mix.left.out": (d,), r + ".out": (d,)})
        else:
            softmax_shapes(p + "mix", m)
            out[p + "mix.temp"] = (m["heads"],)
        if layer.get("mlp"):
            ff = layer["mlp"]["ff"]
            out.update({p + "mlp.gate": (ff, d), p + "mlp.up": (ff, d), p + "mlp.down": (d, ff)})
    out.update({"final.norm": (d,), "head": (cfg["vocab"], d)})
    return out
