"""Plain, slow CPU statement of the Rikanex decoder (test infrastructure only; shares nothing with the product path).

One function per mechanism, numpy float64 throughout.  A sequence is always evaluated whole: no cache, no chunks.
Model = (config dict as in config.json, {tensor name: array}).
"""
from __future__ import annotations

import numpy as np


def bf16_round(a):
    """Nearest bfloat16 (ties to even) of each value, as float32."""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000
    return u.astype(np.uint32).view(np.float32)


def bf16_bits(a):
    return (bf16_round(a).view(np.uint32) >> 16).astype(np.uint16)


def bf16_from_bits(u16):
    return (np.asarray(u16, dtype=np.uint16).astype(np.uint32) << 16).view(np.float32)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def linear(w, h):
    """w [out, in] applied to rows h [T, in]."""
    return h @ w.T


def layer_norm(x, w, b, eps):
    mu = x.mean(-1, keepdims=True)
    var = ((x - mu) ** 2).mean(-1, keepdims=True)
    return (x - mu) / np.sqrt(var + eps) * w + b


def unit_rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def visible(i, j, window):
    """May position i look at position j?  window None: every position up to i."""
    return j <= i and (window is None or i - j < window)


def sink_softmax(scores, sink):
    """Weights of one query over its visible keys; exp(sink) takes part in the denominator only."""
    m = max(scores.max(), sink)
    e = np.exp(scores - m)
    return e / (e.sum() + np.exp(sink - m))


def window_attention(q, k, v, scale, window, sink):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; query head h reads key/value head h // (H // G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        assert visible(i, lo, window) and visible(i, i, window) and (lo == 0 or not visible(i, lo - 1, window))
        for h in range(H):
            g = h // per
            s = (k[lo:i + 1, g] @ q[i, h]) * scale
            out[i, h] = sink_softmax(s, sink[h]) @ v[lo:i + 1, g]
    return out


def mix_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def output_gate(o, z):
    return o * sigmoid(z)


def gated_ff(h, w_gate, w_up, w_down):
    return linear(w_down, silu(linear(w_gate, h)) * linear(w_up, h))


def choose_experts(z, correction, top):
    """Router logits z [E] of one token -> (expert ids, weights): chosen by sigmoid + correction, weighted by the sigmoids."""
    s = sigmoid(z)
    ids = np.argsort(-(s + correction), kind="stable")[:top]
    w = s[ids]
    return ids, w / (w.sum() + 1e-20)


def expert_ff(h, w_router, correction, experts, top):
    """experts: list of (gate, up, down)."""
    z = linear(w_router, h)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        ids, w = choose_experts(z[t], correction, top)
        for e, we in zip(ids, w):
            out[t] += we * gated_ff(h[t:t + 1], *experts[e])[0]
    return out


def mixer(cfg, layer, w, name, h, first_v):
    """Returns (mixer output [T, width], the first mixing layer's values)."""
    mc, eps = layer["mixer"], cfg["norm"]["eps"]
    H, G, dim, vdim, T = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"], h.shape[0]
    q = unit_rms(linear(w[name + ".q"], h).reshape(T, H, dim), eps)
    k = unit_rms(linear(w[name + ".k"], h).reshape(T, G, dim), eps)
    v = linear(w[name + ".v"], h).reshape(T, G, vdim)
    if mc.get("v_mix"):
        if first_v is None:
            first_v = v
        else:
            v = mix_values(v, first_v, float(w[name + ".vmix"]))
    window = mc["mask"]["size"] if mc.get("mask") else None
    o = window_attention(q, k, v, mc["scale"], window, w[name + ".sink"]).reshape(T, H * vdim)
    return linear(w[name + ".o"], output_gate(o, linear(w[name + ".g"], h))), first_v


def feed_forward(layer, w, name, h):
    mlp = layer.get("mlp")
    if mlp is None:
        return 0.0
    if mlp["kind"] == "dense":
        return gated_ff(h, w[name + ".gate"], w[name + ".up"], w[name + ".down"])
    n = mlp["router"]["experts"]
    experts = [tuple(w[f"{name}.e{e}.{p}"] for p in ("gate", "up", "down")) for e in range(n)]
    return expert_ff(h, w[name + ".router"], w[name + ".correction"], experts, mlp["router"]["top"])


def forward(cfg, weights, ids):
    """-> (logits [T, vocab], residual stream after every layer [L, T, width])"""
    w = {k: np.asarray(a, dtype=np.float64) for k, a in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(ids)] * cfg["embedding"]["scale"]
    taps, first_v = [], None
    for i, layer in enumerate(cfg["layers"]):
        h = layer_norm(x, w[f"l{i}.norm1"], w[f"l{i}.norm1.b"], eps)
        a, first_v = mixer(cfg, layer, w, f"l{i}.mix", h, first_v)
        x = x + (a + feed_forward(layer, w, f"l{i}.mlp", h))
        taps.append(x)
    h = layer_norm(x, w["final.norm"], w["final.norm.b"], eps)
    return linear(w["head"], h), np.array(taps)


def tensor_shapes(cfg):
    """Name -> shape of every tensor of a model with this configuration."""
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, layer in enumerate(cfg["layers"]):
        mc, p = layer["mixer"], f"l{i}."
        H, G, dim, vdim = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
        out.update({p + "norm1": (d,), p + "norm1.b": (d,), p + "mix.q": (H * dim, d), p + "mix.k": (G * dim, d), p + "mix.v": (G * vdim, d),
                    p + "mix.sink": (H,), p + "mix.g": (H * vdim, d), p + "mix.o": (d, H * vdim)})
        if mc.get("v_mix"):
            out[p + "mix.vmix"] = ()
        mlp = layer.get("mlp")
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            out.update({p + "mlp.gate": (mlp["ff"], d), p + "mlp.up": (mlp["ff"], d), p + "mlp.down": (d, mlp["ff"])})
        else:
            n, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            for e in range(n):
                out.update({f"{p}mlp.e{e}.gate": (ff, d), f"{p}mlp.e{e}.up": (ff, d), f"{p}mlp.e{e}.down": (d, ff)})
            out.update({p + "mlp.router": (n, d), p + "mlp.correction": (n,)})
    out.update({"final.norm": (d,), "final.norm.b": (d,), "head": (cfg["vocab"], d)})
    return out
