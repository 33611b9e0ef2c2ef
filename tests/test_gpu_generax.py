"""GPU: the Generax decoder through the framework's session against the plain statement of the design (generax_oracle)."""
import copy
import json
import os
import subprocess
import sys

import generax_oracle as G
import numpy as np
import pytest
from decoder_checks import feed, opened, row_errors, rows_close, run
from generax_models import MODELS, ODD, attention, beacon_weights, config, delta, parallel, plain, rotation, softmax_mixer, weights
from rikanex_models import tokens, write_folder

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ("float32", "bfloat16")
# error of a row of logits: root mean square of the difference over that of the logits
LIMIT = {"float32": 2e-5, "bfloat16": 4e-2}
LENGTH = {"odd": 150, "wide": 300, "tall": 90}


def assert_close(got, want, dtype, limit=None):
    ok, text = rows_close(got, want, limit or LIMIT[dtype])
    assert ok, f"{dtype}: {text}"


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """name -> (folder, config, weights, ids, the oracle's logits and residual streams)"""
    out = {}
    for name, cfg in MODELS.items():
        w = weights(cfg)
        ids = tokens(LENGTH[name], cfg["vocab"])
        out[name] = (write_folder(tmp_path_factory.mktemp(name), cfg, w), cfg, w, ids, *G.forward(cfg, w, ids))
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_prompt(moon, ctx, folders, name, dtype):
    path, cfg, w, ids, want, taps = folders[name]
    m = opened(moon, ctx, path, dtype)
    assert_close(m.forward_logits(ids, np.arange(len(ids))), want, dtype)
    assert_close(m.hidden_f32(len(ids)), taps[-1], dtype)
    assert_close(m.logits_f32()[None], want[-1:], dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
@pytest.mark.parametrize("portions", [[1], [2], [3, 1, 7, 2, 30], [64, 1, 65], [17], [16, 15]], ids=str)
def test_portions(moon, ctx, folders, name, dtype, portions):
    path, cfg, w, ids, want, taps = folders[name]
    m = opened(moon, ctx, path, dtype)
    assert_close(feed(m, ids, portions), want, dtype)
    m.close()


@pytest.mark.parametrize("name,dtype", [("odd", "float32"), ("odd", "bfloat16"), ("tall", "float32")])
def test_residual_stream_after_every_layer(moon, ctx, folders, tmp_path, name, dtype):
    path, cfg, w, ids, want, taps = folders[name]
    for k in range(1, len(cfg["layers"]) + 1):
        m = opened(moon, ctx, write_folder(tmp_path / str(k), dict(cfg, layers=cfg["layers"][:k]), w), dtype)
        m.forward(ids)
        assert_close(m.hidden_f32(len(ids)), taps[k - 1], dtype)
        m.reset()
        feed(m, ids[:20], [1])
        assert_close(m.hidden_f32(1), taps[k - 1][19:20], dtype)  # (one token: x ends up in the same place whatever the layers are)
        m.close()


def test_wanted_places_in_any_order(moon, ctx, folders):
    path, cfg, w, ids, want, _ = folders["wide"]
    m = opened(moon, ctx, path, "float32")
    places = [299, 0, 5, 5, 150]
    assert_close(m.forward_logits(ids, places), want[places], "float32")
    m.reset()
    assert_close(m.forward_logits(ids, [298]), want[[298]], "float32")
    m.close()


# ---- every mechanism alone: the session agrees with the statement, and a statement with that mechanism changed does not agree
LEFT, RIGHT = softmax_mixer(4, 2, 16, 24, 6, 0.4, 3), delta(4, 2, 16, 24, 3)
BASE = attention(4, 2, 16, 24, 6, 0.4, rotation(8, 40.0, 1.5))
PLAIN, PARALLEL = config(60, 48, [plain(BASE)]), config(60, 48, [parallel(LEFT, RIGHT)])


def changed(path, value):
    """A configuration with one member replaced."""
    def apply(cfg):
        cfg = copy.deepcopy(cfg)
        at = cfg
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        return cfg
    return apply


def mixer(*path_value):
    return changed(("layers", 0, "mixer") + path_value[:-1], path_value[-1])


def without(name):
    """Weights with one tensor's effect taken out."""
    def apply(w):
        return {k: (np.zeros_like(v) if k.endswith(".b") or k.endswith("_bias") else np.ones_like(v)) if k.endswith(name) else v for k, v in w.items()}
    return apply


F = {name: getattr(G, name) for name in dir(G)}
BORROWS = config(60, 48, [plain(BASE), plain(BASE), plain(dict(BASE, mask=dict(size=11), kv_from=0))])


def _per_head(x, w, eps):
    n = len(w) // 16
    return F["rms_norm"](x.reshape(len(x), n, 16), w.reshape(n, 16), eps).reshape(x.shape)


def _interleaved(x, angle):
    u, v, c, s = x[..., 0::2], x[..., 1::2], np.cos(angle), np.sin(angle)
    return np.stack([u * c - v * s, v * c + u * s], -1).reshape(x.shape)


def _reads_before(S, q, k, v, g, beta):
    new, _ = F["delta_step"](S, q, k, v, g, beta)
    return new, (g[:, None] * S).T @ q


def _decays_late(S, q, k, v, g, beta):
    u = beta * (v - S.T @ k)
    S = g[:, None] * S + np.outer(k, u)
    return S, S.T @ q


def _adds_only(S, q, k, v, g, beta):
    S = g[:, None] * S + np.outer(k, beta * v)
    return S, S.T @ q


def _one_decay(a_log, dt):
    g = F["decay"](a_log, dt)
    return np.broadcast_to(g.mean(-1, keepdims=True), g.shape)


# what -> (configuration, changed configuration, changed function of the statement, changed weights)
MECHANISMS = {
    "norm eps": (changed(("norm", "eps"), 0.3)(PLAIN), changed(("norm", "eps"), 0.2), None, None),
    "norm eps beside the delta rule": (changed(("norm", "eps"), 0.3)(PARALLEL), changed(("norm", "eps"), 0.2), None, None),
    "norm weight": (PLAIN, None, None, without("norm1")),
    "soft cap": (changed(("logit_softcap",), 2.0)(PLAIN), changed(("logit_softcap",), 2.5), None, None),
    "no soft cap": (changed(("logit_softcap",), None)(PLAIN), changed(("logit_softcap",), 3.0), None, None),
    "feed-forward": (config(60, 48, [plain(BASE, 40)]), None, ("gated_ff", lambda h, gate, up, down: G.linear(down, G.linear(gate, h) * G.linear(up, h))), None),
    "feed-forward beside the delta rule": (config(60, 48, [parallel(LEFT, RIGHT, 40)]), lambda c: PARALLEL, None, None),
    "norm of all of q": (PLAIN, None, ("whole_norm", _per_head), None),
    "norm of all of q, blocks": (PARALLEL, None, ("whole_norm", _per_head), None),
    "q norm weight": (PLAIN, None, None, without("q.norm")),
    "k norm weight": (PARALLEL, None, None, without("k.norm")),
    "score scale": (PLAIN, mixer("scale", 0.5), None, None),
    "score scale, blocks": (PARALLEL, mixer("left", "scale", 0.5), None, None),
    "factor per head": (PLAIN, None, None, without("temp")),
    "window one longer": (PLAIN, mixer("mask", dict(size=7)), None, None),
    "window one shorter": (PLAIN, mixer("mask", dict(size=5)), None, None),
    "window before blocks one longer": (PARALLEL, mixer("left", "mask", "size", 7), None, None),
    "window before blocks one shorter": (PARALLEL, mixer("left", "mask", "size", 5), None, None),
    "larger blocks": (PARALLEL, mixer("left", "mask", "pool", 4), None, None),
    "no blocks": (PARALLEL, mixer("left", "mask", dict(size=6)), None, None),
    "blocks one token early": (PARALLEL, None, ("block_visible", lambda i, b, w, p: F["block_visible"](i + 1, b, w, p)), None),
    "blocks one token late": (PARALLEL, None, ("block_visible", lambda i, b, w, p: F["block_visible"](i - 1, b, w, p)), None),
    "sums for means": (PARALLEL, None, ("pooled", lambda x, p: F["pooled"](x, p) * p), None),
    "positions that do not turn": (PLAIN, None, ("frequencies", lambda dims, base, factor: np.zeros(dims // 2)), None),
    "turned dimensions": (PLAIN, mixer("rot", "dims", 10), None, None),
    "rotation base": (PLAIN, mixer("rot", "base", 50.0), None, None),
    "rotation factor": (PLAIN, mixer("rot", "scaling", "factor", 1.0), None, None),
    "no rotation factor": (config(60, 48, [plain(attention(4, 2, 16, 24, 6, 0.4, rotation(16, 40.0)))]), mixer("rot", "scaling", dict(factor=1.25)), None, None),
    "pairs side by side": (PLAIN, None, ("turn", _interleaved), None),
    "values that do not turn": (PLAIN, None, ("rotate_values", lambda v, base: v), None),
    "outputs that do not turn back": (PLAIN, None, ("rotate_back", lambda o, base: o), None),
    "the factor on values": (PLAIN, None, ("frequencies", lambda dims, base, factor: F["frequencies"](dims, base, 1.5)), None),
    "grouped heads": (PLAIN, None, ("attention", lambda q, k, v, *a: F["attention"](q, k[:, ::-1], v[:, ::-1], *a)), None),
    "another layer's keys": (BORROWS, changed(("layers", 2, "mixer", "kv_from"), 1), None, None),
    "the borrower's own window": (BORROWS, changed(("layers", 2, "mixer", "mask", "size"), 6), None, None),
    "convolution order": (PARALLEL, None, ("short_conv", lambda x, w: F["short_conv"](x, w[:, ::-1])), None),
    "convolution": (PARALLEL, None, ("short_conv", lambda x, w: x * w[:, -1]), None),
    "activation behind the convolution": (PARALLEL, None, ("silu", lambda z: z), None),
    "unit vectors": (PARALLEL, None, ("unit", lambda x: x), None),
    "decay": (PARALLEL, None, ("decay", lambda a, dt: np.ones_like(dt)), None),
    "decay per channel": (PARALLEL, None, ("decay", _one_decay), None),
    "decay's own step": (PARALLEL, None, None, without("dt_bias")),
    "step sizes": (PARALLEL, None, None, without("right.b")),
    "read-out behind the write": (PARALLEL, None, ("delta_step", _reads_before), None),
    "decay before the write": (PARALLEL, None, ("delta_step", _decays_late), None),
    "what the state holds is taken off": (PARALLEL, None, ("delta_step", _adds_only), None),
    "norm of a head's output": (PARALLEL, None, None, without("right.norm")),
    "output gate": (PARALLEL, None, None, lambda w: {k: v * 0 if k.endswith("g2") else v for k, v in w.items()}),
    "shared heads of the delta rule": (PARALLEL, None, ("heads_of", lambda x, n: F["heads_of"](x, n)[:, ::-1] if n == 2 else F["heads_of"](x, n)), None),
    "left norm": (PARALLEL, None, None, without("left.out")),
    "right norm": (PARALLEL, None, None, without("right.out")),
    "norms before the sum": (PARALLEL, None, ("join", lambda l, r, a, b, eps: 0.5 * (l * a + r * b)), None),
    "half the sum": (PARALLEL, None, ("join", lambda *a: 2 * F["join"](*a)), None),
}


@pytest.mark.parametrize("what", sorted(MECHANISMS))
def test_mechanism(moon, ctx, tmp_path, monkeypatch, what):
    cfg, other_cfg, patch, other_w = MECHANISMS[what]
    w, ids = weights(cfg, 3), tokens(40, cfg["vocab"], 4)
    want, _ = G.forward(cfg, w, ids)
    if patch:
        monkeypatch.setattr(G, *patch)
    wrong, _ = G.forward(other_cfg(cfg) if other_cfg else cfg, other_w(w) if other_w else w, ids)
    for dtype in DTYPES:
        for portions in ([len(ids)], [1], [13, 2]):
            got = run(moon, ctx, tmp_path, cfg, w, ids, dtype, portions)
            assert_close(got, want, dtype)
            if dtype == "float32":
                assert not rows_close(got, wrong, 5e-3)[0]


# ---- keys just inside and just outside a window or a block, at the first tokens and far away
def beacon_at(cfg, first, count, length, seed):
    ids = np.random.default_rng(seed).permutation(cfg["vocab"] - 2)[:length].astype(np.uint32)
    ids[first:first + count], ids[-1] = cfg["vocab"] - 2, cfg["vocab"] - 1
    return ids


def check_edge(moon, ctx, tmp_path, cfg, w, ids):
    want, _ = G.forward(cfg, w, ids)
    for portions in ([len(ids)], [len(ids) - 1, 1], [len(ids) - 3, 2, 1], [50]):
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "float32", portions), want, "float32")
    for portions in ([len(ids)], [len(ids) - 1, 1]):
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "bfloat16", portions)[-1:], want[-1:], "bfloat16", 0.1)


@pytest.mark.parametrize("window", [2, 63, 64, 65, 129])
def test_window_edge(moon, ctx, tmp_path, window):
    """The last token asks for one earlier token, which sits at the edge of the window."""
    def model(size):
        return config(400, 64, [plain(attention(4, 1, 32, 16, size, 0.6, rotation(2, 1000.0, 30.0)))], softcap=40.0)
    w = beacon_weights(model(window))
    for far in (window - 1, window, window + 1):
        ids = beacon_at(model(window), 39, 1, far + 40, far)
        want, wrong = G.forward(model(window), w, ids)[0], G.forward(model(window + 1), w, ids)[0]
        assert (row_errors(want[-1:], wrong[-1:])[0] > 0.01) == (far == window)  # the case tells the two apart
        check_edge(moon, ctx, tmp_path, model(window), w, ids)


@pytest.mark.parametrize("window,pool", [(1, 1), (1, 4), (6, 4), (3, 7), (64, 5), (40, 64), (130, 3), (20, 2)])
def test_block_edge(moon, ctx, tmp_path, monkeypatch, window, pool):
    """The last token asks for the tokens of one block, whose last one sits at the edge of the window, or far before it."""
    def model(size):
        return config(400, 64, [parallel(softmax_mixer(4, 1, 32, 16, size, 0.6, pool), delta(2, 1, 16, 16, 2))], softcap=40.0)
    w = beacon_weights(model(window))
    w["l0.mix.right.out"] *= 0.25
    first = (40 + pool - 1) // pool * pool
    for behind in (window - 1, window, window + 1, window + 100):  # from the block's last token to the last token
        ids = beacon_at(model(window), first, pool, first + pool + behind, behind)
        want, _ = G.forward(model(window), w, ids)
        with monkeypatch.context() as planted:
            planted.setattr(G, "block_visible", lambda i, b, w, p: F["block_visible"](i - 1, b, w, p))
            wrong, _ = G.forward(model(window), w, ids)
        # seen one token late, the block is missed where it is seen only just
        assert behind != window or row_errors(want[-1:], wrong[-1:])[0] > 0.01
        check_edge(moon, ctx, tmp_path, model(window), w, ids)


def test_far_block_stands_out(moon, ctx, tmp_path):
    """One block among hundreds, thousands of positions back."""
    cfg = config(64, 64, [parallel(softmax_mixer(2, 1, 32, 16, 30, 3.0, 8), delta(2, 1, 16, 16, 2))], softcap=40.0)
    w = beacon_weights(cfg, 2)
    ids = tokens(2600, 62, 5)
    ids[80:88], ids[-1] = 62, 63
    want, _ = G.forward(cfg, w, ids)
    ids2 = ids.copy()
    ids2[80:88] = ids[88:96]
    assert row_errors(want[-1:], G.forward(cfg, w, ids2)[0][-1:])[0] > 0.05
    for portions in ([2600], [2599, 1], [700, 2], [2590, 1]):
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "float32", portions, 2700)[-1:], want[-1:], "float32")


def test_first_tokens(moon, ctx, folders):
    path, cfg, w, ids, want, _ = folders["odd"]
    for dtype in DTYPES:
        m = opened(moon, ctx, path, dtype)
        for n in (1, 2, 3, 5):
            m.reset()
            assert_close(m.forward_logits(ids[:n], np.arange(n)), want[:n], dtype)
        m.close()


def test_scores_that_would_overflow(moon, ctx, tmp_path):
    cfg = config(60, 48, [plain(dict(BASE, scale=40.0)), parallel(dict(LEFT, scale=-40.0), RIGHT)])
    w, ids = weights(cfg, 5), tokens(50, 60, 6)
    w["l0.mix.temp"] = np.array([1.0, -2.0, 0.0, 30.0], np.float32)
    want, _ = G.forward(cfg, w, ids)
    for portions in ([50], [1], [9]):
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "float32", portions), want, "float32", 1e-3)
        assert np.isfinite(run(moon, ctx, tmp_path, cfg, w, ids, "bfloat16", portions)).all()


def test_strong_and_weak_decays(moon, ctx, tmp_path):
    """States that vanish within a token, and states that stay for the whole sequence, beside each other."""
    cfg = config(60, 48, [parallel(LEFT, RIGHT)])
    w, ids = weights(cfg, 8), tokens(200, 60, 9)
    w["l0.mix.right.A_log"] = np.array([6.0, -12.0, 3.0, 0.0], np.float32)
    w["l0.mix.right.dt_bias"][::2] = 40.0
    w["l0.mix.right.dt_bias"][1::2] = -30.0
    want, _ = G.forward(cfg, w, ids)
    for portions in ([200], [1], [33, 2]):
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "float32", portions), want, "float32")
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "bfloat16", portions), want, "bfloat16")


def test_repeated_keys(moon, ctx, tmp_path):
    """The same token again and again with step sizes near 1: every write first takes off what the last one left."""
    cfg = config(60, 48, [parallel(LEFT, RIGHT)])
    w = weights(cfg, 10)
    w["l0.mix.right.b"] *= 8.0
    w["l0.mix.right.dt_bias"][:] = -8.0
    ids = np.repeat(tokens(6, 60, 11), 25)
    want, _ = G.forward(cfg, w, ids)
    for portions in ([150], [1], [47, 16]):
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "float32", portions), want, "float32", 5e-5)


@pytest.mark.parametrize("rank_a,rank_g", [(1, 1), (64, 64), (40, 9), (3, 130)])
def test_ranks_of_the_two_step_projections(moon, ctx, tmp_path, rank_a, rank_g):
    w, ids = weights(PARALLEL, 12, rank_a, rank_g), tokens(40, 60, 13)
    want, _ = G.forward(PARALLEL, w, ids)
    for dtype in DTYPES:
        for portions in ([40], [1], [5]):
            assert_close(run(moon, ctx, tmp_path, PARALLEL, w, ids, dtype, portions), want, dtype)


# ---- cache rows, blocks and states
RING = config(50, 32, [parallel(softmax_mixer(2, 1, 16, 16, 100, 0.5, 9), delta(2, 1, 16, 16, 4), 32), plain(attention(2, 1, 8, 16, 30, 0.7, rotation(4, 3000.0))),
                       plain(attention(2, 1, 8, 16, 77, 0.7, rotation(4, 3000.0), kv_from=1))])


@pytest.mark.parametrize("dtype", DTYPES)
def test_cache_rows_are_used_again(moon, ctx, tmp_path, dtype):
    """A sequence longer than the rows a windowed layer keeps: prompts of several calls' rows, then tokens, around the end of the
    rows; then another sequence in the same session."""
    w, ids = weights(RING, 7), tokens(4500, 50, 8)
    want, _ = G.forward(RING, w, ids)
    m = opened(moon, ctx, write_folder(tmp_path / "m", RING, w), dtype, 5000)
    got = m.forward_logits(ids[:2120], np.arange(2120))  # (2048 rows a call: the rest is a second one)
    assert_close(got, want[:2120], dtype)
    got = feed(m, ids[2120:2180], [1])  # over the end of the first layer's rows
    assert_close(got, want[2120:2180], dtype)
    got = feed(m, ids[2180:], [1000, 1, 3, 700])
    assert_close(got, want[2180:], dtype)
    m.reset()
    short = ids[100:160]
    assert_close(feed(m, short, [20, 1, 1, 38]), G.forward(RING, w, short)[0], dtype)
    m.close()


def test_sequences_do_not_see_each_other(moon, ctx, folders):
    """A long sequence, then short ones in the same session, begun with one token or with several; and two sessions in turn."""
    path, cfg, w, ids, want, _ = folders["odd"]
    m, o = opened(moon, ctx, path, "float32"), opened(moon, ctx, path, "float32", 200)
    other = tokens(30, cfg["vocab"], 77)
    want_other, _ = G.forward(cfg, w, other)
    for first in (1, 2, 30):
        m.reset()
        m.forward(ids)
        m.reset()
        assert_close(feed(m, other, [first, 4]), want_other, "float32")
    m.reset()
    got, got_other = [], []
    for i in range(0, 30, 5):
        got.append(m.forward_logits(ids[i:i + 5], np.arange(5)))
        got_other.append(feed(o, other[i:i + 5], [1, 4]))
    assert_close(np.concatenate(got), want[:30], "float32")
    assert_close(np.concatenate(got_other), want_other, "float32")
    m.close()
    o.close()


def test_full_cache_is_refused(moon, ctx, folders):
    """A refused call changes nothing, also not the recurrent state."""
    path, cfg, w, ids, want, _ = folders["odd"]
    m = opened(moon, ctx, path, "float32", 20)
    m.forward(ids[:18])
    with pytest.raises(moon.SequenceTooLong):
        m.forward(ids[:3])
    with pytest.raises(moon.TokenIdOutOfBounds):
        m.forward([0, cfg["vocab"]])
    assert_close(m.forward_logits(ids[18:20], np.arange(2)), want[18:20], "float32")
    m.close()


def test_cache_shorter_than_a_block(moon, ctx, tmp_path):
    cfg = config(60, 48, [parallel(softmax_mixer(4, 2, 16, 24, 2, 0.4, 64), RIGHT)])
    w, ids = weights(cfg, 3), tokens(10, 60, 4)
    want, _ = G.forward(cfg, w, ids)
    for portions in ([10], [1]):
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "float32", portions, 10), want, "float32")


# ---- generation through the session's loop
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_greedy_generation(moon, ctx, folders, name):
    """Every generated token is the oracle's arg-max at its place (or within rounding of it), over more tokens than the windows hold."""
    path, cfg, w, ids, _, _ = folders[name]
    for dtype in DTYPES:
        m = opened(moon, ctx, path, dtype)
        m.forward(ids[:11])
        out = m.greedy(140)
        assert m.position == 151
        logits, _ = G.forward(cfg, w, np.concatenate([ids[:11], out]))
        at = logits[10:150]
        slack = at.max(-1) - at[np.arange(140), out]
        assert (slack <= 4 * LIMIT[dtype] * at.std()).all(), slack.max()
        m.reset()
        m.forward(ids[:11])
        again = []
        for _ in range(20):
            again.append(m.next_token())
            m.forward([again[-1]])
        assert again == out[:20].tolist()
        m.close()


@pytest.mark.parametrize("sampled", [False, True])
def test_stopped_generation(moon, ctx, folders, sampled):
    """Steps that were queued behind the end of a generation leave no trace in the state."""
    path, cfg, w, ids, _, _ = folders["odd"]
    m = opened(moon, ctx, path, "float32", 200)
    sampler = moon.sampling.sampling_config("top_k", temperature=0.7, top_k=5) if sampled else None
    u = np.random.default_rng(0).random(40).astype(np.float32) if sampled else None
    m.forward(ids[:9])
    out = m.sample(sampler, u) if sampled else m.greedy(40)
    eos = next(int(t) for i, t in enumerate(out) if i >= 3 and t not in out[:i])
    first = out.tolist().index(eos)
    m.reset()
    m.forward(ids[:9])
    got = m.generate(40, eos, sampler, u)
    assert got.tolist() == out[:first].tolist() and m.position == 9 + first
    more = tokens(12, cfg["vocab"], 9)
    want, _ = G.forward(cfg, w, np.concatenate([ids[:9], out[:first], more]))
    assert_close(feed(m, more, [1, 3]), want[-12:], "float32")
    m.close()


def test_random_weights(moon, ctx):
    cfg = config(640, 128, [parallel(softmax_mixer(4, 2, 32, 32, 50, 0.2, 8), delta(4, 2, 32, 32, 4), 192), plain(attention(4, 2, 32, 32, 50, 0.2, rotation(32, 1e4)), 192)])
    m = moon.text_model.TextModel.open_synthetic(cfg, "bfloat16", 256, seed=3, std=0.05, ctx=ctx)
    ids = tokens(70, 640)
    a = m.forward_logits(ids, np.arange(70))
    m.reset()
    assert_close(feed(m, ids, [40, 1]), a, "bfloat16")
    m.close()
    with pytest.raises(moon.MoonError):
        moon.text_model.TextModel.open_synthetic(ODD, ctx=ctx)


# ---- programs
def test_command_line(moon, ctx, folders):
    path, cfg, w, ids, _, _ = folders["odd"]
    m = opened(moon, ctx, path, "float32")
    m.forward(ids[:5])
    want = m.greedy(8).tolist()
    m.close()
    cmd = [sys.executable, os.path.join(ROOT, "moondream-zig_amd"), "generate", "--model", path, "--dtype", "float32", "--ids", ",".join(map(str, ids[:5])),
           "--tokens", "8"]
    r = subprocess.run(cmd, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [int(t) for t in r.stdout.strip().split(",")] == want


def test_trace_program(moon, ctx, folders, tmp_path):
    path, cfg, w, ids, want, _ = folders["odd"]
    toks = [int(t) for t in ids]
    steps = [dict(step=0, entries=[dict(id="a", tokens=toks[:30], want=[0, 29])], end=[]),
             dict(step=1, entries=[dict(id="a", tokens=toks[30:32], want=[])], end=[]),
             dict(step=2, entries=[dict(id="a", tokens=toks[32:33], want=[0])], end=["a"]),
             dict(step=3, entries=[dict(id="b", tokens=toks[:2], want=[1])], end=["b"])]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "40"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    for i, rows in ((0, [0, 29]), (2, [32]), (3, [1])):
        got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(len(rows), cfg["vocab"])
        assert_close(got, want[rows], "float32")
