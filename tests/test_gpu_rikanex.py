"""GPU: the Rikanex decoder through the framework's session against the plain statement of the design (rikanex_oracle)."""
import os
import subprocess
import sys

import numpy as np
import pytest
import rikanex_oracle as R
from decoder_checks import feed, opened, row_errors, rows_close, run
from rikanex_models import (MODELS, ODD, TALL, WIDE, attention, config, dense, beacon_weights, layer, moe, tokens, weights, write_folder)

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ("float32", "bfloat16")
# error of a row of logits: root mean square of the difference over that of the logits
LIMIT = {"float32": 2e-5, "bfloat16": 3e-2}
LENGTH = {"odd": 150, "wide": 300, "tall": 70}


# In bf16 a router's close call may fall the other way (in f32 none of these does): that many rows may be over the limit.
FLIPS = {"float32": 0.0, "bfloat16": 0.03}


def close(got, want, dtype, limit=None):
    return rows_close(got, want, limit or LIMIT[dtype], FLIPS[dtype])


def assert_close(got, want, dtype, limit=None):
    ok, text = close(got, want, dtype, limit)
    assert ok, f"{dtype}: {text}"


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """name -> (folder, config, weights, ids, the oracle's logits and residual streams)"""
    out = {}
    for name, cfg in MODELS.items():
        w = weights(cfg)
        ids = tokens(LENGTH[name], cfg["vocab"])
        out[name] = (write_folder(tmp_path_factory.mktemp(name), cfg, w), cfg, w, ids, *R.forward(cfg, w, ids))
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_prompt(moon, ctx, folders, name, dtype):
    path, cfg, w, ids, want, taps = folders[name]
    m = opened(moon, ctx, path, dtype)
    assert_close(m.forward_logits(ids, np.arange(len(ids))), want, dtype)
    assert_close(m.hidden_f32(len(ids)), taps[-1], dtype)
    assert m.position == len(ids)
    assert_close(m.logits_f32()[None], want[-1:], dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
def test_token_by_token(moon, ctx, folders, name, dtype):
    path, cfg, w, ids, want, taps = folders[name]
    m = opened(moon, ctx, path, dtype)
    assert_close(feed(m, ids, [1]), want, dtype)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(MODELS))
@pytest.mark.parametrize("portions", [[2], [3, 1, 7, 2, 30], [64, 1, 65], [17]], ids=str)
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
        m.close()


def test_wanted_places_in_any_order(moon, ctx, folders):
    path, cfg, w, ids, want, _ = folders["wide"]
    m = opened(moon, ctx, path, "float32")
    places = [299, 0, 5, 5, 150]
    assert_close(m.forward_logits(ids, places), want[places], "float32")
    m.reset()
    assert m.forward_logits(ids, []).shape == (0, cfg["vocab"])
    m.reset()
    assert_close(m.forward_logits(ids, [298]), want[[298]], "float32")
    with pytest.raises(moon.MoonError):
        m.forward_logits(ids[:3], [3])
    m.close()


# ---- every mechanism alone: the session agrees with the statement, and a statement with that mechanism changed does not agree
BASE = attention(4, 2, 16, 24, 6, 0.4)


def one(mixer=BASE, mlp=None, **kw):
    return config(60, 48, [layer(mixer, mlp)], **kw)


def two(mixer, mlp=None):
    return config(60, 48, [layer(mixer, mlp), layer(mixer, mlp)])


def _no_correction(z, correction, top):
    return R_choose(z, 0 * correction, top)


def _corrected_weights(z, correction, top):
    ids, _ = R_choose(z, correction, top)
    s = (R.sigmoid(z) + correction)[ids]
    return ids, s / s.sum()


def _unnormalised(z, correction, top):
    ids, _ = R_choose(z, correction, top)
    return ids, R.sigmoid(z)[ids]


R_choose, R_window, R_norm = R.choose_experts, R.window_attention, R.layer_norm
MECHANISMS = {
    "embedding scale": (one(embed_scale=0.125, eps=0.5), lambda c: dict(c, embedding=dict(scale=0.25)), None),
    "norm eps": (one(eps=0.3), lambda c: dict(c, norm=dict(eps=0.2)), None),
    "norm mean": (one(), None, ("layer_norm", lambda x, w, b, eps: R.unit_rms(x, eps) * w + b)),
    "norm bias": (one(), None, ("layer_norm", lambda x, w, b, eps: R_norm(x, w, 0 * b, eps))),
    "q and k norm": (one(), None, ("unit_rms", lambda x, eps: x)),
    "score scale": (one(), lambda c: one(dict(BASE, scale=0.5)), None),
    "window one longer": (one(), lambda c: one(dict(BASE, mask=dict(size=7))), None),
    "window one shorter": (one(), lambda c: one(dict(BASE, mask=dict(size=5))), None),
    "window of one": (one(dict(BASE, mask=dict(size=1))), lambda c: one(dict(BASE, mask=dict(size=2))), None),
    "sink": (one(), None, ("sink_softmax", lambda s, sink: np.exp(s - s.max()) / np.exp(s - s.max()).sum())),
    "sink not scaled": (one(), None, ("sink_softmax", lambda s, sink: np.exp(s) / (np.exp(s).sum() + np.exp(0.4 * sink)))),
    "grouped heads": (one(), None, ("window_attention", lambda q, k, v, *a: R_window(q, k[:, ::-1], v[:, ::-1], *a))),
    "heads beside groups": (one(), None, ("window_attention", lambda q, k, v, *a: R_window(q, np.tile(k, (1, 2, 1)), np.tile(v, (1, 2, 1)), *a))),
    "value mixing": (two(dict(BASE, v_mix=True)), None, ("mix_values", lambda v, first, lam: v)),
    "value mixing the other way": (two(dict(BASE, v_mix=True)), None, ("mix_values", lambda v, first, lam: lam * v + (1 - lam) * first)),
    "output gate": (one(), None, ("output_gate", lambda o, z: o)),
    "output gate activation": (one(), None, ("output_gate", lambda o, z: o * R.silu(z))),
    "dense feed-forward": (one(mlp=dense(40)), None, ("silu", lambda z: z * (z > 0))),
    "experts": (one(mlp=moe(6, 2, 24)), None, ("silu", lambda z: z * (z > 0))),
    "experts' correction": (one(mlp=moe(6, 2, 24)), None, ("choose_experts", _no_correction)),
    "weights without the correction": (one(mlp=moe(6, 2, 24)), None, ("choose_experts", _corrected_weights)),
    "weights over their sum": (one(mlp=moe(6, 3, 24)), None, ("choose_experts", _unnormalised)),
    "all experts": (one(mlp=moe(3, 3, 8)), lambda c: one(mlp=moe(3, 2, 8)), None),
}


@pytest.mark.parametrize("what", sorted(MECHANISMS))
def test_mechanism(moon, ctx, tmp_path, monkeypatch, what):
    cfg, other_cfg, patch = MECHANISMS[what]
    w, ids = weights(cfg, 3), tokens(40, cfg["vocab"], 4)
    want, _ = R.forward(cfg, w, ids)
    if patch:
        monkeypatch.setattr(R, *patch)
    wrong, _ = R.forward(other_cfg(cfg) if other_cfg else cfg, w, ids)
    for dtype in DTYPES:
        for portions in ([len(ids)], [1], [13, 2]):
            got = run(moon, ctx, tmp_path, cfg, w, ids, dtype, portions)
            assert_close(got, want, dtype)
            assert not close(got, wrong, dtype, 1.2 * LIMIT[dtype])[0]


# ---- keys just inside and just outside a window, at the first tokens and far away
@pytest.mark.parametrize("window", [2, 63, 64, 65, 128, 129, 200])
def test_window_edge(moon, ctx, tmp_path, window):
    """The last token asks for one earlier token, which sits at the edge of the window."""
    cfg = config(400, 64, [layer(attention(4, 1, 32, 16, window, 0.6))])
    w = beacon_weights(cfg)
    for far in (window - 1, window, window + 1):
        ids = np.random.default_rng(far).permutation(398)[: far + 40].astype(np.uint32)
        first = len(ids) - 1 - far
        ids[first], ids[-1] = 398, 399
        want, _ = R.forward(cfg, w, ids)
        with_next, _ = R.forward(dict(cfg, layers=[layer(attention(4, 1, 32, 16, window + 1, 0.6))]), w, ids)
        assert (row_errors(want[-1:], with_next[-1:])[0] > 0.01) == (far == window)  # the case tells the two apart
        for portions in ([len(ids)], [len(ids) - 1, 1], [len(ids) - 3, 2, 1], [50]):
            got = run(moon, ctx, tmp_path, cfg, w, ids, "float32", portions)
            assert_close(got, want, "float32")
        got = run(moon, ctx, tmp_path, cfg, w, ids, "bfloat16", [len(ids) - 1, 1])
        assert_close(got[-1:], want[-1:], "bfloat16", 0.1)
        got = run(moon, ctx, tmp_path, cfg, w, ids, "bfloat16")
        assert_close(got[-1:], want[-1:], "bfloat16", 0.1)


def test_first_tokens(moon, ctx, folders):
    path, cfg, w, ids, want, _ = folders["odd"]
    for dtype in DTYPES:
        m = opened(moon, ctx, path, dtype)
        for n in (1, 2, 3, 5):
            m.reset()
            assert_close(m.forward_logits(ids[:n], np.arange(n)), want[:n], dtype)
        m.close()


def test_scores_that_would_overflow(moon, ctx, tmp_path):
    cfg = config(60, 48, [layer(dict(BASE, scale=40.0)), layer(dict(BASE, scale=-40.0))])
    w, ids = weights(cfg, 5), tokens(50, 60, 6)
    w["l0.mix.sink"] = np.array([300.0, -300.0, 0.0, 88.0], np.float32)
    want, _ = R.forward(cfg, w, ids)
    for portions in ([50], [1], [9]):
        assert_close(run(moon, ctx, tmp_path, cfg, w, ids, "float32", portions), want, "float32", 1e-3)
        assert np.isfinite(run(moon, ctx, tmp_path, cfg, w, ids, "bfloat16", portions)).all()


# ---- cache rows
RING = config(50, 32, [layer(attention(2, 1, 16, 16, 100, 0.5, True), dense(32)), layer(attention(2, 1, 8, 16, 30, 0.7, True))])


@pytest.mark.parametrize("dtype", DTYPES)
def test_cache_rows_are_used_again(moon, ctx, tmp_path, dtype):
    """A sequence longer than the rows a windowed layer keeps: prompts of several calls' rows, then tokens, around the end of the
    rows; then another sequence in the same session."""
    w, ids = weights(RING, 7), tokens(4500, 50, 8)
    want, _ = R.forward(RING, w, ids)
    m = opened(moon, ctx, write_folder(tmp_path / "m", RING, w), dtype, 5000)
    got = m.forward_logits(ids[:2120], np.arange(2120))  # (2048 rows a call: the rest is a second one)
    assert_close(got, want[:2120], dtype)
    got = feed(m, ids[2120:2180], [1])  # over the end of the first layer's rows
    assert_close(got, want[2120:2180], dtype)
    got = feed(m, ids[2180:], [1000, 1, 3, 700])
    assert_close(got, want[2180:], dtype)
    m.reset()
    short = ids[100:160]
    assert_close(feed(m, short, [20, 1, 1, 38]), R.forward(RING, w, short)[0], dtype)
    m.close()


def test_sequences_do_not_see_each_other(moon, ctx, folders):
    """A long sequence, then short ones in the same session; and two sessions whose calls alternate."""
    path, cfg, w, ids, want, _ = folders["odd"]
    m, o = opened(moon, ctx, path, "float32"), opened(moon, ctx, path, "float32", 200)
    m.forward(ids)
    m.reset()
    other = tokens(30, cfg["vocab"], 77)
    want_other, _ = R.forward(cfg, w, other)
    got, got_other = [], []
    for i in range(0, 30, 5):
        got.append(m.forward_logits(ids[i:i + 5], np.arange(5)))
        got_other.append(feed(o, other[i:i + 5], [1, 4]))
    assert_close(np.concatenate(got), want[:30], "float32")
    assert_close(np.concatenate(got_other), want_other, "float32")
    m.close()
    o.close()


def test_full_cache_is_refused(moon, ctx, folders):
    path, cfg, w, ids, want, _ = folders["odd"]
    m = opened(moon, ctx, path, "float32", 20)
    m.forward(ids[:20])
    with pytest.raises(moon.SequenceTooLong):
        m.forward(ids[:1])
    m.reset()
    with pytest.raises(moon.SequenceTooLong):
        m.forward(ids[:21])
    with pytest.raises(moon.TokenIdOutOfBounds):
        m.forward([cfg["vocab"]])
    assert_close(m.forward_logits(ids[:20], np.arange(20)), want[:20], "float32")
    m.close()


# ---- generation through the session's loop
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_greedy_generation(moon, ctx, folders, name):
    """Every generated token is the oracle's arg-max at its place (or within rounding of it), over more tokens than the windows hold."""
    path, cfg, w, ids, _, _ = folders[name]
    for dtype in DTYPES:
        m = opened(moon, ctx, path, dtype)
        m.forward(ids[:11])
        out = m.greedy(90)
        assert m.position == 101
        logits, _ = R.forward(cfg, w, np.concatenate([ids[:11], out]))
        at = logits[10:100]
        slack = at.max(-1) - at[np.arange(90), out]
        assert (slack > 4 * LIMIT[dtype] * at.std()).sum() <= FLIPS[dtype] * 90, slack
        m.reset()
        m.forward(ids[:11])
        again = []
        for _ in range(20):
            again.append(m.next_token())
            m.forward([again[-1]])
        assert again == out[:20].tolist()
        m.close()


def test_sampled_and_stopped_generation(moon, ctx, folders):
    path, cfg, w, ids, _, _ = folders["odd"]
    m = opened(moon, ctx, path, "float32", 200)
    sampler = moon.sampling.sampling_config("top_k", temperature=0.7, top_k=5)
    u = np.random.default_rng(0).random(40).astype(np.float32)
    m.forward(ids[:9])
    out = m.sample(sampler, u)
    m.reset()
    m.forward(ids[:9])
    for i in range(40):
        tok = m.next_token(sampler, float(u[i]))
        assert tok == out[i]
        row = m.logits_f32()
        assert tok in np.argsort(-row)[:6]
        m.forward([tok])
    eos = int(out[25])
    first = out.tolist().index(eos)
    m.reset()
    m.forward(ids[:9])
    got = m.generate(40, eos, sampler, u)
    assert got.tolist() == out[:first].tolist() and m.position == 9 + first
    # the session goes on behind the stop as if nothing had been queued after it
    more = tokens(12, cfg["vocab"], 9)
    want, _ = R.forward(cfg, w, np.concatenate([ids[:9], out[:first], more]))
    assert_close(m.forward_logits(more, np.arange(12)), want[-12:], "float32")
    m.reset()
    m.forward(ids[:150])
    assert len(m.generate(500, eos if eos != 0 else 1)) <= 50  # ends at the last cache position at the latest
    m.close()


def test_calls_of_the_fixed_block_are_refused(moon, ctx, folders):
    path, cfg, w, ids, _, _ = folders["odd"]
    m = opened(moon, ctx, path, "float32")
    m.forward(ids[:4])
    for call in (m.logits, lambda: m.hidden(1), lambda: m.text_encoder(ids[:2]), lambda: m.set_decode_mode(2), lambda: m.greedy_profile(1)):
        with pytest.raises(moon.MoonError):
            call()
    m.close()


def test_wanted_logits_of_the_fixed_block(moon, ctx):
    """The calls that are not tied to a design work on the f16 decoder too."""
    cfg = moon.text_model.make_config(vocab=512, dim=128, hidden_dim=256, n_layers=2, n_heads=2, max_seq=64)
    m = moon.text_model.TextModel(cfg, seed=0, ctx=ctx)
    got = m.forward_logits([1, 2, 3, 4], [3, 0])
    assert np.array_equal(got[0], m.logits().astype(np.float32)) and np.array_equal(got[0], m.logits_f32())
    assert np.array_equal(m.hidden_f32(4), m.hidden(4).astype(np.float32))
    m.reset()
    m.forward([1])
    assert np.abs(m.logits_f32() - got[1]).max() < 0.05
    m.close()


def test_random_weights(moon, ctx):
    cfg = config(640, 128, [layer(attention(4, 2, 32, 32, 50, 0.2, True), dense(192)), layer(attention(4, 2, 32, 32, 50, 0.2, True), moe(64, 4, 64))])
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
    import json

    path, cfg, w, ids, want, _ = folders["tall"]
    toks = [int(t) for t in ids]
    steps = [dict(step=0, entries=[dict(id="a", tokens=toks[:30], want=[0, 29])], end=[]),
             dict(step=1, entries=[dict(id="a", tokens=toks[30:32], want=[])], end=[]),
             dict(step=2, entries=[dict(id="a", tokens=toks[32:33], want=[0])], end=["a"]),
             dict(step=3, entries=[dict(id="b", tokens=toks[:2], want=[1])], end=["b"])]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "40"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert r.stdout.split("\n")[:4] == [f"done {i}" for i in range(4)]
    assert not os.path.exists(tmp_path / "1.f32")
    for i, rows in ((0, [0, 29]), (2, [32]), (3, [1])):
        got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(len(rows), cfg["vocab"])
        assert_close(got, want[rows], "float32")
