"""CPU: the plain Rikanex statement against hand-made cases, and the model-folder reader (no device call)."""
import json
import os
import struct

import numpy as np
import pytest
import rikanex_oracle as R
from rikanex_models import MODELS, ODD, attention, config, dense, layer, tokens, weights, write_folder


def test_bf16_round_ties_to_even():
    x = np.array([1.0, 1.0 + 2**-8, 1.0 + 3 * 2**-8, -1.0 - 2**-8 - 2**-20, 3e38], np.float32)
    assert R.bf16_round(x).tolist() == [1.0, 1.0, 1.0 + 2**-6, -1.0 - 2**-7, float(np.float32(R.bf16_from_bits(np.uint16(0x7F62))))]


def test_window_edges():
    assert R.visible(5, 5, 1) and not R.visible(5, 4, 1) and not R.visible(5, 6, 1)
    assert R.visible(9, 6, 4) and not R.visible(9, 5, 4)
    assert R.visible(9, 0, None) and not R.visible(9, 10, None)


def test_sink_takes_weight_and_has_no_value():
    w = R.sink_softmax(np.array([0.0, 0.0]), 0.0)
    assert np.allclose(w, [1 / 3, 1 / 3])
    assert np.allclose(R.sink_softmax(np.array([1000.0]), -1000.0), [1.0])
    assert np.allclose(R.sink_softmax(np.array([-1000.0]), 1000.0), [0.0])


def test_one_key_without_a_sink_is_its_value():
    q, k, v = np.ones((1, 2, 4)), np.ones((1, 1, 4)), np.arange(3.0).reshape(1, 1, 3)
    out = R.window_attention(q, k, v, 0.5, 4, np.full(2, -np.inf))
    assert np.allclose(out, np.broadcast_to(v, (1, 2, 3)))


def test_query_heads_share_key_value_heads():
    rng = np.random.default_rng(0)
    q, k, v = rng.normal(size=(6, 4, 8)), rng.normal(size=(6, 2, 8)), rng.normal(size=(6, 2, 5))
    out = R.window_attention(q, k, v, 1.0, 3, np.zeros(4))
    for h in range(4):
        alone = R.window_attention(q[:, h:h + 1], k[:, h // 2:h // 2 + 1], v[:, h // 2:h // 2 + 1], 1.0, 3, np.zeros(1))
        assert np.allclose(out[:, h], alone[:, 0])


def test_experts_are_chosen_with_the_correction_and_weighted_without():
    z = np.array([0.0, 1.0, 2.0, -1.0])
    ids, w = R.choose_experts(z, np.array([5.0, 0.0, 0.0, 4.0]), 2)
    s = R.sigmoid(z)
    assert ids.tolist() == [0, 3] and np.allclose(w, [s[0] / (s[0] + s[3]), s[3] / (s[0] + s[3])])


def test_norms():
    x = np.array([[3.0, 4.0]])
    assert np.allclose(R.unit_rms(x, 0.0), x / np.sqrt(12.5))
    y = R.layer_norm(x, np.array([1.0, 2.0]), np.array([0.5, 0.0]), 0.0)
    assert np.allclose(y, [[-0.5, 2.0]])


def test_the_first_mixing_layer_keeps_its_values():
    w = weights(ODD)
    ids = tokens(6, ODD["vocab"])
    a, _ = R.forward(ODD, w, ids)
    w["l1.mix.vmix"] = np.float32(0.0)  # the first mixing layer's own lambda is unused
    b, _ = R.forward(ODD, w, ids)
    w["l3.mix.vmix"] = np.float32(0.0)
    c, _ = R.forward(ODD, w, ids)
    assert np.array_equal(a, b) and not np.allclose(a, c)


# ---- model folders, without a device
@pytest.mark.parametrize("name", sorted(MODELS))
def test_folder_is_accepted(moon, tmp_path, name):
    cfg = MODELS[name]
    design, layers = moon.registry.check_folder(write_folder(tmp_path / name, cfg, weights(cfg)))
    assert (design, layers) == ("Rikanex", len(cfg["layers"]))
    assert design in moon.registry.designs()


def test_folder_errors(moon, tmp_path):
    cfg = config(20, 16, [layer(attention(2, 1, 8, 8, 4, 1.0), dense(8))])
    w = weights(cfg)

    def refused(c, ww, words, name=[0]):
        name[0] += 1
        with pytest.raises(moon.MoonError) as e:
            moon.registry.check_folder(write_folder(tmp_path / str(name[0]), c, ww))
        assert words in str(e.value), str(e.value)

    refused(dict(cfg, architecture="Nothing"), w, "architecture 'Nothing'")
    refused({k: v for k, v in cfg.items() if k != "norm"}, w, "norm")
    refused(dict(cfg, width=15), w, "shape")
    refused(dict(cfg, width=-1), w, "width")
    refused(dict(cfg, layers=[]), w, "layers")
    refused(dict(cfg, layers=[dict(cfg["layers"][0], type="other")]), w, "type")
    refused(dict(cfg, layers=[layer(attention(3, 2, 8, 8, 4, 1.0))]), w, "kv_heads")
    refused(dict(cfg, layers=[layer(attention(2, 1, 8, 8, 0, 1.0))]), w, "mask.size")
    refused(cfg, {k: v for k, v in w.items() if k != "l0.mix.sink"}, "l0.mix.sink")
    refused(cfg, dict(w, **{"l0.mlp.down": w["l0.mlp.down"].T}), "l0.mlp.down") if w["l0.mlp.down"].shape[0] != w["l0.mlp.down"].shape[1] else None


def test_truncated_and_broken_safetensors(moon, tmp_path):
    cfg = config(20, 16, [layer(attention(2, 1, 8, 8, 4, 1.0))])
    path = write_folder(tmp_path / "m", cfg, weights(cfg))
    file = os.path.join(path, "model.safetensors")
    raw = open(file, "rb").read()
    for bad in (raw[:4], raw[:40], raw[:-2], struct.pack("<Q", 1 << 62) + raw[8:], struct.pack("<Q", 2) + b"[]" + raw, struct.pack("<Q", 3) + b'{"a' + raw):
        open(file, "wb").write(bad)
        with pytest.raises(moon.MoonError):
            moon.registry.check_folder(path)
    open(os.path.join(path, "config.json"), "w").write(json.dumps(cfg)[:-1])
    with pytest.raises(moon.MoonError):
        moon.registry.check_folder(path)
