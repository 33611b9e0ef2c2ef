"""CPU: the plain Generax statement against hand-made cases, and the model-folder reader (no device call)."""
import generax_oracle as G
import numpy as np
import pytest
from generax_models import MODELS, attention, config, delta, parallel, plain, rotation, softmax_mixer, weights
from rikanex_models import write_folder


def test_window_and_blocks():
    assert G.visible(9, 6, 4) and not G.visible(9, 5, 4) and not G.visible(3, 4, 4)
    # window 4, blocks of 3: block 1 holds 3, 4, 5 and is seen from position 9 on
    assert G.block_visible(9, 1, 4, 3) and not G.block_visible(8, 1, 4, 3) and not G.block_visible(5, 0, 4, 3) and G.block_visible(6, 0, 4, 3)
    x = np.arange(7.0).reshape(7, 1, 1)
    assert G.pooled(x, 3).ravel().tolist() == [1.0, 4.0]


def test_tokens_between_window_and_block_are_not_seen():
    """Position 8, window 4, blocks of 3: tokens 5 .. 8 and block 0, but neither 3 nor 4."""
    q, k = np.zeros((9, 1, 2)), np.zeros((9, 1, 2))
    out = G.attention(q, k, np.eye(9).reshape(9, 1, 9), np.ones(1), 4, 3)[8, 0]
    assert np.allclose(out, np.array([1 / 3, 1 / 3, 1 / 3, 0, 0, 1, 1, 1, 1]) / 5)


def test_rotation():
    f = G.frequencies(4, 100.0, 2.0)
    assert np.allclose(f, [0.5, 0.05])
    x = np.zeros((2, 1, 6))
    x[1, 0, 0] = x[1, 0, 5] = 1.0
    y = G.rotate_heads(x, 4, 100.0, 2.0)
    assert np.allclose(y[1, 0], [np.cos(0.5), 0, np.sin(0.5), 0, 0, 1])
    v = np.random.default_rng(0).normal(size=(5, 2, 8))
    assert np.allclose(G.rotate_back(G.rotate_values(v, 50.0), 50.0), v)


def test_rotated_values_depend_on_distance_only():
    """One visible key, as far back as the window: the output is its value turned by minus the distance."""
    v = np.random.default_rng(1).normal(size=(4, 1, 4))
    r = G.rotate_back(np.concatenate([G.rotate_values(v, 9.0)[:3][:1]] * 4)[:4], 9.0)
    assert np.allclose(r[3, 0], G.turn(v[0, 0], -3 * G.frequencies(4, 9.0, 1.0)))


def test_short_convolution():
    x, w = np.array([[1.0], [2.0], [4.0]]), np.array([[10.0, 1.0]])
    assert G.short_conv(x, w).ravel().tolist() == [1.0, 12.0, 24.0]
    assert G.short_conv(x, w[:, 1:]).ravel().tolist() == [1.0, 2.0, 4.0]


def test_delta_rule_reads_its_own_write():
    S, o = G.delta_step(np.zeros((2, 3)), np.array([1.0, 0]), np.array([1.0, 0]), np.array([1.0, 2, 3]), np.ones(2), 0.5)
    assert np.allclose(o, [0.5, 1, 1.5])
    S, o = G.delta_step(S, np.array([1.0, 0]), np.array([1.0, 0]), np.array([1.0, 2, 3]), np.array([0.5, 1]), 1.0)  # overwritten
    assert np.allclose(S, [[1, 2, 3], [0, 0, 0]])
    S, o = G.delta_step(S, np.array([1.0, 1]), np.array([0, 1.0]), np.zeros(3), np.array([0.5, 1]), 1.0)
    assert np.allclose(o, [0.5, 1, 1.5])


def test_decay_and_unit():
    g = G.decay(np.array([0.0, 1.0]), np.zeros((1, 2, 3)))
    assert np.allclose(g[0, :, 0], [0.5, 0.5**np.e])
    assert np.allclose(G.unit(np.array([3.0, 4.0])), [0.6, 0.8])


def test_join():
    assert np.allclose(G.join(np.array([2.0, 2.0]), np.array([0.0, 3.0]), 1.0, 2.0, 0.0), [0.5, 0.5 + 2**0.5])


# ---- model folders, without a device
@pytest.mark.parametrize("name", sorted(MODELS))
def test_folder_is_accepted(moon, tmp_path, name):
    cfg = MODELS[name]
    design, layers = moon.registry.check_folder(write_folder(tmp_path / name, cfg, weights(cfg)))
    assert (design, layers) == ("Generax", len(cfg["layers"]))
    assert design in moon.registry.designs()


def test_folder_without_optional_members(moon, tmp_path):
    cfg = {k: v for k, v in config(20, 16, [plain(attention(2, 1, 8, 8, 4, 1.0, rotation(8, 10.0)))]).items() if k != "logit_softcap"}
    moon.registry.check_folder(write_folder(tmp_path, cfg, weights(cfg)))


def test_folder_errors(moon, tmp_path):
    att, left, right = attention(2, 1, 8, 8, 4, 1.0, rotation(8, 10.0)), softmax_mixer(2, 1, 8, 8, 4, 1.0, 3), delta(2, 1, 8, 8, 3)
    cfg = config(20, 16, [plain(att, 8), parallel(left, right)])
    w = weights(cfg)

    def refused(c, ww, words, name=[0]):
        name[0] += 1
        with pytest.raises(moon.MoonError) as e:
            moon.registry.check_folder(write_folder(tmp_path / str(name[0]), c, ww))
        assert words in str(e.value), str(e.value)

    def with_layers(*layers):
        return dict(cfg, layers=list(layers))

    refused({k: v for k, v in cfg.items() if k != "norm"}, w, "norm")
    refused(dict(cfg, logit_softcap=-1.0), w, "logit_softcap")
    refused(dict(cfg, layers=[dict(cfg["layers"][0], type="other")]), w, "type")
    refused(with_layers(plain(dict(att, kv_heads=3))), w, "kv_heads")
    refused(with_layers(plain(dict(att, rot=rotation(7, 10.0)))), w, "rot.dims")
    refused(with_layers(plain(dict(att, rot=rotation(10, 10.0)))), w, "rot.dims")
    refused(with_layers(plain(dict(att, vdim=7))), w, "vdim")
    refused(with_layers(plain(dict(att, kv_from=0))), w, "kv_from")
    refused(with_layers(plain(att), plain(dict(att, kv_from=0, dim=16))), w, "kv_from")
    refused(with_layers(plain(att), plain(dict(att, kv_from=0, rot=rotation(8, 11.0)))), w, "kv_from")
    refused(with_layers(plain(att), plain(dict(att, kv_from=0)), plain(dict(att, kv_from=1))), w, "kv_from")
    refused(with_layers(parallel(left, right), plain(dict(att, kv_from=0))), w, "kv_from")
    refused(with_layers(parallel(dict(left, mask=dict(size=4, pool=0)), right)), w, "mask.pool")
    refused(with_layers(parallel(left, dict(right, conv=0))), w, "right.conv")
    refused(with_layers(parallel(left, dict(right, heads=3, kv_heads=2))), w, "right.kv_heads")
    refused(with_layers(dict(plain(att), mlp=dict(kind="moe"))), w, "mlp.kind")
    for name in ("l0.mix.temp", "l0.mix.k.norm", "l1.mix.right.a1", "l1.mix.right.g2", "l1.mix.left.out", "l1.mix.right.v.conv"):
        refused(cfg, {k: v for k, v in w.items() if k != name}, name)
    refused(cfg, dict(w, **{"l1.mix.right.a2": w["l1.mix.right.a2"][:, 1:]}), "l1.mix.right.a2")

