"""The plain Nusovik oracle (tests/nusovik_oracle.py) pinned by closed forms: each mechanism on inputs whose answer is known by hand, and a demonstration that
switching any mechanism off moves the logits far beyond the tolerance the device path is held to; the configuration reader against the oracle's own tensor
inventory.  CPU only."""
import copy

import numpy as np
import pytest

import nusovik_oracle as no
from test_hip_nusovik import config, mamba, par, tokens, want_of
from tinygpt_amd.desc import stack_desc_from_config


def test_chunks_and_buckets_by_hand():
    c = no.chunk_mask(7, 3)
    assert c[5].tolist() == [False, False, False, True, True, True, False] and c[3].tolist() == [False, False, False, True, False, False, False]
    assert c[2].tolist() == [True, True, True, False, False, False, False]
    assert no.chunk_mask(3, None).tolist() == np.tril(np.ones((3, 3), bool)).tolist()
    # 8 rows up to distance 64: exact 0 .. 3, then 4 * 2^n steps of one row each (ln(n / 4) / ln 16 * 4)
    assert [no.bucket(n, 8, 64) for n in (0, 1, 2, 3, 4, 7, 8, 15, 16, 31, 32, 63, 64, 1000)] == [0, 1, 2, 3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]
    assert [no.bucket(n, 2, 9) for n in (0, 1, 5, 9, 50)] == [0, 1, 1, 1, 1]
    rel = np.arange(16.0).reshape(8, 2)
    np.testing.assert_array_equal(no.distance_bias(rel, 9, 64)[1], [1, 3, 5, 7, 9, 9, 9, 9, 11])


def test_positions_by_hand():
    s = no.sinusoids(4, 6)
    p = np.arange(4)
    np.testing.assert_allclose(s[:, 0], np.sin(p)); np.testing.assert_allclose(s[:, 1], np.cos(p))
    np.testing.assert_allclose(s[:, 4], np.sin(p * 10000.0 ** (-4 / 6))); np.testing.assert_allclose(s[:, 5], np.cos(p * 10000.0 ** (-4 / 6)))


def test_sink_bias_and_groups_by_hand():
    rng = np.random.default_rng(0)
    v = rng.standard_normal((2, 1, 3))
    zero = np.zeros((2, 2, 3))
    # scores 0: one key and a sink of 0 share the weight; the distance bias counts unscaled
    o = no.sink_attention(zero, v, v, no.chunk_mask(2, None), 100.0, np.array([[0.0, -0.7], [0.0, 0.0]]), np.array([0.0, np.log(3.0)]))
    np.testing.assert_allclose(o[0, 0], v[0, 0] / 2); np.testing.assert_allclose(o[0, 1], v[0, 0] / 4)
    e = np.exp(-0.7)
    np.testing.assert_allclose(o[1, 0], (e * v[0, 0] + v[1, 0]) / (2 + e)); np.testing.assert_allclose(o[1, 1], (v[0, 0] + v[1, 0]) / 5)


def test_values_are_the_unnormed_keys():
    eye = np.eye(2)
    t = {"q": eye, "q.b": np.zeros(2), "k": 3 * eye, "k.b": np.array([1.0, -1.0]), "q.norm": np.ones(2), "k.norm": np.ones(2), "rel": np.zeros((2, 1)), "sink": np.array([-1e9]),
         "g": np.zeros((1, 2)), "o": eye}
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "scale": 1.0, "bias_max": 4}
    h = np.array([[1.0, 2.0]])
    np.testing.assert_allclose(no.keys_as_values_attention(h, m, t, "", 1e-5), [[0.5 * 4.0, 0.5 * 5.0]])      # one key: its projection, times the gate's 1/2


def test_short_convolution_by_hand():
    x = np.arange(1.0, 5.0)[:, None]
    np.testing.assert_allclose(no.short_conv(x, np.array([[100.0, 10.0, 1.0]]), np.array([0.5]))[:, 0], [1.5, 12.5, 123.5, 234.5])


def test_scalar_decay_scan_by_hand():
    dt = np.array([[1.0], [0.5]])
    B, C, x = np.array([[[1.0, 2.0]], [[3.0, 0.0]]]), np.array([[[1.0, 1.0]], [[0.0, 1.0]]]), np.array([[[2.0]], [[4.0]]])
    y = no.scalar_decay_scan(dt, np.array([np.log(2.0)]), B, C, x, np.array([10.0]))
    # S_1 = [2, 4]; S_2 = e^-1 [2, 4] + 0.5 * 4 * [3, 0]
    np.testing.assert_allclose(y[:, 0, 0], [6 + 20, 4 * np.exp(-1) + 40])


def test_selective_scan_by_hand():
    dt, x = np.array([[1.0, 2.0], [0.5, 1.0]]), np.array([[3.0, 1.0], [2.0, 5.0]])
    A, B, C = np.array([[-1.0, -2.0], [0.0, -0.5]]), np.array([[1.0, 2.0], [1.0, 0.0]]), np.array([[1.0, 1.0], [1.0, 2.0]])
    y = no.selective_scan(dt, A, B, C, x, np.array([1.0, -1.0]))
    np.testing.assert_allclose(y[0], [3 + 6 + 3, 2 + 4 - 1])
    np.testing.assert_allclose(y[1], [3 * np.exp(-0.5) + 1 + 2 * 6 * np.exp(-1) + 2, 2 + 5 + 2 * 4 * np.exp(-0.5) - 5])


def test_gated_part_norm_and_feed_forward():
    y, z = np.array([[3.0, 4.0, 1.0, 0.0]]), np.array([[50.0, 50.0, 50.0, 50.0]])      # silu(50) = 50
    np.testing.assert_allclose(no.gated_part_norm(y, z, np.array([1.0, 1.0, 2.0, 1.0]), 2, 0.0), [[3 / np.sqrt(12.5), 4 / np.sqrt(12.5), 2 * np.sqrt(2.0), 0.0]])
    np.testing.assert_allclose(no.squared_relu_ff(np.array([[2.0, -3.0]]), np.eye(2), np.array([[1.0, 1.0], [1.0, 0.0]])), [[4.0, 4.0]])


def test_the_norms_stand_behind_the_sublayers():
    """a mixer whose output is scaled does not change the stream (the norm behind it removes the factor); scaling the stream itself does"""
    cfg = config([mamba(), par()], eps=1e-12)
    w = no.random_tensors(cfg, 1)
    toks = tokens(cfg, 12)
    base = want_of(cfg, w, toks)
    np.testing.assert_allclose(want_of(cfg, dict(w, **{"l0.mix.o": w["l0.mix.o"] * 7.0}), toks), base, rtol=1e-6, atol=1e-8)
    assert np.abs(want_of(cfg, dict(w, **{"embed": w["embed"] * 1.5}), toks) - base).max() > 1e-2


def test_every_mechanism_moves_the_logits():
    """the oracle with one mechanism switched off differs far beyond the tolerance: a device path that left it out could not pass"""
    cfg = config()
    w = no.random_tensors(cfg, 3)
    toks = tokens(cfg, 40)
    base = want_of(cfg, w, toks)

    def moved(c2=None, w2=None):
        return np.abs(want_of(c2 or cfg, w2 or w, toks) - base).max() / np.abs(base).max()

    def edit(path, value):
        c2 = copy.deepcopy(cfg)
        node = c2
        for k in path[:-1]:
            node = node[k]
        if value is None:
            node.pop(path[-1], None)
        else:
            node[path[-1]] = value
        return c2

    def swap(name, f):
        return {**w, name: f(w[name])}
    assert moved(edit(["embedding", "scale"], 1.0)) > 1e-2
    assert moved(edit(["logit_scale"], 1.0)) > 1e-2
    assert moved(edit(["norm", "eps"], 1e-2)) > 1e-3
    assert moved(edit(["layers", 1, "mixer", "left", "mask", "size"], 10)) > 1e-3    # chunks one longer
    assert moved(edit(["layers", 1, "mixer", "left", "mask"], None)) > 1e-3
    assert moved(edit(["layers", 1, "mixer", "left", "bias_max"], 6)) > 1e-3
    assert moved(edit(["layers", 1, "mixer", "left", "scale"], 0.4)) > 1e-3
    assert moved(edit(["layers", 1, "mixer", "right_scale"], 0.0)) > 1e-2
    assert moved(edit(["layers", 1, "mixer", "left_scale"], 0.0)) > 1e-2
    assert moved(edit(["layers", 1, "mixer", "right", "norm_groups"], 1)) > 1e-3
    assert moved(edit(["layers", 1, "mlp"], None)) > 1e-2
    for name in ("q.b", "k.b", "rel", "sink", "g"):
        assert moved(w2=swap("l1.mix.left." + name, np.zeros_like)) > 1e-3, name
    for name in ("q.norm", "k.norm"):
        assert moved(w2=swap("l1.mix.left." + name, np.ones_like)) > 1e-3, name
    for name in ("conv.b", "dt_bias", "A_log", "D"):
        assert moved(w2=swap("l1.mix.right." + name, np.zeros_like)) > 1e-3, name
    for name in ("conv.b", "dt.b", "A_log", "D"):
        assert moved(w2=swap("l0.mix." + name, np.zeros_like)) > 1e-3, name
    for name in ("l0.mix.conv", "l1.mix.right.conv"):
        assert moved(w2=swap(name, lambda v: np.roll(v, 1, axis=1))) > 1e-3, name
    for name in ("l0.norm1", "l1.norm2", "l1.mix.right.norm", "final.norm"):
        assert moved(w2=swap(name, np.ones_like)) > 1e-3, name


def test_the_configuration_reader_knows_every_tensor():
    for layers in (None, [mamba(conv=1, state=7, inner=9, dt_rank=2)], [par(left={"heads": 6, "kv_heads": 3, "dim": 5}, right={"groups": 1, "heads": 3, "norm_groups": 3})]):
        cfg = config(layers, width=18, vocab=31)
        want = no.tensor_shapes(cfg, buckets=12)
        d = stack_desc_from_config(cfg, tensor_shapes=want)
        assert d.tensor_shapes() == want
        assert d.family == "nusovik" and d.embed_scale == 2.0 and d.logit_scale == 1.5 and d.norm_eps == 1e-5
    bad = config([{"type": "attention", "mixer": {}, "mlp": None}])
    with pytest.raises(ValueError, match="attention"):
        stack_desc_from_config(bad)
    with pytest.raises(ValueError, match="moe"):
        stack_desc_from_config(config([mamba({"kind": "moe"})]))
