"""The plain Keronex oracle (tests/keronex_oracle.py) pinned by closed forms: each mechanism on inputs whose answer is known by hand, and a demonstration that
switching any mechanism off moves the logits far beyond the tolerance the device path is held to; the configuration reader against the oracle's own tensor
inventory.  CPU only."""
import copy

import numpy as np
import pytest

import keronex_oracle as ko
from test_hip_keronex import attn, cd, config, dense, moe, of, ret, tokens, want_of
from tinygpt_amd.desc import stack_desc_from_config


def test_norm_and_activations_by_hand():
    np.testing.assert_allclose(ko.norm(np.array([[3.0, 4.0]]), np.array([0.0, 1.0]), 0.0), [[3 / np.sqrt(12.5), 8 / np.sqrt(12.5)]])
    np.testing.assert_allclose(ko.norm(np.array([[3.0, 4.0]]), np.array([0.0, 0.0]), 12.5), [[0.6, 0.8]])
    np.testing.assert_allclose(ko.gelu_tanh(np.array([0.0, 1.0, -1.0])), [0.0, 0.841191990608, -0.158808009392], atol=1e-11)
    np.testing.assert_allclose(ko.unit(np.array([[3.0, 4.0]]))[0], [0.6, 0.8], rtol=1e-6)


def test_pair_rows_by_hand():
    b = {"buckets": 10, "mul_prev": 7, "mul_cur": 3}
    assert [ko.bigram_row(None, 5, b), ko.bigram_row(0, 0, b), ko.bigram_row(1, 2, b), ko.bigram_row(2, 1, b), ko.bigram_row(9, 9, b)] == [10, 0, 3, 7, 0]
    t = {"embed": np.array([[1.0], [2.0]]), "bigram": np.arange(11.0)[:, None] * 100}
    np.testing.assert_array_equal(ko.embed([1, 0, 1], {"scale": 3.0, "bigram": b}, t)[:, 0], [6 + 1000, 3 + 700, 6 + 300])      # the pair rows are not scaled


def test_streams_by_hand():
    xs = np.array([[[1.0]], [[10.0]]])
    np.testing.assert_allclose(ko.streams_in(xs, np.array([2.0, 0.5])), [[7.0]])
    # from stream 0 to stream 1 goes mix[0][1]
    np.testing.assert_allclose(ko.streams_out(xs, np.array([[1.0, 3.0], [0.0, 2.0]]), np.array([5.0, 7.0]), np.array([[100.0]]))[:, 0, 0], [1 + 500, 3 + 20 + 700])


def test_rotation_by_hand():
    x = np.zeros((3, 1, 5)); x[..., 0] = 1.0; x[..., 4] = 9.0
    r = ko.rotate(x, {"base": 100.0, "dims": 4})
    np.testing.assert_allclose(r[2, 0], [np.cos(2), 0, np.sin(2), 0, 9.0], atol=1e-15)      # channel 0 turns with channel 2 by the position itself
    x = np.zeros((3, 1, 4)); x[..., 3] = 1.0
    np.testing.assert_allclose(ko.rotate(x, {"base": 100.0, "dims": 4})[2, 0], [0, -np.sin(0.2), 0, np.cos(0.2)], atol=1e-15)


def test_decaying_memory_by_hand():
    q, k, v = np.array([[1.0, 0.0], [1.0, 1.0]]), np.array([[2.0, 3.0], [1.0, 0.0]]), np.array([[5.0], [7.0]])
    np.testing.assert_allclose(ko.decaying_memory(q, k, v, 0.5)[:, 0], [10.0, 0.5 * 25 + 7])


def test_delta_memory_by_hand():
    q, k, v = np.eye(2), np.array([[1.0, 0.0], [1.0, 1.0]]), np.array([[4.0], [10.0]])
    g = np.array([[1.0, 1.0], [0.5, 0.25]])
    # S_1 = [4 b, 0]; the decay halves its first row before the recall; the second write is 0.5 (10 - 2 b)
    o = ko.delta_memory(q, k, v, np.array([0.75, 0.5]), g)[:, 0]
    np.testing.assert_allclose(o, [3.0, 0.5 * (10 - 1.5)])


def test_two_maps_by_hand():
    assert ko.map_weight({"lq1": np.array([1.0, 2.0]), "lk1": np.array([0.5, 0.25]), "lq2": np.zeros(2), "lk2": np.ones(2)}, "", 0.3) == pytest.approx(np.e - 1 + 0.3)
    v = np.array([[1.0, 0.0], [0.0, 1.0]])
    np.testing.assert_allclose(ko.softmax_attention(np.array([[0.0], [1.0]]), np.array([[0.0], [np.log(3.0)]]), v, 1.0), [[1, 0], [0.25, 0.75]])
    np.testing.assert_allclose(ko.softmax_attention(np.zeros((2, 1)), np.zeros((2, 1)), v, 1.0)[1], [0.5, 0.5])


def test_experts_by_hand():
    t = {"router": np.array([[10.0, 0.0], [0.0, np.log(3.0)], [-9.0, -9.0]]), "e0.up": np.eye(2), "e0.down": np.eye(2), "e1.up": np.eye(2), "e1.down": 2 * np.eye(2),
         "shared.up": -np.eye(2), "shared.down": np.eye(2)}
    f = {"router": {"top": 1}, "expert": {"ff": 2}, "shared": None}
    np.testing.assert_allclose(ko.experts_ff(np.array([[-1.0, 1.0]]), f, t, ""), [[0.0, 2 * 0.75 ** 2]])      # the weight 3 / 4 is squared with the input
    np.testing.assert_allclose(ko.experts_ff(np.array([[-1.0, 1.0]]), dict(f, shared={"ff": 2}), t, ""), [[1.0, 2 * 0.75 ** 2]])
    sel, s = ko.chosen_experts(np.array([[-1.0, 1.0]]), t, "", 2)
    assert sel.tolist() == [[1, 2]] and s[0].tolist() == pytest.approx([0.75, 0.5])      # not renormalised


def test_every_mechanism_moves_the_logits():
    """the oracle with one mechanism switched off differs far beyond the tolerance: a device path that left it out could not pass"""
    cfg = config()
    w = ko.random_tensors(cfg, 3)
    toks = tokens(cfg, 40)
    base = want_of(cfg, w, toks)

    def moved(c2=None, w2=None):
        return np.abs(want_of(c2 or cfg, w2 or w, toks) - base).max() / np.abs(base).max()

    def edit(*changes):
        c2 = copy.deepcopy(cfg)
        for path, value in changes:
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
    lay = lambda i, *p: ("layers", i, "mixer") + p
    assert moved(edit((("embedding", "scale"), 1.0))) > 1e-2
    assert moved(edit((("embedding", "bigram"), None))) > 1e-2
    for k in ("mul_prev", "mul_cur"):
        assert moved(edit((("embedding", "bigram", k), 4))) > 1e-2, k
    assert moved(edit((("norm", "eps"), 1e-2))) > 1e-3
    for i in (1, 5):      # (a borrowed layer's own rotation and decays count as well)
        assert moved(edit((lay(i, "rot"), None))) > 1e-3
        assert moved(edit((lay(i, "rot", "base"), 9000.0))) > 1e-4
        assert moved(edit((lay(i, "decay"), [0.875, 0.9]))) > 1e-3
        assert moved(edit((lay(i, "decay"), [0.99, 0.875]))) > 1e-3
    for k, v in (("scale", 0.5), ("diff", 0.2), ("rot", None)):
        assert moved(edit((lay(2, k), v))) > 1e-3, k
    assert moved(edit((("layers", 5, "weights_of"), 4), (("layers", 5, "mlp"), None))) > 1e-2
    assert moved(edit((("layers", 0, "mlp"), None))) > 1e-2
    assert moved(edit((("layers", 1, "mlp", "router", "top"), 1))) > 1e-3
    assert moved(edit((("layers", 1, "mlp", "shared"), None))) > 1e-3
    for n in ("lq1", "lk1", "lq2", "lk2"):
        assert moved(w2=swap("l2.mix." + n, np.zeros_like)) > 1e-3, n
    for n in ("a2", "g2", "A_log", "b"):
        assert moved(w2=swap("l0.mix." + n, np.zeros_like)) > 1e-3, n
    assert moved(w2=swap("l0.mix.dt_bias", np.zeros_like)) > 1e-3
    assert moved(w2=swap("l0.mix.dt_bias", np.flip)) > 1e-4
    for n in ("q", "k", "v"):
        assert moved(w2=swap(f"l0.mix.{n}.conv", lambda v: np.roll(v, 1, axis=1))) > 1e-3, n
    for n in ("l0.norm1", "l1.norm2", "final.norm"):
        assert moved(w2=swap(n, np.zeros_like)) > 1e-3, n
    assert moved(w2=swap("l0.mix.norm", np.ones_like)) > 1e-3
    assert moved(w2=swap("l1.mix.g", lambda v: -v)) > 1e-3
    for n in ("l0.hc1", "l1.hc2", "l4.hc1"):
        assert moved(w2=swap(n + ".mix", np.transpose)) > 1e-3, n
        assert moved(w2=swap(n + ".mix", lambda v: np.eye(len(v)))) > 1e-3, n
        if n != "l0.hc1":                                  # (all streams are equal in front of the first sublayer)
            assert moved(w2=swap(n + ".in", np.flip)) > 1e-3, n
        assert moved(w2=swap(n + ".out", np.flip)) > 1e-3, n


def test_the_configuration_reader_knows_every_tensor():
    for layers in (None, [cd(conv=1, dim=7, vdim=9)], [ret(moe(3, 1, 5, 0)), attn(dense(), heads=6, kv_heads=3, dim=5, rot=None)]):
        cfg = config(layers, width=18, vocab=31)
        want = ko.tensor_shapes(cfg, 3, 11)
        d = stack_desc_from_config(cfg, tensor_shapes=want)
        assert d.tensor_shapes() == want
        assert d.family == "keronex" and d.embed_scale == 2.0 and d.streams == 3 and d.norm_eps == 1e-5 and (d.bigram_buckets, d.bigram_before, d.bigram_cur) == (37, 5, 3)
    layers = [ret(decay=[0.25, 0.5]), attn()]
    layers.append(of(0, layers))
    d = stack_desc_from_config(config(layers))
    assert [l.weights_of for l in d.layers] == [None, None, 0] and d.layers[2].decays == (0.25, 0.5) and d.layers[1].maps == 2
    sd, arr = d.to_c()
    assert arr[2].n_decays == 2 and arr[2].decays[1] == 0.5 and arr[2].weights_of == 1 and sd.streams == 3
    with pytest.raises(ValueError, match="wkv"):
        stack_desc_from_config(config([{"type": "wkv", "mixer": {}, "mlp": None}]))
    with pytest.raises(ValueError, match="other"):
        stack_desc_from_config(config([ret({"kind": "other"})]))
