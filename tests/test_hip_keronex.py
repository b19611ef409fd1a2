"""The Keronex design on the GPU against the plain oracle of tests/keronex_oracle.py: every mechanism on a configuration of its own, prompts against
token-by-token decoding, portions down to two tokens, mixed batches, slots and pages that are used again, far keys and page borders, the pair rows at a portion's
start, long memory through the recurrent states, layers that share weights, and greedy generation through the slot scheduler, tgx_forward / tgx_sample /
tgx_decode, the C++ engine, the command line and bin/trace_run.  Models are config dictionaries of the checkpoint format, so the configuration reader is on the
path of every test.  fp32 storage is the sharp comparison (nothing is rounded: 1e-4 of the largest logit); bf16 storage rounds the cached keys and values (3e-2)."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import keronex_oracle as ko
from test_hip_modepel import write_model_dir
from tinygpt_amd.desc import stack_desc_from_config
from tinygpt_amd.ffi import GREEDY, Model, TgxError
from tinygpt_amd.serving import SlotEngine

pytestmark = pytest.mark.gpu
TOL = {"fp32": 1e-4, "bf16": 3e-2}


# ---- configurations ---------------------------------------------------------------------------------------------------------------
def dense(n=20):
    return {"kind": "dense", "ff": n}


def moe(experts=5, top=2, ff=12, shared=9):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": {"ff": shared} if shared else None}


def ret(mlp=None, **kw):
    m = dict(heads=2, dim=8, vdim=12, decay=[0.875, 0.99], rot={"base": 10000.0, "dims": 6})
    m.update(kw)
    return {"type": "retention", "mixer": {k: v for k, v in m.items() if v is not None}, "mlp": mlp}


def attn(mlp=None, **kw):
    m = dict(heads=4, kv_heads=2, dim=8, vdim=12, scale=0.4, diff=0.3, rot={"base": 5000.0, "dims": 8})
    m.update(kw)
    return {"type": "attention", "mixer": {k: v for k, v in m.items() if v is not None}, "mlp": mlp}


def cd(mlp=None, **kw):
    m = dict(heads=4, kv_heads=2, dim=8, vdim=6, conv=4)
    m.update(kw)
    return {"type": "channel_delta", "mixer": m, "mlp": mlp}


def of(j, layers):
    """another run of layer j's weights"""
    return dict(copy.deepcopy(layers[j]), weights_of=j)


BASE = [cd(dense(13)), ret(moe()), attn(), cd(moe(7, 1)), ret()]
BASE.append(of(1, BASE))
BIGRAM = {"buckets": 37, "mul_prev": 5, "mul_cur": 3}


def config(layers=None, width=24, vocab=67, eps=1e-5, embed=2.0, bigram=BIGRAM, streams=3):
    c = {"architecture": "Keronex", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": embed}, "streams": streams,
         "layers": copy.deepcopy(BASE if layers is None else layers)}
    if bigram:
        c["embedding"]["bigram"] = dict(bigram)
    return c


def engine(cfg, dtype="fp32", seed=0, overrides=None, ranks=(5, 7), options=None, **kw):
    w = ko.random_tensors(cfg, seed, overrides, *ranks)
    kw = dict(dict(max_seqs=4, max_ctx=1024, budget_tokens=2048), **kw)
    eng = SlotEngine(desc=stack_desc_from_config(cfg, dtype, **kw), tensors={k: np.asarray(v, np.float32) for k, v in w.items()})
    for k, v in (options or {}).items():
        eng.model.set_option(k, v)
    return eng, w


def tokens(cfg, n, seed=0):
    return np.random.default_rng(100 + seed).integers(0, cfg["vocab"], n).tolist()


def want_of(cfg, w, toks):
    return ko.forward(cfg, w, toks)


def clear(cfg, w, seqs, seed):
    """router weights whose choices on these sequences are no close calls (a choice that rounding can flip tests nothing): the first of a few seeds of the routers"""
    for k in range(40):
        gap = []

        def watch(h, t, pre, top, f=ko.chosen_experts):
            z = np.sort(-(h @ t[pre + "router"].T), axis=1)
            if top < z.shape[1]:
                gap.append((z[:, top] - z[:, top - 1]).min())
            return f(h, t, pre, top)
        keep = ko.chosen_experts
        ko.chosen_experts = watch
        try:
            want = [want_of(cfg, w, s) for s in seqs]
        finally:
            ko.chosen_experts = keep
        if not gap or min(gap) > 2e-4:
            return want
        rng = np.random.default_rng(1000 * seed + k)
        for n in w:
            if n.endswith(".router"):
                w[n] = ko.bf16_round(rng.standard_normal(w[n].shape) / np.sqrt(w[n].shape[1]))
    raise AssertionError("no router without close calls")


def check(got, want, dtype, what=""):
    err = np.abs(got - want).max() / np.abs(want).max()
    assert err < TOL[dtype], f"{what}: {err:.3e}"


def routed(cfg):
    return any((L.get("mlp") or {}).get("kind") == "moe" for L in cfg["layers"])


def check_rows(got, want, dtype, what="", cfg=None):
    """bf16 with a router: a rounded key or value may flip a close choice at a place; such places are rare, everything else holds the tolerance"""
    err = np.abs(got - want).max(axis=1) / np.abs(want).max()
    if dtype == "fp32" or (cfg and not routed(cfg)):
        assert err.max() < TOL[dtype], f"{what}: {err.max():.3e} at {int(err.argmax())}"
    else:
        assert np.mean(err > TOL[dtype]) <= 0.1, f"{what}: {np.sort(err)[-5:]}"


def run_whole(eng, rid, toks):
    return eng.step([(rid, toks, list(range(len(toks))))], [rid])


# ---- every mechanism on a configuration of its own --------------------------------------------------------------------------------------
MECH = {
    "retention_alone": [ret()],
    "retention_without_rotation": [ret(rot=None)],
    "retention_all_dimensions_turn": [ret(rot={"base": 300.0, "dims": 8})],
    "retention_one_head": [ret(heads=1, decay=[0.97])],
    "retention_no_decay": [ret(decay=[1.0, 0.5])],
    "retention_fast_decay": [ret(decay=[0.01, 0.3])],
    "retention_wide_values": [ret(heads=3, decay=[0.9, 0.95, 0.99], vdim=70, dim=20)],
    "retention_largest_keys": [ret(dim=256, vdim=34, rot={"base": 1e6, "dims": 130})],
    "retention_sizes_off_the_vectors": [ret(heads=3, decay=[0.9, 0.95, 0.99], dim=7, vdim=5, rot={"base": 100.0, "dims": 2})],
    "retention_value_size_one": [ret(vdim=1)],
    "attention_alone": [attn()],
    "attention_without_rotation": [attn(rot=None)],
    "attention_some_dimensions_turn": [attn(rot={"base": 100.0, "dims": 4})],
    "attention_one_head": [attn(heads=1, kv_heads=1)],
    "attention_one_key_head_per_query_head": [attn(kv_heads=4)],
    "attention_one_key_head_for_all": [attn(heads=6, kv_heads=1, dim=10)],
    "attention_three_groups": [attn(heads=6, kv_heads=3, dim=6, rot=None)],
    "attention_wide_heads": [attn(heads=2, kv_heads=1, dim=80, vdim=150, scale=0.1)],
    "attention_widest_heads": [attn(heads=2, kv_heads=2, dim=256, vdim=256, scale=0.05)],
    "attention_values_narrower_than_keys": [attn(dim=16, vdim=4)],
    "attention_no_constant_part": [attn(diff=0.0)],
    "attention_large_constant_part": [attn(diff=0.9)],
    "channel_delta_alone": [cd()],
    "channel_delta_one_head": [cd(heads=1, kv_heads=1)],
    "channel_delta_own_keys": [cd(kv_heads=4)],
    "channel_delta_one_key_head": [cd(heads=6, kv_heads=1)],
    "channel_delta_one_tap": [cd(conv=1)],
    "channel_delta_two_taps": [cd(conv=2)],
    "channel_delta_nine_taps": [cd(conv=9)],
    "channel_delta_more_taps_than_tokens": [cd(conv=40)],
    "channel_delta_wide_values": [cd(heads=2, kv_heads=1, vdim=70)],
    "channel_delta_wide_keys": [cd(heads=2, kv_heads=2, dim=100, vdim=20)],
    "channel_delta_largest_keys": [cd(heads=2, kv_heads=1, dim=256, vdim=33)],
    "channel_delta_sizes_off_the_vectors": [cd(heads=3, kv_heads=1, dim=7, vdim=5, conv=3)],
    "dense_feed_forward": [ret(dense(33)), attn(dense(8))],
    "experts_one_of_many": [attn(moe(16, 1, 10, 6))],
    "experts_all_of_them": [ret(moe(3, 3, 7, 5))],
    "experts_a_single_one": [ret(moe(1, 1, 7, 5))],
    "experts_without_a_shared_one": [cd(moe(6, 2, 9, 0))],
    "experts_wide_shared": [cd(moe(6, 3, 9, 50))],
    "experts_more_than_a_wave": [ret(moe(90, 5, 6, 7))],
    "experts_shared_of_the_same_size": [attn(moe(6, 2, 16, 16))],
    "experts_shared_of_the_same_odd_size": [attn(moe(6, 2, 11, 11))],
    "shared_weights_next_to_each_other": [ret(moe()), dict(ret(moe()), weights_of=0)],
    "shared_weights_of_attention": [attn(dense()), cd(), dict(attn(dense()), weights_of=0)],
    "shared_weights_of_channel_delta": [cd(), attn(), dict(cd(), weights_of=0)],
    "shared_weights_of_a_sharing_layer": [ret(), dict(ret(), weights_of=0), dict(ret(), weights_of=1)],
    "shared_weights_of_a_later_layer": [dict(ret(dense()), weights_of=2), attn(), ret(dense())],
    "one_stream": BASE, "two_streams": BASE, "eight_streams": BASE, "sixteen_streams": [ret(dense()), cd()], "five_streams": [ret(dense()), cd()],
    "plain_residual": BASE,
    "no_pair_rows": BASE,
    "one_pair_bucket": [ret()],
    "large_pair_factors": [ret(), attn()],
    "wide_stream": [ret(dense())],
    "stream_off_the_vectors": BASE,
    "deep": BASE + [attn(moe()), cd(), ret(dense()), attn()],
}
EXTRA = {"one_stream": dict(streams=1), "two_streams": dict(streams=2), "eight_streams": dict(streams=8), "sixteen_streams": dict(streams=16), "five_streams": dict(streams=5),
         "plain_residual": dict(streams=0), "no_pair_rows": dict(bigram=None), "one_pair_bucket": dict(bigram={"buckets": 1, "mul_prev": 3, "mul_cur": 1}),
         "large_pair_factors": dict(bigram={"buckets": 101, "mul_prev": 2147483629, "mul_cur": 1999999973}), "wide_stream": dict(width=4104, vocab=31),
         "stream_off_the_vectors": dict(width=27, vocab=53), "retention_alone": dict(eps=1e-3, embed=1.0), "attention_alone": dict(eps=1e-2)}
RANKS = {"channel_delta_alone": (8, 8), "channel_delta_one_head": (1, 1), "channel_delta_own_keys": (3, 16), "channel_delta_wide_values": (40, 2)}


def oracle_config(cfg):
    """the plain residual written as one stream with unit weights"""
    return cfg if cfg["streams"] else dict(cfg, streams=1)


def plain(cfg, w):
    if cfg["streams"]:
        return w
    w = dict(w)
    for i, L in enumerate(cfg["layers"]):
        for s in ("hc1", "hc2"):
            for n, v in ((".in", np.ones(1)), (".out", np.ones(1)), (".mix", np.ones((1, 1)))):
                w[f"l{i}.{s}{n}"] = v
    return w


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("name", list(MECH))
def test_mechanism(name, dtype):
    cfg = config(MECH[name], **EXTRA.get(name, {}))
    toks = tokens(cfg, 23, seed=len(name))
    w = ko.random_tensors(cfg, len(name), None, *RANKS.get(name, (5, 7)))
    if not cfg["streams"]:
        w = {k: v for k, v in w.items() if ".hc" not in k}
    full = plain(cfg, w)
    want = clear(oracle_config(cfg), full, [toks], len(name))[0]
    w = {k: full[k] for k in w}
    eng = SlotEngine(desc=stack_desc_from_config(cfg, dtype, max_seqs=4, max_ctx=256, budget_tokens=1024), tensors={k: np.asarray(v, np.float32) for k, v in w.items()})
    check_rows(run_whole(eng, "a", toks), want, dtype, name, cfg)
    # ... the same tokens one by one through the cache and the recurrent states
    got = np.concatenate([eng.step([("b", [t], [0])]) for t in toks])
    check_rows(got, want, dtype, name + " by steps", cfg)
    # ... and with the recurrences in blocks whatever the portion's length
    eng.model.set_option("ssd.min", 1)
    check_rows(np.concatenate([eng.step([("c", toks[:3], [0, 1, 2])]), eng.step([("c", toks[3:], list(range(20)))])]), want, dtype, name + " in blocks", cfg)
    eng.close()


# ---- prompts, decoding, portions --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_prompt_then_token_by_token(dtype):
    cfg = config()
    toks = tokens(cfg, 40)
    w = ko.random_tensors(cfg, 1)
    want = clear(cfg, w, [toks], 1)[0]
    eng, _ = engine(cfg, dtype, 1, w)
    got = [eng.step([("r", toks[:9], list(range(9)))])]
    for i in range(9, 40):
        got.append(eng.step([("r", [toks[i]], [0])]))
    check_rows(np.concatenate(got), want, dtype)
    eng.release("r")
    got = np.concatenate([eng.step([("s", [toks[i]], [0])]) for i in range(6)])      # the first tokens of a sequence in a slot that held another one
    check_rows(got, want[:6], dtype, "from the first token")
    eng.close()


@pytest.mark.parametrize("ssd_min", [1, 64, 0])
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("sizes", [[2] * 20, [3, 2, 5, 2, 7, 1, 11, 2, 2], [64, 2, 63, 1], [1, 128, 2, 65], [5, 59, 64, 2], [1, 1, 1, 2, 1, 3, 17], [33, 31, 200, 2]])
def test_portions(sizes, dtype, ssd_min):
    """portions cut through the convolutions' taps, the scans' token groups, the recurrences' blocks and the pairs of neighbouring tokens"""
    cfg = config([cd(dense()), ret(), attn(dense(9)), cd(), ret(dense()), dict(ret(), weights_of=1)])
    eng, w = engine(cfg, dtype, 2, options={"ssd.min": ssd_min})
    toks = tokens(cfg, sum(sizes), seed=len(sizes))
    want = want_of(cfg, w, toks)
    got, at = [], 0
    for n in sizes:
        got.append(eng.step([("r", toks[at:at + n], list(range(n)))]))
        at += n
    check(np.concatenate(got), want, dtype)
    eng.close()


@pytest.mark.parametrize("n", [1, 63, 64, 65, 127, 128, 129, 200])
def test_contexts_around_page_borders(n):
    cfg = config([attn(scale=1.5), ret(), attn(dense(), kv_heads=1), cd()])
    eng, w = engine(cfg, "fp32", 4)
    toks = tokens(cfg, n + 3, seed=n)
    want = want_of(cfg, w, toks)
    got = [eng.step([("r", toks[:n], [n - 1])])]
    got += [eng.step([("r", [toks[n + i]], [0])]) for i in range(3)]      # decoding across the border
    check(np.concatenate(got), want[n - 1:], "fp32")
    eng.close()


# ---- inputs that stand out ------------------------------------------------------------------------------------------------------------------
def loud(cfg, seed, dim, maps=(0,)):
    """weights in which token id 7 carries a key that every query asks for in the given maps of head 0: its embedding row is one loud coordinate (0) that no other
    token has, the key projection turns that coordinate into a large key channel that does not turn, and a coordinate every token shares (1) drives every query there"""
    w0 = ko.random_tensors(cfg, seed)
    p = "l0.mix."
    emb = w0["embed"].copy()
    emb[:, 0] = 0.0; emb[:, 1] = 4.0; emb[7] = 0.0; emb[7, 0] = 12.0; emb[7, 1] = 4.0
    q, k = w0[p + "q"].copy(), w0[p + "k"].copy()
    q[:, :2] = 0.0; k[:, :2] = 0.0
    for i in maps:
        k[i * dim + dim - 1, 0] = 5.0
        q[i * dim + dim - 1, 1] = 4.0
    return {"embed": emb, p + "q": q, p + "k": k}


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("maps", [(0,), (1,)])
@pytest.mark.parametrize("dim,vdim", [(16, 8), (64, 32)])      # (64, 32): the matrix-core kernel in bf16
def test_one_far_key_stands_out(dim, vdim, maps, dtype):
    """the loud key occurs once, at position 3 of 400, and in one map only: every later query must find it among hundreds of keys, across page borders, in portions
    and in decoded tokens, and it must count with that map's weight"""
    cfg = config([attn(heads=2, kv_heads=1, dim=dim, vdim=vdim, scale=dim ** -0.5 * 1.5, rot={"base": 1e4, "dims": dim // 2})], width=16, bigram=None)
    eng, w = engine(cfg, dtype, 8, loud(cfg, 8, dim, maps))
    toks = [t if t != 7 else 8 for t in tokens(cfg, 400)]
    toks[3] = 7
    want = want_of(cfg, w, toks)
    without = list(toks); without[3] = 9
    assert np.abs(want_of(cfg, w, without)[390:] - want[390:]).max() / np.abs(want).max() > 0.05
    got = [eng.step([("r", toks[:200], [2, 3, 4, 199])]), eng.step([("r", toks[200:390], [0, 189])])]
    got += [eng.step([("r", [toks[390 + i]], [0])]) for i in range(10)]
    check(np.concatenate(got), want[[2, 3, 4, 199, 200, 389] + list(range(390, 400))], dtype)
    eng.model.set_option("attn.split_min", 64)            # the keys divided between workgroups
    got = [eng.step([("s", toks[:395], [])])] + [eng.step([("s", [toks[395 + i]], [0])]) for i in range(5)]
    check(np.concatenate(got[1:]), want[395:], dtype, "split")
    eng.close()


@pytest.mark.parametrize("sizes", [[1] * 12, [2] * 6, [5, 1, 6], [12]])
def test_pair_rows_follow_the_token_before(sizes):
    """every pair of neighbouring tokens has a row of its own and the rows are loud: a wrong token before, also across portions, slots and reuse, shows at once"""
    cfg = config([ret()], vocab=11, bigram={"buckets": 121, "mul_prev": 11, "mul_cur": 1})
    w0 = ko.random_tensors(cfg, 3)
    eng, w = engine(cfg, "fp32", 3, {"bigram": w0["bigram"] * 8.0, "embed": w0["embed"] * 0.125})
    seqs = [tokens(cfg, 12, s) for s in range(4)]
    for rnd in range(2):                                   # the second round starts in slots that remember the first one's last tokens
        got, at = [[] for _ in seqs], 0
        for n in sizes:
            order = [0, 2, 1, 3] if (at + rnd) % 2 else [3, 1, 0, 2]
            out = eng.step([(i, seqs[i][at:at + n], list(range(n))) for i in order])
            for k, i in enumerate(order):
                got[i].append(out[k * n:(k + 1) * n])
            at += n
        for i, s in enumerate(seqs):
            check(np.concatenate(got[i]), want_of(cfg, w, s), "fp32", f"round {rnd}, sequence {i}")
            eng.release(i)
    eng.close()


def test_split_keys_form_equals_the_direct_form():
    cfg = config([attn(scale=2.0), attn(kv_heads=1, heads=3)])
    eng, w = engine(cfg, "fp32", 6)
    toks = tokens(cfg, 480)
    want = want_of(cfg, w, toks)
    eng.step([("r", toks[:470], [])])
    eng.model.set_option("attn.split_min", 64)            # steps of few tokens now divide the keys between workgroups
    got = np.concatenate([eng.step([("r", [toks[470 + i]], [0])]) for i in range(10)])
    check(got, want[470:], "fp32")
    eng.close()


@pytest.mark.parametrize("ssd_min", [64, 0])
def test_long_memory_through_the_recurrent_states(ssd_min):
    """decays held near one: both kinds of state still carry the first token after hundreds of steps, through portions and single tokens"""
    cfg = config([cd(dense()), ret(decay=[0.9995, 1.0]), cd()])
    w0 = ko.random_tensors(cfg, 7)
    over = {n: np.full_like(w0[n], -9.0) for n in ("l0.mix.A_log", "l2.mix.A_log")}
    eng, w = engine(cfg, "fp32", 7, over, options={"ssd.min": ssd_min})
    toks = tokens(cfg, 330)
    want = want_of(cfg, w, toks)
    other = want_of(cfg, w, [(toks[0] + 1) % cfg["vocab"]] + toks[1:])
    assert np.abs(other[-1] - want[-1]).max() / np.abs(want).max() > 1e-3      # the first token still matters at the end
    got = [eng.step([("r", toks[:5], [4])]), eng.step([("r", toks[5:130], [0, 124])]), eng.step([("r", toks[130:300], [169])])]
    got += [eng.step([("r", [toks[300 + i]], [0])]) for i in range(30)]
    check(np.concatenate(got), want[[4, 5, 129, 299] + list(range(300, 330))], "fp32")
    eng.close()


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_strong_and_weak_decays(dtype):
    """heads and channels whose state is gone after one token beside ones that forget nothing, through both forms of the recurrences"""
    cfg = config([ret(heads=6, decay=[1e-4, 0.02, 0.4, 0.9, 0.999, 1.0], dim=20, vdim=36), cd(heads=6, kv_heads=3, dim=20, vdim=36)])
    over = {"l1.mix.A_log": np.array([-9.0, -4.0, 0.0, 1.0, 3.0, 5.0]), "l1.mix.dt_bias": np.random.default_rng(0).uniform(-6, 4, 120)}
    toks = tokens(cfg, 270)
    outs = []
    for ssd_min in (1, 0):
        eng, w = engine(cfg, dtype, 9, over, options={"ssd.min": ssd_min})
        outs.append(np.concatenate([eng.step([("r", toks[:100], list(range(100)))]), eng.step([("r", toks[100:269], list(range(169)))]), eng.step([("r", toks[269:], [0])])]))
        eng.close()
    want = want_of(cfg, w, toks)
    check(outs[0], want, dtype)
    check(outs[1], want, dtype)
    assert np.abs(outs[0] - outs[1]).max() / np.abs(outs[1]).max() < 5e-5


def test_a_router_weight_stands_in_front_of_the_square():
    """scores far from one: a weight on an expert's output instead of its input would be off by the score itself"""
    cfg = config([ret(moe(4, 2, 12, 0))])
    w0 = ko.random_tensors(cfg, 5)
    over = {"l0.mlp.router": w0["l0.mlp.router"] - 0.6 * np.sign(w0["l0.mlp.router"].sum(axis=1, keepdims=True)) * 0.5, "l0.hc2.out": w0["l0.hc2.out"] * 6}
    toks = tokens(cfg, 30)
    w = ko.random_tensors(cfg, 5, over)
    want = clear(cfg, w, [toks], 5)[0]
    keep = ko.squared_relu_ff
    eng, _ = engine(cfg, "fp32", 5, w)
    check(run_whole(eng, "a", toks), want, "fp32")
    eng.close()
    out = np.zeros_like(want)
    try:      # the plain form with the weight behind the expert differs by far more than the tolerance
        def behind(h, f, t, pre):
            sel, s = ko.chosen_experts(h, t, pre, f["router"]["top"])
            return np.stack([sum(s[i, k] * keep(h[i], t, f"{pre}e{sel[i, k]}.") for k in range(sel.shape[1])) for i in range(len(h))])
        front, ko.experts_ff = ko.experts_ff, behind
        out = want_of(cfg, w, toks)
    finally:
        ko.experts_ff = front
    assert np.abs(out - want).max() / np.abs(want).max() > 1e-2


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("n", [2, 21, 31, 32, 33, 42, 43, 70])
def test_a_shared_expert_of_the_routed_size(n, dtype):
    """steps of few pairs take the shared expert as one more choice, longer ones compute it by itself: portions on both sides of the border (128 pairs)"""
    cfg = config([ret(moe(5, 3, 16, 16)), cd(moe(9, 2, 24, 24))])
    toks = tokens(cfg, n + 4, seed=n)
    w = ko.random_tensors(cfg, 13)
    want = clear(cfg, w, [toks], 13)[0]
    eng, _ = engine(cfg, dtype, 13, w)
    check_rows(np.concatenate([eng.step([("r", toks[:n], list(range(n)))])] + [eng.step([("r", [t], [0])]) for t in toks[n:]]), want, dtype, "", cfg)
    eng.close()


# ---- batches, slots, pages ----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("ssd_min", [1, 64])
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_unequal_requests_in_one_batch(dtype, ssd_min):
    cfg = config()
    seqs = {"a": tokens(cfg, 170, 1), "b": tokens(cfg, 9, 2), "c": tokens(cfg, 103, 3), "d": tokens(cfg, 1, 4)}
    w = ko.random_tensors(cfg, 7)
    want = dict(zip(seqs, clear(cfg, w, list(seqs.values()), 7)))
    eng, _ = engine(cfg, dtype, 7, w, options={"ssd.min": ssd_min})
    cuts = {"a": [17, 2, 130, 1, 1, 19], "b": [1, 1, 1, 2, 4, 0], "c": [2, 0, 2, 99, 0, 0], "d": [0, 0, 1, 0, 0, 0]}      # 0: the request sits the step out
    got = {k: [] for k in seqs}
    at = {k: 0 for k in seqs}
    for step in range(6):
        entries = []
        for k in seqs:
            n = cuts[k][step]
            if n:
                entries.append((k, seqs[k][at[k]:at[k] + n], list(range(n))))
        out = eng.step(entries)
        o = 0
        for k, tk, _ in entries:
            got[k].append(out[o:o + len(tk)]); o += len(tk); at[k] += len(tk)
    for k in seqs:
        g = np.concatenate(got[k])
        check_rows(g, want[k][:len(g)], dtype, k)
        assert len(g) == min(len(seqs[k]), sum(cuts[k]))
    eng.close()


def test_slots_and_pages_are_used_again():
    """a slot's next request starts from empty states, convolution tails and no token before, whatever the request before left there"""
    cfg = config([cd(dense()), ret(), attn(), dict(attn(), weights_of=2), cd()])
    eng, w = engine(cfg, "fp32", 8, budget_tokens=256, max_ctx=256, max_seqs=2)      # four pages of 64 tokens, two slots
    assert eng.free_tokens == 256
    for rnd in range(5):
        a, b = tokens(cfg, 100 + rnd, 10 + rnd), tokens(cfg, 60 + rnd, 20 + rnd)
        out = eng.step([(("a", rnd), a, [0, 1, 2, len(a) - 1]), (("b", rnd), b[:-1], [])])
        assert eng.free_tokens == 256 - 128 - 64
        with pytest.raises(RuntimeError):      # both slots are taken
            eng.step([(("c", rnd), [1], [])])
        out2 = eng.step([(("b", rnd), b[-1:], [0])], end=[("a", rnd)])
        wa = want_of(cfg, w, a)
        check(np.concatenate([out, out2]), np.stack([wa[0], wa[1], wa[2], wa[-1], want_of(cfg, w, b)[-1]]), "fp32", f"round {rnd}")
        eng.release(("b", rnd))
        assert eng.free_tokens == 256
    eng.step([("big", tokens(cfg, 200), [])])          # the pool refuses what it cannot hold and leaves the slots as they were
    with pytest.raises(TgxError):
        eng.step([("more", tokens(cfg, 100), [])])
    assert eng.length("big") == 200 and eng.length("more") == 0
    eng.close()


def test_a_request_is_the_same_alone_and_beside_others():
    """nothing a token computes reads another entry of the batch; what differs is the summation order of the products (few rows stream the weights,
    many take the matrix-core tiles)"""
    cfg = config([cd(dense()), ret(), attn(dense(9)), ret(dense())])
    eng, w = engine(cfg, "fp32", 9)
    a, b, c = tokens(cfg, 50, 1), tokens(cfg, 20, 2), tokens(cfg, 3, 3)
    alone = np.concatenate([eng.step([("a", a[:31], [30])]), eng.step([("a", a[31:], [18])], ["a"])])
    eng.step([("c", c, [])])
    mixed = np.concatenate([eng.step([("b", b[:7], []), ("a", a[:31], [30])]), eng.step([("a", a[31:], [18]), ("c", [5], []), ("b", b[7:], [])], ["a", "b", "c"])])
    assert np.abs(alone - mixed).max() / np.abs(alone).max() < 1e-5
    eng.close()


# ---- random configurations ------------------------------------------------------------------------------------------------------------------
def random_config(seed):
    r = np.random.default_rng(500 + seed)
    pick = lambda *v: v[int(r.integers(len(v)))]
    layers = []
    for _ in range(int(r.integers(2, 6))):
        e = pick(2, 5, 9)
        mlp = pick(None, dense(int(r.integers(5, 40))), moe(e, int(r.integers(1, e + 1)), int(r.integers(4, 30)), pick(0, 6, 15)))
        kind, g = pick("r", "a", "c"), pick(1, 2, 3)
        if kind == "r":
            d = pick(4, 7, 16, 64)
            layers.append(ret(mlp, heads=g, dim=d, vdim=pick(4, 9, 20), decay=r.uniform(0.3, 1.0, g).tolist(), rot=pick(None, {"base": float(r.uniform(50, 1e5)), "dims": 2 * int(r.integers(1, d // 2 + 1))})))
        elif kind == "a":
            d = pick(4, 6, 16, 64)
            layers.append(attn(mlp, heads=g * pick(1, 2, 4), kv_heads=g, dim=d, vdim=pick(8, 11, 32, 96), scale=float(r.uniform(0.1, 0.5)), diff=float(r.uniform(0, 0.8)), rot=pick(None, {"base": 777.0, "dims": d})))
        else:
            layers.append(cd(mlp, heads=g * pick(1, 2, 3), kv_heads=g, dim=pick(4, 7, 16, 40), vdim=pick(4, 9, 36), conv=pick(1, 2, 4, 6)))
        if len(layers) > 1 and r.integers(4) == 0:
            layers.append(dict(copy.deepcopy(layers[0]), weights_of=0))
    return config(layers, width=int(r.integers(10, 50)), vocab=int(r.integers(30, 90)), eps=pick(1e-6, 1e-5, 1e-3), embed=float(r.uniform(0.5, 4)), streams=pick(1, 2, 3, 4, 6),
                  bigram=pick(None, {"buckets": int(r.integers(1, 200)), "mul_prev": int(r.integers(1, 999)), "mul_cur": int(r.integers(1, 99))})), (int(r.integers(1, 20)), int(r.integers(1, 20)))


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(seed, dtype):
    cfg, ranks = random_config(seed)
    a, b = tokens(cfg, 150, seed), tokens(cfg, 40, seed + 50)
    w = ko.random_tensors(cfg, seed, None, *ranks)
    wa, wb = clear(cfg, w, [a, b], seed)
    eng, _ = engine(cfg, dtype, seed, w, ranks)
    ga, gb = [], []
    out = eng.step([("a", a[:90], list(range(90))), ("b", b[:2], [0, 1])])
    ga.append(out[:90]); gb.append(out[90:])
    out = eng.step([("b", b[2:3], [0]), ("a", a[90:139], list(range(49)))])
    gb.append(out[:1]); ga.append(out[1:])
    for i in range(11):
        out = eng.step([("a", [a[139 + i]], [0]), ("b", b[3 + i:4 + i], [0])])
        ga.append(out[:1]); gb.append(out[1:])
    check_rows(np.concatenate(ga), wa, dtype, "a", cfg); check_rows(np.concatenate(gb), wb[:14], dtype, "b", cfg)
    eng.close()


# ---- generation ---------------------------------------------------------------------------------------------------------------------------
def oracle_greedy(cfg, w, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(np.argmax(want_of(cfg, w, seq)[-1])))
    return seq[len(prompt):]


def test_greedy_generation_through_the_slot_scheduler():
    cfg = config()
    eng, w = engine(cfg, "fp32", 9, max_seqs=2)
    prompts = [tokens(cfg, 11, 1), tokens(cfg, 5, 2), tokens(cfg, 23, 3)]      # three requests on two slots
    want = [oracle_greedy(cfg, w, p, 6) for p in prompts]
    assert eng.generate(prompts, 6) == want
    assert eng.generate(prompts, 6, portion=4) == want
    eng.close()


def test_long_decoding_through_forward_sample_decode():
    cfg = config([cd(dense()), ret(dense()), attn(), dict(ret(dense()), weights_of=1), attn(dense(9))])
    w = ko.random_tensors(cfg, 10)
    m = Model(stack_desc_from_config(cfg, "fp32", max_seqs=2, max_ctx=512)).load_state({k: np.asarray(v, np.float32) for k, v in w.items()}, strict=True).finalize()
    prompts = np.array([tokens(cfg, 7, 1), tokens(cfg, 7, 2)])
    m.forward(prompts)
    first = m.sample(GREEDY)
    rest = np.concatenate([m.decode(75, GREEDY), m.decode(75, GREEDY)])      # crosses two page borders; positions, states, last tokens and their buffer parity (an odd count) advance on the device
    for b in range(2):
        got = [int(first[b])] + rest[:, b].tolist()
        seq = prompts[b].tolist() + got
        lg = want_of(cfg, w, seq[:-1])
        top2 = np.sort(lg[6:], -1)[:, -2:]
        sure = (top2[:, 1] - top2[:, 0]) > 1e-3 * np.abs(lg).max()
        assert (np.argmax(lg[6:], -1)[sure] == np.array(got)[sure]).all()
        assert sure.mean() > 0.9
    assert m.past_length == 7 + 150
    m.close()


# ---- the C++ host engine, the command line, the trace replay ---------------------------------------------------------------------------------
def test_host_engine_and_cli_generate_greedy(tmp_path):
    from host_util import HostEngine, host_lib
    from tinygpt_amd import build
    cfg = config()
    w = ko.random_tensors(cfg, 11)
    write_model_dir(str(tmp_path), cfg, w)
    prompts = [tokens(cfg, 9, 1), tokens(cfg, 4, 2), tokens(cfg, 13, 3)]           # unequal lengths: no padding is fed
    want = [oracle_greedy(cfg, w, p, 5) for p in prompts]
    e = HostEngine(host_lib(), model_dir=str(tmp_path), device="mi355x", dtype=0, max_batch=4)
    assert e.prepare(), e.error()
    e.reconfigure(max_new=5)
    ids, new, fin = e.generate_sync(prompts)
    assert new == 5 and [ids[b, -5:].tolist() for b in range(3)] == want
    e.reconfigure(max_new=5)
    ids2, new2, fin2, seen = e.generate_async(prompts[2])
    assert ids2[-5:].tolist() == want[2]
    e.close()
    build.build_host()
    arg = ";".join(",".join(str(x) for x in p) for p in prompts)
    r = subprocess.run([build.HOST_CLI, "--model", str(tmp_path), "--dtype", "fp32", "--max-tokens", "5", "--temperature", "0", "--top-p", "1", "--prompt-ids", arg,
                        "--context", "256"], capture_output=True, text=True, timeout=120)
    assert r.returncode == 0, r.stderr
    outs = [[int(x) for x in line.split(":")[1].split()] for line in r.stdout.splitlines() if line.startswith("Output ids")]
    assert outs == want


def test_trace_replay_script(tmp_path):
    cfg = config([cd(dense()), attn(), ret(), dict(attn(), weights_of=1)])
    w = ko.random_tensors(cfg, 12)
    mdir, out = tmp_path / "m", tmp_path / "o"
    mdir.mkdir()
    write_model_dir(str(mdir), cfg, w)
    a, b = tokens(cfg, 30, 1), tokens(cfg, 12, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": b[:11], "want": []}, {"id": "x", "tokens": a[20:22], "want": [1]}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[22:], "want": [7]}, {"id": "y", "tokens": b[11:], "want": [0]}], "end": ["x", "y"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    for dtype, tol in (("float32", "fp32"), ("bfloat16", "bf16")):
        r = subprocess.run([sys.executable, f"{root}/bin/trace_run", "--model", str(mdir), "--dtype", dtype, "--out", str(out), "--max-tokens", "128"],
                           input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
        assert r.returncode == 0, r.stderr
        assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
        wa, wb = want_of(cfg, w, a), want_of(cfg, w, b)
        check(np.fromfile(out / "0.f32", "<f4").reshape(2, -1), wa[[0, 19]], tol)
        check(np.fromfile(out / "1.f32", "<f4").reshape(1, -1), wa[[21]], tol)
        check(np.fromfile(out / "2.f32", "<f4").reshape(2, -1), np.stack([wa[29], wb[11]]), tol)


def test_what_the_library_refuses():
    for bad in ([attn(kv_heads=3)],                       # query heads not a multiple of the key heads
                [attn(dim=257)],
                [attn(vdim=257)],
                [attn(rot={"base": 100.0, "dims": 10})],  # more rotated dimensions than there are
                [attn(rot={"base": 100.0, "dims": 3})],
                [ret(decay=[0.5])],                       # a decay per head
                [ret(decay=[0.5, 1.5])],
                [ret(decay=[0.5, 0.0])],
                [ret(dim=257)],
                [cd(heads=4, kv_heads=3)],
                [cd(conv=65)],
                [cd(conv=0)],
                [cd(dim=257)],
                [ret(moe(3, 4))],                         # more choices than experts
                [ret(), dict(ret(vdim=13), weights_of=0)],      # differs from the layer whose weights it uses
                [ret(), dict(ret(), weights_of=1)],       # its own
                [ret(), dict(ret(), weights_of=5)],
                [dict(ret(), weights_of=1), dict(ret(), weights_of=0)]):
        with pytest.raises(TgxError):
            Model(stack_desc_from_config(config(bad), "fp32"))
    with pytest.raises(TgxError):
        Model(stack_desc_from_config(config([ret()], streams=17), "fp32"))
    cfg = config()
    for name in ("l0.mix.a1", "l0.mix.g2", "l2.mix.lk2", "l1.hc2.mix", "l3.mlp.e6.down", "bigram", "head"):
        w = ko.random_tensors(cfg, 0)
        m = Model(stack_desc_from_config(cfg, "fp32"))
        del w[name]
        m.load_state({k: np.asarray(v, np.float32) for k, v in w.items()}, strict=True)
        with pytest.raises(TgxError, match=name):
            m.finalize()
        m.close()
    m = Model(stack_desc_from_config(cfg, "fp32"))
    with pytest.raises(TgxError):                         # a layer on another's weights has no tensors
        m.upload("l5.norm1", np.zeros(cfg["width"], np.float32))
    m.close()


# ---- attention on the matrix cores (16-bit storage; key sizes 64 / 128 / 256) ------------------------------------------------------------------
@pytest.mark.parametrize("heads,kv,dim,vdim", [(4, 1, 64, 128), (8, 2, 128, 64), (6, 3, 64, 96), (2, 2, 256, 256)])
def test_matrix_core_attention_equals_the_lane_kernel(heads, kv, dim, vdim):
    """the same bf16 weights and cached rows through both attention kernels: portions whose 32-row tiles cut through tokens, a mixed batch, decoding, contexts across
    page borders, and the split-keys form"""
    cfg = config([attn(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=1.2 * dim ** -0.5, rot={"base": 1e4, "dims": dim // 2})], width=64)
    w = ko.random_tensors(cfg, heads)
    tens = {k: np.asarray(v, np.float32) for k, v in w.items()}
    mk = lambda: SlotEngine(desc=stack_desc_from_config(cfg, "bf16", max_seqs=4, max_ctx=1024, budget_tokens=2048), tensors=tens)
    fast, slow = mk(), mk()
    slow.model.set_option("attn.mfma", 0)
    a, b, c = tokens(cfg, 200, 1), tokens(cfg, 75, 2), tokens(cfg, 9, 3)
    want = want_of(cfg, w, a)[[0, 1, 69, 130, 131, 199]]
    outs = []
    for eng in (fast, slow):
        o = [eng.step([("a", a[:70], [0, 1, 69]), ("b", b[:3], [2])])]
        o.append(eng.step([("a", a[70:131], [60]), ("c", c, [8]), ("b", b[3:4], [0])]))
        o.append(eng.step([("b", b[4:], [70]), ("a", a[131:132], [0])]))
        o.append(eng.step([("a", a[132:199], [])]))
        eng.model.set_option("attn.split_min", 64)
        o.append(eng.step([("a", a[199:], [0]), ("b", [5], [0])]))
        outs.append(np.concatenate(o))
    assert np.abs(outs[0] - outs[1]).max() / np.abs(outs[1]).max() < 5e-4
    check(outs[0][[0, 1, 2, 4, 8, 9]], want, "bf16")               # a's positions 0, 1, 69, 130, 131, 199 in the order the steps returned them
    check(outs[0][[6, 7]], want_of(cfg, w, b)[[3, 74]], "bf16")
    fast.close(); slow.close()
