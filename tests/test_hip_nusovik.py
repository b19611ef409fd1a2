"""The Nusovik design on the GPU against the plain oracle of tests/nusovik_oracle.py: every mechanism on a configuration of its own, prompts against
token-by-token decoding, portions down to two tokens, mixed batches, slots and pages that are used again, keys just inside and just outside every chunk
(in prompts and in decoding), far keys under the distance bias, page borders, sinks, long decoding through the recurrent states, and greedy generation through
the slot scheduler, tgx_forward / tgx_sample / tgx_decode, the C++ engine, the command line and bin/trace_run.  Models are config dictionaries of the
checkpoint format, so the configuration reader is on the path of every test.  fp32 storage is the sharp comparison (nothing is rounded: 1e-4 of the
largest logit); bf16 storage rounds the cached keys and values (3e-2)."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import nusovik_oracle as no
from test_hip_modepel import write_model_dir
from tinygpt_amd.desc import stack_desc_from_config
from tinygpt_amd.ffi import GREEDY, Model, TgxError
from tinygpt_amd.serving import SlotEngine

pytestmark = pytest.mark.gpu
TOL = {"fp32": 1e-4, "bf16": 3e-2}


# ---- configurations ---------------------------------------------------------------------------------------------------------------
def ff(n=20):
    return {"kind": "dense", "ff": n}


def mamba(mlp=None, **kw):
    m = dict(conv=4, dt_rank=3, inner=28, state=6)
    m.update(kw)
    return {"type": "mamba1", "mixer": m, "mlp": mlp}


def par(mlp=None, left=None, right=None, left_scale=0.8, right_scale=1.3):
    l = dict(heads=4, kv_heads=2, dim=8, vdim=8, mask={"size": 9}, scale=0.5, bias_max=13)
    r = dict(conv=4, groups=2, heads=4, norm_groups=2, state=8, vdim=6)
    l.update(left or {}); r.update(right or {})
    l["vdim"] = l["dim"]
    return {"type": "parallel", "mixer": {"left": {k: v for k, v in l.items() if v is not None}, "right": r, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def config(layers=None, width=24, vocab=67, eps=1e-5, embed=2.0, logits=1.5):
    return {"architecture": "Nusovik", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": embed}, "logit_scale": logits,
            "layers": copy.deepcopy(layers) if layers is not None else [mamba(), par(ff(13)), mamba(ff()), par(), mamba()]}


def engine(cfg, dtype="fp32", seed=0, overrides=None, buckets=8, options=None, **kw):
    w = no.random_tensors(cfg, seed, overrides, buckets)
    kw = dict(dict(max_seqs=4, max_ctx=1024, budget_tokens=2048), **kw)
    eng = SlotEngine(desc=stack_desc_from_config(cfg, dtype, **kw), tensors={k: np.asarray(v, np.float32) for k, v in w.items()})
    for k, v in (options or {}).items():
        eng.model.set_option(k, v)
    return eng, w


def tokens(cfg, n, seed=0):
    return np.random.default_rng(100 + seed).integers(0, cfg["vocab"], n).tolist()


def want_of(cfg, w, toks):
    return no.forward(cfg, w, toks)


def check(got, want, dtype, what=""):
    err = np.abs(got - want).max() / np.abs(want).max()
    assert err < TOL[dtype], f"{what}: {err:.3e}"


def run_whole(eng, rid, toks):
    return eng.step([(rid, toks, list(range(len(toks))))], [rid])


# ---- every mechanism on a configuration of its own --------------------------------------------------------------------------------------
MECH = {
    "mamba1_alone": [mamba()],
    "mamba1_one_state_number": [mamba(state=1)],
    "mamba1_eight_state_numbers": [mamba(state=8)],
    "mamba1_sixteen": [mamba(state=16, inner=40)],
    "mamba1_twenty": [mamba(state=20, inner=37)],
    "mamba1_thirty": [mamba(state=30, inner=17)],
    "mamba1_fifty": [mamba(state=50, inner=33)],
    "mamba1_hundred": [mamba(state=100, inner=19)],
    "mamba1_largest_state": [mamba(state=256, inner=18)],
    "mamba1_rank_one": [mamba(dt_rank=1)],
    "mamba1_rank_sixteen": [mamba(dt_rank=16)],
    "mamba1_many_channels": [mamba(inner=300, state=4)],
    "mamba1_one_channel": [mamba(inner=1)],
    "mamba1_one_tap": [mamba(conv=1)],
    "mamba1_two_taps": [mamba(conv=2)],
    "mamba1_three_taps": [mamba(conv=3)],
    "mamba1_seven_taps": [mamba(conv=7)],
    "mamba1_more_taps_than_tokens": [mamba(conv=40)],
    "mamba1_with_feed_forward": [mamba(ff(17)), mamba()],
    "parallel_alone": [par()],
    "parallel_left_half_only": [par(right_scale=0.0)],
    "parallel_right_half_only": [par(left_scale=0.0)],
    "parallel_scales_of_one": [par(left_scale=1.0, right_scale=1.0)],
    "one_key_head_per_query_head": [par(left={"kv_heads": 4})],
    "one_key_head_for_all": [par(left={"heads": 6, "kv_heads": 1, "dim": 10})],
    "one_head": [par(left={"heads": 1, "kv_heads": 1})],
    "wide_heads": [par(left={"heads": 2, "kv_heads": 1, "dim": 80, "scale": 0.2})],          # more than one channel per lane
    "widest_heads": [par(left={"heads": 2, "kv_heads": 2, "dim": 256, "scale": 0.1})],
    "no_mask": [par(left={"mask": None})],
    "chunks_of_one": [par(left={"mask": {"size": 1}})],
    "chunks_longer_than_the_sequence": [par(left={"mask": {"size": 400}, "bias_max": 9})],
    "distances_beyond_the_table": [par(left={"mask": None, "bias_max": 5})],
    "bias_reaches_past_the_chunk": [par(left={"bias_max": 500})],
    "ssd_one_head": [par(right={"heads": 1, "groups": 1, "norm_groups": 1})],
    "ssd_every_head_its_own_group": [par(right={"heads": 3, "groups": 3, "norm_groups": 1})],
    "ssd_one_group": [par(right={"heads": 6, "groups": 1, "norm_groups": 3})],
    "ssd_norm_parts_across_heads": [par(right={"heads": 4, "vdim": 6, "norm_groups": 8})],
    "ssd_wide_values": [par(right={"heads": 2, "groups": 1, "vdim": 70, "norm_groups": 1})],
    "ssd_large_state": [par(right={"heads": 2, "groups": 2, "state": 132, "vdim": 12, "norm_groups": 2})],
    "ssd_largest_state": [par(right={"heads": 2, "groups": 1, "state": 256, "vdim": 34, "norm_groups": 1})],
    "ssd_sizes_off_the_vectors": [par(right={"heads": 3, "groups": 1, "state": 7, "vdim": 5, "norm_groups": 5})],
    "ssd_one_tap": [par(right={"conv": 1})],
    "ssd_two_taps": [par(right={"conv": 2})],
    "ssd_nine_taps": [par(right={"conv": 9})],
    "ssd_wide_parts": [par(right={"heads": 8, "vdim": 300, "groups": 1, "norm_groups": 1})],      # a part beyond the registers of the norm
    "no_feed_forward_anywhere": [mamba(), par(), mamba()],
    "feed_forward_everywhere": [mamba(ff(33)), par(ff(8)), mamba(ff(19))],
    "ragged_sizes": [mamba(ff(19), inner=23, state=5, dt_rank=2, conv=3), par(ff(11), left={"heads": 6, "kv_heads": 3, "dim": 6}, right={"heads": 5, "groups": 5, "state": 3, "vdim": 7, "conv": 3, "norm_groups": 7})],
    "deep": [mamba(), par(ff(13)), mamba(ff()), par(), mamba(), par(ff()), mamba(), par(ff(13)), mamba(ff()), par()],
}
EXTRA = {"ragged_sizes": dict(width=27, vocab=53), "wide_heads": dict(width=40), "deep": dict(embed=1.0, logits=1.0), "mamba1_alone": dict(eps=1e-3)}
BUCKETS = {"chunks_longer_than_the_sequence": 6, "distances_beyond_the_table": 3, "parallel_alone": 2, "no_mask": 12, "deep": 16}


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("name", list(MECH))
def test_mechanism(name, dtype):
    cfg = config(MECH[name], **EXTRA.get(name, {}))
    toks = tokens(cfg, 23, seed=len(name))
    eng, w = engine(cfg, dtype, seed=len(name), buckets=BUCKETS.get(name, 8))
    want = want_of(cfg, w, toks)
    check(run_whole(eng, "a", toks), want, dtype, name)
    # ... the same tokens one by one through the cache and the recurrent states
    got = np.concatenate([eng.step([("b", [t], [0])]) for t in toks])
    check(got, want, dtype, name + " by steps")
    # ... and with the scalar-decay recurrence in blocks whatever the portion's length
    eng.model.set_option("ssd.min", 1)
    check(np.concatenate([eng.step([("c", toks[:3], [0, 1, 2])]), eng.step([("c", toks[3:], list(range(20)))])]), want, dtype, name + " in blocks")
    eng.close()


# ---- prompts, decoding, portions --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_prompt_then_token_by_token(dtype):
    cfg = config()
    eng, w = engine(cfg, dtype, 1)
    toks = tokens(cfg, 40)
    want = want_of(cfg, w, toks)
    got = [eng.step([("r", toks[:9], list(range(9)))])]
    for i in range(9, 40):
        got.append(eng.step([("r", [toks[i]], [0])]))
    check(np.concatenate(got), want, dtype)
    eng.release("r")
    got = np.concatenate([eng.step([("s", [toks[i]], [0])]) for i in range(6)])      # the first tokens of a sequence in a slot that held another one
    check(got, want[:6], dtype, "from the first token")
    eng.close()


@pytest.mark.parametrize("ssd_min", [1, 64, 0])
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("sizes", [[2] * 20, [3, 2, 5, 2, 7, 1, 11, 2, 2], [64, 2, 63, 1], [1, 128, 2, 65], [5, 59, 64, 2], [1, 1, 1, 2, 1, 3, 17], [33, 31, 200, 2]])
def test_portions(sizes, dtype, ssd_min):
    """portions cut through chunks, the convolutions' taps, the scans' token groups and the blocks of the scalar-decay recurrence"""
    cfg = config()
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
    cfg = config([par(left={"mask": {"size": 70}, "scale": 2.0}), mamba(), par(ff(), left={"mask": {"size": 128}, "bias_max": 100})])
    eng, w = engine(cfg, "fp32", 4)
    toks = tokens(cfg, n + 3, seed=n)
    want = want_of(cfg, w, toks)
    got = [eng.step([("r", toks[:n], [n - 1])])]
    got += [eng.step([("r", [toks[n + i]], [0])]) for i in range(3)]      # decoding across the border
    check(np.concatenate(got), want[n - 1:], "fp32")
    eng.close()


# ---- keys that stand out: a chunk's edge that is one token off, or a far key that is lost, shows as a large error ------------------------------
def loud(cfg, seed, dim):
    """weights in which token id 7 carries a key that every query asks for: its embedding row is one loud coordinate (0) that no other token has, the key
    projection turns that coordinate into a large key channel, and a coordinate that every token shares (1) drives every query towards that channel"""
    w0 = no.random_tensors(cfg, seed)
    p = "l0.mix.left."
    emb = w0["embed"].copy()
    emb[:, 0] = 0.0; emb[:, 1] = 4.0; emb[7] = 0.0; emb[7, 0] = 12.0; emb[7, 1] = 4.0
    k = w0[p + "k"].copy(); k[:, 0] = 0.0; k[:, 1] = 0.0; k[5, 0] = 8.0
    q = w0[p + "q"].copy(); q[:, 0] = 0.0; q[:, 1] = 0.0
    q[5, 1] = 3.0; q[dim + 5, 1] = 3.0
    return {"embed": emb, p + "k": k, p + "q": q, p + "rel": w0[p + "rel"] * 0.5, "l0.norm1": np.full_like(w0["l0.norm1"], 6.0)}


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("dim", [16, 64])      # 64: the matrix-core kernel in bf16
@pytest.mark.parametrize("size,at", [(4, 5), (64, 64), (64, 127), (70, 75), (130, 131), (200, 3)])
def test_chunk_edges_in_prompts_and_in_decoding(size, at, dim, dtype):
    """the loud key sits at position `at`: the rest of its block of `size` positions sees it, the next block's first position does not"""
    cfg = config([par(left={"heads": 2, "kv_heads": 1, "dim": dim, "mask": {"size": size}, "scale": 3.0 * (8 / dim) ** 0.5, "bias_max": 40}, left_scale=1.0, right_scale=0.0)], width=16)
    over = loud(cfg, 7, dim)
    edge = (at // size + 1) * size                         # the first position of the next block
    n = edge + 5
    toks = [t if t != 7 else 8 for t in tokens(cfg, n, seed=size)]
    toks[at] = 7
    for cut in (n, edge - 1, edge, edge + 1, at + 1):
        eng, w = engine(cfg, dtype, 7, over)
        want = want_of(cfg, w, toks)
        if cut == n and edge - 1 > at:
            without = list(toks); without[at] = 9
            other = want_of(cfg, w, without)
            assert np.abs(other[edge - 1] - want[edge - 1]).max() / np.abs(want).max() > 0.05
            assert np.abs(other[edge:] - want[edge:]).max() == 0.0
        places = sorted({p for p in (at, edge - 2, edge - 1, edge, edge + 1, n - 1) if at <= p < n})
        got = [eng.step([("r", toks[:cut], [p for p in places if p < cut])])]
        got += [eng.step([("r", [toks[i]], [0] if i in places else [])]) for i in range(cut, n)]
        check(np.concatenate([g for g in got if len(g)]), want[places], dtype, f"prompt of {cut}")
        eng.close()


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("dim", [16, 64])
def test_one_far_key_stands_out(dim, dtype):
    """the loud key occurs once, at position 3 of 400: every later query must find it among hundreds of keys, across page borders, in portions and in decoded
    tokens, at distances beyond the table's last exact row"""
    cfg = config([par(left={"heads": 2, "kv_heads": 1, "dim": dim, "mask": {"size": 450}, "scale": 3.0 * (8 / dim) ** 0.5, "bias_max": 300}, left_scale=1.0, right_scale=0.0)], width=16)
    over = loud(cfg, 8, dim)
    eng, w = engine(cfg, dtype, 8, over)
    toks = [t if t != 7 else 8 for t in tokens(cfg, 400)]
    toks[3] = 7
    want = want_of(cfg, w, toks)
    without = list(toks); without[3] = 9
    assert np.abs(want_of(cfg, w, without)[390:] - want[390:]).max() / np.abs(want).max() > 0.05
    got = [eng.step([("r", toks[:200], [2, 3, 4, 199])]), eng.step([("r", toks[200:390], [0, 189])])]
    got += [eng.step([("r", [toks[390 + i]], [0])]) for i in range(10)]
    check(np.concatenate(got), want[[2, 3, 4, 199, 200, 389] + list(range(390, 400))], dtype)
    eng.close()


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("dim", [8, 64])
@pytest.mark.parametrize("buckets,bias_max", [(2, 2), (4, 17), (7, 40), (8, 64), (32, 130), (32, 17), (64, 700)])
def test_distance_rows_one_by_one(buckets, bias_max, dim, dtype):
    """scores are zero and every row of the distance table is far from its neighbours: a distance that falls into a wrong row shows at once"""
    cfg = config([par(left={"heads": 2, "kv_heads": 1, "dim": dim, "mask": {"size": 150}, "scale": 1e-3, "bias_max": bias_max}, left_scale=1.0, right_scale=0.0)], width=16)
    rel = np.where(np.arange(buckets)[:, None] % 2 == np.arange(2)[None, :], 3.0, -3.0) + 0.25 * np.arange(buckets)[:, None] / buckets
    over = {"l0.mix.left.rel": rel, "l0.mix.left.sink": np.array([-1.0, 2.0])}
    eng, w = engine(cfg, dtype, 3, over, buckets)
    toks = tokens(cfg, 310, seed=bias_max)
    want = want_of(cfg, w, toks)
    got = [eng.step([("r", toks[:130], list(range(130)))]), eng.step([("r", toks[130:300], list(range(170)))])]
    got += [eng.step([("r", [toks[300 + i]], [0])]) for i in range(10)]
    check(np.concatenate(got), want, dtype)
    eng.model.set_option("attn.split_min", 64)            # the keys divided between workgroups
    got = [eng.step([("s", toks[:290], [])])] + [eng.step([("s", [toks[290 + i]], [0])]) for i in range(10)]
    check(np.concatenate(got[1:]), want[290:300], dtype, "split")
    eng.close()


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("dim", [8, 64])
def test_sinks_decide(dim, dtype):
    """sinks far above the scores mute a head, sinks far below leave it alone: each head follows its own number"""
    cfg = config([par(left={"heads": 4, "kv_heads": 2, "dim": dim, "scale": dim ** -0.5, "mask": {"size": 80}}, left_scale=1.0, right_scale=0.0)], width=16)
    over = {"l0.mix.left.sink": np.array([8.0, -9.0, 1.0, 4.0])}
    eng, w = engine(cfg, dtype, 5, over)
    toks = tokens(cfg, 100)
    want = want_of(cfg, w, toks)
    swapped = want_of(cfg, dict(w, **{"l0.mix.left.sink": np.array([-9.0, 8.0, 4.0, 1.0])}), toks)
    assert np.abs(swapped - want).max() / np.abs(want).max() > 0.1
    check(np.concatenate([eng.step([("r", toks[:70], list(range(70)))]), eng.step([("r", toks[70:98], list(range(28)))]), eng.step([("r", [toks[98]], [0])]), eng.step([("r", [toks[99]], [0])])]),
          want, dtype)
    eng.close()


def test_split_keys_form_equals_the_direct_form():
    cfg = config([par(left={"mask": {"size": 500}, "scale": 2.0, "bias_max": 200}), par(left={"mask": None})])
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
    cfg = config([mamba(ff()), par(left_scale=0.0), mamba()])
    w0 = no.random_tensors(cfg, 7)
    over = {"l0.mix.A_log": np.full_like(w0["l0.mix.A_log"], -9.0), "l2.mix.A_log": np.full_like(w0["l2.mix.A_log"], -9.0), "l1.mix.right.A_log": np.full_like(w0["l1.mix.right.A_log"], -9.0)}
    eng, w = engine(cfg, "fp32", 7, over, options={"ssd.min": ssd_min})
    toks = tokens(cfg, 330)
    want = want_of(cfg, w, toks)
    other = want_of(cfg, w, [toks[0] + 1] + toks[1:])
    assert np.abs(other[-1] - want[-1]).max() / np.abs(want).max() > 1e-3      # the first token still matters at the end
    got = [eng.step([("r", toks[:5], [4])]), eng.step([("r", toks[5:130], [0, 124])]), eng.step([("r", toks[130:300], [169])])]
    got += [eng.step([("r", [toks[300 + i]], [0])]) for i in range(30)]
    check(np.concatenate(got), want[[4, 5, 129, 299] + list(range(300, 330))], "fp32")
    eng.close()


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_strong_and_weak_decays_in_blocks(dtype):
    """heads whose state is gone after one token beside heads that forget nothing: the blocked recurrence's differences of summed logarithms, next to the scan"""
    cfg = config([par(right={"heads": 8, "groups": 2, "state": 20, "vdim": 36, "norm_groups": 4}, left_scale=0.0)])
    over = {"l0.mix.right.A_log": np.array([-9.0, -4.0, -1.0, 0.0, 1.0, 2.0, 3.5, 5.0]), "l0.mix.right.dt_bias": np.array([2.0, -3.0, 0.0, 1.0, -1.0, 2.0, 3.0, 0.0])}
    toks = tokens(cfg, 270)
    outs = []
    for ssd_min in (1, 0):
        eng, w = engine(cfg, dtype, 9, over, options={"ssd.min": ssd_min})
        outs.append(np.concatenate([eng.step([("r", toks[:100], list(range(100)))]), eng.step([("r", toks[100:269], list(range(169)))]), eng.step([("r", toks[269:], [0])])]))
        eng.close()
    want = want_of(cfg, w, toks)
    check(outs[0], want, dtype)
    check(outs[1], want, dtype)
    assert np.abs(outs[0] - outs[1]).max() / np.abs(outs[1]).max() < 2e-5


# ---- batches, slots, pages ----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("ssd_min", [1, 64])
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_unequal_requests_in_one_batch(dtype, ssd_min):
    cfg = config()
    eng, w = engine(cfg, dtype, 7, options={"ssd.min": ssd_min})
    seqs = {"a": tokens(cfg, 170, 1), "b": tokens(cfg, 9, 2), "c": tokens(cfg, 103, 3), "d": tokens(cfg, 1, 4)}
    want = {k: want_of(cfg, w, v) for k, v in seqs.items()}
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
        check(g, want[k][:len(g)], dtype, k)
        assert len(g) == min(len(seqs[k]), sum(cuts[k]))
    eng.close()


def test_slots_and_pages_are_used_again():
    """a slot's next request starts from empty states and convolution tails, whatever the request before left there"""
    cfg = config()
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
    cfg = config()
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
    for _ in range(int(r.integers(2, 5))):
        mlp = ff(int(r.integers(5, 40))) if r.integers(2) else None
        if r.integers(2):
            layers.append(mamba(mlp, conv=pick(1, 2, 3, 4, 5), dt_rank=int(r.integers(1, 12)), inner=int(r.integers(3, 90)), state=int(r.integers(1, 40))))
        else:
            g, d_g, d_per, parts = pick(1, 2, 3), pick(1, 2), pick(1, 2, 3), pick(1, 2, 4)
            layers.append(par(mlp, {"heads": g * pick(1, 2, 4), "kv_heads": g, "dim": pick(4, 7, 16, 64), "mask": {"size": int(r.integers(2, 90))}, "scale": float(r.uniform(0.1, 0.6)), "bias_max": int(r.integers(6, 90))},
                              {"conv": pick(1, 2, 4, 6), "groups": d_g, "heads": d_g * d_per, "state": pick(4, 5, 12, 40, 68), "vdim": 4 * pick(1, 2, 5, 9), "norm_groups": parts},
                              float(r.uniform(0.3, 1.2)), float(r.uniform(0.3, 1.2))))
    return config(layers, width=int(r.integers(10, 50)), vocab=int(r.integers(30, 90)), eps=pick(1e-6, 1e-5, 1e-3), embed=float(r.uniform(0.5, 4)), logits=float(r.uniform(0.5, 3))), pick(4, 6, 9, 10)


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("seed", range(10))
def test_random_configurations(seed, dtype):
    cfg, buckets = random_config(seed)
    eng, w = engine(cfg, dtype, seed, buckets=buckets)
    a, b = tokens(cfg, 150, seed), tokens(cfg, 40, seed + 50)
    wa, wb = want_of(cfg, w, a), want_of(cfg, w, b)
    out = eng.step([("a", a[:90], list(range(90))), ("b", b[:2], [0, 1])])
    check(out[:90], wa[:90], dtype, "a"); check(out[90:], wb[:2], dtype, "b")
    out = eng.step([("b", b[2:3], [0]), ("a", a[90:139], list(range(49)))])
    check(out[:1], wb[2:3], dtype, "b"); check(out[1:], wa[90:139], dtype, "a")
    for i in range(11):
        out = eng.step([("a", [a[139 + i]], [0]), ("b", b[3 + i:4 + i], [0])])
        check(out, np.stack([wa[139 + i], wb[3 + i]]), dtype, f"decoded {i}")
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
    cfg = config([mamba(ff()), par(ff(), left={"mask": {"size": 40}}), mamba(), par(left={"mask": {"size": 90}, "bias_max": 60})])
    w = no.random_tensors(cfg, 10)
    m = Model(stack_desc_from_config(cfg, "fp32", max_seqs=2, max_ctx=512)).load_state({k: np.asarray(v, np.float32) for k, v in w.items()}, strict=True).finalize()
    prompts = np.array([tokens(cfg, 7, 1), tokens(cfg, 7, 2)])
    m.forward(prompts)
    first = m.sample(GREEDY)
    rest = np.concatenate([m.decode(75, GREEDY), m.decode(75, GREEDY)])      # crosses two page borders and many chunks; positions, states and their buffer parity (an odd count) advance on the device
    for b in range(2):
        got = [int(first[b])] + rest[:, b].tolist()
        seq = prompts[b].tolist() + got
        lg = want_of(cfg, w, seq[:-1])
        top2 = np.sort(lg[6:], -1)[:, -2:]
        clear = (top2[:, 1] - top2[:, 0]) > 1e-3 * np.abs(lg).max()
        assert (np.argmax(lg[6:], -1)[clear] == np.array(got)[clear]).all()
        assert clear.mean() > 0.9
    assert m.past_length == 7 + 150
    m.close()


# ---- the C++ host engine, the command line, the trace replay ---------------------------------------------------------------------------------
def test_host_engine_and_cli_generate_greedy(tmp_path):
    from host_util import HostEngine, host_lib
    from tinygpt_amd import build
    cfg = config([mamba(ff()), par(ff()), par(), mamba()])
    w = no.random_tensors(cfg, 11, buckets=6)              # (the C++ reader leaves the rows of the distance table to the tensors)
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
    cfg = config([par(ff()), mamba(), par(), mamba(ff())])
    w = no.random_tensors(cfg, 12, buckets=4)
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
    wrong_values = par()
    wrong_values["mixer"]["left"]["vdim"] = 4             # the keys are the values
    for bad in ([par(left={"kv_heads": 3})],              # query heads not a multiple of the key heads
                [wrong_values],
                [par(left={"mask": {"size": 0}})],
                [par(left={"bias_max": 0})],
                [par(left={"dim": 257})],
                [par(right={"heads": 4, "groups": 3})],
                [par(right={"norm_groups": 5})],          # channels that do not divide into equal parts
                [par(right={"conv": 65})],
                [par(right={"state": 257})],
                [mamba(conv=0)],
                [mamba(state=257)],
                [mamba(dt_rank=0)]):
        with pytest.raises(TgxError):
            Model(stack_desc_from_config(config(bad), "fp32"))
    cfg = config([par(), mamba()])
    for name in ("l0.mix.left.rel", "l0.mix.right.D", "l1.mix.dt.b", "head"):
        w = no.random_tensors(cfg, 0)
        m = Model(stack_desc_from_config(cfg, "fp32"))
        del w[name]
        m.load_state({k: np.asarray(v, np.float32) for k, v in w.items()}, strict=True)
        with pytest.raises(TgxError, match=name):
            m.finalize()
        m.close()
    w = no.random_tensors(cfg, 0, buckets=40)             # every distance below bias_max is an exact row: the logarithmic rows have no range
    m = Model(stack_desc_from_config(cfg, "fp32"))
    with pytest.raises(TgxError, match="rel"):
        m.load_state({k: np.asarray(v, np.float32) for k, v in w.items()}, strict=True)
    m.close()


# ---- attention on the matrix cores (16-bit storage; head sizes 64 / 128 / 256) ------------------------------------------------------------------
@pytest.mark.parametrize("size", [None, 1, 31, 64, 150])
@pytest.mark.parametrize("heads,kv,dim", [(4, 1, 64), (8, 2, 128), (6, 3, 64), (2, 2, 256)])
def test_matrix_core_attention_equals_the_lane_kernel(heads, kv, dim, size):
    """the same bf16 weights and cached rows through both attention kernels: portions whose 32-row tiles cut through tokens, chunks that start inside a key tile,
    a mixed batch, decoding, contexts across page borders, and the split-keys form"""
    cfg = config([par(left=dict(heads=heads, kv_heads=kv, dim=dim, mask={"size": size} if size else None, scale=1.2 * dim ** -0.5, bias_max=70))], width=64)
    w = no.random_tensors(cfg, heads)
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
    assert np.abs(outs[0] - outs[1]).max() / np.abs(outs[1]).max() < 3e-4
    check(outs[0][[0, 1, 2, 4, 8, 9]], want, "bf16")               # a's positions 0, 1, 69, 130, 131, 199 in the order the steps returned them
    check(outs[0][[6, 7]], want_of(cfg, w, b)[[3, 74]], "bf16")
    fast.close(); slow.close()
