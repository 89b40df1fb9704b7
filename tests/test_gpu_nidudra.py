"""GPU tests of the Nidudra model class: the engine (llama_lite over the MI355X backend) against the plain numpy reference of
tests/nidudra_ref.py, on small models with their own sizes and random weights.

f32 serving is the sharp instrument: with 32-bit arithmetic end to end a key wrongly seen or hidden, a missing sink, a convolution tap from the wrong
token, values taken behind the norm instead of in front of it or a lost state moves a logit row by 1e-3 of its spread and more, ten times the gate
(1e-4).  bf16 serving is gated at its rounding level.  Where random data could hide a fault (a key far back among hundreds, a window's edge, the
first tokens, a constant) a test shows that the data discriminate: the same rows are far from the reference computed with the neighbouring rule."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import harness as T
import llama_box_amd as L
import nidudra_ref as R
from llama_box_amd.trace import TraceSession

pytestmark = pytest.mark.gpu

F32_GATE, BF16_GATE = 1e-4, 5e-2


def row_err(got, ref):
    """per row: rms of the difference (means removed) over the rms of the reference row (mean removed)"""
    d = got - ref
    d = d - d.mean(axis=-1, keepdims=True)
    r = ref - ref.mean(axis=-1, keepdims=True)
    return np.sqrt((d * d).mean(axis=-1)) / np.sqrt((r * r).mean(axis=-1))


def within(e, gate, dtype):
    """f32: every row within the gate.  bf16: its rounding now and then turns a router's near-tie the other way — such a row (and, through the states, a few behind it) is
    off by an expert's whole output, which says nothing about the arithmetic (the f32 runs settle the choice) — so the bulk of the rows is within the gate, the median well within"""
    e = np.asarray(e)
    if dtype == "f32":
        return bool(e.max() <= gate)
    return bool(np.quantile(e, 0.85) <= gate and np.median(e) <= gate / 2)


def toks(n, vocab, seed):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


def cfg_a():
    # every mixer and feed-forward; both frequency schedules over a part of the head; two windows over ONE cache (the later layer's is the longer one); 3 query heads per key head;
    # key size != value size; a layer without feed-forward
    return R.make_config(64, 97, [
        R.sink_layer(6, 2, 16, 24, 0.3, R.rot(12, 2000.0, R.banded(4.0, 1.0, 4.0, 128)), R.dense(48)),
        R.window_layer(6, 2, 16, 12, 0.35, R.moe(20, 6, 2, shared=28), size=9, keep_first=2),
        R.parallel_layer(4, 2, 24, 0.25, R.rot(16, 900.0, R.ramped(8.0, 256, 16.0, 1.0)), 3, r_heads=3, r_dim=12, r_vdim=20, tau=9.0, mlp=R.dense(40)),
        R.window_layer(4, 2, 16, 12, 0.3, None, size=37, keep_first=5, kv_from=1),
        R.parallel_layer(3, 1, 8, 0.4, R.rot(8, 50.0), 5, r_heads=2, r_dim=20, r_vdim=8, tau=1.0, mlp=R.moe(16, 5, 1, shared=12)),
    ], softcap=7.0, eps=3e-5)


def cfg_b():
    # rows that are no multiple of 8 (width 52); one head everywhere; no window, no rotation, no frequency scaling; one tap (no history); one expert per token; no shared expert, no cap; the last
    # layer has no feed-forward
    return R.make_config(52, 50, [
        R.window_layer(1, 1, 12, 20, 0.3, R.moe(12, 4, 1)),
        R.parallel_layer(1, 1, 14, 0.4, R.rot(0, 100.0), 1, r_heads=1, r_dim=6, r_vdim=10, tau=3.0, mlp=R.dense(12), rank=1),
        R.sink_layer(2, 1, 8, 8, 0.5, R.rot(8, 300.0), None),
    ], softcap=None, eps=1e-6)


def cfg_c():
    # no recurrence anywhere (no sequence state); three layers over the first one's cache under three different windows, one of them none; every expert chosen
    return R.make_config(48, 257, [
        R.window_layer(4, 4, 8, 16, 0.5, R.moe(16, 8, 8, shared=8), size=6, keep_first=1),
        R.window_layer(4, 4, 8, 16, 0.5, R.dense(24), size=64, keep_first=0, kv_from=0),
        R.window_layer(8, 4, 8, 16, 0.4, None, kv_from=0),
        R.window_layer(4, 4, 8, 16, 0.5, R.dense(24), size=1, keep_first=3, kv_from=0),
    ], softcap=3.0, eps=1e-5)


def cfg_d():
    # heads wider than 128 (the row kernels serve prompts too), value rows beyond 128, key rows of the recurrence beyond 128; many experts
    return R.make_config(96, 120, [
        R.sink_layer(3, 1, 136, 40, 0.09, R.rot(100, 10000.0, R.banded(8.0, 2.0, 6.0, 512)), R.moe(32, 20, 7, shared=24)),
        R.parallel_layer(2, 1, 136, 0.1, R.rot(136, 5000.0, R.ramped(2.0, 100, 4.0, 0.5)), 4, r_heads=2, r_dim=136, r_vdim=72, tau=30.0, mlp=R.dense(40)),
        R.window_layer(4, 2, 40, 136, 0.15, R.dense(32), size=33, keep_first=4),
        R.window_layer(2, 2, 40, 136, 0.2, R.moe(16, 3, 3), size=32, keep_first=4, kv_from=2),
    ], softcap=20.0, eps=1e-6)


def cfg_e():
    # odd sizes everywhere: a width, heads, taps, inner size, ff and vocabulary that are multiples of nothing
    return R.make_config(37, 31, [
        R.parallel_layer(3, 1, 5, 0.6, R.rot(2, 70.0, R.ramped(3.0, 30, 3.0, 0.7)), 6, r_heads=3, r_dim=3, r_vdim=5, tau=2.5, mlp=R.moe(7, 3, 2, shared=5), rank=3),
        R.window_layer(5, 5, 5, 7, 0.6, R.dense(11), size=3, keep_first=1),
        R.sink_layer(9, 3, 7, 3, 0.4, R.rot(6, 11.0, R.banded(2.5, 1.5, 2.0, 40)), R.moe(5, 7, 3)),
        R.window_layer(10, 5, 5, 7, 0.3, R.moe(3, 2, 1, shared=1), size=11, keep_first=7, kv_from=1),
    ], softcap=2.0, eps=1e-6)


def cfg_f():
    # sizes that coincide: one key head per head, key size = value size = taps = experts = window, every expert chosen, tau 1, cap 1, scale 1
    return R.make_config(64, 64, [
        R.window_layer(8, 8, 8, 8, 1.0, R.moe(8, 8, 8, shared=8), size=8, keep_first=8),
        R.parallel_layer(8, 8, 8, 1.0, R.rot(8, 8.0, R.ramped(1.0, 8, 8.0, 8.0)), 8, r_heads=8, r_dim=8, r_vdim=8, tau=1.0, mlp=R.dense(64), rank=8),
        R.sink_layer(8, 8, 8, 8, 1.0, R.rot(8, 8.0, R.banded(1.0, 1.0, 8.0, 8)), R.dense(8)),
    ], softcap=1.0, eps=1e-5)


CONFIGS = {"a": cfg_a, "b": cfg_b, "c": cfg_c, "d": cfg_d, "e": cfg_e, "f": cfg_f}


class Served:
    def __init__(self, backend, tmp_path, cfg, seed, dtype, max_tokens=512, n_ubatch=64, W=None):
        self.cfg, self.W = cfg, W if W is not None else R.random_weights(cfg, seed)
        R.save_model(cfg, self.W, str(tmp_path))
        self.s = TraceSession(str(tmp_path), "float32" if dtype == "f32" else "bfloat16", max_tokens=max_tokens, n_ubatch=n_ubatch, backend=backend)
        self.gate = F32_GATE if dtype == "f32" else BF16_GATE

    def ref(self, tokens):
        return R.forward(self.cfg, self.W, tokens)

    def feed(self, rid, tokens, end=False):
        return self.s.step([{"id": rid, "tokens": list(tokens), "want": list(range(len(tokens)))}], [rid] if end else [])

    def free(self):
        self.s.close()


# ------------------------------------------------------------------------------------------------ whole models through the engine
@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("which", sorted(CONFIGS))
def test_whole_prompt(backend, tmp_path, plog, which, dtype):
    cfg = CONFIGS[which]()
    if dtype == "bf16" and which == "d":  # (7 of 20 experts: the last ones chosen are often nearly tied, and bf16 turns a tenth of them — with all of them the rows show the arithmetic)
        cfg["layers"][0]["mlp"]["router"]["top"] = 20
    s = Served(backend, tmp_path, cfg, 11, dtype)
    t = toks(150, s.cfg["vocab"], 5)  # three micro-batches of 64 / 64 / 22 tokens; every position's logits
    e = row_err(s.feed("w", t, end=True), s.ref(t))
    plog(f"nidudra whole prompt cfg {which} {dtype}: max row error {e.max():.3e}, median {np.median(e):.3e}")
    assert within(e, s.gate, dtype), (int(np.argmax(e)), float(e.max()))
    s.free()


def wind(**kw):
    d = dict(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.4, mlp=None)
    d.update(kw)
    return R.window_layer(**d)


def sink(**kw):
    d = dict(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.4, r=R.rot(16, 500.0), mlp=None)
    d.update(kw)
    return R.sink_layer(**d)


def para(**kw):
    d = dict(heads=4, kv_heads=2, dim=12, scale=0.4, r=R.rot(12, 500.0), conv=3, r_heads=3, r_dim=8, r_vdim=12, tau=6.0, mlp=None)
    d.update(kw)
    return R.parallel_layer(**d)


ONE = {
    "norms_behind": dict(layers=[wind(), wind()]),
    "window": dict(layers=[wind(size=6)]),
    "kept_first": dict(layers=[wind(size=6, keep_first=3)]),
    "shared_cache": dict(layers=[wind(size=6, keep_first=3), wind(size=11, kv_from=0)]),
    "shared_cache_other_heads": dict(layers=[wind(), wind(heads=8, kv_from=0), wind(heads=2, kv_from=0)]),
    "seven_heads": dict(layers=[wind(heads=7, kv_heads=1)]),
    "rotation": dict(layers=[sink()], silent="sink"),
    "rotation_of_a_part": dict(layers=[sink(r=R.rot(6, 500.0))]),
    "no_rotation": dict(layers=[sink(r=R.rot(0, 500.0))]),
    "banded": dict(layers=[sink(r=R.rot(16, 500.0, R.banded(8.0, 1.0, 4.0, 64)))]),
    "sink_and_head_gate": dict(layers=[sink(heads=6, kv_heads=6)]),
    "keys_as_values": dict(layers=[para()], silent="right.o"),
    "ramped": dict(layers=[para(r=R.rot(8, 500.0, R.ramped(8.0, 200, 16.0, 1.0)))], silent="right.o"),
    "many_taps": dict(layers=[para(conv=16)], silent="right.o"),
    "one_tap": dict(layers=[para(conv=1)], silent="right.o"),
    "linear_attention": dict(layers=[para()], silent="left.o"),
    "linear_attention_one_head": dict(layers=[para(r_heads=1, r_dim=20, r_vdim=5, tau=1.0, rank=1)], silent="left.o"),
    "both_branches": dict(layers=[para()]),
    "dense": dict(layers=[wind(mlp=R.dense(24))]),
    "one_expert": dict(layers=[wind(mlp=R.moe(20, 5, 1))]),
    "experts": dict(layers=[wind(mlp=R.moe(20, 7, 3))]),
    "experts_and_shared": dict(layers=[wind(mlp=R.moe(20, 7, 3, shared=12))]),
    "one_expert_and_shared": dict(layers=[wind(mlp=R.moe(20, 5, 1, shared=12))]),
    "all_experts": dict(layers=[wind(mlp=R.moe(20, 4, 4, shared=12))]),
    "cap": dict(layers=[wind()], softcap=0.5),
    "no_cap": dict(layers=[wind()], softcap=None),
}


@pytest.mark.parametrize("case", sorted(ONE))
def test_one_mechanism_at_a_time(backend, tmp_path, case):
    """small models with one mixer and nothing else (or one more part behind a fixed mixer), so that a fault has one place to be; `silent`: a tensor that is zero, so that the other branch is alone"""
    c = ONE[case]
    cfg = R.make_config(48, 40, c["layers"], softcap=c.get("softcap", 9.0))
    W = R.random_weights(cfg, 21)
    if c.get("silent"):
        W["l0.mix." + c["silent"]] = W["l0.mix." + c["silent"]] * 0.0 - (30.0 if c["silent"] == "sink" else 0.0)
    s = Served(backend, tmp_path, cfg, 21, "f32", W=W)
    t = toks(40, 40, 3)
    e = row_err(s.feed("w", t, end=True), s.ref(t))
    assert e.max() <= F32_GATE, (int(np.argmax(e)), float(e.max()))
    e = row_err(np.concatenate([s.feed("x", [tok]) for tok in t]), s.ref(t))
    assert e.max() <= F32_GATE, (int(np.argmax(e)), float(e.max()))
    s.free()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("which", ["a", "d"])
def test_prefill_against_token_by_token(backend, tmp_path, which, dtype):
    s = Served(backend, tmp_path, CONFIGS[which](), 12, dtype)
    t = toks(45, s.cfg["vocab"], 6)
    # the first tokens of a sequence one at a time: position 0 reads no state, no convolution history and an empty cache
    rows = np.concatenate([s.feed("x", [tok]) for tok in t])
    assert within(row_err(rows, s.ref(t)), s.gate, dtype)
    whole = s.feed("y", t, end=True)
    assert within(row_err(whole, rows.astype(np.float64)), 2e-5 if dtype == "f32" else s.gate, dtype)
    s.free()


@pytest.mark.parametrize("which", sorted(CONFIGS))
def test_portions_of_every_size(backend, tmp_path, which):
    s = Served(backend, tmp_path, CONFIGS[which](), 13, "f32")
    t = toks(131, s.cfg["vocab"], 7)
    cuts = [2, 3, 2, 7, 1, 16, 5, 2, 64, 2, 9, 18]  # down to two tokens; cuts fall inside the reach of the convolutions (fewer tokens than taps), inside windows and inside blocks of cells
    assert sum(cuts) == len(t)
    at, rows = 0, []
    for n in cuts:
        rows.append(s.feed("x", t[at:at + n]))
        at += n
    e = row_err(np.concatenate(rows), s.ref(t))
    assert e.max() <= s.gate, (int(np.argmax(e)), float(e.max()))
    s.free()


@pytest.mark.parametrize("sizes", [(9, 37), (64, 256), (257, None)])
def test_long_decoding(backend, tmp_path, sizes):
    """3 prompt tokens, then single steps: the used part of the cache grows past 256 cells, windows pass over decoded tokens (their lengths below, at and above a block of cells, and at its
    border), every state is carried 327 times"""
    cfg = cfg_a()
    cfg["layers"][1]["mixer"]["mask"]["size"] = sizes[0]
    if sizes[1] is None:
        del cfg["layers"][3]["mixer"]["mask"]
    else:
        cfg["layers"][3]["mixer"]["mask"]["size"] = sizes[1]
    s = Served(backend, tmp_path, cfg, 14, "f32", max_tokens=512)
    t = toks(330, s.cfg["vocab"], 8)
    rows = [s.feed("x", t[:3])] + [s.feed("x", [tok]) for tok in t[3:]]
    e = row_err(np.concatenate(rows), s.ref(t))
    assert e.max() <= s.gate, (int(np.argmax(e)), float(e.max()))
    s.free()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_unequal_requests_in_mixed_batches_with_cells_and_slots_used_again(backend, tmp_path, dtype):
    cfg = cfg_a()
    reqs = {name: toks(n, cfg["vocab"], 20 + i) for i, (name, n) in enumerate([("p", 190), ("q", 33), ("r", 1), ("s", 240), ("t", 57), ("u", 175), ("v", 2)])}
    # 256 + 4 x 64 cells for 698 tokens in total: the cells of ended requests are handed out again, as are the four sequence slots with their states
    sv = Served(backend, tmp_path, cfg, 15, dtype, max_tokens=256, n_ubatch=64)
    fed = {k: 0 for k in reqs}
    got = {k: [] for k in reqs}
    plan = [  # (request, tokens) per step: portions beside single tokens, requests left out of steps, ends in between
        [("p", 40), ("q", 2)], [("p", 1), ("q", 30), ("r", 1)], [("p", 1), ("q", 1), ("s", 64), ("v", 2)], [("p", 148), ("s", 3)], [("s", 173)],
        [("t", 20), ("u", 2)], [("t", 1), ("u", 170)], [("u", 1), ("t", 36)], [("u", 2)],
    ]
    for step in plan:
        entries, ends = [], []
        for name, n in step:
            a = fed[name]
            entries.append({"id": name, "tokens": reqs[name][a:a + n], "want": list(range(n))})
            fed[name] = a + n
            if fed[name] == len(reqs[name]):
                ends.append(name)
        rows = sv.s.step(entries, ends)
        at = 0
        for name, n in step:
            got[name].append(rows[at:at + n])
            at += n
    for k in reqs:
        assert fed[k] == len(reqs[k])
        e = row_err(np.concatenate(got[k]), sv.ref(reqs[k]))
        assert within(e, sv.gate, dtype) or (dtype == "bf16" and len(e) < 20), (k, int(np.argmax(e)), float(e.max()))
    sv.free()


def test_batched_requests_give_what_each_gives_alone(backend, tmp_path):
    """the same three requests alone and side by side in one batch, then decoded side by side (one token of each: the short convolutions take their one-token form): the rows agree to
    rounding (a batch changes which mat-mul tiling runs, nothing else)"""
    cfg = cfg_d()
    reqs = [toks(n, cfg["vocab"], 70 + i) for i, n in enumerate((37, 5, 64))]
    more = [toks(6, cfg["vocab"], 80 + i) for i in range(3)]
    s = Served(backend, tmp_path, cfg, 19, "f32")
    alone = [np.concatenate([s.feed("a%d" % i, r)] + [s.feed("a%d" % i, [x]) for x in m]) for i, (r, m) in enumerate(zip(reqs, more))]
    for i in range(3):
        s.s.step([], ["a%d" % i])
    rows = s.s.step([{"id": "b%d" % i, "tokens": r, "want": list(range(len(r)))} for i, r in enumerate(reqs)], [])
    at, got = 0, []
    for r in reqs:
        got.append([rows[at:at + len(r)]])
        at += len(r)
    for k in range(6):
        order = [(i + k) % 3 for i in range(3)]
        rows = s.s.step([{"id": "b%d" % i, "tokens": [more[i][k]], "want": [0]} for i in order], [])
        for j, i in enumerate(order):
            got[i].append(rows[j:j + 1])
    for i in range(3):
        assert row_err(np.concatenate(got[i]), alone[i].astype(np.float64)).max() <= 2e-5
        assert row_err(np.concatenate(got[i]), s.ref(reqs[i] + more[i])).max() <= F32_GATE
    s.free()


def test_only_the_wanted_rows_come_back(backend, tmp_path):
    """a step that asks for some places gives those rows of the step that asks for all; none asked: no rows, and the state has moved on all the same (a last layer with and without feed-forward)"""
    for k, cfg in enumerate((cfg_a(), cfg_b())):
        s = Served(backend, tmp_path / str(k), cfg, 23, "f32")
        t = toks(40, cfg["vocab"], 9)
        ref = s.ref(t)
        rows = s.s.step([{"id": "x", "tokens": t[:20], "want": [3, 11, 19]}], [])
        assert rows.shape[0] == 3 and row_err(rows, ref[[3, 11, 19]]).max() <= F32_GATE
        assert s.s.step([{"id": "x", "tokens": t[20:29], "want": []}], []).shape[0] == 0
        assert row_err(s.s.step([{"id": "x", "tokens": t[29:], "want": [0, 10]}], ["x"]), ref[[29, 39]]).max() <= F32_GATE
        s.free()


def test_a_slot_used_again_starts_from_nothing(backend, tmp_path):
    """a request that takes over the slot (recurrence matrices, convolution history) and the cells of an ended one gives what it gives alone, also when it begins with one token"""
    s = Served(backend, tmp_path, cfg_a(), 16, "f32", max_tokens=64)
    a, b = toks(50, s.cfg["vocab"], 1), toks(60, s.cfg["vocab"], 2)
    s.feed("a", a, end=True)
    rows = np.concatenate([s.feed("b", b[:1]), s.feed("b", b[1:2]), s.feed("b", b[2:7]), s.feed("b", b[7:], end=True)])
    assert row_err(rows, s.ref(b)).max() <= F32_GATE
    s.free()


def test_greedy_generation_through_the_engine(backend, tmp_path, H):
    s = Served(backend, tmp_path, cfg_a(), 17, "f32")
    prompt = toks(9, s.cfg["vocab"], 9)
    s.s.step([{"id": "g", "tokens": prompt, "want": [len(prompt) - 1]}], [])
    seq = list(prompt)
    for _ in range(24):
        tok = H.llm_sample_greedy(s.s.ctx, -1)  # the engine's own sampler on the engine's own logits
        ref_row = s.ref(seq)[-1]
        top2 = np.sort(ref_row)[-2:]
        if top2[1] - top2[0] > 1e-3 * np.abs(ref_row).max():
            assert tok == int(np.argmax(ref_row))
        else:
            tok = int(np.argmax(ref_row))
        seq.append(tok)
        s.s.step([{"id": "g", "tokens": [tok], "want": [0]}], [])
    s.free()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("which", ["a", "c", "d", "e"])
def test_fused_steps_equal_the_unfused_nodes(backend, tmp_path, which, dtype):
    """the fused launches (per-head norms and rotation of queries and keys with both cache stores, bias and convolution with the state's update, the router, the weighted activation, the experts'
    sum with the shared one and the norm behind it, the two branches' blend likewise, the cap): bit for bit what the graph's own nodes give, for a prompt portion and for single tokens"""
    cfg = CONFIGS[which]()
    t = toks(90, cfg["vocab"], 41)
    rows, launches = {}, {}
    for fusion in (1, 0):
        backend.set_option("fusion", fusion)
        s = Served(backend, tmp_path / str(fusion), cfg, 18, dtype)
        before = backend.stat("kernel_launches")
        rows[fusion] = np.concatenate([s.feed("x", t[:70])] + [s.feed("x", [tok]) for tok in t[70:]])
        launches[fusion] = backend.stat("kernel_launches") - before
        s.free()
    backend.set_option("fusion", 1)
    assert np.array_equal(rows[0], rows[1])
    assert launches[1] < 0.7 * launches[0], launches


# ------------------------------------------------------------------------------------------------ the data must show a rule that is one off
def far_from(rows, ref_rows, times=20):
    return row_err(rows, ref_rows).max() > times * F32_GATE


@pytest.mark.parametrize("how", ["prompt", "decoded"])
@pytest.mark.parametrize("size,keep", [(1, 0), (2, 1), (8, 3), (31, 4), (64, 64), (63, 1)])
def test_window_edges_show(backend, tmp_path, how, size, keep):
    """a layer with its own cache and one over it, whose keys count about equally over what they see: the rows match the windows exactly and are far from those that are a token longer or
    shorter, or keep one first token more or less, in a prompt and token by token, also where an edge lies at a block of cells"""
    cfg = R.make_config(48, 40, [wind(scale=0.05, size=size, keep_first=keep), wind(scale=0.05, size=size + 5, keep_first=keep, kv_from=0)])
    s = Served(backend, tmp_path, cfg, 31, "f32")
    t = toks(150, 40, 4)
    rows = s.feed("w", t, end=True) if how == "prompt" else np.concatenate([s.feed("w", t[:5])] + [s.feed("w", [x]) for x in t[5:]])
    assert row_err(rows, s.ref(t)).max() <= F32_GATE
    for il in (0, 1):
        n = cfg["layers"][il]["mixer"]["mask"]["size"]
        for key, off in (("size", -1), ("size", 1), ("keep_first", -1), ("keep_first", 1)):
            c2 = copy.deepcopy(cfg)
            m2 = c2["layers"][il]["mixer"]["mask"]
            m2[key] += off
            if m2["size"] < 1 or m2["keep_first"] < 0:
                continue
            other = R.forward(c2, s.W, t)
            assert far_from(rows[n + keep:], other[n + keep:], 10), (il, key, off)
            assert row_err(rows[:max(n - 1, 1)], other[:max(n - 1, 1)]).max() <= F32_GATE  # (before the window is full nothing changes)
    s.free()


def pointing(W, p, width_entry=0):
    """token 39 alone has entry 0 of the embedding, and its key points where every query points (entry 1 of every token): one score stands far above the rest"""
    W["embed"][:, 0] = 0.0
    W["embed"][39, 0] = 8.0
    W[p + "k"][0, :] = 0.0
    W[p + "k"][0, 0] = 4.0
    W["embed"][:, 1] = 4.0
    W[p + "q"][0, :] = 0.0
    W[p + "q"][0, 1] = 4.0
    return {k: R.bf16_round(v) for k, v in W.items()}


@pytest.mark.parametrize("shared", [False, True])
def test_one_key_inside_and_outside_the_window(backend, tmp_path, shared):
    """a query that points at ONE key (a token that occurs once): with the key just inside the window it carries most of the weight, one token later it is gone — unless it is among the kept
    first tokens.  Every place of the key, across the borders of blocks of cells, f32 and bf16, prompt and decoded; in the layer that owns the cache, or in one over it"""
    layers = [wind(heads=1, kv_heads=1, dim=16, vdim=16, scale=1.5, size=70, keep_first=3)]
    if shared:
        layers = [wind(heads=1, kv_heads=1, dim=16, vdim=16, scale=0.1, size=500)] + [wind(heads=1, kv_heads=1, dim=16, vdim=16, scale=1.5, size=70, keep_first=3, kv_from=0)]
    il = len(layers) - 1
    cfg = R.make_config(48, 40, layers)
    W = R.random_weights(cfg, 43)
    if shared:
        W["l1.mix.q"][0, :] = 0.0
        W["l1.mix.q"][0, 1] = 4.0
        W["l0.norm1"] = W["l0.norm1"] * 0.05  # (the stream the second layer's query reads is about the embedding)
    W = pointing(W, "l0.mix.")
    rng = np.random.default_rng(8)
    for at in (0, 2, 3, 61, 64, 130):
        t = rng.integers(0, 39, 220).tolist()
        t[at] = 39
        ref = R.forward(cfg, W, t)
        edge = at + 69  # the last position whose window holds it
        if at >= 3:
            other = {}
            for n in (69, 71):
                c2 = copy.deepcopy(cfg)
                c2["layers"][il]["mixer"]["mask"]["size"] = n
                other[n] = R.forward(c2, W, t)
            assert row_err(ref[edge:edge + 1], other[69][edge:edge + 1])[0] > 0.3 and row_err(ref[edge + 1:edge + 2], other[71][edge + 1:edge + 2])[0] > 0.3
        else:
            c2 = copy.deepcopy(cfg)
            c2["layers"][il]["mixer"]["mask"]["keep_first"] = at
            assert row_err(ref[edge + 1:edge + 2], R.forward(c2, W, t)[edge + 1:edge + 2])[0] > 0.3  # (a kept token: seen for ever)
        for dtype in ("f32", "bf16"):
            s = Served(backend, tmp_path / ("%d%s" % (at, dtype)), cfg, 0, dtype, W=W)
            gate = F32_GATE if dtype == "f32" else BF16_GATE
            prompt = s.feed("w", t, end=True)
            single = np.concatenate([s.feed("x", t[:edge - 3])] + [s.feed("x", [x]) for x in t[edge - 3:edge + 6]])
            assert row_err(prompt, ref).max() <= gate and row_err(single, ref[:edge + 6]).max() <= gate, (at, dtype)
            s.free()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
@pytest.mark.parametrize("kind", ["sink", "left"])
def test_one_key_far_back_among_hundreds(backend, tmp_path, dtype, kind):
    """no window, 700 tokens, cells past 256 and 512: ONE early key carries the weight of the last queries — with another token there the rows are far off"""
    slow = R.rot(4, 1e9)  # (rotation that leaves the pointing entry — beyond the rotated part — alone)
    if kind == "sink":
        cfg = R.make_config(48, 40, [sink(heads=1, kv_heads=1, dim=16, vdim=16, scale=1.5, r=slow)])
        W, p = R.random_weights(cfg, 44), "l0.mix."
        W["l0.mix.sink"][:] = 1.0
    else:
        cfg = R.make_config(48, 40, [para(heads=1, kv_heads=1, dim=16, scale=1.5, r=slow, conv=2)])
        W, p = R.random_weights(cfg, 44), "l0.mix.left."
        W["l0.mix.right.o"] = W["l0.mix.right.o"] * 0.0
        for n in ("q", "k"):
            W[p + n + ".conv"][:] = [0.0, 1.0]
            W[p + n + ".b"][:] = 0.0
            W[p + n + ".norm"][:] = 1.0
    # entry 8 of the head (not rotated) points; the rest is small
    W["embed"][:, 0] = 0.0
    W["embed"][39, 0] = 8.0
    W["embed"][:, 1] = 4.0
    for n, e in (("k", 0), ("q", 1)):
        W[p + n] *= 0.2
        W[p + n][8, :] = 0.0
        W[p + n][8, e] = 4.0
    W = {k: R.bf16_round(v) for k, v in W.items()}
    rng = np.random.default_rng(5)
    t = rng.integers(0, 39, 700).tolist()
    t[3] = 39
    s = Served(backend, tmp_path, cfg, 0, dtype, W=W, max_tokens=768)
    rows = np.concatenate([s.feed("w", t[:650])] + [s.feed("w", [x]) for x in t[650:]])
    ref = R.forward(cfg, W, t)
    assert row_err(rows, ref).max() <= s.gate
    t2 = list(t)
    t2[3] = 0
    assert row_err(ref[600:], R.forward(cfg, W, t2)[600:]).min() > 4 * s.gate  # (every one of the last rows rests on that key)
    s.free()


def test_a_token_far_back_is_carried_by_the_state(backend, tmp_path):
    """slow decay: the first tokens of a 300-token sequence still move the last rows (the reference says so), and the engine — prompt in portions, then single tokens — agrees with the
    reference that saw the true first tokens"""
    cfg = R.make_config(48, 40, [para(r_dim=64, tau=40.0)])
    W = R.random_weights(cfg, 35)
    W["l0.mix.right.a2.b"] = W["l0.mix.right.a2.b"] * 0 + 3.0
    W["l0.mix.left.o"] = W["l0.mix.left.o"] * 0
    s = Served(backend, tmp_path, cfg, 0, "f32", W=W)
    t = toks(300, 40, 6)
    rows = np.concatenate([s.feed("w", t[:100]), s.feed("w", t[100:280])] + [s.feed("w", [x]) for x in t[280:]])
    assert row_err(rows, s.ref(t)).max() <= F32_GATE
    t2 = [(x + 1) % 40 for x in t[:20]] + t[20:]
    assert far_from(rows[290:], R.forward(cfg, W, t2)[290:], 10)
    s.free()


@pytest.mark.parametrize("how", ["prompt", "decoded"])
def test_constants_and_rules_show(backend, tmp_path, how):
    """the engine's rows are far from the reference computed with a neighbouring constant, weight or rule: scales, rotation bases, dims and both frequency schedules' constants, the factor on sine
    and cosine, tau, cap, eps, the sink, the order of norm and rotation, the values' place, the experts' weights on the output, the shared expert's gate, norms in front instead of behind"""
    cfg = R.make_config(48, 40, [
        sink(r=R.rot(12, 300.0, R.banded(6.0, 1.0, 4.0, 60)), mlp=R.moe(20, 6, 2, shared=12)),
        para(r=R.rot(8, 200.0, R.ramped(6.0, 80, 8.0, 1.0)), mlp=R.dense(16)),
        wind(size=12, keep_first=2), wind(size=20, kv_from=2),
    ], softcap=2.5)
    s = Served(backend, tmp_path, cfg, 37, "f32")
    W, t = s.W, toks(50, 40, 7)
    rows = s.feed("w", t, end=True) if how == "prompt" else np.concatenate([s.feed("w", t[:7])] + [s.feed("w", [x]) for x in t[7:]])
    assert row_err(rows, s.ref(t)).max() <= F32_GATE

    def changed(path, v):
        c2 = copy.deepcopy(cfg)
        o = c2
        keys = path.split("/")
        for k in keys[:-1]:
            o = o[int(k) if k.isdigit() else k]
        o[keys[-1]] = v
        return R.forward(c2, W, t)

    a, b = "layers/0/mixer/", "layers/1/mixer/left/"
    for path, v in ((a + "scale", 0.42), (a + "rot/base", 330.0), (a + "rot/dims", 10), (a + "rot/scaling/factor", 6.5), (a + "rot/scaling/low", 1.4), (a + "rot/scaling/high", 5.0),
                    (a + "rot/scaling/original", 70), (b + "scale", 0.43), (b + "rot/base", 230.0), (b + "rot/dims", 10), (b + "rot/scaling/factor", 6.5), (b + "rot/scaling/fast", 3.0),
                    (b + "rot/scaling/slow", 0.2), (b + "rot/scaling", None), (a + "rot/scaling", None), ("layers/1/mixer/right/tau", 6.5), ("logit_softcap", 2.6), ("norm/eps", 1e-2),
                    ("layers/0/mlp/router/top", 3), ("layers/2/mixer/scale", 0.43), ("layers/3/mixer/scale", 0.43)):
        assert far_from(rows, changed(path, v)), path
    for name, f in (("l0.mix.sink", lambda x: x + 0.1), ("l0.mix.g", lambda x: np.roll(x, 1, axis=0)), ("l0.norm1", lambda x: np.roll(x, 1)), ("l0.norm2", lambda x: np.roll(x, 1)),
                    ("l1.mix.left.q.b", lambda x: x * 0), ("l1.mix.left.k.b", lambda x: x * 0), ("l1.mix.left.q.conv", lambda x: x[:, ::-1]), ("l1.mix.left.k.conv", lambda x: x[:, ::-1]),
                    ("l1.mix.left.q.norm", lambda x: np.roll(x, 1)), ("l1.mix.left.k.norm", lambda x: np.roll(x, 1)), ("l1.mix.left.out", lambda x: np.roll(x, 1)),
                    ("l1.mix.right.out", lambda x: np.roll(x, 1)), ("l1.mix.right.norm", lambda x: np.roll(x, 1)), ("l1.mix.right.a2.b", lambda x: x + 0.2), ("l1.mix.right.g", lambda x: -x),
                    ("l2.mix.q.norm", lambda x: np.roll(x, 1)), ("l2.mix.k.norm", lambda x: np.roll(x, 1)), ("l3.mix.q.norm", lambda x: np.roll(x, 1)), ("l2.mix.g", lambda x: np.roll(x, 1, axis=0)),
                    ("l0.mlp.shared.sg", lambda x: -x), ("final.norm", lambda x: np.roll(x, 1))):
        W2 = dict(W)
        W2[name] = f(W[name])
        assert far_from(rows, R.forward(cfg, W2, t)), name

    def with_rule(name, f):
        saved = getattr(R, name)
        setattr(R, name, f(saved))
        try:
            return s.ref(t)
        finally:
            setattr(R, name, saved)

    def values_behind(h, mx, W_, p, eps):  # the keys as the cache holds them for values
        q = R.heads_of(R.history_taps(h @ W_[p + "q"].T + W_[p + "q.b"], W_[p + "q.conv"]), mx["heads"], mx["dim"])
        k = R.heads_of(R.history_taps(h @ W_[p + "k"].T + W_[p + "k.b"], W_[p + "k.conv"]), mx["kv_heads"], mx["dim"])
        k = R.rotate_halves(R.over_rms(k, eps) * W_[p + "k.norm"], mx["rot"])
        q = R.rotate_halves(R.over_rms(q, eps) * W_[p + "q.norm"], mx["rot"])
        return R.attend(q, k, k, mx["scale"]).reshape(len(h), -1) @ W_[p + "o"].T

    def weigh_output(h, ml, W_, p):
        chosen, wts = R.route(h @ W_[p + "router"].T, ml["router"]["top"])
        out = np.zeros_like(h)
        for i in range(len(h)):
            for e, w in zip(chosen[i], wts[i]):
                out[i] += w * R.gated_ffn(h[i][None], W_, "%se%d." % (p, e))[0]
        return out + R.gated_ffn(h, W_, p + "shared.") * R.squash(h @ W_[p + "shared.sg"].T)

    def normalised(saved):
        def f(z, top):
            chosen, w = saved(z, top)
            return chosen, w / w.sum(axis=-1, keepdims=True)
        return f

    assert far_from(rows, with_rule("keys_as_values", lambda _: values_behind)), "values in front of norm and rotation"
    assert far_from(rows, with_rule("experts_ffn", lambda _: weigh_output)), "weights on the experts' inputs"
    assert far_from(rows, with_rule("route", normalised)), "weights as they are"
    assert far_from(rows, with_rule("attend", lambda f: lambda q, k, v, scale, mask=None, sink=None: f(q, k, v, scale, mask))), "the sink"
    assert far_from(rows, with_rule("rotation", lambda f: lambda r: (f(r)[0], 1.0))), "the factor on sine and cosine"
    assert far_from(rows, with_rule("fading_memory", lambda f: lambda q, k, v, keep: f(q, k, v, np.concatenate([keep[:1], keep[:-1]])))), "a token's own decay"
    s.free()


# ------------------------------------------------------------------------------------------------ the new operations alone, through the C-ABI
def run(backend, build):
    g = T.G(backend)
    outs = build(g)
    res = g.compute(outs if isinstance(outs, list) else [outs])
    g.free()
    return res


@pytest.mark.parametrize("heads,dk,dv,tau", [(4, 16, 8, 16.0), (3, 136, 5, 1.0), (6, 7, 33, 4.0), (1, 64, 200, 2.5), (2, 256, 12, 9.0)])
def test_linear_attention_over_mixed_batches(backend, H, heads, dk, dv, tau):
    """three sequences in two mixed batches against the plain token-by-token loop, the state going through the engine's own state tensor (stale values in the slot of a sequence that starts);
    batches below and above the size from which the decays are computed ahead"""
    rng = np.random.default_rng(dk * 7 + dv)
    S, lens = 4, [(6, 4), (1, 33), (0, 5)]
    data = []
    for n in (a + b for a, b in lens):
        data.append({k: v.astype(np.float32) for k, v in dict(q=rng.standard_normal((n, heads * dk)), k=rng.standard_normal((n, heads * dk)), v=rng.standard_normal((n, heads * dv)),
                                                              g=rng.standard_normal((n, heads * dk)) * 2.0).items()})
    p0 = rng.uniform(-1.0, 2.0, heads * dk).astype(np.float32)
    size = H.ggml_seq_state_size(5, heads, dk, dv)
    state = np.full((S, size), 3.0, np.float32)
    got = [np.zeros((a + b, heads, dv)) for a, b in lens]
    before = [0, 0, 0]
    for step in (0, 1):
        now = [l[step] for l in lens]
        order = [(s, before[s] + i) for i in range(max(now)) for s in range(3) if i < now[s]] if step else [(s, before[s] + i) for s in range(3) for i in range(now[s])]
        at = {sp: i for i, sp in enumerate(order)}
        tok, info = [], []
        for s in range(3):
            if now[s]:
                info.append([len(tok), now[s], s, 1 if before[s] == 0 else 0])
                tok += [at[(s, before[s] + i)] for i in range(now[s])]
        g = T.G(backend)
        t = {a: g.new(L.F32, [data[0][a].shape[1], len(order)], np.stack([data[s][a][p] for s, p in order])) for a in "qkvg"}
        ts = g.new(L.F32, [size, S], state)
        o = H.ggml_seq_linear(g.ctx, t["q"], t["k"], t["v"], t["g"], g.new(L.F32, [heads * dk], p0), ts, g.new(L.I32, [len(order)], np.asarray(tok, np.int32)),
                              g.new(L.I32, [4, len(info)], np.asarray(info, np.int32)), heads, tau)
        y = g.compute([o])[0].reshape(len(order), heads, dv)
        state = g.read(ts).reshape(S, size)
        g.free()
        for i, (s, p) in enumerate(order):
            got[s][p] = y[i]
        before = [b + n for b, n in zip(before, now)]
    for s in range(3):
        d = {a: b.astype(np.float64) for a, b in data[s].items()}
        n = len(d["q"])
        keep = R.fading(d["g"] + p0, tau).reshape(n, heads, dk)
        ref = R.fading_memory(d["q"].reshape(n, heads, dk) * dk ** -0.5, d["k"].reshape(n, heads, dk), d["v"].reshape(n, heads, dv), keep)
        assert np.abs(got[s] - ref).max() <= 2e-5 * max(1.0, np.abs(ref).max()), s


@pytest.mark.parametrize("n,top", [(12, 5), (8, 1), (256, 9), (256, 256), (70, 70), (1, 1), (300, 4)])
def test_router_with_raw_sigmoid_weights(backend, H, n, top):
    """the scores choose and weigh: the fused launch (up to 256 experts) and the graph's own nodes against the reference"""
    rng = np.random.default_rng(n + top)
    z = (rng.standard_normal((19, n)) * 2.0).astype(np.float32)
    z[3, :] = 0.25  # ties: the lower index first
    ref_sel, ref_w = R.route(z.astype(np.float64), top)
    got = {}
    for fusion in (1, 0):
        backend.set_option("fusion", fusion)

        def build(g):
            probs = H.ggml_unary(g.ctx, g.new(L.F32, [n, 19], z), 7)  # GGML_UNARY_OP_SIGMOID
            order = H.ggml_argsort(g.ctx, probs, 1)
            sel = H.ggml_view_2d(g.ctx, order, top, 19, n * 4, 0)
            return [H.ggml_get_rows(g.ctx, H.ggml_reshape_3d(g.ctx, probs, 1, n, 19), sel), H.ggml_cont(g.ctx, sel)]

        before = backend.stat("fused_nodes")
        w, sel = run(backend, build)
        assert (backend.stat("fused_nodes") > before) == (fusion == 1 and n <= 256)
        sel, w = sel.reshape(19, top), w.reshape(19, top)
        clear = np.ones(19, bool) if n == 1 else np.abs(np.diff(np.sort(R.squash(z.astype(np.float64)), axis=1), axis=1)).min(axis=1) > 1e-6
        rows = clear | (np.arange(19) == 3)
        assert np.array_equal(sel[rows], ref_sel[rows])
        assert np.abs(w[rows] - ref_w[rows]).max() <= 1e-6
        got[fusion] = w
    backend.set_option("fusion", 1)
    assert np.array_equal(got[0], got[1])


@pytest.mark.parametrize("n_q,n_kv,heads,kv_heads,dk,dv,kv_type,size,keep", [
    (1, 700, 6, 2, 96, 96, L.BF16, None, 0), (1, 700, 6, 2, 96, 80, L.F32, None, 0), (1, 1300, 1, 1, 16, 16, L.BF16, 300, 5), (3, 900, 8, 8, 64, 64, L.BF16, 70, 4), (1, 65, 4, 1, 40, 24, L.F32, 9, 2),
    (4, 2000, 4, 4, 128, 128, L.BF16, None, 0), (40, 300, 3, 1, 96, 96, L.BF16, None, 0), (33, 130, 4, 2, 80, 48, L.BF16, 33, 4), (65, 257, 2, 2, 112, 112, L.F32, 64, 1), (1, 512, 2, 1, 300, 200, L.F32, None, 0)])
@pytest.mark.parametrize("sinks", [False, True])
def test_attention_with_sinks_over_windows_with_kept_tokens(backend, H, n_q, n_kv, heads, kv_heads, dk, dv, kv_type, size, keep, sinks):
    """every kernel of the 32-bit attention (rows, tiles, matrix cores) at this class's shapes — few queries over a long cache, head sizes between the tilings' — with a sink per head and windows
    that keep the first tokens"""
    rng = np.random.default_rng(n_q * 1000 + n_kv)
    q, k, v = ((rng.standard_normal(s) * f).astype(np.float32) for s, f in (((n_q, heads, dk), 2.0), ((n_kv, kv_heads, dk), 1.0), ((n_kv, kv_heads, dv), 1.0)))
    sk = rng.normal(0, 2.0, heads).astype(np.float32)
    if kv_type == L.BF16:
        q, k, v = (R.bf16_round(x).astype(np.float32) for x in (q, k, v))  # (prompt portions over a bf16 cache round the queries too)
    mask = np.full((64 * ((n_q + 63) // 64), n_kv), -np.inf, np.float32)
    ok = R.seen(n_kv, {"size": size, "keep_first": keep} if size else None)[n_kv - n_q:]
    mask[:n_q][ok] = 0.0
    scale = 1.0 / np.sqrt(dk)
    bits = lambda x: (np.ascontiguousarray(x, np.float32).view(np.uint32) >> 16).astype(np.uint16)

    def build(g):
        esz = 2 if kv_type == L.BF16 else 4
        tk, tv = (g.new(kv_type, [d * kv_heads, n_kv], bits(x) if kv_type == L.BF16 else x) for d, x in ((dk, k), (dv, v)))
        kk = H.ggml_view_3d(g.ctx, tk, dk, n_kv, kv_heads, dk * kv_heads * esz, dk * esz, 0)
        vv = H.ggml_view_3d(g.ctx, tv, dv, n_kv, kv_heads, dv * kv_heads * esz, dv * esz, 0)
        r = H.ggml_flash_attn_ext(g.ctx, H.ggml_permute(g.ctx, g.new(L.F32, [dk, heads, n_q], q), 0, 2, 1, 3), kk, vv, g.new(L.F32, [n_kv, mask.shape[0]], mask), scale, 0.0, 0.0)
        H.ggml_flash_attn_ext_set_prec(r, 10)
        if sinks:
            H.ggml_flash_attn_ext_add_sinks(r, g.new(L.F32, [heads], sk))
        return r

    got = run(backend, build)[0].reshape(n_q, heads, dv)
    f64 = lambda x: x.astype(np.float64)
    ref = np.zeros((n_q, heads, dv))
    for h in range(heads):
        z = np.where(ok, scale * (f64(q[:, h]) @ f64(k[:, h // (heads // kv_heads)]).T), -np.inf)
        top = np.maximum(z.max(axis=1, keepdims=True), sk[h] if sinks else -np.inf)
        w = np.exp(z - top)
        den = w.sum(axis=1, keepdims=True) + (np.exp(sk[h] - top) if sinks else 0.0)
        ref[:, h] = (w / den) @ f64(v[:, h // (heads // kv_heads)])
    assert np.abs(got - ref).max() <= (2e-5 if kv_type == L.F32 else 2e-3) * max(1.0, np.abs(ref).max())


@pytest.mark.parametrize("ff,width,used,experts,T_", [(1024, 96, 1, 1, 1), (2752, 70, 1, 1, 1), (1000, 50, 1, 1, 1), (520, 33, 2, 5, 1), (704, 64, 3, 4, 3), (256, 40, 1, 3, 2), (264, 12, 4, 4, 1), (1376, 24, 2, 3, 9)])
def test_gated_activation_inside_the_down_projection(backend, H, ff, width, used, experts, T_):
    """a decode step's feed-forward: SwiGLU (of rows that carry a factor each) -> bf16 product, as one launch and as the graph's own nodes: the same bits, and the reference's numbers"""
    rng = np.random.default_rng(ff + width)
    gu = rng.standard_normal((T_, used, 2 * ff)).astype(np.float32)
    w = rng.uniform(0.1, 1.0, (T_, used, 1)).astype(np.float32)
    W = R.bf16_round(rng.standard_normal((experts, width, ff)) / np.sqrt(ff))
    ids = np.stack([rng.permutation(experts)[:used] for _ in range(T_)]).astype(np.int32)
    one = experts == 1
    bits = (W.astype(np.float32).view(np.uint32) >> 16).astype(np.uint16)
    got, fused = {}, {}
    for fusion in (1, 0):
        backend.set_option("fusion", fusion)

        def build(g):
            tw = g.new(L.BF16, [ff, width] if one else [ff, width, experts], bits)
            x = H.ggml_scale(g.ctx, g.new(L.F32, [2 * ff, used, T_], gu), 1.0)
            if one:
                return H.ggml_mul_mat(g.ctx, tw, H.ggml_swiglu(g.ctx, H.ggml_reshape_2d(g.ctx, x, 2 * ff, 1)))
            sel = g.new(L.I32, [used, T_], ids)
            y = H.ggml_mul(g.ctx, x, g.new(L.F32, [1, used, T_], w))
            act = H.ggml_swiglu(g.ctx, H.ggml_reshape_2d(g.ctx, y, 2 * ff, used * T_))
            return H.ggml_mul_mat_id(g.ctx, tw, H.ggml_reshape_3d(g.ctx, act, ff, used, T_), sel)

        before = backend.stat("fused_nodes")
        got[fusion] = run(backend, build)[0].reshape(T_, used, width)
        fused[fusion] = backend.stat("fused_nodes") - before
    backend.set_option("fusion", 1)
    assert np.array_equal(got[0], got[1])
    x = gu.astype(np.float64) * (1.0 if one else w.astype(np.float64))
    act = R.bf16_round(R.silu(x[..., :ff]) * x[..., ff:])
    ref = np.stack([[W[0 if one else ids[t, u]] @ act[t, u] for u in range(used)] for t in range(T_)])
    assert np.abs(got[1] - ref).max() <= 4e-3 * np.abs(ref).max()
    assert fused[0] == 0 and (fused[1] > 0) == (not one or width >= 64)


# ------------------------------------------------------------------------------------------------ the program, and random configurations
def test_trace_run_command_line(tmp_path):
    cfg = cfg_b()
    W = R.random_weights(cfg, 51)
    R.save_model(cfg, W, str(tmp_path / "model"))
    t = toks(30, cfg["vocab"], 52)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t[20:21], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": t[21:], "want": [8]}, {"id": "b", "tokens": t[:3], "want": [2]}], "end": ["a", "b"]}]
    exe = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "trace_run")
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, exe, "--model", str(tmp_path / "model"), "--dtype", "float32", "--out", str(out), "--max-tokens", "128"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    ref = R.forward(cfg, W, t)
    r0 = np.fromfile(out / "0.f32", "<f4").reshape(-1, cfg["vocab"])
    r2 = np.fromfile(out / "2.f32", "<f4").reshape(-1, cfg["vocab"])
    assert not (out / "1.f32").exists()
    assert row_err(r0, ref[[0, 19]]).max() <= F32_GATE and row_err(r2, ref[[29, 2]]).max() <= F32_GATE


def random_config(rng, keep_all):
    layers = []
    n = int(rng.integers(1, 6))

    def rotation(dim):
        dims = 2 * int(rng.integers(1, dim // 2 + 1))
        base, k = float(rng.choice([50.0, 1000.0, 20000.0])), rng.random()
        if k < 0.4:
            return R.rot(dims, base, R.banded(float(rng.uniform(1.5, 8.0)), 1.0, float(rng.uniform(2.0, 6.0)), int(rng.integers(20, 300))))
        return R.rot(dims, base, R.ramped(float(rng.uniform(1.5, 8.0)), int(rng.integers(40, 300)), float(rng.uniform(3.0, 20.0)), float(rng.uniform(0.5, 2.0))) if k < 0.8 else None)

    for il in range(n):
        kind = rng.random()
        if kind < 0.25:
            mlp = None
        elif kind < 0.6:
            mlp = R.dense(int(rng.choice([8, 12, 20, 50])))
        else:
            e = int(rng.integers(1, 9))
            mlp = R.moe(int(rng.choice([6, 16, 24])), e, e if keep_all else int(rng.integers(1, e + 1)), shared=int(rng.choice([0, 4, 18])))
        g, k = int(rng.integers(1, 4)), rng.random()
        own = [i for i, l in enumerate(layers) if l["type"] == "attention" and l["mixer"].get("kv_from") is None]
        scale = float(rng.uniform(0.1, 0.5))
        if k < 0.4:
            size = None if rng.random() < 0.25 else int(rng.integers(1, 80))
            keep = int(rng.integers(0, 6))
            if own and rng.random() < 0.5:
                j = int(rng.choice(own))
                o = layers[j]["mixer"]
                layers.append(R.window_layer(o["kv_heads"] * int(rng.integers(1, 5)), o["kv_heads"], o["dim"], o["vdim"], scale, mlp, size=size, keep_first=keep, kv_from=j))
            else:
                layers.append(R.window_layer(g * int(rng.integers(1, 5)), g, int(rng.choice([8, 12, 32])), int(rng.choice([8, 20, 36])), scale, mlp, size=size, keep_first=keep))
        elif k < 0.65:
            d = int(rng.choice([8, 12, 32]))
            layers.append(R.sink_layer(g * int(rng.integers(1, 5)), g, d, int(rng.choice([8, 20, 36])), scale, rotation(d), mlp))
        else:
            d = int(rng.choice([6, 16, 24]))
            layers.append(R.parallel_layer(g * int(rng.integers(1, 4)), g, d, scale, rotation(d), int(rng.integers(1, 7)), int(rng.integers(1, 5)), int(rng.choice([6, 16, 24])), int(rng.choice([4, 12, 40])),
                                           float(rng.uniform(1.0, 20.0)), mlp, rank=int(rng.integers(1, 9))))
    return R.make_config(int(rng.choice([32, 44, 64])), int(rng.integers(30, 90)), layers, softcap=None if rng.random() < 0.2 else float(rng.uniform(1.0, 20.0)), eps=float(rng.choice([1e-6, 1e-5])))


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(backend, tmp_path, seed):
    """random layer orders, sizes, windows, rotations, shared caches and experts: a prompt portion, then portions of 1 .. 40 tokens beside a second request (bf16 runs use every expert, so that no
    near-tie of a router decides a row; the choice itself is what the f32 runs test)"""
    rng = np.random.default_rng(1000 + seed)
    dtype = "f32" if seed % 3 else "bf16"
    cfg = random_config(rng, dtype == "bf16")
    s = Served(backend, tmp_path, cfg, 100 + seed, dtype, max_tokens=320)
    a, b = toks(140, cfg["vocab"], seed), toks(60, cfg["vocab"], seed + 50)
    got_a, got_b = [s.feed("a", a[:31])], []
    at_a, at_b = 31, 0
    while at_a < len(a):
        n = int(rng.integers(1, 41))
        entries = [{"id": "a", "tokens": a[at_a:at_a + n], "want": list(range(len(a[at_a:at_a + n])))}]
        nb = int(rng.integers(0, 9)) if at_b < len(b) else 0
        if nb:
            entries.append({"id": "b", "tokens": b[at_b:at_b + nb], "want": list(range(len(b[at_b:at_b + nb])))})
        rows = s.s.step(entries, [])
        na = len(entries[0]["tokens"])
        got_a.append(rows[:na])
        if nb:
            got_b.append(rows[na:])
        at_a += na
        at_b += len(entries[1]["tokens"]) if nb else 0
    ea = row_err(np.concatenate(got_a), s.ref(a))
    assert within(ea, s.gate, dtype), (json.dumps(cfg), int(np.argmax(ea)), float(ea.max()))
    if got_b:
        eb = row_err(np.concatenate(got_b), s.ref(b)[:at_b])
        assert within(eb, s.gate, dtype), (json.dumps(cfg), int(np.argmax(eb)), float(eb.max()))
    s.free()
