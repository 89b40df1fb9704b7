"""GPU tests of the Pisulorn model class: the engine (llama_lite over the MI355X backend) against the plain numpy reference of
tests/pisulorn_ref.py, on small models with their own sizes and random weights.

f32 serving is the sharp instrument: with 32-bit arithmetic end to end a key wrongly seen or hidden, a wrong slope, a stream mixed the wrong way
round, a convolution tap from the wrong token or a lost state moves a logit row by 1e-3 of its spread and more, ten times the gate (1e-4).  bf16
serving is gated at its rounding level.  Where random data could hide a fault (a key far back among hundreds, a window's edge, the first tokens of
a long sequence, a constant) a test shows that the data discriminate: the same rows are far from the reference computed with the neighbouring rule."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import harness as T
import llama_box_amd as L
import pisulorn_ref as R
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
    # both mixers and both feed-forwards; three streams; the first two of four layers run three times; two windows and two query factors; 3 query heads per key head (slopes over a
    # head count that is no power of two); key size != value size; a layer without feed-forward
    return R.make_config(64, 97, [
        R.delta_layer(heads=4, kv_heads=2, dim=12, vdim=20, conv=3, mlp=R.dense(48)),
        R.attention_layer(heads=6, kv_heads=2, dim=16, vdim=24, scale=0.3, size=9, coef=0.4, every=16, mlp=R.moe(20, 6, 2, 0.7)),
        R.attention_layer(heads=4, kv_heads=4, dim=24, vdim=8, scale=0.2, size=37, coef=0.25, every=50, mlp=None),
        R.delta_layer(heads=3, kv_heads=3, dim=16, vdim=12, conv=5, mlp=R.moe(24, 5, 3, 1.5)),
    ], streams=3, residual_mult=0.4, loop=(0, 2, 3), eps=3e-5)


def cfg_b():
    # ONE stream; rows that are no multiple of 8 (width 52); one head; no window, no query factor; one tap (no history); one expert per token; key rows that are no multiple of 4; the last
    # layer has no feed-forward
    return R.make_config(52, 50, [
        R.attention_layer(heads=1, kv_heads=1, dim=12, vdim=20, scale=0.3, mlp=R.moe(12, 4, 1, 1.0)),
        R.delta_layer(heads=1, kv_heads=1, dim=14, vdim=10, conv=1, mlp=R.dense(12)),
        R.attention_layer(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.5, size=5, mlp=None),
    ], streams=1, residual_mult=0.7, eps=1e-6)


def cfg_c():
    # no attention anywhere (no cells are read, no masks); four streams; the repeated range ends the model
    return R.make_config(48, 257, [
        R.delta_layer(heads=4, kv_heads=4, dim=8, vdim=16, conv=4, mlp=R.dense(24)),
        R.delta_layer(heads=6, kv_heads=2, dim=20, vdim=4, conv=2, mlp=R.moe(16, 8, 8, 2.0)),
    ], streams=4, residual_mult=1.0, loop=(1, 2, 2), eps=1e-5)


def cfg_d():
    # heads wider than 128 (the row kernels serve prompts too), value rows beyond 128, key rows of the recurrence beyond 128; many experts; two streams; the whole model repeats
    return R.make_config(96, 120, [
        R.attention_layer(heads=3, kv_heads=1, dim=136, vdim=40, scale=0.09, size=64, coef=0.5, every=7, mlp=R.moe(32, 20, 7, 0.4)),
        R.delta_layer(heads=2, kv_heads=1, dim=136, vdim=72, conv=4, mlp=R.dense(40)),
        R.attention_layer(heads=4, kv_heads=2, dim=40, vdim=136, scale=0.15, size=33, coef=0.1, every=1, mlp=R.dense(32)),
    ], streams=2, residual_mult=0.3, loop=(0, 3, 2), eps=1e-6)


def cfg_e():
    # odd sizes everywhere: a width, heads, taps, ff, vocabulary and stream count that are multiples of nothing
    return R.make_config(37, 31, [
        R.delta_layer(heads=3, kv_heads=1, dim=3, vdim=5, conv=6, mlp=R.moe(7, 3, 2, 0.9)),
        R.attention_layer(heads=5, kv_heads=5, dim=5, vdim=7, scale=0.6, size=3, coef=1.3, every=3, mlp=R.dense(11)),
        R.attention_layer(heads=9, kv_heads=3, dim=7, vdim=3, scale=0.4, size=1, coef=0.7, every=11, mlp=R.moe(5, 7, 3, 3.0)),
    ], streams=5, residual_mult=0.6, loop=(1, 3, 2), eps=1e-6)


def cfg_f():
    # sizes that coincide: one key head per head, key size = value size = experts = eight streams = taps, every expert chosen, factor 1
    return R.make_config(64, 64, [
        R.attention_layer(heads=8, kv_heads=8, dim=8, vdim=8, scale=1.0, size=8, coef=1.0, every=8, mlp=R.moe(8, 8, 8, 1.0)),
        R.delta_layer(heads=8, kv_heads=8, dim=8, vdim=8, conv=8, mlp=R.dense(64)),
    ], streams=8, residual_mult=1.0, eps=1e-5)


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
    s = Served(backend, tmp_path, CONFIGS[which](), 11, dtype)
    t = toks(150, s.cfg["vocab"], 5)  # three micro-batches of 64 / 64 / 22 tokens; every position's logits
    e = row_err(s.feed("w", t, end=True), s.ref(t))
    plog(f"pisulorn whole prompt cfg {which} {dtype}: max row error {e.max():.3e}, median {np.median(e):.3e}")
    assert within(e, s.gate, dtype), (int(np.argmax(e)), float(e.max()))
    s.free()


def attn(**kw):
    d = dict(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.4, mlp=None)
    d.update(kw)
    return R.attention_layer(**d)


def delt(**kw):
    d = dict(heads=4, kv_heads=2, dim=12, vdim=8, conv=3, mlp=None)
    d.update(kw)
    return R.delta_layer(**d)


@pytest.mark.parametrize("case", ["attention", "window", "query_factor", "every_head_its_own_key", "seven_heads", "delta", "delta_one_tap", "delta_many_taps", "dense", "experts", "one_expert",
                                  "all_experts", "one_stream", "two_streams", "six_streams", "repeated", "factor"])
def test_one_mechanism_at_a_time(backend, tmp_path, case):
    """small models with one mixer and nothing else (or one more part behind a fixed mixer), so that a fault has one place to be"""
    streams, mult, loop = 2, 0.5, None
    layers = [attn()]
    if case == "window":
        layers = [attn(size=6)]
    elif case == "query_factor":
        layers = [attn(coef=0.9, every=4)]
    elif case == "every_head_its_own_key":
        layers = [attn(kv_heads=4, size=11)]
    elif case == "seven_heads":
        layers = [attn(heads=7, kv_heads=1)]
    elif case == "delta":
        layers = [delt()]
    elif case == "delta_one_tap":
        layers = [delt(conv=1, kv_heads=1)]
    elif case == "delta_many_taps":
        layers = [delt(conv=16, heads=5, kv_heads=5)]
    elif case == "dense":
        layers = [delt(mlp=R.dense(24))]
    elif case == "experts":
        layers = [delt(mlp=R.moe(20, 7, 3, 0.6))]
    elif case == "one_expert":
        layers = [attn(mlp=R.moe(20, 5, 1, 2.0))]
    elif case == "all_experts":
        layers = [attn(mlp=R.moe(20, 4, 4, 0.3))]
    elif case == "one_stream":
        streams, layers = 1, [attn(), delt(mlp=R.dense(16))]
    elif case == "two_streams":
        layers = [attn(), delt(mlp=R.dense(16))]
    elif case == "six_streams":
        streams, layers = 6, [attn(), delt(mlp=R.dense(16))]
    elif case == "repeated":
        loop, layers = (1, 3, 3), [delt(), attn(size=7), delt(conv=2)]
    elif case == "factor":
        mult, layers = 1.7, [attn(), delt(mlp=R.dense(16))]
    s = Served(backend, tmp_path, R.make_config(48, 40, layers, streams=streams, residual_mult=mult, loop=loop), 21, "f32")
    t = toks(40, 40, 3)
    e = row_err(s.feed("w", t, end=True), s.ref(t))
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
    for il, n in ((1, sizes[0]), (2, sizes[1])):
        cfg["layers"][il]["mixer"]["mask"] = {"size": n} if n else None
    if sizes[1] is None:
        del cfg["layers"][2]["mixer"]["mask"]
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
    """the same three requests alone and side by side in one batch: the rows agree to rounding (a batch changes which mat-mul tiling runs, nothing else)"""
    cfg = cfg_d()
    reqs = [toks(n, cfg["vocab"], 70 + i) for i, n in enumerate((37, 5, 64))]
    s = Served(backend, tmp_path, cfg, 19, "f32")
    alone = [s.feed("a%d" % i, r, end=True) for i, r in enumerate(reqs)]
    rows = s.s.step([{"id": "b%d" % i, "tokens": r, "want": list(range(len(r)))} for i, r in enumerate(reqs)], ["b0", "b1", "b2"])
    at = 0
    for i, r in enumerate(reqs):
        assert row_err(rows[at:at + len(r)], alone[i].astype(np.float64)).max() <= 2e-5
        at += len(r)
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
    """a request that takes over the slot (recurrence matrices, convolution history) and the cells of an ended one gives what it gives alone"""
    s = Served(backend, tmp_path, cfg_a(), 16, "f32", max_tokens=64)
    a, b = toks(50, s.cfg["vocab"], 1), toks(60, s.cfg["vocab"], 2)
    s.feed("a", a, end=True)
    rows = np.concatenate([s.feed("b", b[:1]), s.feed("b", b[1:7]), s.feed("b", b[7:], end=True)])
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
@pytest.mark.parametrize("which", ["a", "d", "e"])
def test_fused_steps_equal_the_unfused_nodes(backend, tmp_path, which, dtype):
    """the fused launches (the per-head norms of queries and keys with the query factor and both cache stores, the router, the weighted sum over the experts, the per-head norm with gate,
    sibling mat-vecs): bit for bit what the graph's own nodes give, for a prompt portion and for single tokens"""
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
    assert launches[1] < 0.75 * launches[0], launches


# ------------------------------------------------------------------------------------------------ the data must show a rule that is one off
def far_from(rows, ref_rows, times=20):
    return row_err(rows, ref_rows).max() > times * F32_GATE


@pytest.mark.parametrize("how", ["prompt", "decoded"])
@pytest.mark.parametrize("size", [1, 2, 8, 31, 64])
def test_window_edges_show(backend, tmp_path, how, size):
    """one attention layer whose keys count about equally over the window (one head: the flattest slope, small scores): the rows match the window exactly and are far from one that is a token
    longer or shorter, in a prompt and token by token, also where the edge lies at a block of cells"""
    cfg = R.make_config(48, 40, [attn(heads=1, kv_heads=1, scale=0.05, size=size)], streams=2, residual_mult=2.0)
    s = Served(backend, tmp_path, cfg, 31, "f32")
    t = toks(140, 40, 4)
    rows = s.feed("w", t, end=True) if how == "prompt" else np.concatenate([s.feed("w", t[:5])] + [s.feed("w", [x]) for x in t[5:]])
    assert row_err(rows, s.ref(t)).max() <= F32_GATE
    for off in (-1, 1):
        if size + off >= 1:
            c2 = copy.deepcopy(cfg)
            c2["layers"][0]["mixer"]["mask"]["size"] = size + off
            other = R.forward(c2, s.W, t)
            assert far_from(rows[size:], other[size:]), off
            assert row_err(rows[:max(size - 1, 1)], other[:max(size - 1, 1)]).max() <= F32_GATE  # (before the window is full nothing changes)
    s.free()


def test_one_key_inside_and_outside_the_window(backend, tmp_path):
    """a query that points at ONE key (a token that occurs once): with the key just inside the window it carries most of the weight, one token later it is gone.  Every place of the key, across
    the borders of blocks of cells, f32 and bf16, prompt and decoded"""
    cfg = R.make_config(48, 40, [attn(heads=1, kv_heads=1, dim=16, vdim=16, scale=1.5, size=70)], streams=2, residual_mult=1.0)
    W = R.random_weights(cfg, 43)
    # token 39 alone has entry 0, and its key points where every query points
    W["embed"][:, 0] = 0.0
    W["embed"][39, 0] = 8.0
    W["l0.mix.k"][0, :] = 0.0
    W["l0.mix.k"][0, 0] = 4.0
    W["embed"][:, 1] = 4.0
    W["l0.mix.q"][0, :] = 0.0
    W["l0.mix.q"][0, 1] = 4.0
    W = {k: R.bf16_round(v) for k, v in W.items()}
    rng = np.random.default_rng(8)
    for at in (0, 1, 61, 64, 130):
        t = rng.integers(0, 39, 220).tolist()
        t[at] = 39
        ref = R.forward(cfg, W, t)
        c2 = copy.deepcopy(cfg)
        c2["layers"][0]["mixer"]["mask"]["size"] = 69
        c3 = copy.deepcopy(cfg)
        c3["layers"][0]["mixer"]["mask"]["size"] = 71
        edge = at + 69  # the last position that sees it
        assert row_err(ref[edge:edge + 1], R.forward(c2, W, t)[edge:edge + 1])[0] > 0.3 and row_err(ref[edge + 1:edge + 2], R.forward(c3, W, t)[edge + 1:edge + 2])[0] > 0.3
        for dtype in ("f32", "bf16"):
            s = Served(backend, tmp_path / ("%d%s" % (at, dtype)), cfg, 0, dtype, W=W)
            gate = F32_GATE if dtype == "f32" else BF16_GATE
            prompt = s.feed("w", t, end=True)
            single = np.concatenate([s.feed("x", t[:edge - 3])] + [s.feed("x", [x]) for x in t[edge - 3:edge + 6]])
            assert row_err(prompt, ref).max() <= gate and row_err(single, ref[:edge + 6]).max() <= gate, (at, dtype)
            s.free()


@pytest.mark.parametrize("dtype", ["f32", "bf16"])
def test_one_key_far_back_among_hundreds(backend, tmp_path, dtype):
    """no window, 700 tokens, cells past 256 and 512: ONE early key carries the weight of the last queries against its distance penalty — with another token there the rows are far off"""
    cfg = R.make_config(48, 40, [attn(heads=1, kv_heads=1, dim=16, vdim=16, scale=1.5)], streams=2, residual_mult=1.0)
    W = R.random_weights(cfg, 44)
    W["embed"][:, 0] = 0.0
    W["embed"][39, 0] = 8.0
    W["l0.mix.k"][0, :] = 0.0
    W["l0.mix.k"][0, 0] = 4.0
    W["embed"][:, 1] = 4.0
    W["l0.mix.q"][0, :] = 0.0
    W["l0.mix.q"][0, 1] = 4.0
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
    cfg = R.make_config(48, 40, [delt(dim=64)], streams=2)
    W = R.random_weights(cfg, 35)
    W["l0.mix.A_log"] = W["l0.mix.A_log"] * 0 - 6.0
    W["l0.mix.b"] = W["l0.mix.b"] * 0       # beta = 1/2 and 64 key entries: 300 writes leave a tenth of the first token's trace
    s = Served(backend, tmp_path, cfg, 0, "f32", W=W)
    t = toks(300, 40, 6)
    rows = np.concatenate([s.feed("w", t[:100]), s.feed("w", t[100:280])] + [s.feed("w", [x]) for x in t[280:]])
    assert row_err(rows, s.ref(t)).max() <= F32_GATE
    t2 = [(x + 1) % 40 for x in t[:20]] + t[20:]
    assert far_from(rows[290:], R.forward(cfg, W, t2)[290:], 10)
    s.free()


@pytest.mark.parametrize("how", ["prompt", "decoded"])
def test_constants_show(backend, tmp_path, how):
    """the engine's rows are far from the reference computed with a neighbouring constant or weight: slopes, scale, query factor and its first step, streams mixed the other way round, the
    sublayer's share, the factor, the order of the passes, decays, the convolution's tap order, per-head norm weights, the experts' limit, the correction's part"""
    cfg = R.make_config(48, 40, [attn(heads=6, kv_heads=2, size=20, coef=0.8, every=10, mlp=R.moe(20, 6, 2, 0.5)), delt(mlp=R.dense(16))], streams=3, residual_mult=0.8, loop=(0, 2, 2))
    s = Served(backend, tmp_path, cfg, 37, "f32")
    W, t = s.W, toks(50, 40, 7)
    rows = s.feed("w", t, end=True) if how == "prompt" else np.concatenate([s.feed("w", t[:7])] + [s.feed("w", [x]) for x in t[7:]])
    assert row_err(rows, s.ref(t)).max() <= F32_GATE

    def changed(**kw):
        c2 = copy.deepcopy(cfg)
        for path, v in kw.items():
            keys = path.split("__")
            o = c2
            for k in keys[:-1]:
                o = o[int(k) if k.isdigit() else k]
            o[keys[-1]] = v
        return R.forward(c2, W, t)

    assert far_from(rows, changed(layers__0__mixer__scale=0.42)) and far_from(rows, changed(layers__0__mixer__q_temp={"coef": 0.85, "every": 10}))
    e = row_err(rows, changed(layers__0__mixer__q_temp={"coef": 0.8, "every": 11}))
    assert e[9] > 20 * F32_GATE and e[:9].max() <= F32_GATE  # the factor first moves at position every - 1
    assert far_from(rows, changed(residual_mult=0.82)) and far_from(rows, changed(loop={"start": 0, "stop": 2, "times": 1})) and far_from(rows, changed(loop={"start": 0, "stop": 1, "times": 2}))
    assert far_from(rows, changed(layers__0__mlp__expert__limit=0.6)) and far_from(rows, changed(layers__0__mlp__router__top=3)) and far_from(rows, changed(norm={"eps": 3e-2}))
    saved = R.head_slope
    try:
        for f in (lambda h, H: saved(h, 8), lambda h, H: 2.0 ** (-8.0 * h / H), lambda h, H: saved(h // 2, H // 2)):
            R.head_slope = f
            assert far_from(rows, s.ref(t)), "slope"
    finally:
        R.head_slope = saved
    saved = R.route
    try:
        def corrected_weights(z, c, top):
            chosen, _ = saved(z, c, top)
            w = np.take_along_axis(R.logistic(z) + c, chosen, axis=-1)
            return chosen, w / w.sum(axis=-1, keepdims=True)
        R.route = corrected_weights
        assert far_from(rows, s.ref(t)), "the correction in the weights"
        R.route = lambda z, c, top: saved(z, c * 0.0, top)
        assert far_from(rows, s.ref(t)), "no correction"
    finally:
        R.route = saved
    saved = R.limited_glu
    try:
        R.limited_glu = lambda g, u, limit: np.clip(g, -limit, limit) * R.logistic(1.702 * np.clip(g, -limit, limit)) * (np.clip(u, -limit, limit) + 1.0)
        assert far_from(rows, s.ref(t)), "the gate is limited from above only"
    finally:
        R.limited_glu = saved
    for name, f in (("l0.hc1.mix", lambda a: a.T), ("l1.hc2.mix", lambda a: a.T), ("l0.hc1.in", lambda a: np.roll(a, 1)), ("l0.hc2.in", lambda a: np.roll(a, 1)), ("l0.hc1.out", lambda a: np.roll(a, 1)),
                    ("l1.hc2.out", lambda a: np.roll(a, 1)), ("l0.mix.q.norm", lambda a: np.roll(a, 1)), ("l0.mix.k.norm", lambda a: np.roll(a, 1)), ("l1.mix.A_log", lambda a: a + 0.3),
                    ("l1.mix.dt_bias", lambda a: a + 0.3), ("l1.mix.v.conv", lambda a: a[:, ::-1]), ("l1.mix.q.conv", lambda a: a[:, ::-1]), ("l1.mix.norm", lambda a: np.roll(a, 1)),
                    ("l0.norm2", lambda a: np.roll(a, 1)), ("final.norm", lambda a: np.roll(a, 1)), ("l0.mlp.correction", lambda a: np.roll(a, 1))):
        W2 = dict(W)
        W2[name] = f(W[name])
        assert far_from(rows, R.forward(cfg, W2, t)), name
    s.free()


# ------------------------------------------------------------------------------------------------ the new operations alone, through the C-ABI
def run(backend, build):
    g = T.G(backend)
    outs = build(g)
    res = g.compute(outs if isinstance(outs, list) else [outs])
    g.free()
    return res


@pytest.mark.parametrize("E,N,rows", [(64, 2, 5), (64, 1, 3), (37, 3, 7), (2048, 4, 1), (4096, 4, 300), (8192, 2, 2), (516, 8, 9), (130, 5, 1), (16384, 3, 2), (40004, 2, 1), (1, 6, 2), (48, 7, 4)])
def test_stream_step(backend, H, E, N, rows):
    """what lies between two sublayers: the streams' update and the normed weighting in front of the next, against the reference's two functions — with all rows, with chosen rows, at the start (no
    streams yet) and at the end (the plain sum, no streams kept); vector and entry-by-entry forms, rows that take one and several groups per thread"""
    rng = np.random.default_rng(E + N)
    y, X = rng.standard_normal((rows, E)).astype(np.float32), rng.standard_normal((N, rows, E)).astype(np.float32)
    mix, out, a = rng.standard_normal((N, N)).astype(np.float32), rng.standard_normal(N).astype(np.float32), rng.standard_normal(N).astype(np.float32)
    w = rng.uniform(0.5, 1.5, E).astype(np.float32)
    ids = rng.integers(0, rows, max(1, rows // 2)).astype(np.int32)
    mult, eps = 0.6, 1e-3
    f64 = lambda v: v.astype(np.float64)
    newX = R.streams_out(f64(X), f64(y), f64(mix), f64(out), mult)
    for case in ("all", "chosen", "start", "end"):
        def build(g):
            ty, tx = g.new(L.F32, [E, rows], y), g.new(L.F32, [E, rows, N], X)
            tm, to, ti, tw = g.new(L.F32, [N, N], mix), g.new(L.F32, [N], out), g.new(L.F32, [N], a), g.new(L.F32, [E], w)
            tid = g.new(L.I32, [len(ids)], ids) if case == "chosen" else None
            st = H.ggml_stream_step(g.ctx, ty, None if case == "start" else tx, tm, to, None if case == "end" else ti, tw, tid, N, 0 if case == "end" else 1, mult, eps)
            outs = [H.ggml_cont(g.ctx, H.ggml_stream_step_rows(g.ctx, st))]
            if case != "end":
                outs.append(H.ggml_cont(g.ctx, H.ggml_stream_step_streams(g.ctx, st)))
            return outs

        res = run(backend, build)
        ref = np.repeat(f64(y)[None], N, axis=0) if case == "start" else newX
        if case == "chosen":
            ref = ref[:, ids]
        n = ref.shape[1]
        u = R.unit_rms(R.streams_in(ref, f64(a) if case != "end" else np.ones(N)), eps) * f64(w)
        assert np.abs(res[0].reshape(n, E) - u).max() <= 2e-5 * max(1.0, np.abs(u).max()), case
        if case != "end":
            assert np.abs(res[1].reshape(N, n, E) - ref).max() <= 1e-5 * max(1.0, np.abs(ref).max()), case


@pytest.mark.parametrize("kv_type,n_q,n_kv,heads,kv_heads,dk,dv,size", [
    (L.F32, 1, 200, 6, 2, 16, 24, 9), (L.F32, 5, 70, 3, 1, 40, 8, None), (L.F32, 40, 130, 5, 5, 64, 72, 33), (L.F32, 65, 300, 2, 1, 100, 128, 64), (L.F32, 2, 90, 7, 7, 300, 20, 50),
    (L.BF16, 1, 513, 12, 4, 64, 64, 100), (L.BF16, 33, 200, 6, 2, 64, 32, 17), (L.BF16, 128, 256, 3, 3, 128, 128, 128), (L.BF16, 20, 90, 4, 2, 48, 36, 30), (L.BF16, 64, 192, 8, 1, 160, 136, 65),
    (L.BF16, 3, 400, 2, 2, 24, 400, None)])
def test_attention_with_linear_distance(backend, H, kv_type, n_q, n_kv, heads, kv_heads, dk, dv, size):
    """every kernel of the 32-bit attention (rows, tiles, matrix cores, matrix cores over wide rows) with the linear distance penalty of every head, windows and head counts that are no power of two"""
    rng = np.random.default_rng(n_q * 1000 + n_kv)
    q = (rng.standard_normal((n_q, heads, dk)) * 2.0).astype(np.float32)
    k = rng.standard_normal((n_kv, kv_heads, dk)).astype(np.float32)
    v = rng.standard_normal((n_kv, kv_heads, dv)).astype(np.float32)
    slopes = np.asarray([R.head_slope(h, heads) for h in range(heads)], np.float32)
    q_pos = np.arange(n_kv - n_q, n_kv)
    dist = q_pos[:, None] - np.arange(n_kv)[None, :]
    ok = (dist >= 0) & ((dist < size) if size else True)
    mask = np.full((64 * ((n_q + 63) // 64), n_kv), -np.inf, np.float32)
    mask[:n_q][ok] = dist[ok]
    scale = 1.0 / np.sqrt(dk)
    if kv_type == L.BF16:
        q, k, v = (R.bf16_round(x).astype(np.float32) for x in (q, k, v))  # (prompt portions over a bf16 cache round the queries too)
    bits = lambda x: (np.ascontiguousarray(x, np.float32).view(np.uint32) >> 16).astype(np.uint16)

    def build(g):
        tq = g.new(L.F32, [dk, heads, n_q], q)
        tk = g.new(kv_type, [dk * kv_heads, n_kv], bits(k) if kv_type == L.BF16 else k)
        tv = g.new(kv_type, [dv * kv_heads, n_kv], bits(v) if kv_type == L.BF16 else v)
        esz = 2 if kv_type == L.BF16 else 4
        kk = H.ggml_view_3d(g.ctx, tk, dk, n_kv, kv_heads, dk * kv_heads * esz, dk * esz, 0)
        vv = H.ggml_view_3d(g.ctx, tv, dv, n_kv, kv_heads, dv * kv_heads * esz, dv * esz, 0)
        r = H.ggml_flash_attn_ext(g.ctx, H.ggml_permute(g.ctx, tq, 0, 2, 1, 3), kk, vv, g.new(L.F32, [n_kv, mask.shape[0]], mask), scale, 0.0, 0.0)
        H.ggml_flash_attn_ext_set_prec(r, 10)
        H.ggml_flash_attn_ext_add_linear_distance(r, g.new(L.F32, [heads], slopes))
        return r

    got = run(backend, build)[0].reshape(n_q, heads, dv)
    ref = np.zeros((n_q, heads, dv))
    for h in range(heads):
        g_ = h // (heads // kv_heads)
        s = (q[:, h].astype(np.float64) @ k[:, g_].astype(np.float64).T) * scale - R.head_slope(h, heads) * dist
        s = np.where(ok, s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        ref[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, g_].astype(np.float64)
    assert np.abs(got - ref).max() <= (2e-5 if kv_type == L.F32 else 2e-3) * max(1.0, np.abs(ref).max())


@pytest.mark.parametrize("n,top,with_correction", [(12, 5, 1), (6, 2, 1), (8, 1, 0), (256, 9, 1), (256, 256, 0), (70, 70, 1), (3, 3, 1), (300, 4, 1)])
def test_router_with_sigmoid_scores_and_correction(backend, H, n, top, with_correction):
    """choice by corrected scores, weights from the scores themselves divided by their sum: the fused launch (up to 256 experts) and the graph's own nodes against the reference"""
    rng = np.random.default_rng(n + top)
    z = (rng.standard_normal((19, n)) * 2.0).astype(np.float32)
    z[3, :] = 0.25  # ties (without a correction): the lower index first
    corr = (rng.standard_normal(n) * 0.3).astype(np.float32) * with_correction
    ref_sel, ref_w = R.route(z.astype(np.float64), corr.astype(np.float64), top)
    got = {}
    for fusion in (1, 0):
        backend.set_option("fusion", fusion)

        def build(g):
            probs = H.ggml_unary(g.ctx, g.new(L.F32, [n, 19], z), 7)  # GGML_UNARY_OP_SIGMOID
            order = H.ggml_argsort(g.ctx, H.ggml_add(g.ctx, probs, g.new(L.F32, [n], corr)) if with_correction else probs, 1)
            sel = H.ggml_view_2d(g.ctx, order, top, 19, n * 4, 0)
            w = H.ggml_reshape_2d(g.ctx, H.ggml_get_rows(g.ctx, H.ggml_reshape_3d(g.ctx, probs, 1, n, 19), sel), top, 19)
            w = H.ggml_div(g.ctx, w, H.ggml_scale_bias(g.ctx, H.ggml_sum_rows(g.ctx, w), 1.0, 1e-20))
            return [w, H.ggml_cont(g.ctx, sel)]

        before = backend.stat("fused_nodes")
        w, sel = run(backend, build)
        assert (backend.stat("fused_nodes") > before) == (fusion == 1 and n <= 256)
        sel, w = sel.reshape(19, top), w.reshape(19, top)
        clear = np.abs(np.diff(np.sort((R.logistic(z.astype(np.float64)) + corr), axis=1), axis=1)).min(axis=1) > 1e-6 if with_correction else np.arange(19) != 3
        rows = clear | (np.arange(19) == 3)
        assert np.array_equal(sel[rows], ref_sel[rows])
        assert np.abs(w[rows] - ref_w[rows]).max() <= 1e-6
        got[fusion] = w
    backend.set_option("fusion", 1)
    assert np.array_equal(got[0], got[1])


@pytest.mark.parametrize("ff,rows", [(96, 5), (7, 3), (2052, 33)])
def test_limited_gated_activation(backend, H, ff, rows):
    rng = np.random.default_rng(ff)
    x = (rng.standard_normal((rows, 2 * ff)) * 3.0).astype(np.float32)
    ref = R.limited_glu(x[:, :ff].astype(np.float64), x[:, ff:].astype(np.float64), 1.3)
    halves = run(backend, lambda g: H.ggml_swiglu_oai(g.ctx, g.new(L.F32, [2 * ff, rows], x), None, 1.702, 1.3))[0].reshape(rows, ff)
    split = run(backend, lambda g: H.ggml_swiglu_oai(g.ctx, g.new(L.F32, [ff, rows], x[:, :ff]), g.new(L.F32, [ff, rows], x[:, ff:]), 1.702, 1.3))[0].reshape(rows, ff)
    assert np.abs(halves - ref).max() <= 1e-5 and np.array_equal(halves, split)


@pytest.mark.parametrize("shape", [(5, 7), (1, 130), (260, 3), (2, 3, 4, 9)])
def test_sum_rows(backend, H, shape):
    x = np.random.default_rng(len(shape)).standard_normal(shape).astype(np.float32)
    got = run(backend, lambda g: H.ggml_sum_rows(g.ctx, g.new(L.F32, list(shape[::-1]), x)))[0]
    assert np.abs(got.reshape(shape[:-1]) - x.astype(np.float64).sum(axis=-1)).max() <= 1e-5


@pytest.mark.parametrize("heads,kv_heads,dk,dv", [(4, 2, 16, 8), (3, 1, 136, 5), (6, 2, 7, 33), (1, 1, 64, 200)])
def test_delta_recurrence_over_mixed_batches(backend, H, heads, kv_heads, dk, dv):
    """three sequences in two mixed batches against the plain token-by-token loop, the state going through the engine's own state tensor (stale values in the slot of a sequence that starts)"""
    rng = np.random.default_rng(dk * 7 + dv)
    S, lens = 4, [(6, 4), (1, 33), (0, 5)]
    data = []
    for n in (a + b for a, b in lens):
        data.append({k: v.astype(np.float32) for k, v in dict(q=rng.standard_normal((n, kv_heads * dk)), k=rng.standard_normal((n, kv_heads * dk)), v=rng.standard_normal((n, heads * dv)),
                                                              g=rng.standard_normal((n, 2 * heads)) * 2.0).items()})
    p0 = np.concatenate([rng.uniform(-2.0, 0.5, heads), rng.uniform(-1.0, 1.0, heads)]).astype(np.float32)
    size = H.ggml_seq_state_size(1, heads, dk, dv)
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
        o = H.ggml_seq_gated_delta(g.ctx, t["q"], t["k"], t["v"], t["g"], g.new(L.F32, [2 * heads], p0), ts, g.new(L.I32, [len(order)], np.asarray(tok, np.int32)),
                                   g.new(L.I32, [4, len(info)], np.asarray(info, np.int32)), heads, kv_heads)
        y = g.compute([o])[0].reshape(len(order), heads, dv)
        state = g.read(ts).reshape(S, size)
        g.free()
        for i, (s, p) in enumerate(order):
            got[s][p] = y[i]
        before = [b + n for b, n in zip(before, now)]
    for s in range(3):
        d = {a: b.astype(np.float64) for a, b in data[s].items()}
        n = len(d["q"])
        q, k = R.unit_length(d["q"].reshape(n, kv_heads, dk)) * dk ** -0.5, R.unit_length(d["k"].reshape(n, kv_heads, dk))
        decay = np.exp(-np.exp(p0[:heads].astype(np.float64)) * R.log1p_exp(d["g"][:, heads:] + p0[heads:]))
        ref = R.delta_recurrence(q, k, d["v"].reshape(n, heads, dv), R.logistic(d["g"][:, :heads]), decay)
        assert np.abs(got[s] - ref).max() <= 2e-5 * max(1.0, np.abs(ref).max()), s


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
    for _ in range(n):
        kind = rng.random()
        if kind < 0.25:
            mlp = None
        elif kind < 0.6:
            mlp = R.dense(int(rng.choice([8, 12, 20, 50])))
        else:
            e = int(rng.integers(1, 9))
            mlp = R.moe(int(rng.choice([6, 16, 24])), e, e if keep_all else int(rng.integers(1, e + 1)), float(rng.uniform(0.3, 3.0)))
        g = int(rng.integers(1, 4))
        if rng.random() < 0.5:
            size = None if rng.random() < 0.25 else int(rng.integers(1, 80))
            temp = {} if rng.random() < 0.25 else dict(coef=float(rng.uniform(0.05, 1.0)), every=int(rng.integers(1, 40)))
            layers.append(R.attention_layer(g * int(rng.integers(1, 5)), g, int(rng.choice([8, 12, 32])), int(rng.choice([8, 20, 36])), float(rng.uniform(0.1, 0.5)), mlp, size=size, **temp))
        else:
            layers.append(R.delta_layer(g * int(rng.integers(1, 4)), g, int(rng.choice([6, 16, 24])), int(rng.choice([4, 12, 40])), int(rng.integers(1, 7)), mlp))
    start = int(rng.integers(0, n))
    loop = (start, int(rng.integers(start + 1, n + 1)), int(rng.integers(1, 4))) if rng.random() < 0.6 else None
    return R.make_config(int(rng.choice([32, 44, 64])), int(rng.integers(30, 90)), layers, streams=int(rng.integers(1, 6)), residual_mult=float(rng.uniform(0.2, 1.2)), loop=loop,
                         eps=float(rng.choice([1e-6, 1e-5])))


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(backend, tmp_path, seed):
    """random layer orders, sizes, windows, factors, stream counts, repeated ranges and experts: a prompt portion, then portions of 1 .. 40 tokens beside a second request (bf16 runs use every
    expert, so that no near-tie of a router decides a row; the choice itself is what the f32 runs test)"""
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
