"""Host side of the Pisulorn model class, without a GPU: the loader (q, k, v of the delta rule as one projection, the experts' gate and up rows in one tensor, slopes computed per head),
what it refuses, the plain reference's own pieces, the query factors the scheduler uploads, and the graph the engine builds for a mixed batch — one op between two sublayers, which weights
it carries, in which order the nodes that the backend runs as one launch follow one another."""
import ctypes as C
import json

import numpy as np
import pytest

import llama_box_amd as L
import pisulorn_ref as R


def small_cfg():
    return R.make_config(40, 53, [
        R.delta_layer(heads=4, kv_heads=2, dim=8, vdim=12, conv=3, mlp=R.dense(16)),
        R.attention_layer(heads=6, kv_heads=2, dim=8, vdim=12, scale=0.3, size=5, coef=0.3, every=4, mlp=R.moe(16, 6, 2, 0.8)),
        R.attention_layer(heads=2, kv_heads=1, dim=12, vdim=8, scale=0.2, size=7, coef=0.5, every=9, mlp=None),
    ], streams=3, residual_mult=0.4, loop=(0, 2, 2), eps=1e-5)


def _get(H, m, name):
    t = H.llm_model_tensor(m, name.encode())
    assert t, name
    raw = np.empty(H.ggml_nbytes(t), np.uint8)
    H.ggml_backend_tensor_get(t, raw.ctypes.data_as(C.c_void_p), 0, raw.nbytes)
    tt = t.contents
    a = (raw.view(np.uint16).astype(np.uint32) << 16).view(np.float32) if tt.type == L.BF16 else raw.view(np.float32)
    return a.reshape([tt.ne[3], tt.ne[2], tt.ne[1], tt.ne[0]])[0]


def test_loader_reads_a_checkpoint_folder(H, tmp_path):
    cfg = small_cfg()
    W = R.random_weights(cfg, 3)
    R.save_model(cfg, W, str(tmp_path))
    for wtype in (L.BF16, L.F32):
        m = H.llm_model_load_dir(str(tmp_path).encode(), H.ggml_backend_cpu_buffer_type(), wtype)
        assert m
        hp = H.llm_model_hparams(m).contents
        assert (hp.arch, hp.n_layer, hp.n_embd, hp.n_vocab) == (b"pisulorn", 3, 40, 53)
        # streams: the mixture as it is stored, [from][to]; f32 in both modes
        assert np.array_equal(_get(H, m, "blk.0.attn_streams_mix.weight")[0], W["l0.hc1.mix"]) and np.array_equal(_get(H, m, "blk.1.ffn_streams_mix.weight")[0], W["l1.hc2.mix"])
        assert np.array_equal(_get(H, m, "blk.0.ffn_streams_in.weight").reshape(-1), W["l0.hc2.in"]) and np.array_equal(_get(H, m, "blk.2.attn_streams_out.weight").reshape(-1), W["l2.hc1.out"])
        assert not H.llm_model_tensor(m, b"blk.2.ffn_streams_mix.weight") and not H.llm_model_tensor(m, b"blk.2.ffn_norm.weight")  # (no feed-forward)
        # the delta rule: q, k, v of unequal heights follow one another in ONE projection; so do their taps; beta's rows, then the decay's
        assert np.array_equal(_get(H, m, "blk.0.attn_qkv.weight")[0], np.concatenate([W["l0.mix.q"], W["l0.mix.k"], W["l0.mix.v"]]))
        assert np.array_equal(_get(H, m, "blk.0.ssm_conv1d.weight")[0], np.concatenate([W["l0.mix.q.conv"], W["l0.mix.k.conv"], W["l0.mix.v.conv"]]))
        assert np.array_equal(_get(H, m, "blk.0.attn_gates.weight")[0], np.concatenate([W["l0.mix.b"], W["l0.mix.a"]]))
        assert np.array_equal(_get(H, m, "blk.0.attn_gates.param").reshape(-1), np.concatenate([W["l0.mix.A_log"], W["l0.mix.dt_bias"]]))
        # attention: per-head norm rows, slopes 2^(-8 (h + 1) / heads) also for a head count that is no power of two
        assert np.array_equal(_get(H, m, "blk.1.attn_k_norm.weight").reshape(-1), W["l1.mix.k.norm"])
        assert np.allclose(_get(H, m, "blk.1.attn_slopes.weight").reshape(-1), [2.0 ** (-8.0 * h / 6) for h in range(1, 7)], rtol=1e-7)
        # experts: per expert its gate rows, then its up rows; the correction and the router in f32
        gu = _get(H, m, "blk.1.ffn_gate_up_exps.weight")
        assert gu.shape == (6, 32, 40) and np.array_equal(gu[4], np.concatenate([W["l1.mlp.e4.gate"], W["l1.mlp.e4.up"]]))
        assert np.array_equal(_get(H, m, "blk.1.ffn_choice.bias").reshape(-1), W["l1.mlp.correction"])
        assert H.llm_model_tensor(m, b"blk.1.ffn_gate_inp.weight").contents.type == L.F32
        assert np.array_equal(_get(H, m, "output.weight")[0], W["head"])
        H.llm_model_free(m)


@pytest.mark.parametrize("breakage", ["shape", "missing", "heads", "mixer", "kind", "streams", "many_streams", "every", "window", "top", "limit", "loop", "taps", "correction", "mix"])
def test_loader_refuses_what_it_cannot_serve(H, tmp_path, breakage):
    cfg = small_cfg()
    W = R.random_weights(cfg, 4)
    if breakage == "shape":
        W["l0.mix.k.conv"] = W["l0.mix.k.conv"][:, :-1]
    elif breakage == "missing":
        del W["l1.mix.q.norm"]
    elif breakage == "heads":
        cfg["layers"][1]["mixer"]["kv_heads"] = 4
    elif breakage == "mixer":
        cfg["layers"][1]["type"] = "something_else"
    elif breakage == "kind":
        cfg["layers"][0]["mlp"]["kind"] = "gated"
    elif breakage == "streams":
        cfg["streams"] = 2
    elif breakage == "many_streams":
        cfg["streams"] = 9
    elif breakage == "every":
        cfg["layers"][1]["mixer"]["q_temp"]["every"] = 0
    elif breakage == "window":
        cfg["layers"][1]["mixer"]["mask"]["size"] = 0
    elif breakage == "top":
        cfg["layers"][1]["mlp"]["router"]["top"] = 7
    elif breakage == "limit":
        del cfg["layers"][1]["mlp"]["expert"]["limit"]
    elif breakage == "loop":
        cfg["loop"]["stop"] = 4
    elif breakage == "taps":
        cfg["layers"][0]["mixer"]["conv"] = 17
    elif breakage == "correction":
        W["l1.mlp.correction"] = W["l1.mlp.correction"][:-1]
    elif breakage == "mix":
        W["l1.hc2.mix"] = W["l1.hc2.mix"][:, :-1]
    R.save_model(cfg, W, str(tmp_path))
    assert not H.llm_model_load_dir(str(tmp_path).encode(), H.ggml_backend_cpu_buffer_type(), L.F32)


def test_parts_that_are_absent_are_not_needed(H, tmp_path):
    """no loop, no window, no query factor, null instead of an object, one stream: the keys may be missing or null"""
    cfg = R.make_config(24, 19, [R.attention_layer(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.3, mlp=None), R.delta_layer(heads=1, kv_heads=1, dim=4, vdim=4, conv=1, mlp=R.dense(8))], streams=1)
    cfg["loop"] = None
    cfg["layers"][0]["mixer"].update(mask=None, q_temp=None)
    R.save_model(cfg, R.random_weights(cfg, 5), str(tmp_path))
    m = H.llm_model_load_dir(str(tmp_path).encode(), H.ggml_backend_cpu_buffer_type(), L.F32)
    assert m
    H.llm_model_free(m)


def test_reference_pieces():
    # streams: [from, to], the sublayer's share per stream
    X = np.array([[[1.0]], [[10.0]]])
    assert np.allclose(R.streams_in(X, np.array([0.5, 2.0])), [[20.5]])
    new = R.streams_out(X, np.array([[3.0]]), np.array([[1.0, 2.0], [0.0, 0.1]]), np.array([1.0, -1.0]), 0.5)
    assert np.allclose(new[:, 0, 0], [1.0 + 1.5, 2.0 + 1.0 - 1.5])
    # the query factor moves where (p + 1) reaches a multiple of `every`
    f = R.query_temperature(np.arange(9), {"coef": 0.5, "every": 4})
    assert np.allclose(f, [1.0] * 3 + [1.0 + 0.5 * np.log(2.0)] * 4 + [1.0 + 0.5 * np.log(3.0)] * 2)
    assert np.allclose([R.head_slope(h, 3) for h in range(3)], [2.0 ** (-8 / 3), 2.0 ** (-16 / 3), 2.0 ** -8])
    assert R.in_window(5, 2)[3].tolist() == [False, False, True, True, False] and R.in_window(3, None)[2].all()
    # the convolution: last column is the token's own, zeros before the start
    assert np.allclose(R.causal_taps(np.arange(1.0, 5.0)[:, None], np.array([[100.0, 10.0, 1.0]]))[:, 0], [1.0, 12.0, 123.0, 234.0])
    # two tokens of the delta rule by hand: the second token's key is the first's, so its write replaces half of the memory's answer
    o = R.delta_recurrence(np.array([[[1.0, 0.0]]] * 2), np.array([[[1.0, 0.0]]] * 2), np.array([[[2.0]], [[4.0]]]), np.array([[1.0], [0.5]]), np.array([[0.3], [0.5]]))
    assert np.allclose(o[:, 0, 0], [2.0, 1.0 + 0.5 * (4.0 - 1.0)])
    # the choice goes by the corrected scores, the weights by the scores
    sel, w = R.route(np.array([[0.0, 1.0, -1.0]]), np.array([0.0, -1.0, 0.5]), 2)
    s = R.logistic(np.array([0.0, 1.0, -1.0]))
    assert sel[0].tolist() == [2, 0] and np.allclose(w[0], np.array([s[2], s[0]]) / (s[2] + s[0]))
    # limits: the gate from above only, the linear part from both sides
    assert np.allclose(R.limited_glu(np.array([5.0, -5.0]), np.array([3.0, -3.0]), 2.0), [2.0 * R.logistic(3.404) * 3.0, -5.0 * R.logistic(-8.51) * -1.0])
    assert abs(R.gelu_by_tanh(np.array([1.0]))[0] - 0.841192) < 1e-6
    assert R.layer_order({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == [0, 1, 2, 1, 2, 3]


def _probe(H, m, n_ctx, steps, n_ubatch=64, n_seq=4, want=None, inputs=()):
    """llm_decode with a compute callback that records the nodes of every graph (host memory here) and the f32 values of some inputs"""
    seen, values = [], []

    def comp(g, _n):
        gg = g.contents
        nodes, vals = [], {}
        for i in range(gg.n_nodes):
            t = gg.nodes[i].contents
            srcs = [t.src[s].contents.name.decode() if t.src[s] else None for s in range(10)]
            for s in range(10):
                if t.src[s] and t.src[s].contents.name.decode() in inputs:
                    tt = t.src[s].contents
                    n = int(np.prod(list(tt.ne)))
                    vals[tt.name.decode()] = np.ctypeslib.as_array((C.c_float * n).from_address(tt.data)).copy()
            nodes.append((H.ggml_op_name(t.op).decode(), t.name.decode(), srcs, list(t.ne), list(t.op_params)))
        seen.append(nodes)
        values.append(vals)
        return 0

    fn = L.COMPUTE_FN(comp)
    cp = L.ContextParams(n_ctx, n_ubatch, 1, 0, 1, 0, 0, n_seq)
    c = H.llm_context_new(m, None, fn, C.byref(cp))
    assert c
    for toks, pos, seq in steps:
        n = len(toks)
        w = (C.c_int8 * n)(*want) if want is not None and len(want) == n else None
        assert H.llm_decode(c, n, (C.c_int32 * n)(*toks), (C.c_int32 * n)(*pos), (C.c_int32 * n)(*seq), w) == 0
    caches = [bool(H.llm_context_cache_tensor(c, il, 0)) for il in range(5)]
    H.llm_context_free(c)
    return seen, values, caches


def test_graph_of_a_mixed_batch(H):
    cfg = small_cfg()
    m = H.llm_model_synth_config(json.dumps(cfg).encode(), 7, H.ggml_backend_cpu_buffer_type(), L.BF16)
    assert m
    seen, values, caches = _probe(H, m, 256, [([5, 6], [0, 1], [2, 2]), ([20, 21, 30, 22], [0, 1, 2, 2], [0, 0, 2, 0])], want=[0, 1, 0, 1],
                                  inputs=("q_temp-0", "q_temp-1", "KQ_mask", "KQ_mask_chunked-1"))
    nodes, vals = seen[-1], values[-1]
    # five layer runs (two layers twice, one once): three attentions, two recurrences; a cache per pass; one op between two sublayers (five mixers, four feed-forwards, the end)
    ops = {}
    for op, *_ in nodes:
        ops[op] = ops.get(op, 0) + 1
    assert ops["FLASH_ATTN_EXT"] == 3 and ops["GATED_LINEAR_ATTN"] == 2 and ops["CUSTOM"] == 10 and "ROPE" not in ops and "CONCAT" not in ops
    assert caches == [False, True, False, True, True]
    steps = [n for n in nodes if n[0] == "CUSTOM"]
    assert [n[1] for n in steps] == ["streams_attn-0", "streams_ffn-0", "streams_attn-1", "streams_ffn-1", "streams_attn-2", "streams_ffn-2", "streams_attn-3", "streams_ffn-3", "streams_attn-4",
                                     "result_norm"]
    # the first spreads the embedding; every other one carries the mixture of the sublayer behind it and the weights of the one in front; a repeated layer's are its own again
    assert steps[0][2][0] == "inp_embd" and steps[0][2][1] is None and steps[0][2][4] == "blk.0.attn_streams_in.weight"
    assert steps[1][2][2:6] == ["blk.0.attn_streams_mix.weight", "blk.0.attn_streams_out.weight", "blk.0.ffn_streams_in.weight", "blk.0.ffn_norm.weight"]
    assert steps[4][2][2:6] == ["blk.1.ffn_streams_mix.weight", "blk.1.ffn_streams_out.weight", "blk.0.attn_streams_in.weight", "blk.0.attn_norm.weight"]
    assert steps[8][2][2:6] == ["blk.1.ffn_streams_mix.weight", "blk.1.ffn_streams_out.weight", "blk.2.attn_streams_in.weight", "blk.2.attn_norm.weight"]
    # the last one sums the streams under the output norm, for the wanted rows only, and keeps no streams
    assert steps[9][2][2:7] == ["blk.2.attn_streams_mix.weight", "blk.2.attn_streams_out.weight", None, "output_norm.weight", "out_ids"]
    assert steps[9][3][:3] == [40, 2, 1] and steps[0][3][:3] == [40, 4, 4]
    assert [n for n in nodes if n[1] == "result_output"][0][3][:2] == [53, 2]
    # which cache every attention reads and stores
    fa = [n for n in nodes if n[0] == "FLASH_ATTN_EXT"]
    assert [n[2][1].split(" ")[0] for n in fa] == ["cache_k_l-1", "cache_k_l-3", "cache_k_l-4"] and [n[2][5] for n in fa] == ["blk.1.attn_slopes.weight"] * 2 + ["blk.2.attn_slopes.weight"]
    assert [n[1] for n in nodes if n[0] == "SET_ROWS"] == ["k_store-1", "v_store-1", "k_store-3", "v_store-3", "k_store-4", "v_store-4"]
    # the query factors of every token, by its position in its own sequence
    for name, coef, every in (("q_temp-0", 0.3, 4), ("q_temp-1", 0.5, 9)):
        assert np.allclose(vals[name], R.query_temperature([0, 1, 2, 2], {"coef": coef, "every": every}), rtol=1e-6)
    # the masks hold distances of visible pairs (cells 0, 1: sequence 2; cells 2 .. 5: this batch)
    mask = vals["KQ_mask"].reshape(-1, 256)
    assert mask[0, :6].tolist() == [-np.inf, -np.inf, 0.0, -np.inf, -np.inf, -np.inf] and mask[3, :6].tolist() == [-np.inf, -np.inf, 2.0, 1.0, -np.inf, 0.0] and mask[2, :6].tolist() == [
        2.0, 1.0, -np.inf, -np.inf, 0.0, -np.inf]
    # node orders the backend's fused launches rest on (views between them skipped): the three products, then the norms and both stores; the router
    flat = [(n[0], n[1]) for n in nodes if n[0] not in ("RESHAPE", "VIEW", "PERMUTE")]
    at = [n[1] for n in flat].index("Qcur-1")
    assert [n[1] for n in flat[at:at + 10]] == ["Qcur-1", "Kcur-1", "Vcur-1", "Qcur_rnorm-1", "Qcur_normed-1", "Qcur_temp-1", "Kcur_rnorm-1", "Kcur_normed-1", "k_store-1", "v_store-1"]
    at = [n[1] for n in flat].index("ffn_moe_logits-1")
    assert [n[1] for n in flat[at:at + 9]] == ["ffn_moe_logits-1", "ffn_moe_probs-1", "ffn_moe_choice-1", "ffn_moe_order-1", "ffn_moe_sel_probs-1", "ffn_moe_sum-1", "ffn_moe_sum_eps-1",
                                               "ffn_moe_weights-1", "ffn_moe_gate_up-1"]
    H.llm_model_free(m)


def test_query_factor_at_a_step(H):
    """positions around the steps of the factor, far into a sequence"""
    cfg = R.make_config(16, 11, [R.attention_layer(heads=1, kv_heads=1, dim=4, vdim=4, scale=0.5, size=3, coef=0.35, every=200, mlp=None)], streams=2)
    m = H.llm_model_synth_config(json.dumps(cfg).encode(), 7, H.ggml_backend_cpu_buffer_type(), L.F32)
    pos = [0, 198, 199, 200, 398, 399, 599, 100000]
    _, values, _ = _probe(H, m, 256, [([1] * 8, pos, [0] * 8)], inputs=("q_temp-0",))
    assert np.allclose(values[-1]["q_temp-0"], [1.0 + 0.35 * np.log((p + 1) // 200 + 1) for p in pos], rtol=1e-6)
    H.llm_model_free(m)


def test_sequence_ids_beyond_the_state_rows_are_refused(H):
    m = H.llm_model_synth_config(json.dumps(small_cfg()).encode(), 9, H.ggml_backend_cpu_buffer_type(), L.F32)
    fn = L.COMPUTE_FN(lambda g, n: 0)
    cp = L.ContextParams(256, 64, 1, 0, 1, 0, 0, 2)
    c = H.llm_context_new(m, None, fn, C.byref(cp))
    assert H.llm_decode(c, 1, (C.c_int32 * 1)(1), (C.c_int32 * 1)(0), (C.c_int32 * 1)(2), None) == -1
    assert H.llm_decode(c, 1, (C.c_int32 * 1)(1), (C.c_int32 * 1)(0), (C.c_int32 * 1)(1), None) == 0
    H.llm_context_free(c)
    H.llm_model_free(m)
