"""Host side of the Nidudra model class, without a GPU: the loader (projections kept as one matrix, frequency tables, no keys and values where a layer uses another's), what it refuses, the
plain reference's own pieces, and the graph the engine builds for a mixed batch — which layers have cells, which cache every attention reads, where the norms stand, in which order the nodes
that the backend runs as one launch follow one another."""
import ctypes as C
import json
import math

import numpy as np
import pytest

import llama_box_amd as L
import nidudra_ref as R


def small_cfg():
    return R.make_config(40, 53, [
        R.window_layer(4, 2, 8, 12, 0.3, R.dense(16), size=5, keep_first=2),
        R.parallel_layer(4, 2, 12, 0.4, R.rot(8, 500.0, R.ramped(4.0, 64, 8.0, 1.0)), 3, r_heads=3, r_dim=6, r_vdim=10, tau=8.0, mlp=R.moe(12, 6, 2, shared=20), rank=7),
        R.window_layer(6, 2, 8, 12, 0.2, None, size=7, keep_first=1, kv_from=0),
        R.sink_layer(4, 1, 12, 8, 0.5, R.rot(12, 1000.0, R.banded(4.0, 1.0, 4.0, 256)), R.moe(8, 3, 1)),
    ], softcap=9.0, eps=1e-5)


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
    cat = lambda *names: np.concatenate([W[n] for n in names])
    for wtype in (L.BF16, L.F32):
        m = H.llm_model_load_dir(str(tmp_path).encode(), H.ggml_backend_cpu_buffer_type(), wtype)
        assert m
        hp = H.llm_model_hparams(m).contents
        assert (hp.arch, hp.n_layer, hp.n_embd, hp.n_vocab) == (b"nidudra", 4, 40, 53)
        # the norms behind the sublayers, none in front
        assert np.array_equal(_get(H, m, "blk.1.attn_post_norm.weight").reshape(-1), W["l1.norm1"]) and np.array_equal(_get(H, m, "blk.3.ffn_post_norm.weight").reshape(-1), W["l3.norm2"])
        assert not any(H.llm_model_tensor(m, n) for n in (b"blk.0.attn_norm.weight", b"blk.0.ffn_norm.weight", b"blk.2.ffn_post_norm.weight"))
        # the parallel mixer: queries and keys as one projection with one bias and one tensor of taps; the linear attention's q, k, v likewise; the inner size from the checkpoint
        assert np.array_equal(_get(H, m, "blk.1.attn_qkv.weight")[0], cat("l1.mix.left.q", "l1.mix.left.k"))
        assert np.array_equal(_get(H, m, "blk.1.attn_qkv.bias").reshape(-1), cat("l1.mix.left.q.b", "l1.mix.left.k.b"))
        assert np.array_equal(_get(H, m, "blk.1.ssm_conv1d.weight")[0], cat("l1.mix.left.q.conv", "l1.mix.left.k.conv"))
        assert np.array_equal(_get(H, m, "blk.1.linear_qkv.weight")[0], cat("l1.mix.right.q", "l1.mix.right.k", "l1.mix.right.v"))
        assert _get(H, m, "blk.1.linear_a2.weight")[0].shape == (18, 7) and np.array_equal(_get(H, m, "blk.1.linear_a2.bias").reshape(-1), W["l1.mix.right.a2.b"])
        assert np.array_equal(_get(H, m, "blk.1.attn_sub_norm.weight").reshape(-1), W["l1.mix.right.norm"]) and np.array_equal(_get(H, m, "blk.1.mix_right_norm.weight").reshape(-1), W["l1.mix.right.out"])
        # a layer over another's cache: queries, gate and output only
        assert H.llm_model_tensor(m, b"blk.2.attn_q_norm.weight") and not any(H.llm_model_tensor(m, n) for n in (b"blk.2.attn_k.weight", b"blk.2.attn_v.weight", b"blk.2.attn_k_norm.weight"))
        # the sink and one gate row per head
        assert np.array_equal(_get(H, m, "blk.3.attn_sink.weight").reshape(-1), W["l3.mix.sink"]) and _get(H, m, "blk.3.attn_gate.weight")[0].shape == (4, 40)
        # the tables of frequencies, both schedules
        for il, r in ((1, cfg["layers"][1]["mixer"]["left"]["rot"]), (3, cfg["layers"][3]["mixer"]["rot"])):
            assert np.allclose(_get(H, m, "blk.%d.rope_freq.weight" % il).reshape(-1), R.rotation(r)[0], rtol=1e-6)
        # feed-forwards: gate rows, then up rows — dense, per expert, shared; the router in f32
        assert np.array_equal(_get(H, m, "blk.0.ffn_gate_up.weight")[0], cat("l0.mlp.gate", "l0.mlp.up"))
        gu = _get(H, m, "blk.1.ffn_gate_up_exps.weight")
        assert gu.shape == (6, 24, 40) and np.array_equal(gu[5], cat("l1.mlp.e5.gate", "l1.mlp.e5.up"))
        assert np.array_equal(_get(H, m, "blk.1.ffn_gate_up_shexp.weight")[0], cat("l1.mlp.shared.gate", "l1.mlp.shared.up"))
        assert np.array_equal(_get(H, m, "blk.1.ffn_gate_inp_shexp.weight")[0], W["l1.mlp.shared.sg"]) and not H.llm_model_tensor(m, b"blk.3.ffn_down_shexp.weight")
        assert H.llm_model_tensor(m, b"blk.1.ffn_gate_inp.weight").contents.type == L.F32
        assert np.array_equal(_get(H, m, "output.weight")[0], W["head"])
        H.llm_model_free(m)


@pytest.mark.parametrize("breakage", ["shape", "missing", "heads", "mixer", "kind", "window", "top", "taps", "rot", "odd_rot", "scaling", "band", "tau", "values", "later", "itself_shared", "other_sizes",
                                      "other_type", "shared_ff", "cap", "rank", "right"])
def test_loader_refuses_what_it_cannot_serve(H, tmp_path, breakage):
    cfg = small_cfg()
    W = R.random_weights(cfg, 4)
    L0, L1, L2, L3 = cfg["layers"]
    if breakage == "shape":
        W["l1.mix.left.k.conv"] = W["l1.mix.left.k.conv"][:, :-1]
    elif breakage == "missing":
        del W["l3.mix.sink"]
    elif breakage == "heads":
        L0["mixer"]["kv_heads"] = 3
    elif breakage == "mixer":
        L0["type"] = "attention_3"
    elif breakage == "kind":
        L0["mlp"]["kind"] = "gated"
    elif breakage == "window":
        L0["mixer"]["mask"]["size"] = 0
    elif breakage == "top":
        L1["mlp"]["router"]["top"] = 7
    elif breakage == "taps":
        L1["mixer"]["left"]["conv"] = 17
    elif breakage == "rot":
        L3["mixer"]["rot"]["dims"] = 14
    elif breakage == "odd_rot":
        L1["mixer"]["left"]["rot"]["dims"] = 7
    elif breakage == "scaling":
        L1["mixer"]["left"]["rot"]["scaling"]["factor"] = 0
    elif breakage == "band":
        L3["mixer"]["rot"]["scaling"]["high"] = 1.0
    elif breakage == "tau":
        L1["mixer"]["right"]["tau"] = 0
    elif breakage == "values":
        L1["mixer"]["left"]["vdim"] = 10
    elif breakage == "later":
        L2["mixer"]["kv_from"] = 2
    elif breakage == "itself_shared":
        cfg["layers"].append(R.window_layer(4, 2, 8, 12, 0.2, None, size=7, kv_from=2))
        W.update(R.random_weights(cfg, 4))
    elif breakage == "other_sizes":
        L2["mixer"]["kv_heads"] = 6
    elif breakage == "other_type":
        L2["mixer"].update(kv_from=1)
    elif breakage == "shared_ff":
        L1["mlp"]["shared"]["ff"] = 0
    elif breakage == "cap":
        cfg["logit_softcap"] = -1.0
    elif breakage == "rank":
        del W["l1.mix.right.a1"]
    elif breakage == "right":
        del L1["mixer"]["right"]
    if breakage == "right":
        with open(tmp_path / "config.json", "w") as f:
            json.dump(cfg, f)
        R.save_model(small_cfg(), W, str(tmp_path / "w"))
        (tmp_path / "w" / "model.safetensors").rename(tmp_path / "model.safetensors")
    else:
        R.save_model(cfg, W, str(tmp_path))
    assert not H.llm_model_load_dir(str(tmp_path).encode(), H.ggml_backend_cpu_buffer_type(), L.F32)


def test_parts_that_are_absent_are_not_needed(H, tmp_path):
    """no window, no scaling, no rotation, no shared expert, no cap, null instead of an object: the keys may be missing or null"""
    cfg = R.make_config(24, 19, [R.window_layer(2, 1, 8, 8, 0.3, None), R.sink_layer(1, 1, 4, 6, 0.5, R.rot(0, 100.0), R.moe(4, 2, 1)), R.sink_layer(2, 2, 8, 4, 0.5, R.rot(2, 100.0), None)], softcap=None)
    cfg["logit_softcap"] = None
    cfg["layers"][0]["mixer"].update(mask=None, kv_from=None)
    cfg["layers"][2]["mixer"]["rot"]["scaling"] = None
    R.save_model(cfg, R.random_weights(cfg, 5), str(tmp_path))
    m = H.llm_model_load_dir(str(tmp_path).encode(), H.ggml_backend_cpu_buffer_type(), L.F32)
    assert m and not H.llm_model_tensor(m, b"blk.1.rope_freq.weight") and H.llm_model_tensor(m, b"blk.2.rope_freq.weight")
    H.llm_model_free(m)


def test_reference_pieces():
    # window with kept first tokens: both edges
    ok = R.seen(7, {"size": 2, "keep_first": 1})
    assert ok[5].tolist() == [True, False, False, False, True, True, False] and ok[0].tolist() == [True] + [False] * 6 and R.seen(3, None)[2].all()
    # the convolution: last column is the token's own, nothing before the start
    assert np.allclose(R.history_taps(np.arange(1.0, 5.0)[:, None], np.array([[100.0, 10.0, 1.0]]))[:, 0], [1.0, 12.0, 123.0, 234.0])
    # two tokens of the memory by hand: key rows fade one by one, the query reads what the token has added
    o = R.fading_memory(np.array([[[1.0, 1.0]], [[1.0, 2.0]]]), np.array([[[1.0, 3.0]], [[0.0, 1.0]]]), np.array([[[2.0]], [[5.0]]]), np.array([[[0.9, 0.9]], [[0.5, 0.1]]]))
    assert np.allclose(o[:, 0, 0], [8.0, 0.5 * 2.0 + 2.0 * (0.1 * 6.0 + 5.0)])
    assert np.allclose(R.fading(np.array([0.0]), 16.0), 0.5 ** (1 / 16))
    # rotation by halves, a tail that passes, the factor on sine and cosine for one of the schedules only
    x = np.arange(12.0).reshape(2, 1, 6)
    y = R.rotate_halves(x, R.rot(4, 100.0))
    c, s = math.cos(0.1), math.sin(0.1)
    assert np.allclose(y[0], x[0]) and np.allclose(y[1, 0, [1, 3]], [7 * c - 9 * s, 9 * c + 7 * s]) and np.allclose(y[1, 0, 4:], [10, 11])
    assert R.rotation(R.rot(4, 100.0, R.ramped(8.0, 64, 8.0, 1.0)))[1] == 0.1 * math.log(8.0) + 1.0 and R.rotation(R.rot(4, 100.0, R.banded(8.0, 1.0, 4.0, 64)))[1] == 1.0
    # banded: kept, blended, divided
    f = R.plain_frequencies(8, 10000.0)
    g = R.banded_frequencies(f, R.banded(4.0, 1.0, 4.0, 64))
    turns = 64 * f / (2 * math.pi)
    assert turns[0] > 4 > turns[1] > 1 > turns[2] and g[0] == f[0] and g[2] == f[2] / 4.0 and np.isclose(g[1], f[1] * ((1 - (turns[1] - 1) / 3) / 4 + (turns[1] - 1) / 3))
    # ramped: kept in front of the ramp, divided behind it
    g = R.ramped_frequencies(f, 8, 10000.0, R.ramped(4.0, 4096, 32.0, 1.0))
    assert np.allclose(g / f, [1.0, 1.0, 0.5 * 1.0 + 0.5 / 4.0, 0.25])  # (the ramp runs from pair 1 to pair 3)
    # the sink is one more term without a value
    o = R.attend(np.zeros((1, 1, 2)), np.zeros((1, 1, 2)), np.ones((1, 1, 1)), 1.0, sink=np.array([math.log(3.0)]))
    assert np.isclose(o[0, 0, 0], 0.25)
    # the scores weigh as they are
    sel, w = R.route(np.array([[0.0, 1.0, -1.0]]), 2)
    assert sel[0].tolist() == [1, 0] and np.allclose(w[0], [1 / (1 + math.exp(-1.0)), 0.5])
    assert np.isclose(R.capped(np.array(3.0), 2.0), 2.0 * math.tanh(1.5)) and R.capped(5.0, None) == 5.0


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
    caches = [bool(H.llm_context_cache_tensor(c, il, 0)) for il in range(4)]
    H.llm_context_free(c)
    return seen, values, caches


def test_graph_of_a_mixed_batch(H):
    cfg = small_cfg()
    m = H.llm_model_synth_config(json.dumps(cfg).encode(), 7, H.ggml_backend_cpu_buffer_type(), L.BF16)
    assert m
    seen, values, caches = _probe(H, m, 256, [([5, 6], [0, 1], [2, 2]), ([20, 21, 30, 22], [0, 1, 2, 2], [0, 0, 2, 0])], want=[0, 1, 0, 1], inputs=("KQ_mask", "KQ_mask_chunked-1", "KQ_mask_chunked-2"))
    nodes, vals = seen[-1], values[-1]
    ops = {}
    for op, *_ in nodes:
        ops[op] = ops.get(op, 0) + 1
    assert ops["FLASH_ATTN_EXT"] == 4 and ops["GATED_LINEAR_ATTN"] == 1 and ops["SSM_CONV"] == 2 and ops["ROPE"] == 4 and "CUSTOM" not in ops
    # the third layer has no cells and stores nothing: it reads the first layer's, under a mask of its own; the sink is the fourth layer's
    assert caches == [True, True, False, True]
    fa = [n for n in nodes if n[0] == "FLASH_ATTN_EXT"]
    assert [n[2][1].split(" ")[0] for n in fa] == ["cache_k_l-0", "cache_k_l-1", "cache_k_l-0", "cache_k_l-3"] and [n[2][2].split(" ")[0] for n in fa] == ["cache_v_l-0", "cache_v_l-1", "cache_v_l-0", "cache_v_l-3"]
    assert [n[2][3] for n in fa] == ["KQ_mask", "KQ_mask_chunked-1", "KQ_mask_chunked-2", "KQ_mask_chunked-1"] and [n[2][4] for n in fa] == [None, None, None, "blk.3.attn_sink.weight"]
    assert [n[1] for n in nodes if n[0] == "SET_ROWS"] == ["k_store-0", "v_store-0", "k_store-1", "v_store-1", "k_store-3", "v_store-3"]
    # the masks: windows with kept first tokens, and plainly causal (cells 0, 1: sequence 2; cells 2 .. 5: this batch)
    mask = vals["KQ_mask_chunked-1"].reshape(-1, 256)
    assert mask[2, :6].tolist() == [0.0, 0.0, -np.inf, -np.inf, 0.0, -np.inf] and mask[3, :6].tolist() == [-np.inf, -np.inf, 0.0, 0.0, -np.inf, 0.0]
    # the sublayers read the stream itself: the embedding goes into the first products, the norms stand behind the mixers and the feed-forwards
    byname = {n[1]: n for n in nodes}
    assert byname["Qcur-0"][2][1] == "inp_embd" and byname["ffn_gate_up-0"][2][1] == "ffn_inp-0" and byname["linear_qkv-1"][2][1] == "l_out-0" and byname["qk_proj-1"][2][1] == "l_out-0"
    assert byname["ffn_inp-0"][2][:2] == ["attn_post_norm-0", "inp_embd"] and byname["l_out-0"][2][:2] == ["ffn_post_norm-0", "ffn_inp-0"] and byname["l_out-2"][2][:2] == ["attn_post_norm-2", "l_out-1"]
    # the values of the parallel mixer are the convolved keys, ahead of their norm (the cache store reads a part of the convolution's rows)
    assert byname["v_store-1"][3][:2] == [24, 256] and byname["qk_conv-1"][0] == "SSM_CONV" and byname["qk_conv-1"][2][0] == "qk_pre-1" and byname["conv_store-1"][2][0] == "qk_pre-1"
    assert byname["linear_attn-1"][4][:3] == [5, 3, 3] and np.array([byname["linear_attn-1"][4][4]], np.int32).view(np.float32)[0] == 8.0
    # only the wanted rows go through the last feed-forward; the cap is the last thing that happens
    assert byname["ffn_moe_logits-3"][3][:2] == [3, 2] and [n[1] for n in nodes][-4:] == ["result_unscaled", "result_by_cap", "result_tanh", "result_output"] and nodes[-1][3][:2] == [53, 2]
    # node orders the backend's fused launches rest on (views between them skipped)
    flat = [n[1] for n in nodes if n[0] not in ("RESHAPE", "VIEW", "PERMUTE")]

    def follow(first, *rest):
        at = flat.index(first)
        assert flat[at:at + 1 + len(rest)] == [first, *rest]

    follow("Qcur-0", "Kcur-0", "Vcur-0", "attn_gate-0", "Qcur_rnorm-0", "Qcur_normed-0", "Kcur_rnorm-0", "Kcur_normed-0", "k_store-0", "v_store-0", "fattn-0")
    follow("linear_qkv-1", "linear_gate-1", "linear_a_in-1", "qk_proj-1", "qk_pre-1", "qk_conv-1", "conv_store-1", "Qcur_rnorm-1", "Qcur_normed-1", "Qcur_rope-1", "Kcur_rnorm-1", "Kcur_normed-1",
           "Kcur_rope-1", "k_store-1", "v_store-1", "fattn-1", "attn_out-1", "linear_a_pre-1", "linear_attn-1", "head_rnorm-1")
    follow("mix_left_rnorm-1", "mix_left_normed-1", "mix_left-1", "mix_right_rnorm-1", "mix_right_normed-1", "mix_right-1", "mix_sum-1", "rnorm-1", "attn_post_norm-1", "ffn_inp-1", "ffn_moe_logits-1",
           "ffn_moe_probs-1", "ffn_moe_order-1", "ffn_moe_sel_probs-1", "ffn_moe_gate_up-1", "ffn_moe_gate_up_weighted-1", "ffn_moe_act-1", "ffn_moe_down-1", "ffn_shared_gate-1", "ffn_shared_gate_up-1",
           "ffn_shared_act-1", "ffn_shared_out-1", "ffn_shared_sigmoid-1", "ffn_shared_gated-1")
    at = flat.index("ffn_moe_out-1")
    assert flat[at + 1:at + 4] == ["rnorm-1", "ffn_post_norm-1", "l_out-1"]
    follow("Qcur-3", "Kcur-3", "Vcur-3", "attn_gate-3", "Qcur_rope-3", "Qcur_unit-3", "Kcur_rope-3", "Kcur_unit-3", "k_store-3", "v_store-3")
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
