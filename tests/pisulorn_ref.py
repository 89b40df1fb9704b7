"""A plain, slow statement of the Pisulorn design in numpy (float64): one function per mechanism, written from the design's equations and
sharing nothing with the product path.  The GPU tests compare the framework against it.

Notation: T tokens, E = width, N streams, H query (or value) heads, G key heads, Dk per-head key size, Dv per-head value size.
Weights are [out, in] and applied as W @ x.  A model is (cfg, W): cfg is the parsed config.json, W maps tensor names to float64 arrays.
Every sequence starts at position 0 with every state at zero."""
import json
import math
import os
import struct

import numpy as np


# ---------------------------------------------------------------------------------------------------------------- small pieces
def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def unit_length(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def logistic(z):
    return 1.0 / (1.0 + np.exp(-z))


def swish(z):
    return z * logistic(z)


def log1p_exp(z):
    return np.logaddexp(0.0, z)


def gelu_by_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_taps(u, w):
    """u [T, C], w [C, taps]: channel c of token t is sum_d w[c, taps - 1 - d] u[t - d, c]; tokens before the start count as zero."""
    T, taps = u.shape[0], w.shape[1]
    y = np.zeros_like(u)
    for d in range(min(taps, T)):
        y[d:] += u[:T - d] * w[:, taps - 1 - d]
    return y


# ---------------------------------------------------------------------------------------------------------------- attention's parts
def head_slope(h, H):
    """what a key loses per token of distance in head h of H"""
    return 2.0 ** (-8.0 * (h + 1) / H)


def query_temperature(pos, temp):
    """the factor on the query of a position: grows by coef times the logarithm of how many whole stretches of `every` tokens have passed"""
    if not temp:
        return np.ones(len(pos))
    return np.asarray([1.0 + temp["coef"] * math.log((p + 1) // temp["every"] + 1.0) for p in pos])


def in_window(T, size):
    """[T, T]: does position i see position j?  size None: every earlier position and itself"""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    ok = j <= i
    return ok if size is None else ok & (i - j < size)


def attention(h, mx, W, p, eps):
    H, G, Dk, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    pos = np.arange(T)
    q = unit_rms((h @ W[p + "q"].T).reshape(T, H, Dk), eps) * W[p + "q.norm"]
    k = unit_rms((h @ W[p + "k"].T).reshape(T, G, Dk), eps) * W[p + "k.norm"]
    v = (h @ W[p + "v"].T).reshape(T, G, Dv)
    q = q * query_temperature(pos, mx.get("q_temp"))[:, None, None]
    ok = in_window(T, mx["mask"]["size"] if mx.get("mask") else None)
    dist = (pos[:, None] - pos[None, :]).astype(np.float64)
    out = np.zeros((T, H, Dv))
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * mx["scale"] - head_slope(hd, H) * dist
        s = np.where(ok, s, -np.inf)
        w = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, hd] = (w / w.sum(axis=1, keepdims=True)) @ v[:, g]
    return out.reshape(T, H * Dv) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------------------------------- the delta rule
def delta_recurrence(q, k, v, beta, decay):
    """q, k [T, G, Dk]; v [T, H, Dv]; beta, decay [T, H] -> [T, H, Dv], token by token from an empty memory.  The memory fades, what it returns for the
    key is replaced by a share beta of the new value, and the query reads the memory that already holds it."""
    T, H, Dv = v.shape
    G, Dk = k.shape[1], k.shape[2]
    o = np.zeros((T, H, Dv))
    for h in range(H):
        g = h // (H // G)
        M = np.zeros((Dk, Dv))
        for t in range(T):
            M = M * decay[t, h]
            M = M + np.outer(k[t, g], beta[t, h] * (v[t, h] - k[t, g] @ M))
            o[t, h] = q[t, g] @ M
    return o


def delta(h, mx, W, p, eps):
    H, G, Dk, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    T = h.shape[0]
    q, k, v = (swish(causal_taps(h @ W[p + n].T, W[p + n + ".conv"])) for n in "qkv")
    q = unit_length(q.reshape(T, G, Dk)) * Dk ** -0.5
    k = unit_length(k.reshape(T, G, Dk))
    beta = logistic(h @ W[p + "b"].T)
    decay = np.exp(-np.exp(W[p + "A_log"]) * log1p_exp(h @ W[p + "a"].T + W[p + "dt_bias"]))
    o = delta_recurrence(q, k, v.reshape(T, H, Dv), beta, decay)
    o = unit_rms(o, eps) * W[p + "norm"] * swish(h @ W[p + "g"].T).reshape(T, H, Dv)
    return o.reshape(T, H * Dv) @ W[p + "o"].T


MIXERS = {"attention": attention, "delta": delta}


# ---------------------------------------------------------------------------------------------------------------- feed-forward
def dense_ffn(h, W, p):
    return gelu_by_tanh(h @ W[p + "up"].T) @ W[p + "down"].T


def route(z, correction, top):
    """z [T, experts] -> (chosen [T, top], weights [T, top]): chosen by the corrected scores, weighted by the scores themselves"""
    s = logistic(z)
    chosen = np.argsort(-(s + correction), axis=-1, kind="stable")[:, :top]
    w = np.take_along_axis(s, chosen, axis=-1)
    return chosen, w / (w.sum(axis=-1, keepdims=True) + 1e-20)


def limited_glu(g, u, limit):
    g = np.minimum(g, limit)
    return g * logistic(1.702 * g) * (np.clip(u, -limit, limit) + 1.0)


def experts_ffn(h, ml, W, p):
    chosen, wts = route(h @ W[p + "router"].T, W[p + "correction"], ml["router"]["top"])
    out = np.zeros_like(h)
    for e in range(ml["router"]["experts"]):
        t, slot = np.nonzero(chosen == e)
        if len(t):
            pe = "%se%d." % (p, e)
            y = limited_glu(h[t] @ W[pe + "gate"].T, h[t] @ W[pe + "up"].T, ml["expert"]["limit"]) @ W[pe + "down"].T
            out[t] += wts[t, slot][:, None] * y
    return out


def feed_forward(h, ml, W, p):
    return dense_ffn(h, W, p) if ml["kind"] == "dense" else experts_ffn(h, ml, W, p)


# ---------------------------------------------------------------------------------------------------------------- streams
def streams_in(X, a):
    """X [N, T, E] -> what a sublayer reads: the streams weighted by a [N]"""
    return np.einsum("n,nte->te", a, X)


def streams_out(X, y, mix, out, mult):
    """every stream becomes a mixture of the old ones (mix[from, to]) plus mult out[to] times the sublayer's output"""
    return np.einsum("ab,ate->bte", mix, X) + mult * out[:, None, None] * y[None]


# ---------------------------------------------------------------------------------------------------------------- the model
def layer(X, cfg, W, il):
    L, eps, p = cfg["layers"][il], cfg["norm"]["eps"], "l%d." % il
    mult = cfg["residual_mult"]
    subs = [("1", lambda h: MIXERS[L["type"]](h, L["mixer"], W, p + "mix.", eps))]
    if L.get("mlp"):
        subs.append(("2", lambda h: feed_forward(h, L["mlp"], W, p + "mlp.")))
    for n, f in subs:
        hc = p + "hc" + n + "."
        y = f(unit_rms(streams_in(X, W[hc + "in"]), eps) * W[p + "norm" + n])
        X = streams_out(X, y, W[hc + "mix"], W[hc + "out"], mult)
    return X


def layer_order(cfg):
    n, lp = len(cfg["layers"]), cfg.get("loop")
    order = list(range(n))
    if lp:
        order = order[:lp["start"]] + order[lp["start"]:lp["stop"]] * lp["times"] + order[lp["stop"]:]
    return order


def forward(cfg, W, tokens, residuals=None):
    """logits [T, vocab] of one sequence from position 0; `residuals` (a list) receives the sum of the streams after every layer run."""
    x = W["embed"][np.asarray(tokens)]
    X = np.repeat(x[None], cfg["streams"], axis=0)
    for il in layer_order(cfg):
        X = layer(X, cfg, W, il)
        if residuals is not None:
            residuals.append(X.sum(axis=0))
    return unit_rms(X.sum(axis=0), cfg["norm"]["eps"]) * W["final.norm"] @ W["head"].T


# ---------------------------------------------------------------------------------------------------------------- making models
def bf16_round(a):
    """float array -> the nearest bfloat16 values (round to nearest even), as float64."""
    b = np.asarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    b = ((b + 0x7FFF + ((b >> 16) & 1)) >> 16 << 16).astype(np.uint32)
    return b.view(np.float32).astype(np.float64)


def tensor_shapes(cfg):
    E, V, N = cfg["width"], cfg["vocab"], cfg["streams"]
    sh = {"embed": (V, E), "head": (V, E), "final.norm": (E,)}
    for il, L in enumerate(cfg["layers"]):
        p, mx, ml = "l%d." % il, L["mixer"], L.get("mlp")
        m, f = p + "mix.", p + "mlp."
        H, G, Dk, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        for n in ("1", "2") if ml else ("1",):
            sh.update({p + "norm" + n: (E,), p + "hc" + n + ".in": (N,), p + "hc" + n + ".out": (N,), p + "hc" + n + ".mix": (N, N)})
        if L["type"] == "attention":
            sh.update({m + "q": (H * Dk, E), m + "k": (G * Dk, E), m + "v": (G * Dv, E), m + "q.norm": (Dk,), m + "k.norm": (Dk,), m + "o": (E, H * Dv)})
        else:
            taps = mx["conv"]
            sh.update({m + "q": (G * Dk, E), m + "k": (G * Dk, E), m + "v": (H * Dv, E), m + "q.conv": (G * Dk, taps), m + "k.conv": (G * Dk, taps),
                       m + "v.conv": (H * Dv, taps), m + "b": (H, E), m + "a": (H, E), m + "A_log": (H,), m + "dt_bias": (H,), m + "norm": (Dv,),
                       m + "g": (H * Dv, E), m + "o": (E, H * Dv)})
        if ml and ml["kind"] == "dense":
            sh.update({f + "up": (ml["ff"], E), f + "down": (E, ml["ff"])})
        elif ml:
            n_e, ff = ml["router"]["experts"], ml["expert"]["ff"]
            sh.update({f + "router": (n_e, E), f + "correction": (n_e,)})
            for e in range(n_e):
                pe = "%se%d." % (f, e)
                sh.update({pe + "gate": (ff, E), pe + "up": (ff, E), pe + "down": (E, ff)})
    return sh


def random_weights(cfg, seed):
    """bf16-representable random weights with magnitudes that keep every mechanism alive (decays away from 0 and 1, unequal streams, experts that reach their limit)."""
    rng = np.random.default_rng(seed)
    N = cfg["streams"]
    W = {}
    for name, s in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        if leaf in ("norm1", "norm2", "norm"):
            a = rng.uniform(0.7, 1.4, s)
        elif leaf == "in":
            a = rng.uniform(0.2, 1.0, s)
        elif leaf == "out":
            a = rng.uniform(0.5, 1.5, s)
        elif leaf == "mix":
            a = np.eye(N) * 0.7 + rng.uniform(-0.2, 0.4, s)
        elif leaf == "conv":
            a = rng.normal(0, 0.5, s)
        elif leaf == "A_log":
            a = rng.uniform(-2.0, 0.5, s)
        elif leaf == "dt_bias":
            a = rng.uniform(-1.0, 1.0, s)
        elif leaf == "correction":
            a = rng.normal(0, 0.2, s)
        elif name == "embed":
            a = rng.normal(0, 1.0, s)
        elif leaf in ("router", "gate", "up", "a", "b"):
            a = rng.normal(0, 2.0 / math.sqrt(s[-1]), s)
        else:
            a = rng.normal(0, 1.0 / math.sqrt(s[-1]), s)
        W[name] = bf16_round(a)
    return W


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, limit):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def attention_layer(heads, kv_heads, dim, vdim, scale, mlp, size=None, coef=None, every=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        mx["mask"] = {"size": size}
    if every is not None:
        mx["q_temp"] = {"coef": coef, "every": every}
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def delta_layer(heads, kv_heads, dim, vdim, conv, mlp):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def make_config(width, vocab, layers, streams, residual_mult=0.5, loop=None, eps=1e-5):
    cfg = {"architecture": "Pisulorn", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers, "streams": streams, "residual_mult": residual_mult}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def save_model(cfg, W, folder):
    """config.json + model.safetensors with every tensor as bf16."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, at = {}, [], 0
    for name, a in W.items():
        b = (np.asarray(a, dtype=np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    hj = json.dumps(head).encode()
    hj += b" " * (-len(hj) % 8)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(hj)) + hj + b"".join(blobs))
