"""A plain, slow statement of the Nidudra design in numpy (float64): one function per mechanism, written from the design's equations and
sharing nothing with the product path.  The GPU tests compare the framework against it.

Notation: T tokens, E = width, H query heads, G key/value heads, Dk per-head key size, Dv per-head value size.
Weights are [out, in] and applied as W @ x.  A model is (cfg, W): cfg is the parsed config.json, W maps tensor names to float64 arrays.
Every sequence starts at position 0 with every state at zero."""
import json
import math
import os
import struct

import numpy as np


# ---------------------------------------------------------------------------------------------------------------- small pieces
def over_rms(x, eps):
    return x / np.sqrt((x ** 2).mean(axis=-1, keepdims=True) + eps)


def squash(z):
    """the logistic function, exact in relative terms on both sides (a decay is a root of it)"""
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0, e) / (1.0 + e)


def silu(z):
    return z * squash(z)


def capped(z, cap):
    return cap * np.tanh(z / cap) if cap else z


def history_taps(u, w):
    """u [T, C], w [C, taps]: the last tap multiplies the token's own input, the one before it the previous token's; before the start there is nothing."""
    T, taps = u.shape[0], w.shape[1]
    y = np.zeros_like(u)
    for t in range(T):
        for back in range(min(taps, t + 1)):
            y[t] += w[:, taps - 1 - back] * u[t - back]
    return y


# ---------------------------------------------------------------------------------------------------------------- positions
def plain_frequencies(dims, base):
    return np.asarray([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)])


def banded_frequencies(f, sc):
    """by wavelength: short ones stay, long ones are divided by `factor`, those between two bounds are blended linearly in original / wavelength"""
    out = []
    for fi in f:
        turns = sc["original"] * fi / (2.0 * math.pi)  # how often the pair turns within the original length
        if turns > sc["high"]:
            out.append(fi)
        elif turns < sc["low"]:
            out.append(fi / sc["factor"])
        else:
            s = (turns - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1.0 - s) * fi / sc["factor"] + s * fi)
    return np.asarray(out)


def ramped_frequencies(f, dims, base, sc):
    """by index: between the pair that turns `fast` times and the pair that turns `slow` times within the original length, a ramp from kept to divided"""
    def index_of(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(index_of(sc["fast"])), 0)
    hi = min(math.ceil(index_of(sc["slow"])), dims - 1)
    ramp = np.clip((np.arange(len(f)) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp)


def rotation(rot):
    """-> (frequencies, factor on sine and cosine)"""
    f = plain_frequencies(rot["dims"], rot["base"])
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    if "low" in sc:
        return banded_frequencies(f, sc), 1.0
    return ramped_frequencies(f, rot["dims"], rot["base"], sc), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_halves(x, rot):
    """x [T, heads, D], row t at position t: entry i of the first half of the leading dims turns with entry i of the second half"""
    f, mag = rotation(rot)
    half = len(f)
    a = np.arange(x.shape[0])[:, None, None] * f
    c, s = mag * np.cos(a), mag * np.sin(a)
    u, v = x[..., :half], x[..., half:2 * half]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * half:]], axis=-1)


# ---------------------------------------------------------------------------------------------------------------- attention
def seen(T, mask):
    """[T, T]: does position i see position j?  A window over the last `size` positions, and besides the first `keep_first` of the sequence"""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    ok = j <= i
    if mask:
        ok = ok & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    return ok


def attend(q, k, v, scale, mask=None, sink=None):
    """q [T, H, Dk], k [T, G, Dk], v [T, G, Dv] -> [T, H, Dv]; `sink` [H]: one more term exp(sink) in the denominator"""
    T, H, _ = q.shape
    per = H // k.shape[1]
    ok = seen(T, mask)
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        z = np.where(ok, scale * (q[:, h] @ k[:, h // per].T), -np.inf)
        top = z.max(axis=1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink[h])
        w = np.exp(z - top)
        den = w.sum(axis=1, keepdims=True)
        if sink is not None:
            den = den + np.exp(sink[h] - top)
        out[:, h] = (w / den) @ v[:, h // per]
    return out


def heads_of(y, n, d):
    return y.reshape(y.shape[0], n, d)


def windowed(h, mx, W, p, eps, kept):
    """normed queries and keys, no positions, a window with kept first tokens, a gate per value entry; `kept`: keys and values of the layers so far (None: own ones).
    Returns (output, (keys, values))"""
    H, G, Dk, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = over_rms(heads_of(h @ W[p + "q"].T, H, Dk), eps) * W[p + "q.norm"]
    if kept is None:
        k = over_rms(heads_of(h @ W[p + "k"].T, G, Dk), eps) * W[p + "k.norm"]
        kept = k, heads_of(h @ W[p + "v"].T, G, Dv)
    o = attend(q, kept[0], kept[1], mx["scale"], mx.get("mask")).reshape(len(h), H * Dv)
    return (o * squash(h @ W[p + "g"].T)) @ W[p + "o"].T, kept


def rotated_with_sink(h, mx, W, p, eps):
    """rotated queries and keys, then made unit by their root mean square (no weight); a learned sink; one gate per head"""
    H, G, Dk, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = over_rms(rotate_halves(heads_of(h @ W[p + "q"].T, H, Dk), mx["rot"]), eps)
    k = over_rms(rotate_halves(heads_of(h @ W[p + "k"].T, G, Dk), mx["rot"]), eps)
    v = heads_of(h @ W[p + "v"].T, G, Dv)
    o = attend(q, k, v, mx["scale"], sink=W[p + "sink"]) * squash(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(len(h), H * Dv) @ W[p + "o"].T


def keys_as_values(h, mx, W, p, eps):
    """biased projections of queries and keys behind short convolutions; the convolved keys ARE the values; normed, then rotated queries and keys"""
    H, G, Dk = mx["heads"], mx["kv_heads"], mx["dim"]
    q = heads_of(history_taps(h @ W[p + "q"].T + W[p + "q.b"], W[p + "q.conv"]), H, Dk)
    v = heads_of(history_taps(h @ W[p + "k"].T + W[p + "k.b"], W[p + "k.conv"]), G, Dk)
    k = rotate_halves(over_rms(v, eps) * W[p + "k.norm"], mx["rot"])
    q = rotate_halves(over_rms(q, eps) * W[p + "q.norm"], mx["rot"])
    return attend(q, k, v, mx["scale"]).reshape(len(h), H * Dk) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------------------------------- gated linear attention
def fading_memory(q, k, v, keep):
    """q, k, keep [T, H, Dk], v [T, H, Dv] -> [T, H, Dv]: every key row of a head's memory fades by its own factor, the token's pair is added, the query reads"""
    T, H, Dv = v.shape
    o = np.zeros((T, H, Dv))
    for h in range(H):
        M = np.zeros((q.shape[2], Dv))
        for t in range(T):
            M = keep[t, h][:, None] * M + k[t, h][:, None] * v[t, h][None, :]
            o[t, h] = q[t, h] @ M
    return o


def fading(z, tau):
    return squash(z) ** (1.0 / tau)


def linear_attention(h, mx, W, p, eps):
    H, Dk, Dv = mx["heads"], mx["dim"], mx["vdim"]
    q = heads_of(h @ W[p + "q"].T, H, Dk) * Dk ** -0.5
    k = heads_of(h @ W[p + "k"].T, H, Dk)
    v = heads_of(h @ W[p + "v"].T, H, Dv)
    keep = heads_of(fading((h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"], mx["tau"]), H, Dk)
    o = over_rms(fading_memory(q, k, v, keep), eps) * W[p + "norm"]
    return (o.reshape(len(h), H * Dv) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def side_by_side(h, mx, W, p, eps):
    a = keys_as_values(h, mx["left"], W, p + "left.", eps)
    b = linear_attention(h, mx["right"], W, p + "right.", eps)
    return 0.5 * (over_rms(a, eps) * W[p + "left.out"] + over_rms(b, eps) * W[p + "right.out"])


# ---------------------------------------------------------------------------------------------------------------- feed-forward
def gated_ffn(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(z, top):
    """z [T, experts] -> (chosen [T, top], weights [T, top]): the logistic scores choose and weigh, as they are"""
    s = squash(z)
    chosen = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=-1)


def experts_ffn(h, ml, W, p):
    """an expert reads its weight times the token; one more runs for every token, behind a gate of its own"""
    chosen, wts = route(h @ W[p + "router"].T, ml["router"]["top"])
    out = np.zeros_like(h)
    for t in range(len(h)):
        for e, w in zip(chosen[t], wts[t]):
            out[t] += gated_ffn(w * h[t][None], W, "%se%d." % (p, e))[0]
    if ml.get("shared"):
        out += gated_ffn(h, W, p + "shared.") * squash(h @ W[p + "shared.sg"].T)
    return out


# ---------------------------------------------------------------------------------------------------------------- the model
def forward(cfg, W, tokens, residuals=None):
    """logits [T, vocab] of one sequence from position 0; `residuals` (a list) receives the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][np.asarray(tokens)]
    kept = {}
    for il, L in enumerate(cfg["layers"]):
        p, mx, ml = "l%d." % il, L["mixer"], L.get("mlp")
        if L["type"] == "attention":
            m, kept[il] = windowed(x, mx, W, p + "mix.", eps, kept[mx["kv_from"]] if mx.get("kv_from") is not None else None)
        elif L["type"] == "attention_2":
            m = rotated_with_sink(x, mx, W, p + "mix.", eps)
        else:
            m = side_by_side(x, mx, W, p + "mix.", eps)
        x = x + over_rms(m, eps) * W[p + "norm1"]
        if ml:
            f = gated_ffn(x, W, p + "mlp.") if ml["kind"] == "dense" else experts_ffn(x, ml, W, p + "mlp.")
            x = x + over_rms(f, eps) * W[p + "norm2"]
        if residuals is not None:
            residuals.append(x.copy())
    return capped((over_rms(x, eps) * W["final.norm"]) @ W["head"].T, cfg.get("logit_softcap"))


# ---------------------------------------------------------------------------------------------------------------- making models
def bf16_round(a):
    """float array -> the nearest bfloat16 values (round to nearest even), as float64."""
    b = np.asarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    b = ((b + 0x7FFF + ((b >> 16) & 1)) >> 16 << 16).astype(np.uint32)
    return b.view(np.float32).astype(np.float64)


def tensor_shapes(cfg):
    E, V = cfg["width"], cfg["vocab"]
    sh = {"embed": (V, E), "head": (V, E), "final.norm": (E,)}
    for il, L in enumerate(cfg["layers"]):
        p, mx, ml = "l%d." % il, L["mixer"], L.get("mlp")
        m, f = p + "mix.", p + "mlp."
        sh[p + "norm1"] = (E,)
        if L["type"] == "parallel":
            a, r = mx["left"], mx["right"]
            H, G, D, taps = a["heads"], a["kv_heads"], a["dim"], a["conv"]
            m1, m2 = m + "left.", m + "right."
            sh.update({m1 + "q": (H * D, E), m1 + "q.b": (H * D,), m1 + "k": (G * D, E), m1 + "k.b": (G * D,), m1 + "q.norm": (D,), m1 + "k.norm": (D,),
                       m1 + "q.conv": (H * D, taps), m1 + "k.conv": (G * D, taps), m1 + "o": (E, H * D), m1 + "out": (E,)})
            H, Dk, Dv, rank = r["heads"], r["dim"], r["vdim"], r.get("rank", 5)
            sh.update({m2 + "q": (H * Dk, E), m2 + "k": (H * Dk, E), m2 + "v": (H * Dv, E), m2 + "g": (H * Dv, E), m2 + "o": (E, H * Dv), m2 + "norm": (Dv,),
                       m2 + "a1": (rank, E), m2 + "a2": (H * Dk, rank), m2 + "a2.b": (H * Dk,), m2 + "out": (E,)})
        else:
            H, G, Dk, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
            own = mx.get("kv_from") is None
            sh.update({m + "q": (H * Dk, E), m + "o": (E, H * Dv)})
            if own:
                sh.update({m + "k": (G * Dk, E), m + "v": (G * Dv, E)})
            if L["type"] == "attention":
                sh.update({m + "q.norm": (Dk,), m + "g": (H * Dv, E)})
                if own:
                    sh[m + "k.norm"] = (Dk,)
            else:
                sh.update({m + "sink": (H,), m + "g": (H, E)})
        if not ml:
            continue
        sh[p + "norm2"] = (E,)
        parts = {f: ml["ff"]} if ml["kind"] == "dense" else {"%se%d." % (f, e): ml["expert"]["ff"] for e in range(ml["router"]["experts"])}
        if ml["kind"] != "dense":
            sh[f + "router"] = (ml["router"]["experts"], E)
            if ml.get("shared"):
                parts[f + "shared."] = ml["shared"]["ff"]
                sh[f + "shared.sg"] = (1, E)
        for q, ff in parts.items():
            sh.update({q + "gate": (ff, E), q + "up": (ff, E), q + "down": (E, ff)})
    return sh


def random_weights(cfg, seed):
    """bf16-representable random weights with magnitudes that keep every mechanism alive (decays that differ per channel, sinks that matter, experts that differ)."""
    rng = np.random.default_rng(seed)
    W = {}
    for name, s in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        if leaf in ("norm1", "norm2", "norm", "out"):
            a = rng.uniform(0.6, 1.4, s)
        elif leaf == "conv":
            a = rng.normal(0, 0.6, s)
        elif leaf == "sink":
            a = rng.normal(0, 1.5, s)
        elif name.endswith("a2.b"):
            a = rng.normal(0.5, 1.5, s)
        elif leaf == "b":
            a = rng.normal(0, 0.3, s)
        elif name == "embed":
            a = rng.normal(0, 1.0, s)
        elif leaf in ("router", "gate", "up", "sg", "a1", "a2"):
            a = rng.normal(0, 1.5 / math.sqrt(s[-1]), s)
        else:
            a = rng.normal(0, 1.0 / math.sqrt(s[-1]), s)
        W[name] = bf16_round(a)
    return W


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, shared=None):
    ml = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        ml["shared"] = {"ff": shared}
    return ml


def banded(factor, low, high, original):
    return {"factor": factor, "low": low, "high": high, "original": original}


def ramped(factor, original, fast, slow):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def rot(dims, base, scaling=None):
    r = {"dims": dims, "base": base}
    if scaling:
        r["scaling"] = scaling
    return r


def window_layer(heads, kv_heads, dim, vdim, scale, mlp, size=None, keep_first=0, kv_from=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        mx["mask"] = {"size": size, "keep_first": keep_first}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def sink_layer(heads, kv_heads, dim, vdim, scale, r, mlp):
    return {"type": "attention_2", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": r}, "mlp": mlp}


def parallel_layer(heads, kv_heads, dim, scale, r, conv, r_heads, r_dim, r_vdim, tau, mlp, rank=5):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "rot": r, "conv": conv}
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "tau": tau, "rank": rank}}, "mlp": mlp}


def make_config(width, vocab, layers, softcap=12.0, eps=1e-5):
    cfg = {"architecture": "Nidudra", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}
    if softcap:
        cfg["logit_softcap"] = softcap
    return cfg


def save_model(cfg, W, folder):
    """config.json (the helper key 'rank' is left out: the tensors' shapes give it) + model.safetensors with every tensor as bf16."""
    os.makedirs(folder, exist_ok=True)
    out = json.loads(json.dumps(cfg))
    for L in out["layers"]:
        if L["type"] == "parallel":
            L["mixer"]["right"].pop("rank", None)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(out, f)
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
