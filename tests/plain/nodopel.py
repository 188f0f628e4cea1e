"""Plain Nodopel: whole sequences, no cache and no state carried between calls, float64 throughout, one function per
mechanism, written from the design's equations. It shares nothing with the engine.

Notation: T tokens, h the width, S streams, H query heads, G key/value heads, d a map's size, e a value head's size.
``store`` is applied wherever the engine keeps a bfloat16 tensor between kernels (the identity by default;
``to_bfloat16`` to measure what that rounding alone does)."""
from __future__ import annotations

import json
import math
from pathlib import Path

import numpy as np


def read_config(model_dir) -> dict:
    return json.loads((Path(model_dir) / "config.json").read_text())


def read_weights(model_dir) -> dict:
    """name -> float64 array, read with the safetensors library (the engine has a reader of its own)."""
    import torch
    from safetensors.torch import load_file
    return {name: t.to(torch.float64).numpy() for name, t in load_file(str(Path(model_dir) / "model.safetensors")).items()}


def to_bfloat16(x: np.ndarray) -> np.ndarray:
    """Round to nearest even at 8 bits of mantissa, through float32."""
    bits = np.asarray(x, dtype=np.float32).view(np.uint32).astype(np.uint64)
    bits = (bits + 0x7FFF + ((bits >> 16) & 1)) & 0xFFFF0000
    return bits.astype(np.uint32).view(np.float32).astype(np.float64)


def _keep(x):
    return x


# ------------------------------------------------------------------ norms and activations

def unit_rms(x, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def silu(z):
    e = np.exp(-np.abs(z))
    return z * np.where(z >= 0, 1.0, e) / (1.0 + e)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------------ positions

def frequencies(n, base, scaling=None) -> np.ndarray:
    """The n/2 angular frequencies of a turned part of n channels. With ``scaling``: as they are where ``original`` tokens hold
    more than ``high`` turns, divided by ``factor`` where they hold fewer than ``low``, and in between a blend of the two that is
    linear in the count of turns."""
    f = np.array([base ** (-2.0 * i / n) for i in range(n // 2)])
    if scaling is None:
        return f
    out = []
    for x in f:
        length = 2.0 * math.pi / x
        if length < scaling["original"] / scaling["high"]:
            out.append(x)
        elif length > scaling["original"] / scaling["low"]:
            out.append(x / scaling["factor"])
        else:
            s = (scaling["original"] / length - scaling["low"]) / (scaling["high"] - scaling["low"])
            out.append((1.0 - s) * x / scaling["factor"] + s * x)
    return np.array(out)


def turn(x, positions, rot):
    """x [T, heads, d]: the first ``dims`` channels in pairs (i, i + dims/2), turned by their row's position (a 32-bit angle); the rest pass."""
    n = rot["dims"]
    f = frequencies(n, rot["base"], rot.get("scaling")).astype(np.float32)
    a = (np.asarray(positions, dtype=np.float32)[:, None] * f[None, :]).astype(np.float64)[:, None, :]
    u, v = x[..., :n // 2], x[..., n // 2:n]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), x[..., n:]], axis=-1)


# ------------------------------------------------------------------ attention

def visible(T, mask):
    """[T, T]: row i sees j up to itself, within the last ``size`` or among the first ``keep_first`` of the sequence."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    if mask is None:
        return j <= i
    return (j <= i) & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))


def capped(s, cap):
    return s if cap is None else cap * np.tanh(s / cap)


def softmax_over(s, seen):
    s = np.where(seen, s, -np.inf)
    p = np.exp(s - s.max(axis=-1, keepdims=True))
    return p / p.sum(axis=-1, keepdims=True)


def mixing_number(W, pre, diff):
    """lambda, one number for the layer."""
    return math.exp(float((W[pre + "lq1"] * W[pre + "lk1"]).sum())) - math.exp(float((W[pre + "lq2"] * W[pre + "lk2"]).sum())) + diff


def combine_maps(a1, a2, lam, diff, eps):
    """What a head gives, from its two maps' outputs [..., e]."""
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def pieces(x, W, pre, m, store=_keep):
    """(q [T, H, 2, d], k [T, G, 2, d], turned; v [T, G, e])."""
    T, H, G, d, e = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = store(x @ W[pre + "q"].T + W[pre + "q.b"]).reshape(T, 2 * H, d)
    k = store(x @ W[pre + "k"].T + W[pre + "k.b"]).reshape(T, 2 * G, d)
    v = store(x @ W[pre + "v"].T + W[pre + "v.b"]).reshape(T, G, e)
    where = np.arange(T)
    return store(turn(q, where, m["rot"])).reshape(T, H, 2, d), store(turn(k, where, m["rot"])).reshape(T, G, 2, d), v


def differential_attention(x, W, pre, m, eps, store=_keep):
    T, H, G, e = x.shape[0], m["heads"], m["kv_heads"], m["vdim"]
    q, k, v = pieces(x, W, pre, m, store)
    seen, lam = visible(T, m.get("mask")), mixing_number(W, pre, m["diff"])
    out = np.zeros((T, H, e))
    for a in range(H):
        g = a // (H // G)
        maps = [softmax_over(capped(q[:, a, n] @ k[:, g, n].T * m["scale"], m.get("softcap")), seen) @ v[:, g] for n in range(2)]
        out[:, a] = combine_maps(maps[0], maps[1], lam, m["diff"], eps)
    return store(out.reshape(T, H * e)) @ W[pre + "o"].T


# ------------------------------------------------------------------ feed-forwards

def gated_ff(x, w_gate, w_up, w_down, act, weight=1.0, store=_keep):
    return store(weight * act(x @ w_gate.T) * (x @ w_up.T)) @ w_down.T


def route(x, w_router, correction, top):
    """(chosen [T, top], weights [T, top]): the largest softmax score + correction, the lower index among equals; their scores, made to sum to one."""
    z = x @ w_router.T
    s = np.exp(z - z.max(axis=-1, keepdims=True))
    s = s / s.sum(axis=-1, keepdims=True)
    chosen = np.argsort(-(s + correction), axis=-1, kind="stable")[:, :top]
    w = np.take_along_axis(s, chosen, axis=-1)
    return chosen, w / (w.sum(axis=-1, keepdims=True) + 1e-20)


def mixture(x, W, pre, mlp, store=_keep):
    r = mlp["router"]
    chosen, weights = route(x, W[pre + "router"], W[pre + "correction"], r["top"])
    out = np.zeros_like(x)
    for e in range(r["experts"] + r.get("identity", 0)):
        rows, place = np.nonzero(chosen == e)
        if not len(rows):
            continue
        w = weights[rows, place][:, None]
        if e >= r["experts"]:      # the row itself, handed on
            out[rows] += w * x[rows]
        else:
            out[rows] += gated_ff(x[rows], W[f"{pre}e{e}.gate"], W[f"{pre}e{e}.up"], W[f"{pre}e{e}.down"], silu, w, store)
    if mlp.get("shared"):
        out += gated_ff(x, W[pre + "shared.gate"], W[pre + "shared.up"], W[pre + "shared.down"], silu, 1.0, store)
    return out


# ------------------------------------------------------------------ streams

def read_streams(X, w_in):
    """X [T, S, h] -> what a sub-layer reads, [T, h]."""
    return np.einsum("s,tsh->th", w_in, X)


def write_streams(X, y, mix, w_out):
    """All streams at once from the old ones: stream t takes mix[s, t] of stream s, and w_out[t] of the sub-layer's result."""
    return np.einsum("st,nsh->nth", mix, X) + w_out[None, :, None] * y[:, None, :]


# ------------------------------------------------------------------ the model

def order(cfg) -> list:
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def layer(X, W, cfg, i, store=_keep):
    l, p, eps = cfg["layers"][i], f"l{i}.", cfg["norm"]["eps"]
    u = store(rms_norm(read_streams(X, W[p + "hc1.in"]), W[p + "norm1"], eps))
    X = write_streams(X, differential_attention(u, W, p + "mix.", l["mixer"], eps, store), W[p + "hc1.mix"], W[p + "hc1.out"])
    mlp = l["mlp"]
    if mlp is None:
        return X
    u = store(rms_norm(read_streams(X, W[p + "hc2.in"]), W[p + "norm2"], eps))
    if mlp["kind"] == "dense":
        y = gated_ff(u, W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"], gelu_tanh, 1.0, store)
    else:
        y = mixture(u, W, p + "mlp.", mlp, store)
    return write_streams(X, y, W[p + "hc2.mix"], W[p + "hc2.out"])


def forward_hidden(W, cfg, ids, store=_keep) -> list:
    """The sum of the streams after every layer that is run (a layer in the loop as often as it is passed), [T, h] each."""
    X, out = np.repeat(W["embed"][np.asarray(ids)][:, None, :], cfg["streams"], axis=1), []
    for i in order(cfg):
        X = layer(X, W, cfg, i, store)
        out.append(X.sum(axis=1))
    return out


def forward_logits(W, cfg, ids, store=_keep) -> np.ndarray:
    x = forward_hidden(W, cfg, ids, store)[-1]
    return store(rms_norm(x, W["final.norm"], cfg["norm"]["eps"])) @ W["embed"].T


def greedy(W, cfg, prompt, n_new) -> list:
    """n_new tokens, each the first index of the highest logit after everything before it."""
    ids, out = list(prompt), []
    for _ in range(n_new):
        out.append(int(np.argmax(forward_logits(W, cfg, ids)[-1])))
        ids.append(out[-1])
    return out


def router_margins(W, cfg, ids) -> np.ndarray:
    """Per position the smallest gap, over all passes of layers with a router, between the last choice score that is taken and the
    first that is not, in units of the two experts' softmax scores (what moves a score by rounding is proportional to it; infinite where nothing
    is left out). Positions with a small gap are the ones where rounding may change which experts a token takes."""
    out = np.full(len(ids), np.inf)
    X, eps = np.repeat(W["embed"][np.asarray(ids)][:, None, :], cfg["streams"], axis=1), cfg["norm"]["eps"]
    for i in order(cfg):
        l, p = cfg["layers"][i], f"l{i}."
        mlp = l["mlp"]
        if mlp is not None and mlp["kind"] == "moe" and mlp["router"]["top"] < len(W[p + "mlp.correction"]):
            u = rms_norm(read_streams(X, W[p + "hc1.in"]), W[p + "norm1"], eps)
            mid = write_streams(X, differential_attention(u, W, p + "mix.", l["mixer"], eps), W[p + "hc1.mix"], W[p + "hc1.out"])
            z = rms_norm(read_streams(mid, W[p + "hc2.in"]), W[p + "norm2"], eps) @ W[p + "mlp.router"].T
            s = np.exp(z - z.max(axis=-1, keepdims=True))
            s = s / s.sum(axis=-1, keepdims=True)
            by = np.argsort(-(s + W[p + "mlp.correction"]), axis=-1, kind="stable")
            c = np.take_along_axis(s + W[p + "mlp.correction"], by, axis=-1)
            s = np.take_along_axis(s, by, axis=-1)
            top = mlp["router"]["top"]
            # (any expert that is left out may be the one that comes in)
            gap = (c[:, top - 1:top] - c[:, top:]) / (s[:, top - 1:top] + s[:, top:] + 1e-30)
            out = np.minimum(out, gap.min(axis=-1))
        X = layer(X, W, cfg, i)
    return out
