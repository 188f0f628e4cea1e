"""Plain Lalepel: whole sequences, no cache and no state carried between calls, float64 throughout, one function per
mechanism, written from the design's equations. It shares nothing with the engine.

Notation: T tokens, h the width, H heads, r the size of the keys' latent, n the size of a head's turned part.
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


# ------------------------------------------------------------------ mechanisms

def unit_rms(x, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def frequencies(n, base, scaling=None) -> np.ndarray:
    """The n/2 angular frequencies of a turned part of n channels; with ``scaling``, long wavelengths are slowed down by
    ``factor``, short ones are not, with a straight ramp over the pair's number in between."""
    f = np.array([base ** (-2.0 * i / n) for i in range(n // 2)])
    if scaling is None:
        return f

    def pair_that_turns(times):
        return n * math.log(scaling["original"] / (2.0 * math.pi * times)) / (2.0 * math.log(base))
    lo = max(math.floor(pair_that_turns(scaling["fast"])), 0)
    hi = min(math.ceil(pair_that_turns(scaling["slow"])), n - 1)
    ramp = np.clip((np.arange(n // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1.0 - ramp)


def turn(x, positions, base, scaling=None):
    """x [T, ..., n]: neighbours (2i, 2i + 1) turned by their row's position; the angle is a 32-bit number."""
    n = x.shape[-1]
    f = frequencies(n, base, scaling).astype(np.float32)
    a = (np.asarray(positions, dtype=np.float32)[:, None] * f[None, :]).astype(np.float64)
    m = 1.0 if scaling is None else 0.1 * math.log(scaling["factor"]) + 1.0
    shape = (x.shape[0],) + (1,) * (x.ndim - 2) + (n // 2,)
    c, s = (m * np.cos(a)).reshape(shape), (m * np.sin(a)).reshape(shape)
    u, v = x[..., 0::2], x[..., 1::2]
    out = np.empty_like(x)
    out[..., 0::2], out[..., 1::2] = u * c - v * s, v * c + u * s
    return out


def latent_pieces(x, W, pre, m, eps, store=_keep):
    """(queries [T, H, dim], turned queries [T, H, n], the latents [T, r], the turned key part [T, n] that all heads share)."""
    T, H, dim, n, r = x.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    base, scaling, where = m["rot"]["base"], m["rot"].get("scaling"), np.arange(T)
    cq = store(rms_norm(store(x @ W[pre + "dq"].T), W[pre + "dq.norm"], eps))
    q = store(cq @ W[pre + "uq"].T).reshape(T, H, dim + n)
    down = store(x @ W[pre + "dkv"].T)
    c = store(rms_norm(down[:, :r], W[pre + "dkv.norm"], eps))
    return q[:, :, :dim], store(turn(q[:, :, dim:], where, base, scaling)), c, store(turn(down[:, r:], where, base, scaling))


def latent_attention(x, W, pre, m, eps, store=_keep):
    """Queries through a normed latent; keys and values made of another latent, plus one turned key part for all heads; a row
    sees itself and the size - 1 tokens before it; exp(sink) of the head joins the softmax's denominator."""
    T, H, dim, dv = x.shape[0], m["heads"], m["dim"], m["vdim"]
    qn, qr, c, kr = latent_pieces(x, W, pre, m, eps, store)
    kn = store(c @ W[pre + "uk"].T).reshape(T, H, dim)
    v = store(c @ W[pre + "uv"].T).reshape(T, H, dv)
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    size = m["mask"]["size"] if m.get("mask") else T
    seen = (i - j >= 0) & (i - j < size)
    out = np.zeros((T, H, dv))
    for a in range(H):
        s = np.where(seen, (qn[:, a] @ kn[:, a].T + qr[:, a] @ kr.T) * m["scale"], -np.inf)
        sink = W[pre + "sink"][a]
        top = np.maximum(s.max(axis=1), sink)
        p = np.exp(s - top[:, None])
        out[:, a] = (p / (p.sum(axis=1) + np.exp(sink - top))[:, None]) @ v[:, a]
    return store(out.reshape(T, H * dv)) @ W[pre + "o"].T


def retention(x, W, pre, m, eps, store=_keep):
    """S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, one decay per head; o over its root mean square, times silu(g)."""
    T, H, dk, dv = x.shape[0], m["heads"], m["dim"], m["vdim"]
    q = store(x @ W[pre + "q"].T).reshape(T, H, dk)
    k = store(x @ W[pre + "k"].T).reshape(T, H, dk) * dk ** -0.5
    v = store(x @ W[pre + "v"].T).reshape(T, H, dv)
    decay = np.asarray(m["decay"], dtype=np.float64)[:, None, None]
    S, o = np.zeros((H, dk, dv)), np.zeros((T, H, dv))
    for t in range(T):
        S = decay * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(axis=1)
    g = store(x @ W[pre + "g"].T)
    return store(unit_rms(o, eps).reshape(T, H * dv) * silu(g)) @ W[pre + "o"].T


def gated_ff(x, w_gate, w_up, w_down, store=_keep):
    return store(silu(x @ w_gate.T) * (x @ w_up.T)) @ w_down.T


def expert(x, w_up, w_down, weight=1.0, store=_keep):
    """weight * down(max(up x, 0)^2)"""
    return store(weight * np.maximum(x @ w_up.T, 0.0) ** 2) @ w_down.T


def route(x, w_router, bias, top):
    """(chosen [T, top], weights [T, top]): the largest logits, the lower index among equals; the softmax over those alone."""
    z = x @ w_router.T + bias
    chosen = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    zc = np.take_along_axis(z, chosen, axis=-1)
    e = np.exp(zc - zc.max(axis=-1, keepdims=True))
    return chosen, e / e.sum(axis=-1, keepdims=True)


def mixture(x, W, pre, mlp, store=_keep):
    chosen, weights = route(x, W[pre + "router"], W[pre + "router.b"], mlp["router"]["top"])
    out = np.zeros_like(x)
    for e in range(mlp["router"]["experts"]):
        rows, place = np.nonzero(chosen == e)
        if len(rows):
            out[rows] += expert(x[rows], W[f"{pre}e{e}.up"], W[f"{pre}e{e}.down"], weights[rows, place][:, None], store)
    if mlp.get("shared"):
        gate = sigmoid(x @ W[pre + "shared.sg"].T)
        out += expert(x, W[pre + "shared.up"], W[pre + "shared.down"], gate, store)
    return out


# ------------------------------------------------------------------ the model

MIXERS = {"latent_attention": latent_attention, "retention": retention}


def layer(x, W, cfg, i, store=_keep):
    l, p, eps = cfg["layers"][i], f"l{i}.", cfg["norm"]["eps"]
    y = MIXERS[l["type"]](store(x), W, p + "mix.", l["mixer"], eps, store)
    x = x + rms_norm(y, W[p + "norm1"], eps)
    mlp = l["mlp"]
    if mlp is None:
        return x
    if mlp["kind"] == "dense":
        y = gated_ff(store(x), W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"], store)
    else:
        y = mixture(store(x), W, p + "mlp.", mlp, store)
    return x + rms_norm(y, W[p + "norm2"], eps)


def forward_hidden(W, cfg, ids, store=_keep) -> list:
    """The stream after every layer, [T, h] each."""
    x, out = W["embed"][np.asarray(ids)], []
    for i in range(len(cfg["layers"])):
        x = layer(x, W, cfg, i, store)
        out.append(x)
    return out


def forward_logits(W, cfg, ids, store=_keep) -> np.ndarray:
    x = forward_hidden(W, cfg, ids, store)[-1]
    return store(rms_norm(x, W["final.norm"], cfg["norm"]["eps"])) @ W["head"].T


def greedy(W, cfg, prompt, n_new) -> list:
    """n_new tokens, each the first index of the highest logit after everything before it."""
    ids, out = list(prompt), []
    for _ in range(n_new):
        out.append(int(np.argmax(forward_logits(W, cfg, ids)[-1])))
        ids.append(out[-1])
    return out


def router_margins(W, cfg, ids) -> np.ndarray:
    """Per position the smallest gap, over all layers with a router, between the last router product that is taken and the
    first that is not, in units of the products' spread at that position (infinite where nothing is left out). Positions
    with a small gap are the ones where rounding may change which experts a token takes."""
    out = np.full(len(ids), np.inf)
    x, eps = W["embed"][np.asarray(ids)], cfg["norm"]["eps"]
    for i, l in enumerate(cfg["layers"]):
        p, mlp = f"l{i}.", l["mlp"]
        if mlp is not None and mlp["kind"] == "moe" and mlp["router"]["top"] < mlp["router"]["experts"]:
            mid = x + rms_norm(MIXERS[l["type"]](x, W, p + "mix.", l["mixer"], eps), W[p + "norm1"], eps)
            z = np.sort(mid @ W[p + "mlp.router"].T + W[p + "mlp.router.b"], axis=-1)[:, ::-1]
            top = mlp["router"]["top"]
            out = np.minimum(out, (z[:, top - 1] - z[:, top]) / (z.std(axis=-1) + 1e-30))
        x = layer(x, W, cfg, i)
    return out
