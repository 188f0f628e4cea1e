"""Small Lalepel configurations for the tests, different in every size and option, and their plain logits."""
import functools

import numpy as np

from helpers import Reference
from plain import lalepel as pl


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, base, scale, window, scaling=None):
    rot = {"base": base, "dims": rot_dim}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return "latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "rot": rot, "scale": scale,
                                "mask": {"size": window}}


def _retention(dim, vdim, *decay):
    return "retention", {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, ff, shared=None):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, **({"shared": {"ff": shared}} if shared else {})}


def _config(vocab, width, eps, layers):
    return {"architecture": "Lalepel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": [{"type": t, "mixer": m, "mlp": mlp} for (t, m), mlp in layers]}


LALEPEL = {
    # every mixer and feed-forward once; values wider than keys and narrower; a layer without a feed-forward
    "A": _config(211, 64, 1e-6, [
        (_latent(3, 16, 8, 24, 40, 32, 10000.0, 0.21, 20, (4.0, 64, 8.0, 1.0)), _dense(96)),
        (_retention(16, 24, 0.9, 0.99), _moe(6, 2, 24, 40)),
        (_latent(4, 24, 16, 16, 24, 48, 700.0, 0.15, 37), None),
        (_retention(32, 16, 0.5, 0.97, 0.999), _dense(72))]),
    # nothing a multiple of eight; one head; a turned part of one pair; every expert taken (top = experts), no shared expert; one key in the window
    "B": _config(97, 52, 1e-4, [
        (_retention(7, 5, 0.8, 0.95, 0.99), _moe(3, 3, 14)),
        (_latent(1, 5, 2, 7, 9, 13, 50.0, 0.4, 11), _dense(30)),
        (_latent(3, 9, 6, 11, 10, 18, 300.0, 0.3, 1, (2.0, 16, 2.0, 1.5)), _moe(5, 1, 10, 6)),
        (_retention(10, 30, 0.99), None)]),
    # heads that run on the matrix cores: more than a block of the decode kernel takes, and few enough to share tiles; one expert per token
    "C": _config(157, 128, 1e-5, [
        (_latent(20, 16, 24, 32, 64, 40, 20000.0, 0.16, 33, (3.0, 128, 16.0, 2.0)), _moe(12, 1, 32, 48)),
        (_latent(8, 32, 32, 16, 48, 96, 5000.0, 0.12, 17), _dense(64)),
        (_retention(64, 32, 0.97, 0.99, 0.999, 0.9), _moe(4, 2, 40)),
        (_latent(7, 8, 16, 8, 16, 16, 900.0, 0.3, 50, (5.0, 32, 3.0, 1.0)), _moe(8, 3, 16, 16))]),
    # latents too wide to be a head of the attention kernels (the pages then hold every head's keys and values): heads of one size that no prefill
    # kernel is built for, values wider than keys, and an odd size
    "D": _config(130, 64, 1e-6, [
        (_latent(2, 48, 32, 80, 32, 264, 10000.0, 0.12, 25, (4.0, 64, 8.0, 1.0)), _dense(48)),
        (_latent(3, 16, 8, 40, 20, 300, 600.0, 0.25, 18), _moe(4, 2, 16, 16)),
        (_latent(2, 9, 4, 6, 12, 257, 80.0, 0.3, 40), None)]),
    # wider, in another order: a head of 256 channels, four experts of sixteen, a long window
    "E": _config(401, 320, 1e-5, [
        (_retention(48, 80, 0.95, 0.99, 0.995, 0.9985, 0.9999), _moe(16, 4, 72, 104)),
        (_latent(7, 64, 48, 96, 128, 200, 150000.0, 0.09, 130, (6.0, 512, 24.0, 2.0)), _moe(16, 4, 72, 104)),
        (_latent(10, 32, 32, 48, 96, 64, 30000.0, 0.13, 65), _dense(384)),
        (_retention(128, 64, 0.98, 0.999), _moe(10, 5, 64, 40))]),
}


@functools.lru_cache(maxsize=None)
def plain_model(model_dir):
    return pl.read_config(model_dir), pl.read_weights(model_dir)


@functools.lru_cache(maxsize=64)
def _logits(model_dir, ids, rounded):
    cfg, w = plain_model(model_dir)
    return pl.forward_logits(w, cfg, list(ids), store=pl.to_bfloat16 if rounded else (lambda x: x)).astype(np.float32)


def plain_logits(model_dir, ids):
    ref = _logits(str(model_dir), tuple(ids), False).view(Reference)
    ref._rounded = lambda: _logits(str(model_dir), tuple(ids), True)
    return ref


@functools.lru_cache(maxsize=64)
def _margins(model_dir, ids):
    cfg, w = plain_model(model_dir)
    return pl.router_margins(w, cfg, list(ids))


def clear_calls(model_dir, ids, dtype, threshold=0.04):
    """The positions to compare: all of them in float32; in bfloat16 those at which no router's call is so close that rounding the
    activations may change which experts the token takes (such a change is no fault, and moves logits by far more than the bound measured
    from rounding allows)."""
    if dtype == "float32":
        return np.arange(len(ids))
    return np.flatnonzero(_margins(str(model_dir), tuple(ids)) >= threshold)
