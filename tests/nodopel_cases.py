"""Small Nodopel configurations for the tests, different in every size and option, and their plain logits."""
import functools

import numpy as np

from helpers import Reference
from plain import nodopel as pl


def _mixer(heads, kv, dim, vdim, dims, base, scale, diff, cap=None, window=None, keep=0, scaling=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff, "rot": {"base": base, "dims": dims}}
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    if cap is not None:
        m["softcap"] = cap
    if window is not None:
        m["mask"] = {"size": window, "keep_first": keep}
    return m


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, ff, identity=0, shared=None):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "identity": identity}, "expert": {"ff": ff}, **({"shared": {"ff": shared}} if shared else {})}


def _config(vocab, width, eps, streams, loop, layers):
    return {"architecture": "Nodopel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "streams": streams,
            **({"loop": dict(zip(("start", "stop", "times"), loop))} if loop else {}), "layers": [{"type": "attention", "mixer": m, "mlp": mlp} for m, mlp in layers]}


NODOPEL = {
    # a head of the matrix-core kernels; a loop in the middle; every feed-forward, and none; frequencies kept, blended and slowed down
    "A": _config(211, 64, 1e-6, 3, (1, 3, 2), [
        (_mixer(4, 2, 16, 32, 12, 500.0, 0.3, 0.25, 20.0, 20, 5, (3.0, 1.0, 4.0, 64)), _dense(96)),
        (_mixer(6, 3, 16, 32, 16, 10000.0, 0.22, 0.5, 50.0, 37, 21, (8.0, 2.0, 6.0, 256)), _moe(6, 2, 24, 2, 40)),
        (_mixer(4, 4, 16, 32, 8, 100.0, 0.25, 0.8, None, 16, 16), None),
        (_mixer(2, 1, 16, 32, 16, 3000.0, 0.2, 0.1, 90.0, 33), _moe(8, 3, 16, 1))]),
    # nothing a multiple of eight, odd heads; one copy of the stream; no loop; every expert taken, no identity expert; a window of one key with kept ones, and no window at all
    "B": _config(97, 52, 1e-4, 1, None, [
        (_mixer(3, 1, 7, 9, 6, 50.0, 0.45, 0.3, 8.0, 11, 18, (2.0, 0.5, 2.0, 24)), _moe(3, 3, 14)),
        (_mixer(2, 2, 5, 13, 2, 300.0, 0.5, 0.6, 30.0, 1, 3), _dense(30)),
        (_mixer(5, 5, 10, 6, 4, 80.0, 0.3, 0.2), _moe(5, 1, 10, 2, 6))]),
    # more heads a key head than a decode block takes; the whole model in a loop; two copies
    "C": _config(157, 128, 1e-5, 2, (0, 3, 3), [
        (_mixer(20, 1, 16, 32, 16, 20000.0, 0.2, 0.3, 40.0, 33, 4, (4.0, 1.0, 4.0, 128)), _dense(64)),
        (_mixer(8, 2, 32, 64, 24, 5000.0, 0.16, 0.45, 60.0, 17, 40), _moe(12, 3, 32, 4, 48)),
        (_mixer(6, 6, 24, 48, 16, 900.0, 0.18, 0.2, 25.0, 50, 16, (5.0, 1.5, 3.0, 32)), _dense(72))]),
    # values narrower and wider than both maps (widened heads), a map too wide for the matrix-core kernels; four copies; kept tokens and no loop
    "D": _config(130, 64, 1e-6, 4, None, [
        (_mixer(2, 1, 40, 80, 40, 10000.0, 0.15, 0.3, 35.0, 25, 7, (4.0, 1.0, 4.0, 64)), _dense(48)),
        (_mixer(3, 3, 16, 72, 8, 600.0, 0.25, 0.4, 50.0, 18, 30), _moe(4, 2, 16, 1, 16)),
        (_mixer(4, 2, 48, 16, 30, 80.0, 0.12, 0.3, 20.0, 40, 9), _dense(40)),
        (_mixer(2, 1, 132, 20, 64, 2000.0, 0.1, 0.35, 50.0, 30, 6), None)]),
    # wider, heads of 128, 192 and 256 channels, sixteen experts of which a token takes four, a long window
    "E": _config(401, 320, 1e-5, 4, (1, 2, 2), [
        (_mixer(4, 2, 64, 128, 64, 150000.0, 0.11, 0.3, 50.0, 130, 20, (6.0, 1.0, 4.0, 512)), _dense(384)),
        (_mixer(8, 2, 64, 128, 32, 30000.0, 0.12, 0.5, 30.0, 65, 70), _moe(16, 4, 72, 4, 104)),
        (_mixer(2, 1, 96, 192, 96, 10000.0, 0.1, 0.2, None, 100, 33), _moe(16, 4, 40)),
        (_mixer(2, 2, 128, 256, 128, 500000.0, 0.09, 0.3, 45.0, 90, 50), _dense(200))]),
}


def write_model(cfg, out_dir, seed, change=None):
    """A model folder with random weights whose routers' corrections are far apart, so that they decide many calls and few are close;
    ``change``(weights) may alter more."""
    import torch
    from alofa_amd.weights import write_random_model
    from safetensors.torch import load_file, save_file
    d = write_random_model(cfg, out_dir, seed=seed)
    w = load_file(str(d / "model.safetensors"))
    for n in w:
        if n.endswith("correction"):
            w[n] = (0.12 * torch.argsort(w[n].float(), stable=True).float()).to(w[n].dtype)
    if change is not None:
        change(w)
    save_file(w, str(d / "model.safetensors"))
    return d


# per configuration a seed with which rounding the activations changes no router's call in the main tests' prompts
SEEDS = {"A": 121, "B": 8, "C": 22, "D": 15, "E": 3}


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


def clear_calls(model_dir, ids, dtype, threshold=0.03):
    """The positions to compare: all of them in float32; in bfloat16 those at which no router's call is so close that rounding the
    activations may change which experts the token takes (such a change is no fault, and moves logits by far more than the bound measured
    from rounding allows)."""
    if dtype == "float32":
        return np.arange(len(ids))
    return np.flatnonzero(_margins(str(model_dir), tuple(ids)) >= threshold)
