"""Lalepel: a decoder whose layers are listed one by one in config.json; every layer has one of two mixers (softmax attention over latents
within a window, with a turned key part that all heads share and a sink; a linear attention with a constant decay per head) and an optional
feed-forward, dense or routed; norms stand behind the sub-layers only.

config.json: ``architecture`` "Lalepel"; ``vocab``, ``width``; ``norm.eps``; ``layers``: a list of {``type``, ``mixer``, ``mlp``}. Tensor names:
``embed``, ``l<i>.`` + ``norm1``, ``norm2``, ``mix.*``, ``mlp.*``; ``final.norm``, ``head``.

The model: a token's row of ``embed``. A layer: x += norm1(mixer(x)), then, unless ``mlp`` is null, x += norm2(mlp(x)), RMS norms with a weight.
The logits are the head's product of the final norm's rows.

Mixers by ``type``:
  latent_attention  ``heads`` heads of ``dim`` channels as projected and ``rot_dim`` turned ones, values of ``vdim``; queries through a latent of
                    ``q_rank`` channels, keys and values from one of ``kv_rank``; the turned channels in pairs (2i, 2i + 1) by ``rot.base``, frequencies
                    stretched by wavelength as ``rot.scaling`` {factor, original, fast, slow} says; scores times ``scale``; a row sees the last
                    ``mask.size`` keys; ``sink`` per head in the softmax's denominator.
  retention         ``heads`` x (``dim``, ``vdim``), one ``decay`` per head, no positions, a silu gate.
Feed-forward by ``mlp.kind`` (``mlp`` null: none):
  dense  gate, up and down with silu, ``ff`` wide.
  moe    ``router.experts`` experts of ``expert.ff`` channels (two matrices, the square of relu between them), of which a token takes the
         ``router.top`` with the largest logits (a bias per expert), weighted by the softmax over those; and optionally one of the same form
         that every token takes (``shared.ff``), weighted by a sigmoid of its own."""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Optional

from ..config.base import LayerSpec, ModelConfig, ModelSpec, PartSpec, RunEntry
from ..errors import AlofaError
from .tugalix import _get, _positive

MIXERS = ("latent_attention", "retention")


def _latent(m: dict, where: str) -> dict:
    out = {k: _get(m, k, int, where) for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")}
    _positive(where, **out)
    out["scale"] = _get(m, "scale", float, where)
    rot = _get(m, "rot", dict, where)
    r = {"base": _get(rot, "base", float, where), "dims": _get(rot, "dims", int, where)}
    _positive(where, base=r["base"])
    if r["dims"] != out["rot_dim"] or r["dims"] % 2:
        raise AlofaError("parse", "rot.dims is even and the size of a head's turned part", f"dims={r['dims']} rot_dim={out['rot_dim']} config={where}")
    if rot.get("scaling") is not None:
        r["scaling"] = {k: _get(rot["scaling"], k, float, where) for k in ("factor", "original", "fast", "slow")}
        _positive(where, **r["scaling"])
    out["rot"] = r
    if m.get("mask") is not None:
        out["mask"] = {"size": _get(m["mask"], "size", int, where)}
        _positive(where, size=out["mask"]["size"])
    return out


def _retention(m: dict, where: str) -> dict:
    out = {k: _get(m, k, int, where) for k in ("heads", "dim", "vdim")}
    _positive(where, **out)
    out["decay"] = [float(x) for x in _get(m, "decay", list, where)]
    if len(out["decay"]) != out["heads"]:
        raise AlofaError("parse", "one decay per head", f"heads={out['heads']} decay={len(out['decay'])} config={where}")
    return out


def _mlp(mlp, where: str):
    if mlp is None:
        return None
    kind = _get(mlp, "kind", str, where)
    if kind == "dense":
        ff = _get(mlp, "ff", int, where)
        _positive(where, ff=ff)
        return {"kind": "dense", "ff": ff}
    if kind != "moe":
        raise AlofaError("unsupported", "no such feed-forward in this design", f"kind={kind} config={where}")
    r = _get(mlp, "router", dict, where)
    router = {"experts": _get(r, "experts", int, where), "top": _get(r, "top", int, where)}
    _positive(where, **router)
    if router["top"] > router["experts"]:
        raise AlofaError("parse", "a token cannot take more experts than there are", f"top={router['top']} experts={router['experts']} config={where}")

    def sized(e):
        ff = _get(e, "ff", int, where)
        _positive(where, ff=ff)
        return {"ff": ff}
    shared = mlp.get("shared")
    return {"kind": "moe", "router": router, "expert": sized(_get(mlp, "expert", dict, where)), "shared": None if shared is None else sized(shared)}


@dataclass(frozen=True)
class LalepelConfig(ModelConfig):
    vocab: int
    width: int
    eps: float
    layers: tuple      # per layer a dict {type, mixer, mlp}, checked

    architecture = "Lalepel"

    @classmethod
    def from_dict(cls, raw: dict, where: str = "<dict>") -> "LalepelConfig":
        layers = []
        for i, l in enumerate(_get(raw, "layers", list, where)):
            at = f"{where} layers[{i}]"
            kind = _get(l, "type", str, at)
            if kind not in MIXERS:
                raise AlofaError("unsupported", "no such mixer in this design", f"type={kind} known={','.join(MIXERS)} config={at}")
            m = _get(l, "mixer", dict, at)
            layers.append({"type": kind, "mixer": _latent(m, at) if kind == "latent_attention" else _retention(m, at), "mlp": _mlp(l.get("mlp"), at)})
        if not layers:
            raise AlofaError("parse", "a model has at least one layer", f"config={where}")
        cfg = cls(vocab=_get(raw, "vocab", int, where), width=_get(raw, "width", int, where), eps=_get(_get(raw, "norm", dict, where), "eps", float, where), layers=tuple(layers))
        _positive(where, vocab=cfg.vocab, width=cfg.width, eps=cfg.eps)
        return cfg

    def to_dict(self) -> dict:
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps}, "layers": copy.deepcopy(list(self.layers))}

    # ---- the model as data
    def _norm(self, name: str, width: Optional[int] = None) -> PartSpec:
        return PartSpec("rmsnorm", {"name": name, "width": width or self.width, "eps": self.eps})

    def _mixer_spec(self, kind: str, m: dict, pre: str) -> PartSpec:
        h = self.width
        if kind == "retention":
            return PartSpec("retention", {"prefix": pre, "hidden": h, "heads": m["heads"], "key_dim": m["dim"], "value_dim": m["vdim"], "decay": tuple(m["decay"]),
                                          "position": None, "eps": self.eps})
        rot = m["rot"]
        return PartSpec("latent_attention", {
            "prefix": pre, "hidden": h, "heads": m["heads"], "head_dim": m["dim"], "v_head_dim": m["vdim"], "latent": m["kv_rank"], "scale": m["scale"],
            "latent_norm": self._norm(pre + "dkv.norm", m["kv_rank"]), "q_latent": {"rank": m["q_rank"], "norm": self._norm(pre + "dq.norm", m["q_rank"])},
            "turned": {"size": m["rot_dim"], "position": PartSpec("rotary", {"theta": rot["base"], "head_dim": m["rot_dim"], "pairing": "neighbours",
                                                                             "frequencies": "direct", "stretch": rot.get("scaling")})},
            "window": m["mask"]["size"] if m.get("mask") is not None else None, "sink": True, "gate": None,
            "names": {"q_down": "dq", "q": "uq", "down": "dkv", "up_k": "uk", "up_v": "uv", "o": "o", "sink": "sink"}})

    def _feed_forward(self, mlp, pre: str) -> Optional[PartSpec]:
        h = self.width
        if mlp is None:
            return None
        if mlp["kind"] == "dense":
            return PartSpec("swiglu", {"prefix": pre, "hidden": h, "intermediate": mlp["ff"], "names": {"gate": "gate", "up": "up", "down": "down"}, "init": "fan_in"})
        r, shared = mlp["router"], mlp["shared"]
        return PartSpec("routed_experts", {
            "prefix": pre, "hidden": h, "experts": r["experts"], "top": r["top"], "score": "softmax_chosen", "router_bias": "router.b",
            "expert": {"intermediate": mlp["expert"]["ff"]}, "shared": None if shared is None else {"intermediate": shared["ff"]},
            "shared_gate": None if shared is None else "shared.sg", "activation": "relu_squared",
            "names": {"router": "router", "expert": "e{}", "shared": "shared", "up": "up", "down": "down"}})

    def spec(self) -> ModelSpec:
        h = self.width
        layers = []
        for i, l in enumerate(self.layers):
            p = f"l{i}."
            ff = self._feed_forward(l["mlp"], p + "mlp.")
            layers.append(LayerSpec(prefix=p, block=PartSpec("postnorm", {"hidden": h}),
                                    parts=dict(mixer=self._mixer_spec(l["type"], l["mixer"], p + "mix."), feed_forward=ff,
                                               norms=tuple(self._norm(p + f"norm{s + 1}") for s in range(1 if ff is None else 2)))))
        return ModelSpec(
            hidden_size=h, vocab_size=self.vocab, max_positions=1 << 30,
            embedding=PartSpec("token_embedding", {"name": "embed", "vocab": self.vocab, "width": h, "init": "unit"}),
            layers=tuple(layers), order=tuple(RunEntry(i) for i in range(len(layers))), final_norm=self._norm("final.norm"),
            head=PartSpec("lm_head", {"name": "head", "tied_to": None, "vocab": self.vocab, "width": h, "init": "fan_in"}))
