"""Nodopel: a decoder whose layers are listed one by one in config.json, on several copies of the residual stream that every sub-layer reads as a weighted
sum and writes by mixing; attention with two maps per head, one taken from the other, within a window that keeps the sequence's first tokens in sight; dense or
routed feed-forwards; a run of layers that is passed through several times.

config.json: ``architecture`` "Nodopel"; ``vocab``, ``width``; ``norm.eps``; ``streams``; ``loop``: {``start``, ``stop``, ``times``}; ``layers``: a list of {``type``,
``mixer``, ``mlp``}. Tensor names: ``embed``, ``l<i>.`` + ``norm1``, ``norm2``, ``hc1.*``, ``hc2.*`` (``in``, ``mix``, ``out``), ``mix.*``, ``mlp.*``; ``final.norm``.

The model: ``streams`` copies of a token's row of ``embed``. A sub-layer q (1: mixer, 2: feed-forward) reads norm<q>(sum_s in[s] x_s), and what it gives, y, goes
into x_v <- sum_s mix[s, v] x_s + out[v] y. The layers ``loop.start`` .. ``loop.stop`` - 1 run ``loop.times`` times one after the other with the same weights, every pass
with a cache of its own. The logits are the embedding table's product with the final norm of the copies' sum.

Mixer by ``type``:
  attention  ``heads`` query and ``kv_heads`` key/value heads; queries and keys in two maps of ``dim`` channels, values of ``vdim``; biases on all three; the first ``rot.dims``
             channels of every map turned in pairs (i, i + dims/2) by ``rot.base``, frequencies blended by their turns as ``rot.scaling`` {factor, low, high, original} says;
             scores times ``scale``, capped by ``softcap``; a row sees the last ``mask.size`` keys and the sequence's first ``mask.keep_first``; ``diff`` in the maps' difference.
Feed-forward by ``mlp.kind`` (``mlp`` null: none):
  dense  gate, up and down with the tanh form of gelu, ``ff`` wide.
  moe    ``router.experts`` experts with silu gates, ``expert.ff`` wide, and ``router.identity`` ones behind them that hand the row on, of which a token takes the
         ``router.top`` with the largest softmax score + ``correction``, weighted by their scores made to sum to one; and optionally one that every token takes (``shared.ff``)."""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Optional

from ..config.base import LayerSpec, ModelConfig, ModelSpec, PartSpec, RunEntry
from ..errors import AlofaError
from .tugalix import _get, _positive

MIXERS = ("attention",)


def _attention(m: dict, where: str) -> dict:
    out = {k: _get(m, k, int, where) for k in ("heads", "kv_heads", "dim", "vdim")}
    _positive(where, **out)
    if out["heads"] % out["kv_heads"]:
        raise AlofaError("parse", "kv_heads must divide heads", f"heads={out['heads']} kv_heads={out['kv_heads']} config={where}")
    out["scale"], out["diff"] = _get(m, "scale", float, where), _get(m, "diff", float, where)
    if m.get("softcap") is not None:
        out["softcap"] = _get(m, "softcap", float, where)
        _positive(where, softcap=out["softcap"])
    rot = _get(m, "rot", dict, where)
    r = {"base": _get(rot, "base", float, where), "dims": _get(rot, "dims", int, where)}
    _positive(where, base=r["base"], dims=r["dims"])
    if r["dims"] % 2 or r["dims"] > out["dim"]:
        raise AlofaError("parse", "rot.dims is even and at most the head's size", f"dims={r['dims']} dim={out['dim']} config={where}")
    if rot.get("scaling") is not None:
        r["scaling"] = {k: _get(rot["scaling"], k, float, where) for k in ("factor", "low", "high", "original")}
        _positive(where, **r["scaling"])
        if r["scaling"]["low"] > r["scaling"]["high"]:
            raise AlofaError("parse", "the scaling's low bound lies below the high one", f"low={r['scaling']['low']} high={r['scaling']['high']} config={where}")
    out["rot"] = r
    if m.get("mask") is not None:
        mask = {"size": _get(m["mask"], "size", int, where), "keep_first": _get(m["mask"], "keep_first", int, where) if m["mask"].get("keep_first") is not None else 0}
        _positive(where, size=mask["size"])
        if mask["keep_first"] < 0:
            raise AlofaError("parse", "a count of kept tokens is not negative", f"keep_first={mask['keep_first']} config={where}")
        out["mask"] = mask
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
    router["identity"] = _get(r, "identity", int, where) if r.get("identity") is not None else 0
    if router["identity"] < 0 or router["top"] > router["experts"] + router["identity"]:
        raise AlofaError("parse", "a token cannot take more experts than there are", f"top={router['top']} experts={router['experts']} identity={router['identity']} config={where}")

    def sized(e):
        ff = _get(e, "ff", int, where)
        _positive(where, ff=ff)
        return {"ff": ff}
    shared = mlp.get("shared")
    return {"kind": "moe", "router": router, "expert": sized(_get(mlp, "expert", dict, where)), "shared": None if shared is None else sized(shared)}


@dataclass(frozen=True)
class NodopelConfig(ModelConfig):
    vocab: int
    width: int
    eps: float
    streams: int
    loop: Optional[tuple]        # (start, stop, times), or None: every layer once
    layers: tuple                # per layer a dict {type, mixer, mlp}, checked

    architecture = "Nodopel"

    @classmethod
    def from_dict(cls, raw: dict, where: str = "<dict>") -> "NodopelConfig":
        layers = []
        for i, l in enumerate(_get(raw, "layers", list, where)):
            at = f"{where} layers[{i}]"
            kind = _get(l, "type", str, at)
            if kind not in MIXERS:
                raise AlofaError("unsupported", "no such mixer in this design", f"type={kind} known={','.join(MIXERS)} config={at}")
            layers.append({"type": kind, "mixer": _attention(_get(l, "mixer", dict, at), at), "mlp": _mlp(l.get("mlp"), at)})
        if not layers:
            raise AlofaError("parse", "a model has at least one layer", f"config={where}")
        loop = raw.get("loop")
        if loop is not None:
            loop = (_get(loop, "start", int, where), _get(loop, "stop", int, where), _get(loop, "times", int, where))
            if not (0 <= loop[0] < loop[1] <= len(layers) and loop[2] >= 1):
                raise AlofaError("parse", "loop names a run of existing layers and a positive count", f"loop={loop} layers={len(layers)} config={where}")
        cfg = cls(vocab=_get(raw, "vocab", int, where), width=_get(raw, "width", int, where), eps=_get(_get(raw, "norm", dict, where), "eps", float, where),
                  streams=_get(raw, "streams", int, where), loop=loop, layers=tuple(layers))
        _positive(where, vocab=cfg.vocab, width=cfg.width, eps=cfg.eps, streams=cfg.streams)
        return cfg

    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps}, "streams": self.streams, "layers": copy.deepcopy(list(self.layers))}
        if self.loop is not None:
            out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return out

    # ---- the model as data
    def _norm(self, name: str) -> PartSpec:
        return PartSpec("rmsnorm", {"name": name, "width": self.width, "eps": self.eps})

    def _mixer_spec(self, m: dict, pre: str) -> PartSpec:
        rot, mask = m["rot"], m.get("mask") or {}
        return PartSpec("differential_attention", {
            "prefix": pre, "hidden": self.width, "heads": m["heads"], "kv_heads": m["kv_heads"], "head_dim": m["dim"], "v_head_dim": m["vdim"], "scale": m["scale"],
            "window": mask.get("size"), "keep_first": mask.get("keep_first", 0), "softcap": m.get("softcap"), "diff": m["diff"], "eps": self.eps, "biases": True,
            "position": PartSpec("rotary", {"theta": rot["base"], "head_dim": m["dim"] + m["dim"] % 2, "dims": rot["dims"], "pairing": "half", "frequencies": "direct", "blend": rot.get("scaling")})})

    def _feed_forward(self, mlp, pre: str) -> Optional[PartSpec]:
        if mlp is None:
            return None
        if mlp["kind"] == "dense":
            return PartSpec("swiglu", {"prefix": pre, "hidden": self.width, "intermediate": mlp["ff"], "activation": "gelu_tanh", "names": {"gate": "gate", "up": "up", "down": "down"}, "init": "fan_in"})
        r, shared = mlp["router"], mlp["shared"]
        return PartSpec("routed_experts", {
            "prefix": pre, "hidden": self.width, "experts": r["experts"], "top": r["top"], "score": "softmax", "correction": "correction", "passing": r["identity"], "renormalize": True,
            "expert": {"intermediate": mlp["expert"]["ff"]}, "shared": None if shared is None else {"intermediate": shared["ff"]}, "activation": "silu_glu",
            "names": {"router": "router", "expert": "e{}", "shared": "shared", "gate": "gate", "up": "up", "down": "down"}})

    def _order(self) -> tuple:
        n = len(self.layers)
        if self.loop is None:
            return tuple(RunEntry(i) for i in range(n))
        a, b, times = self.loop
        return tuple(RunEntry(i) for i in (*range(a), *(i for _ in range(times) for i in range(a, b)), *range(b, n)))

    def spec(self) -> ModelSpec:
        h = self.width
        layers = []
        for i, l in enumerate(self.layers):
            p = f"l{i}."
            ff = self._feed_forward(l["mlp"], p + "mlp.")
            subs = range(1, 2 if ff is None else 3)
            layers.append(LayerSpec(
                prefix=p, block=PartSpec("hyper_connected", {"hidden": h, "streams": self.streams, "names": tuple(tuple(f"{p}hc{q}.{n}" for n in ("in", "mix", "out")) for q in subs)}),
                parts=dict(mixer=self._mixer_spec(l["mixer"], p + "mix."), feed_forward=ff, norms=tuple(self._norm(f"{p}norm{q}") for q in subs))))
        return ModelSpec(
            hidden_size=h, vocab_size=self.vocab, max_positions=1 << 30,
            embedding=PartSpec("token_embedding", {"name": "embed", "vocab": self.vocab, "width": h, "init": "unit"}),
            layers=tuple(layers), order=self._order(), final_norm=self._norm("final.norm"),
            head=PartSpec("lm_head", {"name": "head", "tied_to": "embed", "vocab": self.vocab, "width": h}), streams=self.streams)
