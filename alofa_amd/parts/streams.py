"""Several copies of the residual stream instead of one (hyper-connections).

A model of S copies (``ModelSpec.streams``) starts every copy as the embedding's output. Around every sub-layer:
  u = sum_s in[s] x_s;  y = sub-layer(norm(u));  x_v <- sum_s mix[s, v] x_s + out[v] y, all copies at once from the old ones
with vectors ``in`` and ``out`` [S] and a matrix ``mix`` [S, S] (from, to) per sub-layer. What leaves the last layer is the sum of the copies.

The copies are float32 and lie side by side, [T, S, h]. A sub-layer leaves its result apart, and one launch mixes it in and leaves what the next
reader starts from (``StreamRead``): the next sub-layer's normed rows, the next block's, or, behind the last block, the sum of the copies."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from .. import ops
from ..errors import AlofaError
from ..weights.loader import TensorRule
from .base import Block, build_part, register_part, tensors_of


@dataclass(frozen=True)
class StreamRead:
    """How a reader sees the copies: their weighted sum, through an RMSNorm (weight, eps) or as it is. ``last``: nobody reads the copies again."""
    weights: torch.Tensor
    norm: Optional[tuple] = None
    last: bool = False


class HyperConnectedBlock(Block):
    """Pre-norm sub-layers on several copies of the stream. It reads the layer's parts ``mixer``, ``feed_forward`` (may be None) and ``norms``
    (one RMSNorm per sub-layer). params: hidden, streams, names: per sub-layer the tensors' names (in, mix, out)."""
    on_streams = True
    takes_normed = True

    @classmethod
    def layer_tensors(cls, layer) -> dict:
        out = {}
        for n in layer.part("norms"):
            out.update(tensors_of("norm", n))
        out.update(tensors_of("mixer", layer.part("mixer")))
        if layer.part("feed_forward") is not None:
            out.update(tensors_of("feed_forward", layer.part("feed_forward")))
        s = layer.block.params["streams"]
        for w_in, mix, w_out in layer.block.params["names"]:
            out.update({w_in: TensorRule((s,), "average"), mix: TensorRule((s, s), "head_mix"), w_out: TensorRule((s,), "near_one")})
        return out

    def __init__(self, layer, weights, rt):
        super().__init__(layer, weights, rt)
        ff, norms, names = layer.part("feed_forward"), layer.part("norms"), layer.block.params["names"]
        subs = 1 if ff is None else 2
        self.streams = int(layer.block.params["streams"])
        if len(norms) != subs or len(names) != subs:
            raise AlofaError("invalid_argument", "one norm and one set of mixing weights per sub-layer", f"prefix={layer.prefix} sub-layers={subs} norms={len(norms)} mixes={len(names)}")
        if not 1 <= self.streams <= ops.MAX_STREAMS:
            raise AlofaError("unsupported", f"one to {ops.MAX_STREAMS} copies of the stream", f"prefix={layer.prefix} streams={self.streams}")
        self.norms = [build_part("norm", n, weights, rt) for n in norms]
        if any(n.as_rmsnorm() is None for n in self.norms):
            raise AlofaError("unsupported", "copies of the stream are read through an RMSNorm", f"prefix={layer.prefix}")
        self.mixer = build_part("mixer", layer.part("mixer"), weights, rt)
        self.feed_forward = build_part("feed_forward", ff, weights, rt) if ff is not None else None
        self.mix = [rt.vector(weights[m]) for _, m, _ in names]
        self.w_out = [rt.vector(weights[o]) for _, _, o in names]
        self.w_in = [rt.vector(weights[i]) for i, _, _ in names]
        self.reads = [StreamRead(w, n.as_rmsnorm()) for w, n in zip(self.w_in, self.norms)]
        self.parts = [p for p in (*self.norms, self.mixer, self.feed_forward) if p is not None]

    def mixers(self):
        return self.mixer.stateful_parts()

    def wants_normed(self, rows):
        return self.reads[0]

    def can_leave(self, norm):
        return isinstance(norm, StreamRead)

    def _write(self, x, y, sub, read=None, rows=None, slots=None):
        """The sub-layer's result (``y``, or a mixture's ``slots``) into the copies; ``rows`` afterwards holds what ``read`` sees of them."""
        ops.streams_step(x, y=None if slots is not None else y, slots=slots, mix=self.mix[sub], w_out=self.w_out[sub], w_in=read.weights if read else None, norm=read.norm if read else None, out=rows,
                         write=read is None or not read.last, exact=self.rt.exact)

    def forward(self, ctx, entry, x, normed=None, then=None):
        """``x``: the copies [T, S, h]. ``normed``: the first sub-layer's rows, where the step before has left them; ``then`` = (read, rows): what
        the next reader starts from, to be left in ``rows``. Returns whether that was done."""
        shape = (x.shape[0], x.shape[2])
        buf, apart = ctx.scratch("normed", shape, self.rt.dtype), ctx.scratch("sub_out", shape, torch.float32)
        if normed is None:
            ops.streams_step(x, w_in=self.w_in[0], norm=self.reads[0].norm, out=buf, write=False, exact=self.rt.exact)
            normed = buf
        slots = None
        self.mixer.forward(ctx, (entry, 0), normed, apart, out=apart)
        if self.feed_forward is not None:
            self._write(x, apart, 0, self.reads[1], buf)
            if hasattr(self.feed_forward, "forward_slots"):      # (the launch that mixes the result in adds the experts' results up)
                slots = self.feed_forward.forward_slots(ctx, buf, apart)
            else:
                self.feed_forward.forward(ctx, buf, apart, out=apart)
        self._write(x, apart, len(self.mix) - 1, *(then or (None, None)), slots=slots)
        return then is not None


register_part("block", "hyper_connected", HyperConnectedBlock)
