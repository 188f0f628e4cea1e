"""Feed-forwards of which a token takes a few: a router scores the experts, the token takes the best ``top`` of them, and
what they give is summed with weights that follow from the scores; an expert that every token takes may stand beside them.

Router: z = x W_r^T in float32; the score is sigmoid(z); the ``top`` largest are taken (the lower index among equals);
the weights are the taken scores (made to sum to one first where the design says so) times ``weight_scale``.
Expert ("clamped_glu"): a = min(gate(x), limit), b = clamp(up(x), -limit, limit); down(a sigmoid(slope a) (b + 1)).

Another router ("softmax"): the score is softmax(z) over all experts; the choice goes by score + ``correction`` (a tensor), within the
``groups.keep`` best of ``groups.count`` groups of neighbouring experts (a group's score: its largest member's); the weights are the
scores themselves. The last ``passing`` experts of such a router have no matrices: they hand the row on, times their weight.
A third router ("softmax_chosen"): the ``top`` largest z + ``router_bias`` (a tensor) are taken; the weights are the softmax over those alone.
Another expert ("silu_glu"): down(silu(gate(x)) up(x)). A third ("relu_squared"): down(max(up(x), 0)^2), no gate matrix.
The expert that every token takes may have a gate of its own (``shared_gate``, a tensor [1, hidden]): it is then weighted by sigmoid(gate x),
which the router's product forms beside the scores.

The experts' matrices lie side by side in one tensor each (gate and up by rows, down by columns, the shared expert's
last), so that every expert is a slice of them."""
from __future__ import annotations

import os

import torch

from .. import ops
from ..errors import AlofaError
from ..weights.loader import TensorRule
from .base import FeedForward, register_part


SPARSE_EXPERTS = os.environ.get("ALOFA_SPARSE_EXPERTS", "1") != "0"      # 0 (for measurements): every expert against every row


class RoutedExperts(FeedForward):
    """params: prefix, hidden, experts, top, score ("sigmoid"), weight_scale, renormalize, expert {intermediate, limit},
    shared (the same, or None), activation ("clamped_glu"), slope, names (after the prefix: router; expert, a pattern with {}
    for the expert's number; shared; gate, up, down after an expert's name and a dot).
    Optional: correction (a tensor's name after the prefix, [experts + passing]), groups {count, keep}, passing (experts without
    matrices behind the others; the router has experts + passing outputs), router_init (the rule random router weights are drawn by), router_bias and shared_gate (tensor names after the prefix).
    ``forward(..., scale=)`` with a float32 vector: what is added to the stream is multiplied by it channel by channel;
    ``forward(..., out=)``: the result is stored there (float32, the stream's shape) and the stream left alone;
    ``forward(..., post=)`` (weight, eps, rows or None): the result passes this RMSNorm before it joins the stream, whose new rows are left in
    ``rows`` in the activation dtype."""
    capturable = True
    takes_channel_scale = True
    takes_post_norm = True

    @staticmethod
    def _expert_names(p, e) -> dict:
        n = p["names"]
        stem = p["prefix"] + (n["shared"] if e is None else n["expert"].format(e)) + "."
        return {k: stem + n[k] for k in (("up", "down") if p.get("activation") == "relu_squared" else ("gate", "up", "down"))}

    @staticmethod
    def _expert_rules(names, i, h) -> dict:
        return {name: TensorRule((h, i) if k == "down" else (i, h), "fan_in") for k, name in names.items()}

    @classmethod
    def tensors(cls, spec):
        p = spec.params
        h = p["hidden"]
        out = {}
        for e in range(p["experts"]):
            out.update(cls._expert_rules(cls._expert_names(p, e), p["expert"]["intermediate"], h))
        out[p["prefix"] + p["names"]["router"]] = TensorRule((p["experts"] + int(p.get("passing", 0)), h), p.get("router_init", "fan_in"))
        if p.get("router_bias") is not None:
            out[p["prefix"] + p["router_bias"]] = TensorRule((p["experts"],), "unit")
        if p.get("correction") is not None:
            out[p["prefix"] + p["correction"]] = TensorRule((p["experts"] + int(p.get("passing", 0)),), "bias")
        if p.get("shared") is not None:
            out.update(cls._expert_rules(cls._expert_names(p, None), p["shared"]["intermediate"], h))
            if p.get("shared_gate") is not None:
                out[p["prefix"] + p["shared_gate"]] = TensorRule((1, h), "fan_in")
        return out

    def __init__(self, spec, weights, rt):
        super().__init__(spec, weights, rt)
        p = spec.params
        self.score, self.activation = p.get("score", "sigmoid"), p.get("activation", "clamped_glu")
        if self.score not in ("sigmoid", "softmax", "softmax_chosen") or self.activation not in ("clamped_glu", "silu_glu", "relu_squared"):
            raise AlofaError("unsupported", "no such router score or expert activation is built", f"score={p.get('score')} activation={p.get('activation')}")
        self.hidden, self.experts, self.top = int(p["hidden"]), int(p["experts"]), int(p["top"])
        self.passing = int(p.get("passing", 0))
        groups = p.get("groups") or {"count": 1, "keep": 1}
        self.groups, self.keep = int(groups["count"]), int(groups["keep"])
        routed = self.experts + self.passing
        if not 0 < self.top <= routed <= ops.MAX_EXPERTS or self.experts <= 0 or self.passing < 0:
            raise AlofaError("unsupported", f"a token takes 1..experts experts of at most {ops.MAX_EXPERTS}", f"experts={self.experts} passing={self.passing} top={self.top}")
        if self.score != "softmax" and (self.passing or self.groups != 1 or p.get("correction") is not None):
            raise AlofaError("unsupported", "groups, a correction and experts without matrices go with the softmax router", f"score={self.score}")
        if self.groups < 1 or routed % self.groups or not 1 <= self.keep <= self.groups or self.top > self.keep * (routed // self.groups):
            raise AlofaError("invalid_argument", "equal groups, of which the kept ones hold at least the experts a token takes", f"experts={routed} groups={self.groups} keep={self.keep} top={self.top}")
        self.weight_scale, self.renormalize, self.slope = float(p.get("weight_scale", 1.0)), bool(p.get("renormalize", False)), float(p.get("slope", 1.0))
        # silu(g) u is the clamped form without limits, with slope one and nothing added to u
        unbounded = self.activation != "clamped_glu"
        self.offset = 0.0 if unbounded else 1.0
        self.ff, self.limit = int(p["expert"]["intermediate"]), float("inf") if unbounded else float(p["expert"]["limit"])
        shared = p.get("shared")
        self.shared_ff, self.shared_limit = (int(shared["intermediate"]), float("inf") if unbounded else float(shared["limit"])) if shared is not None else (0, 0.0)
        self.correction = rt.vector(weights[p["prefix"] + p["correction"]]) if p.get("correction") is not None else None
        who = list(range(self.experts)) + ([None] if shared is not None else [])
        names = [self._expert_names(p, e) for e in who]
        self.w_gate = rt.matrix(torch.cat([weights[n["gate"]] for n in names], dim=0)) if self.activation != "relu_squared" else None
        self.w_up = rt.matrix(torch.cat([weights[n["up"]] for n in names], dim=0))
        self.w_down = rt.matrix(torch.cat([weights[n["down"]] for n in names], dim=1))
        w_router = weights[p["prefix"] + p["names"]["router"]]
        self.b_router = rt.vector(weights[p["prefix"] + p["router_bias"]]) if p.get("router_bias") is not None else None
        self.shared_gate = shared is not None and p.get("shared_gate") is not None
        if (self.shared_gate or self.b_router is not None) and self.score == "softmax":
            raise AlofaError("unsupported", "a gate of the shared expert and a bias of the router go with the other routers", f"score={self.score}")
        if self.shared_gate and self.activation != "relu_squared":
            raise AlofaError("unsupported", "a gate of the shared expert goes with experts that have no gate matrix", f"activation={self.activation}")
        if self.shared_gate:      # one output more of the router's product
            gate = weights[p["prefix"] + p["shared_gate"]]
            if gate.dtype is not w_router.dtype:
                gate, w_router = gate.float(), w_router.float()
            w_router = torch.cat([w_router, gate], dim=0)
            if self.b_router is not None:
                self.b_router = torch.cat([self.b_router, self.b_router.new_zeros(1)])
        self.w_router = rt.matrix(w_router)
        self.channels = self.experts * self.ff + self.shared_ff

    def route(self, ctx, x):
        """(dense [T, E], chosen [T, top], weights [T, top], and, with experts that hand the row on, their summed weight [T] or None) of the step's rows.
        The shared expert's weights, where it has a gate, are left in the scratch buffer ``router_shared``."""
        T = x.shape[0]
        z = ctx.scratch("router_z", (T, self.w_router.shape[0]), torch.float32)
        ops.gemm(z, x, self.w_router, self.b_router, exact=self.rt.exact)
        dense = ctx.scratch("router_dense", (T, self.experts), torch.float32)
        chosen, weights = ctx.scratch("router_chosen", (T, self.top), torch.int32), ctx.scratch("router_weights", (T, self.top), torch.float32)
        if self.score != "softmax":
            ops.route_top(z, dense, chosen, weights, self.top, self.weight_scale, self.renormalize, self.rt.exact, softmax=self.score == "softmax_chosen",
                          shared_weight=self._shared_weight(ctx, T))
            return dense, chosen, weights, None
        passed = ctx.scratch("router_passed", (T,), torch.float32)
        ops.route_groups(z, self.correction, dense, chosen, weights, passed, self.top, self.passing, self.groups, self.keep, self.weight_scale,
                         self.renormalize, self.rt.exact)
        return dense, chosen, weights, passed if self.passing else None

    def _shared_weight(self, ctx, T):
        return ctx.scratch("router_shared", (T,), torch.float32) if self.shared_gate else None

    def sparse(self, x) -> bool:
        """Whether the experts run slot by slot (every row against the experts it takes only) rather than all of them against
        every row with weights of zero: where a token leaves at least half of the experts out, and the kernel takes the sizes."""
        return (SPARSE_EXPERTS and not self.rt.exact and 2 * self.top <= self.experts
                and ops.can_group_experts(x, self.w_up, self.ff, self.shared_ff))

    def forward_slots(self, ctx, x, out):
        """The mixture's results slot by slot, (y, ``ExpertRows``, None or (weight, rows)), for a reader that adds them up itself; where the experts do not run
        slot by slot the result is stored in ``out`` and None returned."""
        return self.forward(ctx, x, out, out=out, slots=True)

    def forward(self, ctx, x, residual, scale=None, out=None, post=None, slots=False):
        T, exact = residual.shape[0], self.rt.exact
        dense, chosen, weights, passed = self.route(ctx, x)
        if passed is not None and scale is not None:
            raise AlofaError("unsupported", "experts that hand the row on do not go with a channel scale")
        if post is not None and (scale is not None or out is not None or passed is not None):
            raise AlofaError("unsupported", "a norm behind the mixture goes with neither a channel scale, a result apart nor experts that hand the row on")
        shared_weight = self._shared_weight(ctx, T)
        if self.sparse(x):
            rows = ops.ExpertRows(T, self.top, self.experts, self.shared_ff > 0, ctx.scratch)
            ops.expert_rows(rows, chosen, weights, shared_weight)
            act = ctx.scratch("experts_act", (rows.slots, (max(self.ff, self.shared_ff) + 7) // 8 * 8), torch.bfloat16)
            if self.activation == "relu_squared":
                ops.experts_up(act, x, self.w_up, rows, self.ff, self.shared_ff)
            else:
                ops.experts_gate_up(act, x, self.w_gate, self.w_up, rows, self.ff, self.shared_ff, self.limit, self.shared_limit, self.slope, self.offset)
            y = ctx.scratch("experts_out", (rows.slots, self.hidden), torch.float32)
            ops.experts_down(y, act, self.w_down, rows, self.ff, self.shared_ff)
            if slots:
                return y, rows, None if passed is None else (passed, x)
            if post is not None:
                ops.experts_sum_norm(residual, y, rows, *post, scratch=ctx.scratch)
                return
            ops.experts_sum(residual if out is None else out, y, rows, scale, passed=None if passed is None else (passed, x), assign=out is not None)
            return
        # every expert's gate and up for every row, the rows an expert is not taken by weighted with zero
        u, act = ctx.scratch("experts_up", (T, self.channels), self.rt.dtype), ctx.scratch("ff_act", (T, self.channels), self.rt.dtype)
        ops.gemm(u, x, self.w_up, exact=exact)
        if self.activation == "relu_squared":
            ops.weighted_relu_squared(act, u, dense, shared_weight, self.experts, self.ff, self.shared_ff, exact)
        else:
            g = ctx.scratch("experts_gate", (T, self.channels), self.rt.dtype)
            ops.gemm(g, x, self.w_gate, exact=exact)
            ops.clamped_glu(act, g, u, dense, self.experts, self.ff, self.shared_ff, self.limit, self.shared_limit, self.slope, exact, self.offset)
        if post is not None:
            apart = ctx.scratch("sub_out", tuple(residual.shape), torch.float32)
            ops.gemm(apart, act, self.w_down, exact=exact)
            ops.rmsnorm_add(residual, apart, *post, exact=exact)
            return
        if out is not None:
            ops.gemm(out, act, self.w_down, exact=exact)
            if scale is not None:
                out.mul_(scale)
            if passed is not None:
                ops.add_row_scaled(out, x, passed, exact)
        elif scale is None:
            ops.gemm(residual, act, self.w_down, add_to_out=True, exact=exact)
            if passed is not None:
                ops.add_row_scaled(residual, x, passed, exact)
        else:
            ops.gemm_channel_scaled(residual, act, self.w_down, scale, ctx.scratch("sub_out", tuple(residual.shape), torch.float32), exact)


register_part("feed_forward", "routed_experts", RoutedExperts)
