"""Differential attention over a paged cache: two softmax maps per head over the same values, one taken from the other.

q = Wq x + bq (``heads`` x [map 1, map 2] of ``head_dim`` channels each), k = Wk x + bk (``kv_heads`` x the same), v = Wv x + bv (``kv_heads`` x
``v_head_dim``); every map's queries and keys take the position encoding, values do not; query head h reads key/value head h // (heads / kv_heads).
Map m's scores are ``scale`` q_m . k_m, then (``softcap`` c) c tanh(score / c); row i sees the keys j <= i with i - j < ``window`` or j < ``keep_first``
(``window`` None: all of them). With a1, a2 the maps' sums and lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + ``diff`` (one number, formed when the weights are
loaded) a head gives (a1 - lambda a2) over its root mean square over its channels (plus eps), times 1 - ``diff``; then the output projection.

The pages hold a key as two key heads of one half each, [2 kv_heads, slot, d / 2], and values transposed; d is the size both halves of a key and a value
are widened to with zeros. Keys of the first ``keep_first`` tokens stay in their pages for good, the others go as the window passes. In bfloat16, with sizes
the matrix-core kernels are built for, portions of prompts and single tokens take one launch each from turned queries to the heads' ends (single tokens of
heads in steps of 128 channels: from the projection on); every other case
runs the always-valid window kernel on both maps and the kernel that ends the heads. Softmax weights are 32-bit numbers: on the matrix cores each meets
the values as two bfloat16 numbers."""
from __future__ import annotations

import math
import os

import torch

from .. import ops
from ..errors import AlofaError
from ..weights.loader import TensorRule
from .attention import RowPlan, _padded_heads
from .base import SLOT, CacheNeed, CacheTensor, Mixer, build_part, part_class, register_part

NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "lq1": "lq1", "lk1": "lk1", "lq2": "lq2", "lk2": "lk2"}

TURN_IN_DECODE = os.environ.get("ALOFA_TURN_IN_DECODE", "1") != "0"      # 0 (for measurements): a launch of its own turns and writes single tokens too


class DifferentialAttention(Mixer):
    """params: prefix, hidden, heads, kv_heads, head_dim (of one map), v_head_dim, scale, window (None or a count of keys), keep_first, softcap (None or a positive
    number), position (PartSpec of an encoding with a table, for one map's head), diff, eps, biases (bool), names, init."""
    capturable = True

    @classmethod
    def tensors(cls, spec):
        p = spec.params
        n, init = {**NAMES, **p.get("names", {})}, p.get("init", "fan_in")
        pre, h, H, G, d, e = p["prefix"], p["hidden"], p["heads"], p["kv_heads"], p["head_dim"], p["v_head_dim"]
        out = {pre + n["q"]: TensorRule((2 * H * d, h), init), pre + n["k"]: TensorRule((2 * G * d, h), init), pre + n["v"]: TensorRule((G * e, h), init)}
        if p.get("biases", False):
            out.update({pre + n["q_bias"]: TensorRule((2 * H * d,), "filter"), pre + n["k_bias"]: TensorRule((2 * G * d,), "filter"), pre + n["v_bias"]: TensorRule((G * e,), "filter")})
        out.update({pre + n[k]: TensorRule((d,), "filter") for k in ("lq1", "lk1", "lq2", "lk2")})
        out[pre + n["o"]] = TensorRule((h, H * e), init)
        return out

    @staticmethod
    def stored_sizes(d: int, e: int) -> tuple:
        """(channels a map, channels a value) that the pages hold: the smallest head of the matrix-core kernels that takes both, or, beyond those, even sizes."""
        size = next((n for n in ops.MAPS_HEAD_DIMS if n >= max(2 * d, e)), None)
        return (size // 2, size) if size is not None else (d + d % 2, e + e % 2)

    def __init__(self, spec, weights, rt):
        super().__init__(spec, weights, rt)
        p = spec.params
        self.hidden, self.heads, self.kv_heads = int(p["hidden"]), int(p["heads"]), int(p["kv_heads"])
        self.map_dim, self.v_dim = int(p["head_dim"]), int(p["v_head_dim"])
        self.dm, self.d = self.stored_sizes(self.map_dim, self.v_dim)
        self.window, self.keep_first = p.get("window"), int(p.get("keep_first") or 0)
        self.scale, self.softcap = float(p["scale"]), p.get("softcap")
        diff, eps = float(p["diff"]), float(p["eps"])
        if self.kv_heads <= 0 or self.heads % self.kv_heads:
            raise AlofaError("unsupported", "kv_heads must be positive and divide heads", f"heads={self.heads} kv_heads={self.kv_heads}")
        if not 0 < self.dm <= ops.MAX_HEAD_DIM or not 0 < self.d <= ops.MAX_HEAD_DIM:
            raise AlofaError("unsupported", f"the attention kernels take maps and values of up to {ops.MAX_HEAD_DIM} channels", f"head_dim={self.map_dim} v_head_dim={self.v_dim}")
        if (self.window is not None and self.window <= 0) or self.keep_first < 0 or (self.softcap is not None and not self.softcap > 0):
            raise AlofaError("invalid_argument", "a window and a cap of scores are positive, a count of kept tokens is not negative", f"window={self.window} keep_first={self.keep_first} softcap={self.softcap}")
        if self.window is None:
            self.keep_first = 0      # (every key is seen anyway)
        pre, n = p["prefix"], {**NAMES, **p.get("names", {})}
        position = p["position"]
        if self.dm != self.map_dim:
            position = part_class("position", position.kind).for_head(position, self.dm)
        self.position = build_part("position", position, weights, rt)
        if self.position.table(1) is None:
            raise AlofaError("unsupported", "this mixer takes position encodings that give a table of angles", f"position={position.kind}")
        order = self.position.channel_order()
        H, G = self.heads, self.kv_heads
        sizes = {"q": (2 * H, self.map_dim, self.dm, order), "k": (2 * G, self.map_dim, self.dm, order), "v": (G, self.v_dim, self.d, None)}
        mats = [_padded_heads(weights[pre + n[k]], *sizes[k]) for k in sizes]
        if len({m.dtype for m in mats}) > 1:
            mats = [m.float() for m in mats]
        self.width = sum(m.shape[0] for m in mats)
        if self.width % 8:      # (rows of the projection stay 16-byte aligned)
            mats.append(torch.zeros((8 - self.width % 8, self.hidden), dtype=mats[0].dtype, device=mats[0].device))
        self.w_in = rt.matrix(torch.cat(mats, dim=0))
        self.b_in = None
        if p.get("biases", False):
            b = torch.cat([_padded_heads(weights[pre + n[k + "_bias"]].float(), *sizes[k]) for k in sizes])
            self.b_in = rt.vector(torch.cat([b, b.new_zeros(self.w_in.shape[0] - self.width)]))
        w_o = weights[pre + n["o"]]
        if self.d != self.v_dim:      # zero columns where the value heads were widened
            w_o = _padded_heads(w_o.t(), H, self.v_dim, self.d).t()
        self.w_o = rt.matrix(w_o)
        lq1, lk1, lq2, lk2 = (weights[pre + n[k]].double() for k in ("lq1", "lk1", "lq2", "lk2"))
        lam = math.exp(float((lq1 * lk1).sum())) - math.exp(float((lq2 * lk2).sum())) + diff
        self.end = ops.HeadEnd(lam, 1.0 - diff, eps, self.v_dim)

    def cache_need(self):
        # (a value head of d channels is stored as two of d / 2, which lie as it does: keys and values then take the same count of heads)
        return CacheNeed((CacheTensor("k", (2 * self.kv_heads, SLOT, self.dm)), CacheTensor("v", (2 * self.kv_heads, self.d // 2, SLOT))), self.window, self.keep_first)

    def prepare(self, n_positions):
        self.position.table(n_positions)

    def forward(self, ctx, where, x, residual, out=None):
        T, exact = residual.shape[0], self.rt.exact
        kv = ctx.kv(where)
        H, G, D = self.heads, self.kv_heads, self.d
        proj = ctx.scratch("maps_proj", (T, self.w_in.shape[0]), self.rt.dtype)
        ops.gemm(proj, x, self.w_in, self.b_in, exact=exact)
        table, qkv = self.position.table(ctx.n_positions), proj[:, :self.width]
        fast = not exact and ops.maps_attention_fast(D, self.dm, kv.k.shape[2], self.keep_first, self.rt.dtype)
        plan = ctx.memo("gqa_attention.rows", lambda: RowPlan(ctx)) if fast else None
        # one new token per request: the decode kernel turns it and writes its cache slot itself
        turns = fast and TURN_IN_DECODE and ctx.max_q_len == 1 and plan.long_runs is None and ops.can_turn_in_maps_decode(D)
        if turns:
            pass
        elif 2 * self.dm == D:
            ops.rope_kv_write(qkv, *table, ctx.positions, 2 * H, 2 * G, self.dm, kv.slots, kv.k, kv.v)
        else:
            ops.norm_turn_write(qkv, ctx.positions, table, 2 * H, 2 * G, self.dm, D // 2, ops.NORM_NONE, None, None, 0.0, exact, kv.slots, kv.k, kv.v)
        attn = ctx.scratch("maps_out", (T, H * D), self.rt.dtype)
        self._attend(ctx, qkv if turns else proj[:, :2 * H * self.dm], kv, attn, plan, (*table, kv.slots) if turns else None)
        if out is not None:
            ops.gemm(out, attn, self.w_o, exact=exact)
        else:
            ops.gemm(residual, attn, self.w_o, add_to_out=True, exact=exact)

    def _attend(self, ctx, q, kv, attn, plan, rope) -> None:
        T, H, G, D = q.shape[0], self.heads, self.kv_heads, self.d
        if plan is None:
            # the exact path, and page or head sizes the bfloat16 kernels are not built for
            sums = ctx.scratch("maps_sums", (T, 2 * H * D), torch.float32)
            ops.span_attention(sums, q, kv.k, kv.v, kv.block_table, ctx.req_of_token, ctx.positions, 2 * H, 2 * G, self.dm, D, self.window, self.scale, self.rt.exact,
                               keep_first=self.keep_first, softcap=self.softcap, maps=2)
            ops.combine_maps(attn, sums, H, D, self.end, self.rt.exact)
            return
        common = (H, G, D, self.window, self.keep_first, self.scale, self.softcap, self.end)
        if plan.long_runs is not None:      # portions of prompts
            tiles = ctx.memo("runs of 64 rows", lambda: torch.tensor(plan.long_runs, dtype=torch.int32, device=ctx.device))
            ops.maps_prefill(attn, q, kv.k, kv.v, kv.block_table, tiles, *common)
        if plan.n_short:                    # single tokens and very short portions
            parts = ops.maps_decode_plan(plan.n_short, H, G, D, ctx.max_context, self.window, self.keep_first)
            scratch = ctx.scratch("attn_partial", (parts[2],), torch.float32) if parts[2] else None
            sums = ctx.scratch("maps_sums", (T, 2 * H * D), torch.float32) if parts[2] else None
            # (one token per request and nothing else in the step: token i is request i)
            one_each = ctx.max_q_len == 1 and plan.short_rows is None and plan.long_runs is None
            ops.maps_decode(attn, q, kv.k, kv.v, kv.block_table, None if one_each else ctx.req_of_token, ctx.positions, *common, ctx.max_context, scratch, sums,
                            plan.short_rows, parts, rope)


register_part("mixer", "differential_attention", DifferentialAttention)
