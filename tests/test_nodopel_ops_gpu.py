"""Each kernel behind Nodopel's parts alone, against the plain functions (float64 on the host): the copies of the stream, gelu-gated products, the choice of experts,
attention of two maps with kept tokens and capped scores (the always-valid kernel, the kernels for prompts and for single tokens), the heads' end. What a
row may not see is filled with NaN in the pages, so that anything read from there and used shows."""
import numpy as np
import pytest
import torch

from plain import nodopel as pl

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
BF, F32 = torch.bfloat16, torch.float32


def b16(x):
    return pl.to_bfloat16(np.asarray(x, dtype=np.float64))


def f32(x):
    return np.asarray(x, dtype=np.float32).astype(np.float64)


def dev(x, dtype=F32):
    return torch.tensor(np.asarray(x), device=DEV).to(dtype)


def back(t):
    return t.detach().float().cpu().numpy().astype(np.float64)


def near(got, want, dtype, what, factor=1.0):
    got = back(got)
    assert np.isfinite(got).all(), f"{what}: not finite"
    err = np.abs(got - want).max()
    assert err <= factor * (1e-5 if dtype is F32 else 2.0 ** -7) * max(1.0, np.abs(want).max()), f"{what}: {err}"


# ------------------------------------------------------------------ copies of the stream

@pytest.mark.parametrize("dtype, exact", [(F32, True), (F32, False), (BF, False)])
@pytest.mark.parametrize("S, h", [(1, 64), (2, 52), (3, 96), (4, 2048), (4, 1030), (2, 4100), (4, 3072), (6, 320), (16, 132), (16, 1027), (5, 5000)])
def test_streams(S, h, dtype, exact):
    from alofa_amd import ops
    rng = np.random.default_rng(S * h)
    T, eps = 5, 1e-5
    X, y, source = f32(rng.normal(0, 2, (T, S, h))), f32(rng.normal(0, 3, (T, h))), f32(rng.normal(0, 1, (T, h)))
    mix, wo, wi, w = f32(rng.normal(0, 0.7, (S, S))), f32(rng.normal(1, 0.5, S)), f32(rng.normal(0.5, 0.5, S)), f32(rng.normal(1, 0.2, h))
    new = pl.write_streams(X, y, mix, wo)
    args = dict(y=dev(y), mix=dev(mix), w_out=dev(wo), exact=exact)
    x = dev(X)
    ops.streams_step(x, **args)      # written, nobody reads
    near(x, new, F32, "copies")
    x, out = dev(X), torch.full((T, h), 7.0, dtype=dtype, device=DEV)
    ops.streams_step(x, **args, w_in=dev(wi), norm=(dev(w), eps), out=out)
    near(x, new, F32, "copies beside what is read")
    near(out, pl.rms_norm(pl.read_streams(new, wi), w, eps), dtype, "normed")
    x, out = dev(X), torch.full((T, h), 7.0, dtype=F32, device=DEV)
    ops.streams_step(x, **args, w_in=dev(np.ones(S)), out=out, write=False)      # the sum at the end of a pass; the copies are left alone
    near(out, new.sum(axis=1), F32, "sum")
    assert (back(x) == X).all()
    out = torch.full((T, h), 7.0, dtype=dtype, device=DEV)
    ops.streams_step(x, w_in=dev(wi), norm=(dev(w), eps), out=out, write=False, exact=exact)      # read as they are
    near(out, pl.rms_norm(pl.read_streams(X, wi), w, eps), dtype, "read")
    assert (back(x) == X).all()
    x = torch.full((T, S, h), 5.0, device=DEV)
    ops.streams_step(x, source=dev(source), w_in=dev(wi), norm=(dev(w), eps), out=out, exact=exact)      # spread and read
    assert (back(x) == source[:, None, :]).all()
    near(out, pl.rms_norm(source * wi.sum(), w, eps), dtype, "read from the source", 2.0)


@pytest.mark.parametrize("out_dtype", [F32, BF])
@pytest.mark.parametrize("S, h, top, shared, passing", [(4, 2048, 4, True, 2), (2, 96, 3, False, 0), (3, 1030, 7, True, 1), (1, 4100, 5, True, 3), (8, 320, 1, False, 1), (2, 3000, 11, True, 2)])
def test_streams_take_a_mixture_slot_by_slot(S, h, top, shared, passing, out_dtype):
    from alofa_amd import ops
    rng = np.random.default_rng(h)
    T, experts, eps = 9, 12, 1e-5
    chosen = np.stack([rng.permutation(experts + passing)[:top] for _ in range(T)])
    rows = ops.ExpertRows(T, top, experts, shared, lambda name, shape, dtype: torch.zeros(shape, dtype=dtype, device=DEV))
    ops.expert_rows(rows, dev(chosen, torch.int32), dev(rng.random((T, top))))
    y, px, pw = f32(rng.normal(0, 1, (rows.slots, h))), b16(rng.normal(0, 1, (T, h))), f32(rng.random(T))
    of = rows.slot_of.cpu().numpy()
    want = np.zeros((T, h))
    for t in range(T):
        for k in range(top):
            assert (of[t * top + k] < 0) == (chosen[t, k] >= experts)
            if of[t * top + k] >= 0:
                want[t] += y[of[t * top + k]]
        if shared:
            want[t] += y[of[T * top + t]]
    if passing:
        want += pw[:, None] * px
    X, mix, wo, wi, w = f32(rng.normal(0, 2, (T, S, h))), f32(rng.normal(0, 0.7, (S, S))), f32(rng.normal(1, 0.5, S)), f32(rng.normal(0.5, 0.5, S)), f32(rng.normal(1, 0.2, h))
    x, out = dev(X), torch.full((T, h), 7.0, dtype=out_dtype, device=DEV)
    ops.streams_step(x, slots=(dev(y), rows, (dev(pw), dev(px, BF)) if passing else None), mix=dev(mix), w_out=dev(wo), w_in=dev(wi), norm=(dev(w), eps), out=out)
    new = pl.write_streams(X, want, mix, wo)
    near(x, new, F32, "copies")
    near(out, pl.rms_norm(pl.read_streams(new, wi), w, eps), out_dtype, "normed")


def test_streams_refuses_what_does_not_fit():
    from alofa_amd import ops
    from alofa_amd.errors import AlofaError
    x = torch.zeros((2, 3, 8), device=DEV)
    with pytest.raises(AlofaError, match="do not fit"):
        ops.streams_step(x, y=torch.zeros((2, 8), device=DEV), mix=torch.zeros((2, 2), device=DEV), w_out=torch.zeros(3, device=DEV))
    with pytest.raises(AlofaError, match="copies"):
        ops.streams_step(torch.zeros((2, 17, 8), device=DEV))


# ------------------------------------------------------------------ feed-forwards

@pytest.mark.parametrize("M, N, K, kernel", [(1, 72, 128, "rows"), (3, 40, 64, "rows"), (8, 136, 512, "rows"), (5, 96, 256, "stream"), (40, 200, 320, "stream"), (64, 64, 128, "stream"),
                                             (17, 300, 448, "tiled"), (130, 264, 128, "tiled"), (300, 520, 2048, "tiled"), (520, 8200, 128, "tiled"), (40, 2600, 2048, "tiled"), (260, 512, 96, "wide"),
                                             (9, 30, 52, None), (2, 13, 7, None)])
def test_gelu_gated_products(M, N, K, kernel):
    from alofa_amd import ops
    rng = np.random.default_rng(N)
    a, wg, wu = b16(rng.normal(0, 1, (M, K))), b16(rng.normal(0, 1.5 / K ** 0.5, (N, K))), b16(rng.normal(0, 1 / K ** 0.5, (N, K)))
    want = pl.gelu_tanh(a @ wg.T) * (a @ wu.T)
    out = torch.full((M, N), 3.0, dtype=BF, device=DEV)
    ops.gemm_swiglu(out, dev(a, BF), dev(wg, BF), dev(wu, BF), kernel=kernel, act="gelu_tanh")
    near(out, want, BF, "bfloat16")
    out = torch.full((M, N), 3.0, dtype=F32, device=DEV)
    ops.gemm_swiglu(out, dev(a), dev(wg), dev(wu), exact=True, act="gelu_tanh")
    near(out, want, F32, "float32")
    if kernel in ("rows", "stream") and M <= 8:
        x, w = f32(rng.normal(0, 2, (M, K))), f32(rng.normal(1, 0.1, K))
        out = torch.full((M, N), 3.0, dtype=BF, device=DEV)
        if ops.can_fuse_norm(M, dev(wg, BF), BF, swiglu=True, kernel=kernel):
            ops.gemm_swiglu(out, dev(x), dev(wg, BF), dev(wu, BF), kernel=kernel, norm=(dev(w), 1e-5), act="gelu_tanh")
            n = b16(pl.rms_norm(x, w, 1e-5))
            near(out, pl.gelu_tanh(n @ wg.T) * (n @ wu.T), BF, "with the norm", 2.0)


@pytest.mark.parametrize("exact", [True, False])
@pytest.mark.parametrize("experts, passing, top, groups, keep", [(6, 2, 3, 1, 1), (3, 0, 3, 1, 1), (16, 4, 4, 1, 1), (60, 4, 9, 1, 1), (64, 0, 1, 1, 1), (90, 7, 12, 1, 1), (500, 12, 20, 1, 1),
                                                                 (12, 4, 5, 4, 2), (30, 2, 4, 8, 3), (120, 8, 6, 16, 4)])
def test_the_choice_of_experts(experts, passing, top, groups, keep, exact):
    from alofa_amd import ops
    rng = np.random.default_rng(experts)
    T, E = 37, experts + passing
    z, corr = f32(rng.normal(0, 2, (T, E))), f32(rng.normal(0, 0.2, E))
    chosen, weights = torch.zeros((T, top), dtype=torch.int32, device=DEV), torch.zeros((T, top), device=DEV)
    dense, passed = torch.full((T, experts), 9.0, device=DEV), torch.full((T,), 9.0, device=DEV)
    ops.route_groups(dev(z), dev(corr), dense, chosen, weights, passed, top, passing, groups, keep, renormalize=True, exact=exact)
    s = np.exp(z - z.max(axis=1, keepdims=True))
    s = s / s.sum(axis=1, keepdims=True)
    c = s + corr
    by_group = c.reshape(T, groups, -1).max(axis=2)
    kept = np.zeros((T, groups), dtype=bool)
    np.put_along_axis(kept, np.argsort(-by_group, axis=1, kind="stable")[:, :keep], True, axis=1)
    want = np.argsort(-np.where(np.repeat(kept, E // groups, axis=1), c, -np.inf), axis=1, kind="stable")[:, :top]
    assert (back(chosen) == want).all()
    w = np.take_along_axis(s, want, axis=1)
    w = w / w.sum(axis=1, keepdims=True)
    near(weights, w, F32, "weights")
    full = np.zeros((T, E))
    np.put_along_axis(full, want, w, axis=1)
    near(dense, full[:, :experts], F32, "dense")
    near(passed, full[:, experts:].sum(axis=1), F32, "passed")


def test_scores_that_are_all_next_to_nothing():
    """The correction picks experts whose scores underflow: their weights are zeros, not NaN."""
    from alofa_amd import ops
    z = torch.tensor([[300.0, 0.0, 0.0, 0.0]], device=DEV)
    chosen, weights = torch.zeros((1, 2), dtype=torch.int32, device=DEV), torch.full((1, 2), 9.0, device=DEV)
    ops.route_groups(z, torch.tensor([0.0, 5.0, 6.0, 0.0], device=DEV), torch.zeros((1, 3), device=DEV), chosen, weights, torch.zeros(1, device=DEV), 2, 1, renormalize=True)
    assert chosen.tolist() == [[2, 1]] and weights.tolist() == [[0.0, 0.0]]


# ------------------------------------------------------------------ attention

class Requests:
    """Requests of some length whose last ``rows`` tokens are served: keys and values in shuffled pages, NaN wherever no served row may look, no page (-1) where
    the window has passed one."""

    def __init__(self, spans, G, dm, d, page, window, keep, dtype, seed):
        rng = np.random.default_rng(seed)
        self.spans, self.G, self.dm, self.d = spans, G, dm, d
        blocks = [(n + page - 1) // page for n, _ in spans]
        order = list(rng.permutation(sum(blocks) + 4))
        self.k = [b16(rng.normal(0, 1, (n, G, 2, dm))) for n, _ in spans]
        self.v = [b16(rng.normal(0, 1, (n, G, d))) for n, _ in spans]
        kc = np.full((len(order), 2 * G, page, dm), np.nan)
        vc = np.full((len(order), G, d, page), np.nan)
        table = np.full((len(spans), max(blocks)), -1)
        for r, (n, rows) in enumerate(spans):
            first = 0 if window is None else max(0, n - rows - window + 1)
            for j in range(n):
                if j < first and j >= keep:
                    continue
                if table[r, j // page] < 0:
                    table[r, j // page] = order.pop()
                kc[table[r, j // page], :, j % page] = self.k[r][j].reshape(2 * G, dm)
                vc[table[r, j // page], :, :, j % page] = self.v[r][j]
        self.kc, self.vc = dev(kc, dtype).contiguous(), dev(vc.reshape(len(vc), 2 * G, d // 2, page), dtype).contiguous()
        self.table = dev(table, torch.int32)
        self.positions = dev(np.concatenate([np.arange(n - rows, n) for n, rows in spans]), torch.int32)
        self.request = dev(np.concatenate([np.full(rows, r) for r, (_, rows) in enumerate(spans)]), torch.int32)
        self.T = sum(rows for _, rows in spans)

    def sums(self, q, H, window, keep, scale, cap):
        """Both maps' sums of every served row, [T, H, 2, d]."""
        out, at = np.zeros((self.T, H, 2, self.d)), 0
        for r, (n, rows) in enumerate(self.spans):
            seen = pl.visible(n, None if window is None else {"size": window, "keep_first": keep})[n - rows:]
            for h in range(H):
                g = h // (H // self.G)
                for m in range(2):
                    s = pl.capped(q[at:at + rows, h, m] @ self.k[r][:, g, m].T * scale, cap)
                    out[at:at + rows, h, m] = pl.softmax_over(s, seen) @ self.v[r][:, g]
            at += rows
        return out


LAM, DIFF, EPS = 0.42, 0.3, 1e-5


def ends(sums, true_d):
    return pl.combine_maps(sums[:, :, 0, :true_d], sums[:, :, 1, :true_d], LAM, DIFF, EPS)


def padded(y, d):
    return np.concatenate([y, np.zeros((*y.shape[:-1], d - y.shape[-1]))], axis=-1).reshape(y.shape[0], -1)


# d, query heads, key heads, page, window, kept tokens, cap, scale
SIZES = [(32, 4, 2, 16, 20, 5, 20.0, 0.5), (32, 20, 1, 16, 33, 40, None, 0.4), (64, 3, 3, 8, 17, 100, 60.0, 0.3), (96, 4, 1, 16, 40, 20, 50.0, 0.3), (128, 8, 2, 16, 100, 17, 30.0, 0.25),
         (128, 2, 1, 32, None, 0, 50.0, 0.25), (48, 2, 2, 16, 1, 3, 15.0, 0.5), (16, 5, 1, 8, 64, 64, None, 0.6), (192, 4, 2, 16, 70, 9, 90.0, 0.2), (256, 3, 1, 16, 50, 33, 45.0, 0.2),
         (64, 4, 2, 16, 16, 16, 25.0, 0.4), (64, 4, 2, 16, 15, 1, None, 0.4), (32, 2, 1, 64, 200, 130, 40.0, 0.5)]


def head_end(true_d):
    from alofa_amd import ops
    return ops.HeadEnd(LAM, 1.0 - DIFF, EPS, true_d)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("d, H, G, page, window, keep, cap, scale", SIZES + [(14, 3, 1, 5, 9, 7, 12.0, 0.5), (22, 4, 2, 6, 13, 30, None, 0.4)])
def test_always_valid_attention_of_two_maps(d, H, G, page, window, keep, cap, scale, dtype):
    from alofa_amd import ops
    exact, dm = dtype is F32, d // 2 + (d % 4 == 2)      # (also maps that are no half of a value head)
    r = Requests([(3, 3), (150, 1), (97, 30), (40, 5)], G, dm, d, page, window, keep, dtype, d)
    q = b16(np.random.default_rng(1).normal(0, 1, (r.T, H, 2, dm)))
    sums, out = torch.full((r.T, 2 * H * d), 9.0, device=DEV), torch.full((r.T, H * d), 9.0, dtype=dtype, device=DEV)
    ops.span_attention(sums, dev(q.reshape(r.T, -1), dtype), r.kc, r.vc, r.table, r.request, r.positions, 2 * H, 2 * G, dm, d, window, scale, exact, keep_first=keep, softcap=cap, maps=2)
    want = r.sums(q, H, window, keep, scale, cap)
    near(sums, want.reshape(r.T, -1), F32, "sums", 1.0 if exact else 5.0)
    end = head_end(d - 3)
    ops.combine_maps(out, sums, H, d, end, exact)
    near(out, padded(ends(want, d - 3), d), dtype, "ends", 3.0)


@pytest.mark.parametrize("d, H, G, page, window, keep, cap, scale", SIZES)
def test_two_maps_for_portions_of_prompts(d, H, G, page, window, keep, cap, scale):
    from alofa_amd import ops
    spans = [(7, 7), (64, 64), (230, 100), (131, 2), (300, 65), (200, 1), (129, 129)]
    r = Requests(spans, G, d // 2, d, page, window, keep, BF, d + 1)
    q = b16(np.random.default_rng(2).normal(0, 1, (r.T, H, 2, d // 2)))
    tiles, row = [], 0
    for i, (n, rows) in enumerate(spans):
        tiles += [(i, row + a, min(64, rows - a), n - rows + a) for a in range(0, rows, 64)]
        row += rows
    out = torch.full((r.T, H * d), 9.0, dtype=BF, device=DEV)
    wide = torch.full((r.T, H * d + 8), 5.0, dtype=BF, device=DEV)      # (rows of queries that lie in a wider projection)
    wide[:, :H * d] = dev(q.reshape(r.T, -1), BF)
    ops.maps_prefill(out, wide[:, :H * d], r.kc, r.vc, r.table, dev(tiles, torch.int32), H, G, d, window, keep, scale, cap, head_end(d))
    near(out, ends(r.sums(q, H, window, keep, scale, cap), d).reshape(r.T, -1), BF, "prompts", 1.5)


@pytest.mark.parametrize("plan", [None, (1, False), (3, True), (8, True), (5, False), (20, False)])
@pytest.mark.parametrize("d, H, G, page, window, keep, cap, scale", SIZES)
def test_two_maps_for_single_tokens(d, H, G, page, window, keep, cap, scale, plan):
    from alofa_amd import ops
    spans = [(n, rows) for n, rows in ((1, 1), (2, 1), (17, 4), (64, 1), (163, 3), (299, 1), (481, 1))]
    r = Requests(spans, G, d // 2, d, page, window, keep, BF, d + 2)
    q = b16(np.random.default_rng(3).normal(0, 1, (r.T, H, 2, d // 2)))
    want = ends(r.sums(q, H, window, keep, scale, cap), d).reshape(r.T, -1)

    def run(rows):
        n = r.T if rows is None else len(rows)
        p = ops.maps_decode_plan(n, H, G, d, 512, window, keep) if plan is None else (*plan, n * 2 * H * plan[0] * (d + 2) if plan[0] > 1 and not plan[1] else 0)
        out = torch.full((r.T, H * d), 9.0, dtype=BF, device=DEV)
        scratch, sums = (torch.empty(p[2], device=DEV), torch.empty((r.T, 2 * H * d), device=DEV)) if p[2] else (None, None)
        ops.maps_decode(out, dev(q.reshape(r.T, -1), BF), r.kc, r.vc, r.table, r.request, r.positions, H, G, d, window, keep, scale, cap, head_end(d), 512, scratch, sums,
                        None if rows is None else dev(rows, torch.int32), p)
        return out
    near(run(None), want, BF, "all rows", 1.5)
    rows = [0, 4, 5, r.T - 1]
    got = back(run(rows))
    near(dev(got[rows]), want[rows], BF, "some rows", 1.5)
    assert (np.delete(got, rows, axis=0) == 9.0).all()


@pytest.mark.parametrize("plan", [None, (1, False), (4, True), (6, False)])
@pytest.mark.parametrize("d, H, G, page, window, keep, cap, scale", [z for z in SIZES if z[0] % 128 == 0] + [(128, 20, 1, 16, 17, 16, 50.0, 0.25), (128, 3, 3, 8, 1, 0, None, 0.3)])
def test_single_tokens_turned_and_written_on_the_way(d, H, G, page, window, keep, cap, scale, plan):
    """One new token per request, straight from the projection: as turned by the plain function, and written to its slot."""
    from alofa_amd import ops
    spans = [(n, 1) for n in (1, 2, 16, 17, 100, 163, 481, 64)]
    r = Requests(spans, G, d // 2, d, page, window, keep, BF, d + 3)
    rng = np.random.default_rng(7)
    T, dims, base = r.T, d // 2, 300.0
    q, k, v = (b16(rng.normal(0, 1, shape)) for shape in ((T, H, 2, d // 2), (T, G, 2, d // 2), (T, G, d)))
    at = np.array([n - 1 for n, _ in spans])
    turned_q, turned_k = (b16(pl.turn(x.reshape(T, -1, d // 2), at, {"base": base, "dims": dims})).reshape(x.shape) for x in (q, k))
    table, slots = r.table.cpu().numpy(), []
    for i, (n, _) in enumerate(spans):      # (the new token's slot holds nothing yet)
        b, o = table[i, (n - 1) // page], (n - 1) % page
        slots.append(b * page + o)
        r.kc[b, :, o] = float("nan")
        r.vc[b, :, :, o] = float("nan")
        r.k[i][n - 1], r.v[i][n - 1] = turned_k[i], v[i]
    angles = np.arange(512)[:, None].astype(np.float32) * pl.frequencies(dims, base).astype(np.float32)
    rope = (dev(np.cos(angles.astype(np.float64))), dev(np.sin(angles.astype(np.float64))), dev(slots, torch.int64))
    rows = dev(np.concatenate([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], axis=1), BF)
    p = ops.maps_decode_plan(T, H, G, d, 512, window, keep) if plan is None else (*plan, T * 2 * H * plan[0] * (d + 2) if plan[0] > 1 and not plan[1] else 0)
    scratch, sums = (torch.empty(p[2], device=DEV), torch.empty((T, 2 * H * d), device=DEV)) if p[2] else (None, None)
    out = torch.full((T, H * d), 9.0, dtype=BF, device=DEV)
    ops.maps_decode(out, rows, r.kc, r.vc, r.table, None, r.positions, H, G, d, window, keep, scale, cap, head_end(d), 512, scratch, sums, None, p, rope)
    near(out, ends(r.sums(turned_q, H, window, keep, scale, cap), d).reshape(T, -1), BF, "turned here", 2.0)
    for i, s in enumerate(slots):
        near(r.kc[s // page, :, s % page], turned_k[i].reshape(2 * G, d // 2), BF, "the new key")
        assert (back(r.vc.reshape(len(r.vc), G, d, page)[s // page, :, :, s % page]) == v[i]).all()


def test_prompts_and_single_tokens_give_a_row_the_same():
    """The same rows through both kernels, and through the kernel for prompts in other runs."""
    from alofa_amd import ops
    d, H, G, window, keep = 128, 4, 1, 50, 21
    r = Requests([(190, 100)], G, d // 2, d, 16, window, keep, BF, 5)
    q = dev(b16(np.random.default_rng(4).normal(0, 1, (r.T, H * d))), BF)
    outs = []
    for cuts in ([0, 64], [0, 2, 40, 77], None):
        out = torch.full((r.T, H * d), 9.0, dtype=BF, device=DEV)
        common = (H, G, d, window, keep, 0.3, 40.0, head_end(d))
        if cuts is None:
            ops.maps_decode(out, q, r.kc, r.vc, r.table, r.request, r.positions, *common, 256, plan=(1, False, 0))
        else:
            ops.maps_prefill(out, q, r.kc, r.vc, r.table, dev([(0, a, b - a, 90 + a) for a, b in zip(cuts, cuts[1:] + [100])], torch.int32), *common)
        outs.append(back(out))
    assert np.abs(outs[0] - outs[1]).max() <= 2.0 ** -7 * 4 and np.abs(outs[0] - outs[2]).max() <= 2.0 ** -7 * 4


def test_what_the_kernels_refuse():
    from alofa_amd import ops
    from alofa_amd.errors import AlofaError
    r = Requests([(20, 20)], 1, 16, 32, 16, 8, 4, BF, 6)
    q, out = torch.zeros((20, 64), dtype=BF, device=DEV), torch.zeros((20, 64), dtype=BF, device=DEV)
    tiles = dev([(0, 0, 20, 0)], torch.int32)
    with pytest.raises(AlofaError, match="takes these sizes"):      # (kept tokens in more pages than the kernels hold)
        ops.maps_prefill(out, q, r.kc, r.vc, r.table, tiles, 2, 1, 32, 8, 64 * 16 + 1, 0.3, None, head_end(32))
    with pytest.raises(AlofaError, match="cap of scores"):
        ops.maps_prefill(out, q, r.kc, r.vc, r.table, tiles, 2, 1, 32, 8, 4, 0.3, -1.0, head_end(32))
    with pytest.raises(AlofaError, match="do not fit"):
        ops.maps_prefill(out, q, r.kc, r.vc, r.table, tiles, 3, 1, 32, 8, 4, 0.3, None, head_end(32))
