"""Each kernel behind Lalepel's parts alone, against the plain functions (float64 on the host): latents on their way into the pages, turned pairs,
the choice of experts and the experts with a gated shared one, the norm behind a sub-layer, attention with a sink on the matrix cores."""
import numpy as np
import pytest
import torch

from plain import lalepel as pl

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
BF = torch.bfloat16


def b16(x):
    return pl.to_bfloat16(np.asarray(x, dtype=np.float64))


def dev(x, dtype=torch.float32):
    return torch.tensor(np.asarray(x), device=DEV).to(dtype)


def back(t):
    return t.detach().float().cpu().numpy().astype(np.float64)


def near(got, want, dtype, what, factor=1.0):
    err = np.abs(back(got) - want).max()
    assert err <= factor * (1e-5 if dtype is torch.float32 else 2.0 ** -7) * max(1.0, np.abs(want).max()), f"{what}: {err}"


def table_of(n, base, scaling, upto=600):
    a = np.arange(upto)
    one = np.zeros((upto, n))
    one[:, 0::2] = 1.0
    t = pl.turn(one, a, base, scaling)
    return dev(t[:, 0::2]), dev(t[:, 1::2])


SCALING = {"factor": 3.0, "original": 100, "fast": 8.0, "slow": 1.0}


@pytest.mark.parametrize("dtype", [torch.float32, BF])
@pytest.mark.parametrize("q_rank, r, n, d, page", [(40, 32, 8, 48, 16), (9, 13, 2, 16, 16), (700, 200, 48, 256, 32), (0, 64, 0, 64, 8), (16, 600, 24, 640, 16), (128, 5, 6, 12, 5)])
def test_latents_on_their_way_into_pages(q_rank, r, n, d, page, dtype):
    from alofa_amd import ops
    rng = np.random.default_rng(r)
    T, eps, exact = 11, 1e-5, dtype is torch.float32
    x = b16(rng.normal(0.2, 1.5, (T, q_rank + r + n + 3)))
    wq, wk = rng.normal(1, 0.2, max(q_rank, 1)).astype(np.float32), rng.normal(1, 0.2, r).astype(np.float32)
    pos = rng.integers(0, 600, T)
    slots = rng.permutation(6 * page)[:T]
    k, v = torch.full((6, 1, page, d), 7.0, dtype=dtype, device=DEV), torch.full((6, 1, d, page), 7.0, dtype=dtype, device=DEV)
    cq = torch.full((T, q_rank), 5.0, dtype=dtype, device=DEV) if q_rank else None
    ops.latent_rows(dev(x, dtype), (0, dev(wq), eps, cq) if q_rank else None, (q_rank, dev(wk), eps), n, dev(pos, torch.int32) if n else None,
                    table_of(n, 100.0, SCALING) if n else None, pages=(dev(slots, torch.int64), k, v), exact=exact)
    if q_rank:
        near(cq, pl.rms_norm(x[:, :q_rank], wq.astype(np.float64), eps), dtype, "queries' latent")
    c = pl.rms_norm(x[:, q_rank:q_rank + r], wk.astype(np.float64), eps)
    want = np.zeros((T, d))
    if n:
        want[:, :n] = pl.turn(x[:, q_rank + r:q_rank + r + n], pos, 100.0, SCALING)
    want[:, n:n + r] = c
    at = (slots // page, slots % page)
    kc, vc = k.permute(0, 2, 1, 3)[:, :, 0], v.permute(0, 3, 1, 2)[:, :, 0]      # [pages, place, d]
    near(kc[at], want, dtype, "keys")
    want[:, :n] = 0.0
    near(vc[at], want, dtype, "values")
    untouched = np.ones((6, page), dtype=bool)
    untouched[at] = False
    assert (back(kc)[untouched] == 7.0).all() and (back(vc)[untouched] == 7.0).all()
    rows = torch.full((T, 5 + r + n + 2), 3.0, dtype=dtype, device=DEV)      # the other form: side by side in rows, the turned part as it is
    ops.latent_rows(dev(x, dtype), None, (q_rank, dev(wk), eps), n, rows=rows[:, 5:], exact=exact)
    near(rows[:, 5:], np.concatenate([c, x[:, q_rank + r:q_rank + r + n], np.zeros((T, 2))], axis=1), dtype, "rows")
    assert (back(rows)[:, :5] == 3.0).all()


@pytest.mark.parametrize("dtype", [torch.float32, BF])
@pytest.mark.parametrize("heads, size, first, n", [(3, 24, 16, 8), (1, 7, 5, 2), (20, 40, 0, 24)])
def test_turned_pairs(heads, size, first, n, dtype):
    from alofa_amd import ops
    rng = np.random.default_rng(n)
    x, pos = b16(rng.normal(0, 1, (13, heads * size + 8))), rng.integers(0, 600, 13)
    xs = dev(x, dtype)
    ops.turn_pairs(xs[:, :heads * size], dev(pos, torch.int32), table_of(n, 50.0, None), heads, first, dtype is torch.float32)
    want = x.copy()
    h = want[:, :heads * size].reshape(13, heads, size)
    h[:, :, first:first + n] = pl.turn(h[:, :, first:first + n], pos, 50.0)
    want[:, :heads * size] = h.reshape(13, -1)
    near(xs, want, dtype, "turned")


@pytest.mark.parametrize("dtype", [torch.float32, BF])
@pytest.mark.parametrize("heads, din, dout, n, rows", [(6, 64, 64, 16, 5), (3, 40, 48, 24, 1), (5, 15, 16, 2, 70), (20, 16, 64, 8, 300), (2, 128, 256, 64, 33)])
def test_a_projection_per_head_whose_first_outputs_are_turned(heads, din, dout, n, rows, dtype):
    from alofa_amd import ops
    rng = np.random.default_rng(heads)
    exact = dtype is torch.float32
    x, w, pos = b16(rng.normal(0, 1, (rows, heads * din))), b16(rng.normal(0, din ** -0.5, (heads, dout, din))), rng.integers(0, 600, rows)
    out = torch.full((rows, heads * dout + 8), 5.0, dtype=dtype, device=DEV)
    ops.head_project(out[:, 8:], dev(x, dtype), dev(w, dtype), exact, turn=(dev(pos, torch.int32), *table_of(n, 70.0, SCALING)))
    want = np.einsum("tai,aoi->tao", x.reshape(rows, heads, din), w)
    want[:, :, :n] = pl.turn(want[:, :, :n], pos, 70.0, SCALING)
    near(out[:, 8:], want.reshape(rows, -1), dtype, "projected and turned", 2.0)
    assert (back(out)[:, :8] == 5.0).all()


@pytest.mark.parametrize("exact", [True, False])
@pytest.mark.parametrize("experts, top, shared", [(8, 3, True), (5, 5, False), (3, 1, True), (64, 6, True), (100, 7, False), (300, 2, True)])
def test_the_choice_of_experts(experts, top, shared, exact):
    from alofa_amd import ops
    rng = np.random.default_rng(experts)
    z = rng.normal(0, 3, (37, experts + 1)).astype(np.float32)
    z[3, :experts] = 0.25                        # all equal: the lowest indices win
    z[4, :experts] *= 40.0                       # far apart: the weights of all but the first vanish without overflow
    dense, chosen, weights = torch.empty(37, experts, device=DEV), torch.empty(37, top, dtype=torch.int32, device=DEV), torch.empty(37, top, device=DEV)
    sw = torch.empty(37, device=DEV) if shared else None
    zs = dev(z)
    ops.route_top(zs if shared else zs[:, :experts], dense, chosen, weights, top, exact=exact, softmax=True, shared_weight=sw)
    want_e, want_w = pl.route(z[:, :experts].astype(np.float64), np.eye(experts), np.zeros(experts), top)
    assert (chosen.cpu().numpy() == want_e).all()
    assert np.abs(back(weights) - want_w).max() <= 1e-6 and chosen[3].tolist() == list(range(top))
    d = np.zeros((37, experts))
    np.put_along_axis(d, want_e, back(weights), -1)
    assert (back(dense) == d).all()
    if shared:
        assert np.abs(back(sw) - pl.sigmoid(z[:, experts].astype(np.float64))).max() <= 1e-6


def _mixture_weights(rng, h, E, ff, sff):
    W = {"router": b16(rng.normal(0, 0.5, (E, h))), "router.b": b16(rng.normal(0, 1, E))}
    for e in range(E):
        W[f"e{e}.up"], W[f"e{e}.down"] = b16(rng.normal(0, 0.3, (ff, h))), b16(rng.normal(0, 0.3, (h, ff)))
    if sff:
        W["shared.up"], W["shared.down"], W["shared.sg"] = b16(rng.normal(0, 0.3, (sff, h))), b16(rng.normal(0, 0.3, (h, sff))), b16(rng.normal(0, 0.3, (1, h)))
    return W


def _routed(ops, x, W, E, top, sff, dtype, exact):
    T = x.shape[0]
    router = np.concatenate([W["router"], W["shared.sg"]]) if sff else W["router"]
    bias = np.concatenate([W["router.b"], [0.0]]) if sff else W["router.b"]
    z = torch.empty(T, len(router), device=DEV)
    ops.gemm(z, x, dev(router, dtype), dev(bias), exact=exact)
    dense, chosen, weights = torch.empty(T, E, device=DEV), torch.empty(T, top, dtype=torch.int32, device=DEV), torch.empty(T, top, device=DEV)
    sw = torch.empty(T, device=DEV) if sff else None
    ops.route_top(z, dense, chosen, weights, top, exact=exact, softmax=True, shared_weight=sw)
    names = [f"e{e}" for e in range(E)] + (["shared"] if sff else [])
    up = dev(np.concatenate([W[n + ".up"] for n in names]), dtype)
    down = dev(np.concatenate([W[n + ".down"] for n in names], axis=1), dtype)
    return dense, chosen, weights, sw, up, down


@pytest.mark.parametrize("dtype", [torch.float32, BF])
@pytest.mark.parametrize("E, top, ff, sff", [(5, 2, 12, 20), (3, 3, 7, 0), (4, 1, 16, 16)])
def test_the_mixture_as_one_product(E, top, ff, sff, dtype):
    """Every expert against every row, the experts a row does not take weighted with zero."""
    from alofa_amd import ops
    rng = np.random.default_rng(E)
    T, h, exact = 21, 40, dtype is torch.float32
    hn, W = b16(rng.normal(0, 1, (T, h))), _mixture_weights(rng, h, E, ff, sff)
    want = pl.mixture(hn, W, "", {"router": {"experts": E, "top": top}, "shared": {"ff": sff} if sff else None})
    x = dev(hn, dtype)
    dense, chosen, weights, sw, up, down = _routed(ops, x, W, E, top, sff, dtype, exact)
    u, act = torch.empty(T, E * ff + sff, dtype=dtype, device=DEV), torch.empty(T, E * ff + sff, dtype=dtype, device=DEV)
    ops.gemm(u, x, up, exact=exact)
    ops.weighted_relu_squared(act, u, dense, sw, E, ff, sff, exact)
    out = torch.empty(T, h, device=DEV)
    ops.gemm(out, act, down, exact=exact)
    near(out, want, dtype, "mixture", 4.0)


@pytest.mark.parametrize("T, h, E, top, ff, sff", [(21, 40, 5, 2, 16, 24), (1, 64, 8, 3, 96, 96), (150, 72, 16, 4, 8, 0), (64, 48, 4, 1, 40, 8), (300, 64, 4, 2, 72, 40),
                                                  (700, 40, 6, 3, 16, 0), (9, 4104, 4, 2, 16, 24)])
def test_the_mixture_slot_by_slot_with_the_norm_behind_it(T, h, E, top, ff, sff):
    from alofa_amd import ops
    rng = np.random.default_rng(T)
    hn, W = b16(rng.normal(0, 1, (T, h))), _mixture_weights(rng, h, E, ff, sff)
    want = pl.mixture(hn, W, "", {"router": {"experts": E, "top": top}, "shared": {"ff": sff} if sff else None})
    x = dev(hn, BF)
    dense, chosen, weights, sw, up, down = _routed(ops, x, W, E, top, sff, BF, False)

    def room(name, shape, dtype):
        return torch.empty(shape, dtype=dtype, device=DEV)
    rows = ops.ExpertRows(T, top, E, sff > 0, room)
    ops.expert_rows(rows, chosen, weights, sw)
    act = torch.zeros(rows.slots, (max(ff, sff) + 7) // 8 * 8, dtype=BF, device=DEV)
    ops.experts_up(act, x, up, rows, ff, sff)
    y = torch.empty(rows.slots, h, device=DEV)
    ops.experts_down(y, act, down, rows, ff, sff)
    plainly = torch.empty(T, h, device=DEV)
    ops.experts_sum(plainly, y, rows, assign=True)
    near(plainly, want, BF, "sum", 4.0)
    stream, w = rng.normal(0, 1, (T, h)).astype(np.float32), rng.normal(1, 0.3, h).astype(np.float32)
    out, left = dev(stream), torch.empty(T, h, dtype=BF, device=DEV)
    ops.experts_sum_norm(out, y, rows, dev(w), 1e-5, left, room)
    assert np.abs(back(out) - (stream + pl.rms_norm(back(plainly), w.astype(np.float64), 1e-5))).max() <= 2e-5
    assert (back(left) == b16(back(out))).all()
    again = dev(stream)
    ops.experts_sum_norm(again, y, rows, dev(w), 1e-5, None, room)
    assert torch.equal(again, out)


@pytest.mark.parametrize("width", [24, 52, 2048, 2056, 5001])
@pytest.mark.parametrize("dtype, exact", [(torch.float32, True), (torch.float32, False), (BF, False)])
def test_the_norm_behind_a_sub_layer(width, dtype, exact):
    from alofa_amd import ops
    rng = np.random.default_rng(width)
    stream, x, w = rng.normal(0, 3, (6, width)).astype(np.float32), rng.normal(0.1, 20, (6, width)).astype(np.float32), rng.normal(1, 0.3, width).astype(np.float32)
    want = stream.astype(np.float64) + pl.rms_norm(x.astype(np.float64), w.astype(np.float64), 1e-4)
    out, rows = dev(stream), torch.empty(6, width, dtype=dtype, device=DEV)
    ops.rmsnorm_add(out, dev(x), dev(w), 1e-4, rows, exact)
    assert np.abs(back(out) - want).max() <= 4e-6
    assert torch.equal(rows, out.to(dtype))
    alone = dev(stream)
    ops.rmsnorm_add(alone, dev(x), dev(w), 1e-4, None, exact)
    assert torch.equal(alone, out)
    if dtype is BF:
        ops.to_bfloat16(rows, dev(x))
        assert torch.equal(rows, dev(x).to(BF))


# ---- attention with a sink on the matrix cores

class Pages:
    """Keys and values of a few requests scattered over pages in a shuffled order, with the tables the kernels read."""

    def __init__(self, lengths, G, d, S, seed):
        rng = np.random.default_rng(seed)
        n_pages = sum((n + S - 1) // S for n in lengths) + 3
        order = rng.permutation(n_pages).tolist()
        table = np.full((len(lengths), max((n + S - 1) // S for n in lengths)), -1, dtype=np.int32)
        self.k, self.v = ([b16(rng.normal(0, 1, (n, G, d))) for n in lengths] for _ in range(2))
        kc, vc = np.full((n_pages, G, S, d), 50.0), np.full((n_pages, G, d, S), 50.0)
        for r, n in enumerate(lengths):
            for b in range((n + S - 1) // S):
                table[r, b] = page = order.pop()
                m = min(n, (b + 1) * S) - b * S
                kc[page, :, :m] = self.k[r][b * S:b * S + m].transpose(1, 0, 2)
                vc[page, :, :, :m] = self.v[r][b * S:b * S + m].transpose(1, 2, 0)
        self.table, self.kc, self.vc = dev(table, torch.int32), dev(kc, BF), dev(vc, BF)

    def attend(self, q, r, p, heads, window, scale, sink):
        """One row of request r at position p: [heads, d]."""
        lo = max(0, p - window + 1) if window else 0
        out = []
        for a in range(heads):
            g = a // (heads // self.k[r].shape[1])
            s = self.k[r][lo:p + 1, g] @ q[a] * scale
            top = max(s.max(), sink[a])
            e = np.exp(s - top)
            out.append(e @ self.v[r][lo:p + 1, g] / (e.sum() + np.exp(sink[a] - top)))
        return np.stack(out)


SINKS = (6.0, -40.0, 0.0, 2.0, 15.0, -1.0, 3.0)


ALONE = [(6, 1, 64), (7, 1, 96), (8, 1, 128), (20, 1, 48), (12, 2, 32), (4, 4, 64), (5, 1, 256), (3, 1, 16)]
SHARING = [(6, 1, 64), (7, 1, 96), (8, 1, 128), (20, 1, 48), (12, 2, 32), (7, 1, 16)]


@pytest.mark.parametrize("heads, kv_heads, d, shared", [(*s, False) for s in ALONE] + [(*s, True) for s in SHARING])
@pytest.mark.parametrize("window", [None, 1, 33, 64, 100])
def test_prompt_rows_with_a_sink(heads, kv_heads, d, window, shared):
    """The prefill kernel with sixteen bits of every weight, each head with blocks of its own and six to eight heads sharing their tiles."""
    from alofa_amd import ops
    group = heads // kv_heads
    chunks = -(-group // 8)
    share = -(-group // chunks) if shared else 0
    lengths, new = [150, 70, 200], [150, 20, 65]
    pages = Pages(lengths, kv_heads, d, 16, heads + d)
    rng = np.random.default_rng(3)
    T = sum(new)
    q = b16(rng.normal(0, 1, (T, heads * d)))
    sink = np.array([SINKS[a % len(SINKS)] for a in range(heads)])
    runs, row = [], 0
    for r, (n, m) in enumerate(zip(lengths, new)):
        runs += [(r, row + i, min(64, m - i), n - m + i) for i in range(0, m, 64)]
        row += m
    tiles = dev(ops.pair_tiles(runs, window, ops.prefill_blocks_per_run(heads, kv_heads, share)), torch.int32)
    out = torch.empty(T, heads * d, dtype=BF, device=DEV)
    ops.attention_prefill(out, dev(q, BF), pages.kc, pages.vc, pages.table, tiles, heads, kv_heads, d, window, 0.3, share=share, fine_weights=True, sink=dev(sink))
    got, row = back(out).reshape(T, heads, d), 0
    for r, (n, m) in enumerate(zip(lengths, new)):
        for i in range(m):
            want = pages.attend(q[row].reshape(heads, d), r, n - m + i, heads, window, 0.3, sink)
            assert np.abs(got[row] - want).max() <= 2.0 ** -7 * max(1.0, np.abs(want).max()), (r, i)
            row += 1


@pytest.mark.parametrize("heads, kv_heads, d", [(6, 1, 64), (20, 1, 96), (16, 1, 256), (12, 2, 80), (4, 4, 32)])
@pytest.mark.parametrize("window", [None, 1, 33, 300])
@pytest.mark.parametrize("splits, hand_over, block_heads", [(1, False, 16), (3, False, 16), (4, True, 16), (20, False, 16), (40, False, 16), (1, False, 4), (4, True, 2), (6, True, 4),
                                                           (5, False, 8), (3, True, 3)])
def test_single_rows_with_a_sink(heads, kv_heads, d, window, splits, hand_over, block_heads):
    """The decode kernel: one part, parts that meet in the workspace, parts a second kernel combines: the sink counts once in each; and heads dealt out over
    blocks."""
    from alofa_amd import ops
    lengths = [1, 40, 333, 700]
    pages = Pages(lengths, kv_heads, d, 16, heads + d)
    q = b16(np.random.default_rng(5).normal(0, 1, (4, heads * d)))
    sink = np.array([SINKS[a % len(SINKS)] for a in range(heads)])
    out = torch.empty(4, heads * d, dtype=BF, device=DEV)
    room = torch.empty(4 * heads * splits * (d + 2), device=DEV)
    ops.attention_decode(out, dev(q, BF), pages.kc, pages.vc, pages.table, None, dev([n - 1 for n in lengths], torch.int32), heads, kv_heads, d, window, 0.3, 1024, room,
                         n_splits=splits, hand_over=hand_over, fine_weights=True, sink=dev(sink), block_heads=block_heads)
    got = back(out).reshape(4, heads, d)
    for r, n in enumerate(lengths):
        want = pages.attend(q[r].reshape(heads, d), r, n - 1, heads, window, 0.3, sink)
        assert np.abs(got[r] - want).max() <= 2.0 ** -7 * max(1.0, np.abs(want).max()), r


# ---- the recurrence in chunks

@pytest.mark.parametrize("heads, dk, dv", [(2, 16, 24), (3, 64, 64), (1, 128, 80), (5, 40, 7), (2, 200, 130)])
@pytest.mark.parametrize("spans", [[64], [65], [1], [63, 1, 200], [130, 64, 2, 17], [700]])
def test_a_constant_decay_in_chunks(heads, dk, dv, spans):
    """Requests of unequal lengths in one call, twice (the second call goes on from the states the first left), against the recurrence row by row."""
    from alofa_amd import ops
    from test_recurrent_ops_gpu import rows_of
    rng = np.random.default_rng(dk + sum(spans))
    decay = np.array([0.5, 1.0, 0.999, 0.97, 0.0])[:heads].astype(np.float32)
    T, slots = sum(spans), [4, 1, 3, 0][:len(spans)]
    state = dev(rng.normal(0, 1, (6, heads, dk, dv)))
    S = back(state)
    untouched = S[[s for s in range(6) if s not in slots]].copy()
    row0 = np.cumsum([0] + spans)
    chunks = ops.Chunks(list(zip(row0[:-1].tolist(), spans)), DEV)
    assert chunks.count == sum(-(-n // 64) for n in spans)
    rows = rows_of(list(zip(slots, spans)), 6)
    powers = ops.decay_powers(dev(decay))
    for call in range(2):
        proj = b16(rng.normal(0, 1, (T, heads * (2 * dk + dv) + 8)))
        q, k, v = proj[:, :heads * dk], proj[:, heads * dk:2 * heads * dk], proj[:, 2 * heads * dk:2 * heads * dk + heads * dv]
        wide = (proj.shape[1] + 7) // 8 * 8
        p = torch.zeros(T, wide, dtype=BF, device=DEV)
        p[:, :proj.shape[1]] = dev(proj, BF)
        out, added = torch.full((T, heads * dv), 9.0, device=DEV), torch.empty(chunks.count, heads, dk, dv, device=DEV)
        assert ops.can_chunk(p[:, :heads * dk], p[:, heads * dk:2 * heads * dk], dk, 1000)
        ops.chunked_recurrence(out, p[:, :heads * dk], p[:, heads * dk:2 * heads * dk], p[:, 2 * heads * dk:2 * heads * dk + heads * dv], state, rows, chunks, heads, dk, dv, powers, added,
                               q_scale=0.7, k_scale=dk ** -0.5)
        want = np.zeros((T, heads, dv))
        for r, (s, n) in enumerate(zip(slots, spans)):
            for t in range(row0[r], row0[r] + n):
                S[s] = decay.astype(np.float64)[:, None, None] * S[s] + dk ** -0.5 * k[t].reshape(heads, dk)[:, :, None] * v[t].reshape(heads, dv)[:, None, :]
                want[t] = (S[s] * 0.7 * q[t].reshape(heads, dk)[:, :, None]).sum(axis=1)
        err = np.abs(back(out) - want.reshape(T, -1)).max()
        assert err <= 2e-5 * max(1.0, np.abs(want).max()), (call, err)
        assert np.abs(back(state)[slots] - S[slots]).max() <= 2e-5 * max(1.0, np.abs(S[slots]).max())
    assert (back(state)[[s for s in range(6) if s not in slots]] == untouched).all()
