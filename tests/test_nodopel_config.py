"""Nodopel without a GPU: the configuration's keys and checks, the tensor list, the run order, what every layer keeps per token, the table of angles, pages of kept
tokens in the cache manager, and the plain implementation's own consistency."""
import copy
import json

import numpy as np
import pytest

from alofa_amd.cache.manager import CacheManager, blocks_for
from alofa_amd.config.base import PartSpec
from alofa_amd.config.registry import config_from_dict, load_config
from alofa_amd.errors import AlofaError
from alofa_amd.model import check_spec, expected_tensors
from alofa_amd.parts.base import CacheNeed, CacheTensor, SLOT
from nodopel_cases import NODOPEL, write_model
from plain import nodopel as pl


@pytest.mark.parametrize("name", list(NODOPEL))
def test_config_round_trip_and_tensor_list(name, tmp_path):
    cfg = config_from_dict(NODOPEL[name])
    assert config_from_dict(cfg.to_dict()) == cfg
    spec = cfg.spec()
    check_spec(spec)
    write_model(NODOPEL[name], tmp_path, 1)
    assert load_config(tmp_path) == cfg
    w = pl.read_weights(tmp_path)
    expected = expected_tensors(spec)
    assert set(w) == {n for n, r in expected.items() if not r.optional}
    assert all(tuple(w[n].shape) == tuple(expected[n].shape) for n in w)
    h, s = NODOPEL[name]["width"], NODOPEL[name]["streams"]
    for i, l in enumerate(NODOPEL[name]["layers"]):
        p, m, mlp = f"l{i}.", l["mixer"], l["mlp"]
        assert w[p + "norm1"].shape == (h,) and (p + "norm2" in w) == (p + "hc2.mix" in w) == (mlp is not None)
        assert w[p + "hc1.in"].shape == w[p + "hc1.out"].shape == (s,) and w[p + "hc1.mix"].shape == (s, s)
        assert w[p + "mix.q"].shape == (m["heads"] * 2 * m["dim"], h) and w[p + "mix.k"].shape == (m["kv_heads"] * 2 * m["dim"], h)
        assert w[p + "mix.v.b"].shape == (m["kv_heads"] * m["vdim"],) and w[p + "mix.lq1"].shape == (m["dim"],) and w[p + "mix.o"].shape == (h, m["heads"] * m["vdim"])
        if mlp is not None and mlp["kind"] == "moe":
            r = mlp["router"]
            assert w[p + "mlp.router"].shape == (r["experts"] + r["identity"], h) and w[p + "mlp.correction"].shape == (r["experts"] + r["identity"],)
            assert f"{p}mlp.e{r['experts'] - 1}.gate" in w and f"{p}mlp.e{r['experts']}.gate" not in w and (p + "mlp.shared.up" in w) == ("shared" in mlp)
    assert "head" not in w


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="retention"), "no such mixer"),
    (lambda c: c["layers"][1]["mlp"].update(kind="glu"), "no such feed-forward"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "more experts than there are"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads must divide heads"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims is even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "rot.dims is even"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=5.0), "low bound"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("high"), "lacks a required key"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "must be positive"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1), "is not negative"),
    (lambda c: c["layers"][0]["mixer"].update(softcap=0.0), "must be positive"),
    (lambda c: c["layers"][0]["mixer"].pop("diff"), "lacks a required key"),
    (lambda c: c.update(streams=0), "must be positive"),
    (lambda c: c["loop"].update(stop=5), "a run of existing layers"),
    (lambda c: c.update(layers=[]), "at least one layer"),
])
def test_what_the_configuration_refuses(change, message):
    raw = copy.deepcopy(NODOPEL["A"])
    change(raw)
    with pytest.raises(AlofaError, match=message):
        config_from_dict(raw)


def test_weights_that_do_not_fit_are_named(tmp_path):
    from alofa_amd.weights.loader import load_weights
    write_model(NODOPEL["A"], tmp_path, 1)
    raw = json.loads((tmp_path / "config.json").read_text())
    raw["streams"] = 2
    (tmp_path / "config.json").write_text(json.dumps(raw))
    with pytest.raises(AlofaError, match=r"l0\.hc1\.in"):
        load_weights(tmp_path, expected_tensors(load_config(tmp_path).spec()))


@pytest.mark.parametrize("name", list(NODOPEL))
def test_the_run_order_is_the_plain_one(name):
    spec = config_from_dict(NODOPEL[name]).spec()
    assert [e.layer for e in spec.order] == pl.order(NODOPEL[name])
    assert all(e.cache_of is None and e.join is None for e in spec.order) and spec.streams == NODOPEL[name]["streams"]


def test_sizes_as_the_pages_store_them():
    from alofa_amd.parts.differential import DifferentialAttention as D
    assert D.stored_sizes(16, 32) == (16, 32) and D.stored_sizes(40, 80) == (48, 96) and D.stored_sizes(16, 72) == (48, 96) and D.stored_sizes(48, 16) == (48, 96)
    assert D.stored_sizes(7, 9) == (8, 16) and D.stored_sizes(5, 13) == (8, 16) and D.stored_sizes(132, 21) == (132, 22) and D.stored_sizes(128, 256) == (128, 256)


@pytest.mark.parametrize("n, base, scaling", [(8, 10000.0, None), (24, 20000.0, (3.0, 1.0, 4.0, 128)), (2, 50.0, (4.0, 2.0, 2.0, 16)), (6, 300.0, (2.0, 1.0, 8.0, 16)),
                                              (64, 500000.0, (8.0, 1.0, 4.0, 512)), (16, 100.0, (8.0, 0.5, 3.0, 64)), (4, 9.0, (4.0, 20.0, 30.0, 8))])
def test_the_table_of_angles_is_the_plain_one(n, base, scaling):
    from alofa_amd.parts.position import Rotary
    s = None if scaling is None else dict(zip(("factor", "low", "high", "original"), scaling))
    cos, sin = Rotary(PartSpec("rotary", {"theta": base, "head_dim": n + 4, "dims": n, "pairing": "half", "frequencies": "direct", "blend": s}), {}, None).host_table(900)
    assert cos.shape == (900, n // 2 + 2) and (cos[:, n // 2:] == 1).all() and (sin[:, n // 2:] == 0).all()
    one = np.zeros((900, 1, n + 4))
    one[:, 0, :n // 2] = 1.0      # a pair (1, 0) turns to (cos, sin)
    turned = pl.turn(one, np.arange(900), {"base": base, "dims": n, **({"scaling": s} if s else {})})[:, 0]
    assert np.abs(turned[:, :n // 2] - cos[:, :n // 2]).max() < 1e-6 and np.abs(turned[:, n // 2:n] - sin[:, :n // 2]).max() < 1e-6


def test_frequencies_by_their_turns():
    """Within 64 tokens: more than four turns stay, fewer than one are slowed down eight times, in between a straight blend of the two."""
    f = pl.frequencies(4, 10.0, None)
    s = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}
    turns = 64 * f / (2 * np.pi)
    assert turns[0] > 4 > turns[1] > 1
    got = pl.frequencies(4, 10.0, s)
    share = (turns[1] - 1.0) / 3.0
    assert got[0] == f[0] and np.isclose(got[1], share * f[1] + (1 - share) * f[1] / 8.0)
    assert np.allclose(pl.frequencies(4, 10.0, dict(s, original=2)), f / 8.0)


# ---- pages of kept tokens

def _manager(needs, n_blocks, bs):
    return CacheManager(needs, {}, n_blocks, block_size=bs, max_requests=4)


def _need(window, keep):
    return CacheNeed((CacheTensor("k", (1, SLOT, 2)),), window, keep)


def test_pages_of_kept_tokens_stay_while_the_window_goes_on():
    m = _manager([_need(8, 6), _need(8, 0), _need(8, 6)], 12, 4)
    assert [(g.window, g.keep_first, g.entries) for g in m.groups] == [(8, 6, [0, 2]), (8, 0, [1])]      # (what differs in kept tokens shares no tables)
    m.admit("a"), m.reserve("a", 3), m.commit("a", 3)
    m.reserve("a", 21), m.commit("a", 21)
    # the next row, at 21, sees 14 .. 21 and the first 6: blocks 0 and 1 stay, 2 goes
    assert [b >= 0 for b in m.table("a", 0)] == [True, True, False, True, True, True] and [b >= 0 for b in m.table("a", 1)] == [False, False, False, True, True, True]
    assert m.slots("a", 0, 0, 6) and m.slots("a", 0, 14, 7)
    m.reserve("a", 40), m.commit("a", 40)
    assert [i for i, b in enumerate(m.table("a", 0)) if b >= 0] == [0, 1, 8, 9]
    m.check()
    m.free("a")
    m.check()
    assert m.groups[0].pool.n_free == 12


@pytest.mark.parametrize("bs, window, keep", [(4, 5, 1), (4, 5, 4), (8, 17, 9), (16, 3, 40), (8, 1, 0)])
def test_what_a_request_holds_stays_within_what_is_counted(bs, window, keep):
    need = _need(window, keep)
    for step in (1, 3, 2 * bs):
        bound = CacheManager.pages_for(need.group, 1, 10_000, step, bs)
        m = _manager([need], bound, bs)
        m.admit("a")
        at = 0
        for _ in range(60):      # (no page more than the bound is ever asked for: reserve would refuse)
            m.reserve("a", at + step), m.commit("a", at + step)
            at += step
            held = [i for i, b in enumerate(m.table("a", 0)) if b >= 0]
            assert set(range(min(blocks_for(keep, bs), len(m.table("a", 0))))) <= set(held) and len(held) <= blocks_for(keep, bs) + blocks_for(window, bs) + 1
            m.check()
        rule = m.group_rules(step)[0]
        assert rule == (bound, window + step + 2 * bs + blocks_for(keep, bs) * bs)


def test_pools_by_group():
    needs = {0: _need(None, 0), 1: _need(16, 5), 2: _need(16, 0)}
    assert CacheManager.windows_of(needs) == [None, (16, 5), 16]
    m = _manager(needs, {None: 30, (16, 5): 7, 16: 5}, 8)
    assert [g.pool.n_blocks for g in m.groups] == [30, 7, 5]
    assert CacheManager.page_bytes(needs, 8) == {None: 32, (16, 5): 32, 16: 32}
    with pytest.raises(AlofaError, match="no page count"):
        _manager(needs, {None: 30, 16: 5}, 8)


# ---- the plain implementation against itself

@pytest.fixture(scope="module")
def model_a(tmp_path_factory):
    d = tmp_path_factory.mktemp("plain_a")
    write_model(NODOPEL["A"], d, 5)
    return pl.read_config(d), pl.read_weights(d)


def test_a_position_depends_on_nothing_after_it(model_a):
    cfg, w = model_a
    ids = [int(t) for t in np.random.default_rng(0).integers(0, cfg["vocab"], 40)]
    full = pl.forward_logits(w, cfg, ids)
    assert np.abs(pl.forward_logits(w, cfg, ids[:17]) - full[:17]).max() < 1e-9
    other = ids[:30] + [(ids[30] + 1) % cfg["vocab"]] + ids[31:]
    moved = np.abs(pl.forward_logits(w, cfg, other) - full).max(axis=1)
    assert moved[:30].max() < 1e-9 and moved[30:].min() > 1e-6


def test_one_head_written_out():
    """One key head, two query heads, key by key: each map has a softmax of its own, the window counts the row itself, the first tokens stay at their positions."""
    rng = np.random.default_rng(1)
    h, m = 6, {"heads": 2, "kv_heads": 1, "dim": 3, "vdim": 4, "rot": {"base": 10.0, "dims": 2}, "scale": 0.7, "softcap": 1.5, "diff": 0.4, "mask": {"size": 3, "keep_first": 2}}
    W = {k: rng.normal(0, 1, s) for k, s in {"q": (12, h), "k": (6, h), "v": (4, h), "o": (h, 8), "q.b": (12,), "k.b": (6,), "v.b": (4,), "lq1": (3,), "lk1": (3,), "lq2": (3,), "lk2": (3,)}.items()}
    x = rng.normal(0, 1, (9, h))
    got = pl.differential_attention(x, W, "", m, 1e-6)

    def turn(v, p):
        return np.array([v[0] * np.cos(p) - v[1] * np.sin(p), v[1] * np.cos(p) + v[0] * np.sin(p), v[2]])
    lam = np.exp(W["lq1"] @ W["lk1"]) - np.exp(W["lq2"] @ W["lk2"]) + 0.4
    for i in range(9):
        seen = [j for j in range(i + 1) if i - j < 3 or j < 2]
        heads = []
        for a in range(2):
            maps = []
            for n in range(2):
                q = turn((W["q"] @ x[i] + W["q.b"])[6 * a + 3 * n:][:3], i)
                e = [np.exp(1.5 * np.tanh(0.7 * (q @ turn((W["k"] @ x[j] + W["k.b"])[3 * n:][:3], j)) / 1.5)) for j in seen]
                maps.append(sum(y * (W["v"] @ x[j] + W["v.b"]) for y, j in zip(e, seen)) / sum(e))
            o = maps[0] - lam * maps[1]
            heads.append(o / np.sqrt(np.mean(o ** 2) + 1e-6) * 0.6)
        assert np.allclose(got[i], W["o"] @ np.concatenate(heads), atol=1e-7)      # (angles are 32-bit numbers)


def test_copies_of_the_stream_are_mixed_from_the_old_ones():
    X = np.arange(12.0).reshape(1, 2, 6)
    y = np.full((1, 6), 100.0)
    mix, out = np.array([[0.5, 2.0], [0.0, 3.0]]), np.array([1.0, -1.0])
    got = pl.write_streams(X, y, mix, out)
    assert np.allclose(got[0, 0], 0.5 * X[0, 0] + 100.0) and np.allclose(got[0, 1], 2.0 * X[0, 0] + 3.0 * X[0, 1] - 100.0)
    assert np.allclose(pl.read_streams(X, np.array([2.0, -1.0])), 2 * X[:, 0] - X[:, 1])


def test_the_choice_of_experts():
    x = np.array([[1.0, 0.0], [0.0, 1.0]])
    w_router = np.array([[0.5, 2.0], [3.0, 2.0], [0.5, -1.0], [2.0, 0.0]])
    chosen, weights = pl.route(x, w_router, np.array([0.0, 0.0, 0.7, 0.0]), 2)      # the correction lifts expert 2 but does not weigh it
    assert chosen.tolist() == [[2, 1], [2, 0]]
    e = np.exp(w_router @ x[0])
    assert np.allclose(weights[0], [e[2] / (e[1] + e[2]), e[1] / (e[1] + e[2])])


def test_an_identity_expert_hands_the_row_on():
    rng = np.random.default_rng(3)
    x = rng.normal(0, 1, (4, 6))
    mlp = {"router": {"experts": 1, "identity": 1, "top": 1}, "shared": {"ff": 3}}
    W = {"router": np.zeros((2, 6)), "correction": np.array([0.0, 1.0]), "shared.gate": rng.normal(0, 1, (3, 6)), "shared.up": rng.normal(0, 1, (3, 6)), "shared.down": rng.normal(0, 1, (6, 3))}
    z = x @ W["shared.gate"].T
    assert np.allclose(pl.mixture(x, W, "", mlp), x + (z / (1 + np.exp(-z)) * (x @ W["shared.up"].T)) @ W["shared.down"].T)
