"""Lalepel without a GPU: the configuration's keys and checks, the tensor list, what every layer keeps per token and per request, the table
of angles, and the plain implementation's own consistency."""
import copy
import json

import numpy as np
import pytest

from alofa_amd.config.base import PartSpec
from alofa_amd.config.registry import config_from_dict, load_config
from alofa_amd.errors import AlofaError
from alofa_amd.model import check_spec, expected_tensors
from alofa_amd.weights import write_random_model
from lalepel_cases import LALEPEL
from plain import lalepel as pl


@pytest.mark.parametrize("name", list(LALEPEL))
def test_config_round_trip_and_tensor_list(name, tmp_path):
    cfg = config_from_dict(LALEPEL[name])
    assert config_from_dict(cfg.to_dict()) == cfg
    spec = cfg.spec()
    check_spec(spec)
    write_random_model(LALEPEL[name], tmp_path, seed=1)
    assert load_config(tmp_path) == cfg
    w = pl.read_weights(tmp_path)
    expected = expected_tensors(spec)
    assert set(w) == {n for n, r in expected.items() if not r.optional}
    assert all(tuple(w[n].shape) == tuple(expected[n].shape) for n in w)
    h = LALEPEL[name]["width"]
    for i, l in enumerate(LALEPEL[name]["layers"]):
        p, m, mlp = f"l{i}.", l["mixer"], l["mlp"]
        assert w[p + "norm1"].shape == (h,) and (p + "norm2" in w) == (mlp is not None)
        if l["type"] == "latent_attention":
            assert w[p + "mix.dq"].shape == (m["q_rank"], h) and w[p + "mix.uq"].shape == (m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"])
            assert w[p + "mix.dkv"].shape == (m["kv_rank"] + m["rot_dim"], h) and w[p + "mix.dkv.norm"].shape == (m["kv_rank"],)
            assert w[p + "mix.uk"].shape == (m["heads"] * m["dim"], m["kv_rank"]) and w[p + "mix.uv"].shape == (m["heads"] * m["vdim"], m["kv_rank"])
            assert w[p + "mix.sink"].shape == (m["heads"],) and p + "mix.g" not in w
        else:
            assert w[p + "mix.g"].shape == (m["heads"] * m["vdim"], h) and p + "mix.sink" not in w
        if mlp is not None and mlp["kind"] == "moe":
            assert w[p + "mlp.router.b"].shape == (mlp["router"]["experts"],) and p + "mlp.e0.gate" not in w
            assert (p + "mlp.shared.sg" in w) == (p + "mlp.shared.up" in w) == ("shared" in mlp)


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="attention"), "no such mixer"),
    (lambda c: c["layers"][1]["mlp"].update(kind="glu"), "no such feed-forward"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "more experts than there are"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6), "the size of a head's turned part"),
    (lambda c: c["layers"][0]["mixer"].update(rot_dim=7), "the size of a head's turned part"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "must be positive"),
    (lambda c: c["layers"][0]["mixer"].pop("q_rank"), "lacks a required key"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("fast"), "lacks a required key"),
    (lambda c: c["layers"][1]["mixer"]["decay"].append(0.5), "one decay per head"),
    (lambda c: c["layers"][1]["mlp"]["shared"].update(ff=0), "must be positive"),
    (lambda c: c.update(layers=[]), "at least one layer"),
])
def test_what_the_configuration_refuses(change, message):
    raw = copy.deepcopy(LALEPEL["A"])
    change(raw)
    with pytest.raises(AlofaError, match=message):
        config_from_dict(raw)


def test_weights_that_do_not_fit_are_named(tmp_path):
    from alofa_amd.weights.loader import load_weights
    write_random_model(LALEPEL["A"], tmp_path, seed=1)
    raw = json.loads((tmp_path / "config.json").read_text())
    raw["layers"][0]["mixer"]["q_rank"] = 41
    (tmp_path / "config.json").write_text(json.dumps(raw))
    with pytest.raises(AlofaError, match=r"l0\.mix\.dq"):
        load_weights(tmp_path, expected_tensors(load_config(tmp_path).spec()))


def test_every_layer_reads_the_stream_and_norms_what_it_adds():
    spec = config_from_dict(LALEPEL["A"]).spec()
    assert [l.block.kind for l in spec.layers] == ["postnorm"] * 4
    assert [len(l.parts["norms"]) for l in spec.layers] == [2, 2, 1, 2]
    assert [l.parts["mixer"].kind for l in spec.layers] == ["latent_attention", "retention", "latent_attention", "retention"]
    assert spec.layers[0].parts["mixer"].params["window"] == 20 and spec.layers[1].parts["mixer"].params["position"] is None


@pytest.mark.parametrize("n, base, scaling", [(8, 10000.0, None), (24, 20000.0, (3.0, 128, 16.0, 2.0)), (2, 50.0, None), (6, 300.0, (2.0, 16, 2.0, 1.5)),
                                              (48, 150000.0, (6.0, 512, 24.0, 2.0)), (16, 100.0, (8.0, 4096, 0.5, 0.1)), (2, 9.0, (4.0, 8, 1.0, 0.9))])
def test_the_table_of_angles_is_the_plain_one(n, base, scaling):
    from alofa_amd.parts.position import Rotary
    s = None if scaling is None else dict(zip(("factor", "original", "fast", "slow"), scaling))
    cos, sin = Rotary(PartSpec("rotary", {"theta": base, "head_dim": n, "pairing": "neighbours", "frequencies": "direct", "stretch": s}), {}, None).host_table(900)
    assert cos.shape == (900, n // 2)
    one = np.zeros((900, n))
    one[:, 0::2] = 1.0      # a pair (1, 0) turns to (cos, sin)
    turned = pl.turn(one, np.arange(900), base, s)
    assert np.abs(turned[:, 0::2] - cos).max() < 1e-6 and np.abs(turned[:, 1::2] - sin).max() < 1e-6


# ---- the plain implementation against itself

@pytest.fixture(scope="module")
def model_a(tmp_path_factory):
    d = tmp_path_factory.mktemp("plain_a")
    write_random_model(LALEPEL["A"], d, seed=5)
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
    """Latent attention with one head, key by key: the score is the sum of both products, the window counts the row itself, the sink stands
    in the denominator alone."""
    rng = np.random.default_rng(1)
    h, m = 6, {"heads": 1, "dim": 3, "rot_dim": 2, "vdim": 4, "q_rank": 5, "kv_rank": 4, "rot": {"base": 10.0, "dims": 2}, "scale": 0.7, "mask": {"size": 3}}
    W = {k: rng.normal(0, 1, s) for k, s in {"dq": (5, h), "dq.norm": (5,), "uq": (5, 5), "dkv": (6, h), "dkv.norm": (4,), "uk": (3, 4), "uv": (4, 4), "sink": (1,), "o": (h, 4)}.items()}
    x = rng.normal(0, 1, (9, h))
    got = pl.latent_attention(x, W, "", m, 1e-6)

    def normed(v, w):
        return v / np.sqrt(np.mean(v ** 2) + 1e-6) * w

    def turn(v, p):
        return np.array([v[0] * np.cos(p) - v[1] * np.sin(p), v[1] * np.cos(p) + v[0] * np.sin(p)])
    q = [W["uq"] @ normed(W["dq"] @ r, W["dq.norm"]) for r in x]
    down = [W["dkv"] @ r for r in x]
    c = [normed(d[:4], W["dkv.norm"]) for d in down]
    for i in range(9):
        seen = [j for j in range(9) if 0 <= i - j < 3]
        e = [np.exp(0.7 * (q[i][:3] @ (W["uk"] @ c[j]) + turn(q[i][3:], i) @ turn(down[j][4:], j))) for j in seen]
        out = sum(a * (W["uv"] @ c[j]) for a, j in zip(e, seen)) / (sum(e) + np.exp(W["sink"][0]))
        assert np.allclose(got[i], W["o"] @ out, atol=1e-9)


def test_retention_is_its_unrolled_sum():
    rng = np.random.default_rng(2)
    m = {"heads": 2, "dim": 3, "vdim": 4, "decay": [0.5, 0.9]}
    W = {k: rng.normal(0, 1, s) for k, s in {"q": (6, 5), "k": (6, 5), "v": (8, 5), "g": (8, 5), "o": (5, 8)}.items()}
    x = rng.normal(0, 1, (7, 5))
    q, k, v = ((x @ W[n].T).reshape(7, 2, -1) for n in "qkv")
    y = np.zeros((7, 8))
    for t in range(7):
        for a in range(2):
            o = sum(m["decay"][a] ** (t - s) * (q[t, a] @ k[s, a]) / np.sqrt(3) * v[s, a] for s in range(t + 1))
            y[t, 4 * a:4 * a + 4] = o / np.sqrt(np.mean(o ** 2) + 1e-5)
    z = x @ W["g"].T
    assert np.allclose(pl.retention(x, W, "", m, 1e-5), (y * z / (1 + np.exp(-z))) @ W["o"].T, atol=1e-9)


def test_the_choice_of_experts():
    x = np.array([[1.0, 0.0], [0.0, 1.0]])
    w_router = np.array([[0.5, 2.0], [3.0, 2.0], [0.5, -1.0], [2.0, 0.0]])
    chosen, weights = pl.route(x, w_router, np.array([0.0, 0.0, 0.0, 1.0]), 2)      # the bias lifts expert 3 level with expert 1
    assert chosen.tolist() == [[1, 3], [0, 1]]
    assert np.allclose(weights, [[0.5, 0.5], [0.5, 0.5]])
    _, weights = pl.route(x, w_router, np.array([0.0, 0.0, 0.0, 0.0]), 2)
    assert np.allclose(weights[0], [1 / (1 + np.exp(-1.0)), 1 / (1 + np.exp(1.0))])      # (over the chosen two alone)


def test_the_shared_expert_is_gated():
    rng = np.random.default_rng(3)
    x = rng.normal(0, 1, (4, 6))
    mlp = {"router": {"experts": 2, "top": 1}, "shared": {"ff": 3}}
    W = {"router": rng.normal(0, 1, (2, 6)), "router.b": np.array([1e6, 0.0]), "e0.up": rng.normal(0, 1, (5, 6)), "e0.down": rng.normal(0, 1, (6, 5)),
         "e1.up": np.zeros((5, 6)), "e1.down": np.zeros((6, 5)), "shared.up": rng.normal(0, 1, (3, 6)), "shared.down": rng.normal(0, 1, (6, 3)), "shared.sg": rng.normal(0, 1, (1, 6))}
    one = np.maximum(x @ W["e0.up"].T, 0) ** 2 @ W["e0.down"].T
    two = np.maximum(x @ W["shared.up"].T, 0) ** 2 @ W["shared.down"].T
    assert np.allclose(pl.mixture(x, W, "", mlp), one + two / (1 + np.exp(-(x @ W["shared.sg"].T))))
