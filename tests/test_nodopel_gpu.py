"""Nodopel through the engine against the plain implementation, in float32 and bfloat16: whole prompts, the stream after every layer run, every layer alone, decoding
token by token, portions down to two tokens, unequal requests in one batch, slots and pages that are used again, windows whose edges and kept tokens fall on, before and behind
page borders, weights made so that single keys, kept tokens, the cap, the second map, the turn or the copies of the stream decide, and greedy generation through the engine's
own loop."""
import copy
import json

import numpy as np
import pytest
import torch

from helpers import Reference, assert_close, bulk_and_tail, collect, mixed, portions, random_ids, whole
from nodopel_cases import NODOPEL, clear_calls, plain_logits, plain_model, write_model
from plain import nodopel as pl

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]
LENGTHS = {"A": 110, "B": 80, "C": 130, "D": 90, "E": 200}


@pytest.fixture(scope="module")
def replayers(nodopel_dirs):
    from alofa_amd.replay import Replayer
    made = {}

    def get(name, dtype, max_tokens=512):
        key = (name, dtype, max_tokens)
        if key not in made:
            made[key] = Replayer(nodopel_dirs[name], dtype, max_tokens, max_requests=4)
        r = made[key]
        assert not r.cache.requests, "a test left requests behind"
        return r
    return get


def ids_of(name, n=None, seed=7):
    return random_ids(seed, n or LENGTHS[name], NODOPEL[name]["vocab"])


def compare(got, model_dir, ids, dtype, what):
    rows = clear_calls(model_dir, ids, dtype)
    assert len(rows) >= max(8, 0.2 * len(ids)), f"{what}: too few positions are left to compare ({len(rows)} of {len(ids)})"
    assert_close(np.asarray(got)[rows], plain_logits(model_dir, tuple(ids))[rows], dtype, what)


def compare_together(results, model_dir, dtype, what):
    """Several requests of one model measured as one sample: what rounding alone does is an average."""
    picked = [(np.asarray(got)[rows], plain_logits(model_dir, tuple(ids)), rows) for got, ids in results for rows in [clear_calls(model_dir, ids, dtype)]]
    ref = np.concatenate([np.asarray(r)[rows] for _, r, rows in picked]).view(Reference)
    ref._rounded = lambda: np.concatenate([r.rounded()[rows] for _, r, rows in picked])
    assert len(ref) >= 60
    assert_close(np.concatenate([g for g, _, _ in picked]), ref, dtype, what)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(NODOPEL))
def test_whole_prompt(replayers, nodopel_dirs, name, dtype):
    ids = ids_of(name)
    compare(collect(replayers(name, dtype), whole("w", ids))["w"], nodopel_dirs[name], ids, dtype, f"{name} whole")


@pytest.mark.parametrize("name", list(NODOPEL))
def test_the_stream_after_every_layer_run(replayers, nodopel_dirs, name):
    """The sum of the copies, a looped layer as often as it is passed; and looking on changes nothing."""
    ids = ids_of(name, 45)
    r = replayers(name, "float32")
    seen = []
    r.fn.watch = lambda i, hidden: seen.append(hidden.detach().cpu().numpy().astype(np.float64))
    try:
        watched = collect(r, whole("w", ids))["w"]
    finally:
        r.fn.watch = None
    cfg, w = plain_model(str(nodopel_dirs[name]))
    want = pl.forward_hidden(w, cfg, ids)
    assert len(seen) == len(want) == len(pl.order(cfg))
    for i, (a, b) in enumerate(zip(seen, want)):
        assert np.abs(a - b).max() <= 1e-5 * max(1.0, np.abs(b).max()), f"layer run {i}"
    assert np.abs(watched - collect(r, whole("w", ids))["w"]).max() <= 1e-6 * max(1.0, np.abs(watched).max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,layer", [(n, i) for n in NODOPEL for i in range(len(NODOPEL[n]["layers"]))])
def test_every_layer_alone(tmp_path, name, layer, dtype):
    """One layer: whole, then token by token, then in portions."""
    from alofa_amd.replay import Replayer
    cfg = copy.deepcopy(NODOPEL[name])
    cfg["layers"] = [cfg["layers"][layer]]
    cfg.pop("loop", None)
    d = write_model(cfg, tmp_path / "m", 77 + layer)
    ids = ids_of(name, 75, seed=3)
    r = Replayer(d, dtype, 256, max_requests=2)
    for what, steps in (("whole", whole("a", ids)), ("decoding", bulk_and_tail("a", ids, tail=55)), ("portions", portions("a", ids))):
        compare(collect(r, steps)["a"], d, ids, dtype, f"{name} layer {layer} alone, {what}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(NODOPEL))
def test_prompt_then_token_by_token(replayers, nodopel_dirs, name, dtype):
    ids = ids_of(name)
    got = collect(replayers(name, dtype), bulk_and_tail("t", ids, tail=60))["t"]
    compare(got, nodopel_dirs[name], ids, dtype, f"{name} bulk+tail")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_from_the_first_token_one_by_one(replayers, nodopel_dirs, name, dtype):
    """Long decoding from nothing: single tokens only, past the kept tokens and every window of the configuration."""
    ids = ids_of(name, 80)
    got = collect(replayers(name, dtype), bulk_and_tail("t", ids, tail=79))["t"]
    compare(got, nodopel_dirs[name], ids, dtype, f"{name} one by one")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(NODOPEL))
def test_portions_of_changing_size(replayers, nodopel_dirs, name, dtype):
    ids = ids_of(name)
    steps = portions("p", ids)
    assert min(len(s["entries"][0]["tokens"]) for s in steps) == 2
    got = collect(replayers(name, dtype), steps)["p"]
    compare(got, nodopel_dirs[name], ids, dtype, f"{name} portions")
    other = collect(replayers(name, dtype), portions("q", ids, sizes=(2, 19, 2, 2, 33, 3, 17)))["q"]
    compare(other, nodopel_dirs[name], ids, dtype, f"{name} other portions")
    if dtype == "float32":      # the cut changes nothing beyond rounding
        assert np.abs(other - got).max() <= 4e-6 * max(1.0, np.abs(got).max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(NODOPEL))
def test_unequal_requests_together_with_slots_and_pages_used_again(nodopel_dirs, name, dtype):
    """Up to four live requests, seven in all: portions beside single tokens, a request left out now and then; a slot and its
    pages go to the next request as soon as one ends. Every request must come out as it does alone."""
    from alofa_amd.replay import Replayer
    top = LENGTHS[name]
    requests = {f"r{i}": ids_of(name, n, seed=200 + i) for i, n in enumerate([top, 37, top - 23, 64, 35, top - 9, 50])}
    steps, peak = mixed(requests, seed=9, tail=20)
    assert max(len(s["entries"]) for s in steps) >= 3
    r = Replayer(nodopel_dirs[name], dtype, peak, max_requests=4)
    got = collect(r, steps)
    r.cache.check()
    assert not r.cache.requests
    if dtype == "float32":
        for req, ids in requests.items():
            compare(got[req], nodopel_dirs[name], ids, dtype, f"{name} mixed {req}")
    else:
        compare_together([(got[req], ids) for req, ids in requests.items()], nodopel_dirs[name], dtype, f"{name} mixed")


def test_pools_of_what_the_windows_need(nodopel_dirs):
    """Pools that hold the windows and the kept tokens' pages and little more: pages come back behind the windows and go to whoever needs them next."""
    from alofa_amd.replay import Replayer
    requests = {f"r{i}": ids_of("E", n, seed=300 + i) for i, n in enumerate([300, 260, 310, 240, 280])}
    steps, _ = mixed(requests, seed=4, tail=150, max_live=3)
    longest = max(len(e["tokens"]) for s in steps for e in s["entries"])
    need = max(130 + 32, 65 + 80, 100 + 48, 90 + 64) + longest + 2 * 16
    r = Replayer(nodopel_dirs["E"], "float32", 3 * 320, blocks=3 * -(-need // 16), max_requests=3)
    got = collect(r, steps)
    r.cache.check()
    for req, ids in requests.items():
        compare(got[req], nodopel_dirs["E"], ids, "float32", f"small pools {req}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_and_long_decoding(nodopel_dirs, dtype):
    """Hundreds of tokens through the wider model: many tiles of keys behind the kept ones, steps of more rows than the experts' small tiles take, decoding across
    page borders and windows' edges."""
    from alofa_amd.replay import Replayer
    ids = ids_of("E", 700, seed=31)
    r = Replayer(nodopel_dirs["E"], dtype, 1408, max_requests=2)
    compare(collect(r, portions("p", ids, sizes=(300, 2, 150, 17, 3, 64, 5)))["p"], nodopel_dirs["E"], ids, dtype, "long, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=120))["t"], nodopel_dirs["E"], ids, dtype, "long, decoding")
    r.cache.check()


def test_a_slot_used_again_starts_from_nothing(replayers, nodopel_dirs):
    name = "A"
    r = replayers(name, "float32")
    a, b = ids_of(name, 60, seed=1), ids_of(name, 75, seed=2)
    first = collect(r, whole("a", a))["a"]
    collect(r, whole("b", b))
    again = collect(r, portions("a", a, sizes=(3, 2, 9)))["a"]
    assert np.abs(again - first).max() <= 4e-6 * max(1.0, np.abs(first).max())
    assert_close(again, plain_logits(nodopel_dirs[name], tuple(a)), "float32", "slot used again")


def _variant(base, out_dir, seed, change, weights=None):
    cfg = copy.deepcopy(NODOPEL[base])
    change(cfg)
    return write_model(cfg, out_dir, seed, weights)


def _only_attention(cfg, layers=None):
    cfg.pop("loop", None)
    cfg["layers"] = [cfg["layers"][i] for i in (layers or range(len(cfg["layers"])))]
    for l in cfg["layers"]:
        l["mlp"] = None


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window, keep", [(15, 16), (16, 15), (17, 17), (31, 1), (33, 32), (64, 33), (1, 4), (2, 0), (20, 64)])
@pytest.mark.parametrize("base", ["A", "C", "D"])      # (C: twenty query heads on one key head; D: widened heads, and a map for the always-valid kernel)
def test_windows_and_kept_tokens_around_page_borders_with_keys_that_decide(tmp_path, base, window, keep, dtype):
    """Scores scaled up until single keys carry much of the weight, and windows and kept tokens that end on a page's border, one before and one behind
    (pages of 16): a key too many or too few at a window's edge or at the end of the kept ones shows, in prompts' portions and in decoding."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        _only_attention(cfg)
        for l in cfg["layers"]:
            l["mixer"]["mask"] = {"size": window, "keep_first": keep}
            l["mixer"]["scale"] *= 3.0
            l["mixer"]["softcap"] = 60.0
    d = _variant(base, tmp_path / "w", 500 + window, change)
    ids = ids_of(base, 150, seed=11)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids, sizes=(67, 2, 16, 17, 3, 15)))["p"], d, ids, dtype, f"window {window} keep {keep}, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=70))["t"], d, ids, dtype, f"window {window} keep {keep}, decoding")
    cfg, w = plain_model(str(d))
    full = pl.forward_logits(w, cfg, ids)
    for key, other in (("size", window - 1), ("size", window + 1), ("keep_first", keep - 1), ("keep_first", keep + 1)):      # (one key more or less does show)
        if other > 0 or (key == "keep_first" and other == 0):
            moved = copy.deepcopy(cfg)
            for l in moved["layers"]:
                l["mixer"]["mask"][key] = other
            assert np.abs(pl.forward_logits(w, moved, ids) - full).max() > 0.05 * np.abs(full).max(), (key, other)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("place", ["kept", "edge"])
def test_a_far_key_that_decides(tmp_path, place, dtype):
    """One key hundreds of tokens back carries the weight of the last rows: among the kept first tokens, or at the far edge of a long window. With one kept token
    less, or the window one shorter, it is out of sight."""
    from alofa_amd.replay import Replayer
    n, logits = 341, {}
    at = 18 if place == "kept" else n - 1 - 200
    for inside in (True, False):
        mask = {"size": 40, "keep_first": 19 - (not inside)} if place == "kept" else {"size": 201 - (not inside), "keep_first": 3}

        def change(cfg):
            _only_attention(cfg, [0])
            cfg["layers"][0]["mixer"].update(scale=2.0, mask=mask, softcap=50.0)

        def weights(w):      # (the turned channels hardly count, so that scores hardly depend on positions)
            for t, heads in (("q", 4), ("k", 2)):
                for name in (f"l0.mix.{t}", f"l0.mix.{t}.b"):
                    x = w[name].float().reshape(heads * 2, 16, -1).clone()
                    x[:, :12] *= 0.1
                    x[:, 12:] *= 2.5
                    w[name] = x.reshape(w[name].shape).to(w[name].dtype)
        d = _variant("A", tmp_path / f"far{inside}", 950, change, weights)
        cfg, w = plain_model(str(d))
        m, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
        X = np.repeat(w["embed"][:, None], cfg["streams"], axis=1)
        u = pl.rms_norm(pl.read_streams(X, w["l0.hc1.in"]), w["l0.norm1"], eps)      # (every token of the vocabulary as if it stood at position 0)
        q, k = ((u @ w[f"l0.mix.{t}"].T + w[f"l0.mix.{t}.b"]).reshape(len(u), -1, 2, 16)[..., 12:] for t in "qk")
        ids = ids_of("A", n, seed=17)
        liked = k[:, 0, 0] @ q[ids[-1], 0, 0]
        liked[ids[-1]] = -1e9
        marker = int(liked.argmax())
        ids = [t if t != marker else (t + 1) % cfg["vocab"] for t in ids]
        ids[at] = marker
        r = Replayer(d, dtype, 384, max_requests=2)
        compare(collect(r, portions("p", ids, sizes=(150, 2, 61, 17, 3)))["p"], d, ids, dtype, f"far key {place} {inside}, portions")
        compare(collect(r, bulk_and_tail("t", ids, tail=30))["t"], d, ids, dtype, f"far key {place} {inside}, decoding")
        logits[inside] = pl.forward_logits(w, cfg, ids)[-1]
    assert np.abs(logits[True] - logits[False]).max() > 0.1 * np.abs(logits[True]).max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cap", [1.5, 54.0, 70.0])      # (up to 55 the kernels need no running maximum)
@pytest.mark.parametrize("base", ["A", "D"])
def test_the_cap_decides(tmp_path, base, cap, dtype):
    """Scores several times the cap: without it, or with it in another place, the weights are others."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        _only_attention(cfg)
        for l in cfg["layers"]:
            l["mixer"]["softcap"] = cap
            l["mixer"]["scale"] *= 1.0 if cap < 10 else 30.0      # (scores of a few, against a small cap, or beyond the large ones)
    d = _variant(base, tmp_path / "cap", 955, change)
    ids = ids_of(base, 100, seed=13)
    r = Replayer(d, dtype, 256, max_requests=2)
    if dtype == "float32" or cap < 10:
        compare(collect(r, portions("p", ids, sizes=(2, 47, 2, 16, 17, 3, 15)))["p"], d, ids, dtype, "cap, portions")
        compare(collect(r, bulk_and_tail("t", ids, tail=80))["t"], d, ids, dtype, "cap, decoding")
    else:      # (scores of a hundred turn rounding of queries and keys into other choices: finite, and the cuts agree about most rows)
        a, b = collect(r, portions("p", ids, sizes=(2, 47, 2, 16, 17, 3, 15)))["p"], collect(r, bulk_and_tail("t", ids, tail=80))["t"]
        assert np.isfinite(a).all() and np.isfinite(b).all()
    cfg, w = plain_model(str(d))
    other = copy.deepcopy(cfg)
    for l in other["layers"]:
        l["mixer"]["softcap"] = None
    full = pl.forward_logits(w, cfg, ids)
    assert np.abs(pl.forward_logits(w, other, ids) - full).max() > 0.03 * np.abs(full).max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("base", ["A", "C", "D"])
def test_the_second_map_and_the_biases_decide(tmp_path, base, dtype):
    """A large lambda (the second map outweighs the first), large biases: maps that change places, a lambda or a bias left out, show."""
    from alofa_amd.replay import Replayer

    def weights(w):
        for n in w:
            if n.endswith(("lq1", "lk1")):
                w[n] = torch.full_like(w[n], 0.2)
            if n.endswith((".q.b", ".k.b", ".v.b")):
                w[n] = w[n] * 3.0
    d = _variant(base, tmp_path / "lambda", 960, lambda cfg: _only_attention(cfg), weights)
    ids = ids_of(base, 100, seed=19)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids, sizes=(2, 47, 2, 16, 17, 3, 15)))["p"], d, ids, dtype, "lambda, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=99))["t"], d, ids, dtype, "lambda, decoding")
    cfg, w = plain_model(str(d))
    full = pl.forward_logits(w, cfg, ids)
    for gone in ("lq1", "q.b", "k.b", "v.b"):
        changed = {n: v * 0 if n.endswith("." + gone) else v for n, v in w.items()}
        assert np.abs(pl.forward_logits(changed, cfg, ids) - full).max() > 0.02 * np.abs(full).max(), gone


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("base", ["A", "C"])
def test_the_turn_decides(tmp_path, base, dtype):
    """Scores that are mostly the turned channels': positions one off, another pairing, frequencies that are not blended, show; and kept tokens stand at their true positions."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        _only_attention(cfg, [0])
        cfg["layers"][0]["mixer"]["scale"] *= 4.0
    d = _variant(base, tmp_path / "turned", 965, change)
    ids = ids_of(base, 140, seed=41)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids, sizes=(67, 2, 16, 17, 3, 15)))["p"], d, ids, dtype, "turned, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=60))["t"], d, ids, dtype, "turned, decoding")
    cfg, w = plain_model(str(d))
    plainly = copy.deepcopy(cfg)
    del plainly["layers"][0]["mixer"]["rot"]["scaling"]
    full = pl.forward_logits(w, cfg, ids)
    assert np.abs(pl.forward_logits(w, plainly, ids) - full).max() > 0.1 * np.abs(full).max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("streams", [1, 2, 5, 9])
def test_other_counts_of_copies(tmp_path, streams, dtype):
    """Mixing matrices far from the identity and from symmetry: one that is transposed, or copies that are mixed one after the other, show."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        cfg["streams"] = streams
        for l in cfg["layers"]:
            if l["mlp"] is not None:
                l["mlp"] = {"kind": "dense", "ff": 80}

    def weights(w):
        g = torch.Generator().manual_seed(streams)
        for n in w:
            if ".hc" in n:
                w[n] = (torch.randn(w[n].shape, generator=g) * 0.8 / streams ** 0.5 + (0.3 if n.endswith("in") else 0.0)).to(w[n].dtype)
    d = _variant("A", tmp_path / "copies", 968, change, weights)
    ids = ids_of("A", 70, seed=45)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids))["p"], d, ids, dtype, f"{streams} copies, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=30))["t"], d, ids, dtype, f"{streams} copies, decoding")
    if streams > 1:
        cfg, w = plain_model(str(d))
        full = pl.forward_logits(w, cfg, ids)
        turned = {n: v.T if n.endswith("mix") and ".hc" in n else v for n, v in w.items()}
        assert np.abs(pl.forward_logits(turned, cfg, ids) - full).max() > 0.05 * np.abs(full).max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("loop", [None, (0, 4, 1), (0, 1, 3), (3, 4, 2), (1, 4, 2)])
def test_loops(tmp_path, loop, dtype):
    """Every pass keeps pages of its own."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        cfg.pop("loop")
        if loop:
            cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
        for l in cfg["layers"]:
            if l["mlp"] is not None:
                l["mlp"] = {"kind": "dense", "ff": 72}
    d = _variant("A", tmp_path / "loop", 972, change)
    ids = ids_of("A", 70, seed=47)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids))["p"], d, ids, dtype, f"loop {loop}, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=30))["t"], d, ids, dtype, f"loop {loop}, decoding")


@pytest.mark.parametrize("dtype", DTYPES)
def test_no_window_no_cap_no_shared_expert_no_identity_expert(tmp_path, dtype):
    from alofa_amd.replay import Replayer

    def change(cfg):
        for l in cfg["layers"]:
            l["mixer"].pop("mask", None)
            l["mixer"].pop("softcap", None)
            if l["mlp"] is not None and l["mlp"]["kind"] == "moe":
                l["mlp"].pop("shared", None)
                l["mlp"]["router"].pop("identity")
    d = _variant("A", tmp_path / "open", 975, change)
    ids = ids_of("A", 150, seed=43)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids))["p"], d, ids, dtype, "open, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=50))["t"], d, ids, dtype, "open, decoding")


@pytest.mark.parametrize("page", [5, 8, 64])
def test_other_pages(nodopel_dirs, page):
    from alofa_amd.replay import Replayer
    for name, dtype in (("A", "float32"), ("A", "bfloat16"), ("C", "bfloat16")):
        ids = ids_of(name)
        r = Replayer(nodopel_dirs[name], dtype, 320, block_size=page, max_requests=2)
        compare(collect(r, portions("p", ids))["p"], nodopel_dirs[name], ids, dtype, f"{name} pages of {page}, portions")
        compare(collect(r, bulk_and_tail("t", ids, tail=40))["t"], nodopel_dirs[name], ids, dtype, f"{name} pages of {page}, decoding")


def test_which_kernels_serve_which_layer(replayers, monkeypatch):
    """In bfloat16 portions and single tokens go through the kernels for two maps; float32 and maps too wide for them go through the kernel that takes a wavefront per row
    and map."""
    from alofa_amd import ops
    calls = {}

    def counted(name):
        real = getattr(ops, name)

        def call(*a, **k):
            calls[name] = calls.get(name, 0) + 1
            return real(*a, **k)
        return call
    for name in ("maps_prefill", "maps_decode", "span_attention", "combine_maps", "experts_gate_up", "clamped_glu"):
        monkeypatch.setattr(ops, name, counted(name))

    def run(model, dtype, steps):
        calls.clear()
        collect(replayers(model, dtype), steps)
        return dict(calls)
    one = [{"step": 0, "entries": [{"id": "m", "tokens": [1], "want": []}], "end": ["m"]}]
    assert run("C", "bfloat16", whole("m", ids_of("C", 70))) == {"maps_prefill": 9, "experts_gate_up": 3}
    assert run("C", "bfloat16", one) == {"maps_decode": 9, "experts_gate_up": 3}
    assert run("C", "float32", whole("m", ids_of("C", 70))) == {"span_attention": 9, "combine_maps": 9, "clamped_glu": 3}
    assert run("D", "bfloat16", whole("m", ids_of("D", 70))) == {"maps_prefill": 3, "span_attention": 1, "combine_maps": 1, "experts_gate_up": 1}
    both = [{"step": 0, "entries": [{"id": "m", "tokens": ids_of("C", 30), "want": []}, {"id": "n", "tokens": [5, 6], "want": []}], "end": ["m", "n"]}]
    assert run("C", "bfloat16", both) == {"maps_prefill": 9, "maps_decode": 9, "experts_gate_up": 3}


def test_greedy_generation_through_the_engine(nodopel_dirs):
    """The engine's own loop and scheduler: prompts of unequal length, more than a batch holds at once, longer than the windows."""
    from alofa_amd import Engine
    for name in ("A", "B", "C"):
        cfg, w = plain_model(str(nodopel_dirs[name]))
        prompts = [random_ids(300 + i, n, cfg["vocab"]) for i, n in enumerate((5, 23, 2, 61, 17, 44))]
        want = [pl.greedy(w, cfg, p, 8) for p in prompts]
        engine = Engine(nodopel_dirs[name], dtype="float32", max_tokens=96, max_batch=4, token_budget=48, max_chunk=16)
        assert engine.generate(prompts, max_new=8) == want, name
        engine.cache.check()
        got = Engine(nodopel_dirs[name], dtype="bfloat16", max_tokens=96, max_batch=4).generate(prompts, max_new=8)
        agree = sum(a == b for g, r in zip(got, want) for a, b in zip(g, r))
        assert agree >= 30, f"{name}: {agree}/48 greedy tokens agree with the plain model in bfloat16"


def test_decode_steps_replay_a_captured_graph(replayers, nodopel_dirs):
    """Every replay must fill the next slot of the pages; other requests' eager steps lie between."""
    for name in ("A", "C", "D", "E"):
        r = replayers(name, "bfloat16")
        if not r.fn.use_graphs:
            pytest.skip("graphs are switched off")
        ids = ids_of(name, 90)
        before = r.fn.graph_replays
        steps = bulk_and_tail("t", ids, tail=50)
        other = portions("o", ids_of(name, 40, seed=2), sizes=(5, 2, 9))
        woven = []
        for i, s in enumerate(steps):
            woven.append(s)
            if i % 4 == 3 and other:
                woven.append(other.pop(0))
        got = collect(r, woven + other)["t"]
        assert r.fn.graph_replays > before
        compare(got, nodopel_dirs[name], ids, "bfloat16", f"{name} graph decode")


def test_the_programs_take_the_design_by_its_config(nodopel_dirs, tmp_path):
    """bin/generate and bin/trace_run on a folder of this design."""
    import os
    import subprocess
    from conftest import ROOT
    d = nodopel_dirs["A"]
    cfg, w = plain_model(str(d))
    prompts = [random_ids(1, 5, cfg["vocab"]), random_ids(2, 19, cfg["vocab"])]
    want = [pl.greedy(w, cfg, p, 5) for p in prompts]
    env = dict(os.environ, ALOFA_WEIGHTS=str(d), ALOFA_DTYPE="float32", ALOFA_MAX_NEW="5", ALOFA_MAX_TOKENS="64",
               ALOFA_PROMPT_IDS=";".join(",".join(map(str, p)) for p in prompts))
    p = subprocess.run([str(ROOT / "bin" / "generate")], env=env, capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [[int(t) for t in line.split(",")] for line in p.stdout.strip().splitlines()] == want
    ids = random_ids(12, 70, cfg["vocab"])
    steps = portions("a", ids, sizes=(33, 2, 1, 1, 20, 1))
    text = "".join(json.dumps(s) + "\n" for s in steps)
    p = subprocess.run([str(ROOT / "bin" / "trace_run"), "--model", str(d), "--dtype", "float32", "--out", str(tmp_path / "out"), "--max-tokens", "128"],
                       input=text, capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert p.stdout.split("\n")[:-1] == [f"done {s['step']}" for s in steps]
    got = np.concatenate([np.fromfile(tmp_path / "out" / f"{s['step']}.f32", dtype="<f4").reshape(-1, cfg["vocab"]) for s in steps])
    assert_close(got, plain_logits(d, tuple(ids)), "float32", "program")
