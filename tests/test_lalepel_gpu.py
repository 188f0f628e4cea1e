"""Lalepel through the engine against the plain implementation, in float32 and bfloat16: whole prompts, the stream after every layer, every
mixer alone, decoding token by token, portions down to two tokens, unequal requests in one batch, slots and pages that are used again,
windows whose edges fall on, before and behind page borders, weights made so that single keys, the sink, the turned part or an old token
decide, and greedy generation through the engine's own loop."""
import copy
import json

import numpy as np
import pytest

from helpers import Reference, assert_close, bulk_and_tail, collect, mixed, portions, random_ids, whole
from lalepel_cases import LALEPEL, clear_calls, plain_logits, plain_model
from plain import lalepel as pl

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]
LENGTHS = {"A": 110, "B": 80, "C": 130, "D": 90, "E": 200}


@pytest.fixture(scope="module")
def replayers(lalepel_dirs):
    from alofa_amd.replay import Replayer
    made = {}

    def get(name, dtype, max_tokens=512):
        key = (name, dtype, max_tokens)
        if key not in made:
            made[key] = Replayer(lalepel_dirs[name], dtype, max_tokens, max_requests=4)
        r = made[key]
        assert not r.cache.requests, "a test left requests behind"
        return r
    return get


def ids_of(name, n=None, seed=7):
    return random_ids(seed, n or LENGTHS[name], LALEPEL[name]["vocab"])


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
@pytest.mark.parametrize("name", list(LALEPEL))
def test_whole_prompt(replayers, lalepel_dirs, name, dtype):
    ids = ids_of(name)
    compare(collect(replayers(name, dtype), whole("w", ids))["w"], lalepel_dirs[name], ids, dtype, f"{name} whole")


@pytest.mark.parametrize("name", list(LALEPEL))
def test_the_stream_after_every_layer(replayers, lalepel_dirs, name):
    ids = ids_of(name, 45)
    r = replayers(name, "float32")
    seen = []
    r.fn.watch = lambda i, hidden: seen.append(hidden.detach().cpu().numpy().astype(np.float64))
    try:
        collect(r, whole("w", ids))
    finally:
        r.fn.watch = None
    cfg, w = plain_model(str(lalepel_dirs[name]))
    want = pl.forward_hidden(w, cfg, ids)
    assert len(seen) == len(want) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(seen, want)):
        assert np.abs(a - b).max() <= 1e-5 * max(1.0, np.abs(b).max()), f"layer {i} ({cfg['layers'][i]['type']})"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,layer", [(n, i) for n in LALEPEL for i in range(len(LALEPEL[n]["layers"]))])
def test_every_layer_alone(tmp_path, name, layer, dtype):
    """One layer: whole, then token by token, then in portions."""
    from alofa_amd.replay import Replayer
    from alofa_amd.weights import write_random_model
    cfg = copy.deepcopy(LALEPEL[name])
    cfg["layers"] = [cfg["layers"][layer]]
    d = write_random_model(cfg, tmp_path / "m", seed=77 + layer)
    ids = ids_of(name, 75, seed=3)
    r = Replayer(d, dtype, 256, max_requests=2)
    for what, steps in (("whole", whole("a", ids)), ("decoding", bulk_and_tail("a", ids, tail=55)), ("portions", portions("a", ids))):
        compare(collect(r, steps)["a"], d, ids, dtype, f"{name} layer {layer} alone, {what}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(LALEPEL))
def test_prompt_then_token_by_token(replayers, lalepel_dirs, name, dtype):
    ids = ids_of(name)
    got = collect(replayers(name, dtype), bulk_and_tail("t", ids, tail=60))["t"]
    compare(got, lalepel_dirs[name], ids, dtype, f"{name} bulk+tail")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_from_the_first_token_one_by_one(replayers, lalepel_dirs, name, dtype):
    """Long decoding from nothing: single tokens only, past every window of the configuration."""
    ids = ids_of(name, 80)
    got = collect(replayers(name, dtype), bulk_and_tail("t", ids, tail=79))["t"]
    compare(got, lalepel_dirs[name], ids, dtype, f"{name} one by one")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(LALEPEL))
def test_portions_of_changing_size(replayers, lalepel_dirs, name, dtype):
    ids = ids_of(name)
    steps = portions("p", ids)
    assert min(len(s["entries"][0]["tokens"]) for s in steps) == 2
    got = collect(replayers(name, dtype), steps)["p"]
    compare(got, lalepel_dirs[name], ids, dtype, f"{name} portions")
    other = collect(replayers(name, dtype), portions("q", ids, sizes=(2, 19, 2, 2, 33, 3, 17)))["q"]
    compare(other, lalepel_dirs[name], ids, dtype, f"{name} other portions")
    if dtype == "float32":      # the cut changes nothing beyond rounding
        assert np.abs(other - got).max() <= 4e-6 * max(1.0, np.abs(got).max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(LALEPEL))
def test_unequal_requests_together_with_slots_and_pages_used_again(lalepel_dirs, name, dtype):
    """Up to four live requests, seven in all: portions beside single tokens, a request left out now and then; a slot and its
    pages go to the next request as soon as one ends. Every request must come out as it does alone."""
    from alofa_amd.replay import Replayer
    top = LENGTHS[name]
    requests = {f"r{i}": ids_of(name, n, seed=200 + i) for i, n in enumerate([top, 37, top - 23, 64, 35, top - 9, 50])}
    steps, peak = mixed(requests, seed=9, tail=20)
    assert max(len(s["entries"]) for s in steps) >= 3
    r = Replayer(lalepel_dirs[name], dtype, peak, max_requests=4)
    got = collect(r, steps)
    r.cache.check()
    assert not r.cache.requests
    if dtype == "float32":
        for req, ids in requests.items():
            compare(got[req], lalepel_dirs[name], ids, dtype, f"{name} mixed {req}")
    else:
        compare_together([(got[req], ids) for req, ids in requests.items()], lalepel_dirs[name], dtype, f"{name} mixed")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_and_long_decoding(lalepel_dirs, dtype):
    """Hundreds of tokens through the wider model: several tiles of keys a row, steps of more rows than the experts' small tiles take, decoding across
    page borders and windows' edges."""
    from alofa_amd.replay import Replayer
    ids = ids_of("E", 700, seed=31)
    r = Replayer(lalepel_dirs["E"], dtype, 1408, max_requests=2)
    compare(collect(r, portions("p", ids, sizes=(300, 2, 150, 17, 3, 64, 5)))["p"], lalepel_dirs["E"], ids, dtype, "long, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=120))["t"], lalepel_dirs["E"], ids, dtype, "long, decoding")
    r.cache.check()


def test_a_slot_used_again_starts_from_nothing(replayers, lalepel_dirs):
    """The same request twice in the same slot, a different one between them: the state and the pages that an earlier owner left must not show."""
    name = "A"
    r = replayers(name, "float32")
    a, b = ids_of(name, 60, seed=1), ids_of(name, 75, seed=2)
    first = collect(r, whole("a", a))["a"]
    collect(r, whole("b", b))
    again = collect(r, portions("a", a, sizes=(3, 2, 9)))["a"]
    assert np.abs(again - first).max() <= 4e-6 * max(1.0, np.abs(first).max())
    assert_close(again, plain_logits(lalepel_dirs[name], tuple(a)), "float32", "slot used again")


def _variant(cfg, out_dir, seed, change, weights=None):
    from alofa_amd.weights import write_random_model
    cfg = copy.deepcopy(cfg)
    change(cfg)
    d = write_random_model(cfg, out_dir, seed=seed)
    if weights is not None:
        from safetensors.torch import load_file, save_file
        w = load_file(str(d / "model.safetensors"))
        weights(w)
        save_file(w, str(d / "model.safetensors"))
    return d


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [15, 16, 17, 31, 33, 64, 1, 2])
@pytest.mark.parametrize("base", ["A", "C", "D"])      # (C: twenty heads and seven that share tiles; D: every head's keys in the pages)
def test_windows_around_page_borders_with_keys_that_decide(tmp_path, base, window, dtype):
    """Scores scaled up until single keys carry much of the weight, sinks made small, and windows that end on a page's border, one before
    and one behind (pages of 16), and of one and two keys: a key too many or too few at a window's edge shows in every logit, in prompts'
    portions and in decoding."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        cfg["layers"] = [l for l in cfg["layers"] if l["type"] == "latent_attention"]
        for l in cfg["layers"]:
            l["mixer"]["mask"]["size"] = window
            l["mixer"]["scale"] *= 3.0
            l["mlp"] = None

    def weights(w):
        for n in w:
            if n.endswith("sink"):
                w[n] = w[n] - 4.0
    d = _variant(LALEPEL[base], tmp_path / "w", 500 + window, change, weights)
    ids = ids_of(base, 150, seed=11)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids, sizes=(67, 2, 16, 17, 3, 15)))["p"], d, ids, dtype, f"window {window}, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=70))["t"], d, ids, dtype, f"window {window}, decoding")
    cfg, w = plain_model(str(d))
    full = pl.forward_logits(w, cfg, ids)
    for other in (window - 1, window + 1):      # (one key more or less does show: far above the rounding that is allowed for)
        if other:
            moved = copy.deepcopy(cfg)
            for l in moved["layers"]:
                l["mixer"]["mask"]["size"] = other
            assert np.abs(pl.forward_logits(w, moved, ids) - full).max() > 0.05 * np.abs(full).max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("far", [127, 128, 300])
def test_a_far_key_that_decides(tmp_path, far, dtype):
    """One key at the far edge of a long window carries the weight: the unturned part of queries and keys is scaled up, and the token there is
    the one of the vocabulary whose key the last token's query likes best. Inside the window it decides the last logits; with the window one
    shorter it is out of it."""
    from alofa_amd.replay import Replayer

    def layout(size):
        def change(cfg):
            cfg["layers"] = [cfg["layers"][0]]
            cfg["layers"][0]["mixer"].update(scale=2.0)
            cfg["layers"][0]["mixer"]["mask"]["size"] = size
            cfg["layers"][0]["mlp"] = None
        return change

    def weights(w):
        w["l0.mix.sink"] = w["l0.mix.sink"] - 8.0
        q = w["l0.mix.uq"].float().view(3, 24, -1)
        q[:, 16:] *= 0.1                       # (the turned part hardly counts, so that scores hardly depend on positions)
        w["l0.mix.uq"] = q.view(72, -1).to(w["l0.mix.uq"].dtype)
    logits = {}
    for size in (far, far + 1):
        d = _variant(LALEPEL["A"], tmp_path / f"far{size}", 950, layout(size), weights)
        cfg, w = plain_model(str(d))
        m, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
        qn, _, c, _ = pl.latent_pieces(w["embed"], w, "l0.mix.", m, eps)       # (every token of the vocabulary as if it were a sequence: only what is not turned is used)
        kn = (c @ w["l0.mix.uk"].T).reshape(-1, m["heads"], m["dim"])
        ids = ids_of("A", far + 40, seed=17)
        liked = (kn[:, 0] @ qn[ids[-1], 0])
        liked[ids[-1]] = -1e9
        marker = int(liked.argmax())
        ids = [t if t != marker else (t + 1) % cfg["vocab"] for t in ids]
        ids[len(ids) - 1 - far] = marker
        r = Replayer(d, dtype, 384, max_requests=2)
        compare(collect(r, portions("p", ids, sizes=(150, 2, 61, 17, 3)))["p"], d, ids, dtype, f"far key {size}, portions")
        compare(collect(r, bulk_and_tail("t", ids, tail=30))["t"], d, ids, dtype, f"far key {size}, decoding")
        logits[size] = pl.forward_logits(w, cfg, ids)[-1]
    assert np.abs(logits[far] - logits[far + 1]).max() > 0.1 * np.abs(logits[far]).max()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("base", ["A", "C", "D"])
def test_the_sink_decides(tmp_path, base, dtype):
    """Sinks made large (nearly all the weight leaves through them) in some heads and very negative in others: a sink left out, counted twice,
    once per part of the keys, or scaled, shows; also for the first tokens, where there is little beside it."""
    from alofa_amd.replay import Replayer
    import torch

    def change(cfg):
        cfg["layers"] = [l for l in cfg["layers"] if l["type"] == "latent_attention"]
        for l in cfg["layers"]:
            l["mlp"] = None

    def weights(w):
        for n in w:
            if n.endswith("sink"):
                w[n] = torch.tensor([(5.0, -30.0, 2.0, 0.0, 9.0)[i % 5] for i in range(len(w[n]))], dtype=w[n].dtype)
    d = _variant(LALEPEL[base], tmp_path / "sink", 960, change, weights)
    ids = ids_of(base, 100, seed=19)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids, sizes=(2, 47, 2, 16, 17, 3, 15)))["p"], d, ids, dtype, "sink, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=99))["t"], d, ids, dtype, "sink, decoding")
    cfg, w = plain_model(str(d))
    full = pl.forward_logits(w, cfg, ids)
    for other in (-1e9, np.log(2.0)):      # without the sinks, and with every one counted twice
        changed = {n: v if not n.endswith("sink") else (v + other if other > 0 else np.full_like(v, other)) for n, v in w.items()}
        assert np.abs(pl.forward_logits(changed, cfg, ids) - full).max() > 0.05


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("base", ["A", "D"])
def test_the_turned_part_decides(tmp_path, base, dtype):
    """The turned part scaled up until it makes most of the score: positions one off, a pair taken the wrong way round, a stretch or its factor
    left out, show."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        cfg["layers"] = [cfg["layers"][0]]
        cfg["layers"][0]["mlp"] = None

    def weights(w):
        m = LALEPEL[base]["layers"][0]["mixer"]
        q = w["l0.mix.uq"].float().view(m["heads"], m["dim"] + m["rot_dim"], -1)
        q[:, m["dim"]:] *= 4.0
        w["l0.mix.uq"] = q.reshape(w["l0.mix.uq"].shape).to(w["l0.mix.uq"].dtype)
    d = _variant(LALEPEL[base], tmp_path / "turned", 965, change, weights)
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
def test_an_old_token_in_the_state(tmp_path, dtype):
    """Decays near one: what the first tokens wrote still decides hundreds of tokens later, through portions, decoding and a slot that another
    request used between."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        cfg["layers"] = [cfg["layers"][1], cfg["layers"][3]]
        cfg["layers"][0]["mixer"]["decay"] = [1.0, 0.99951171875]
        cfg["layers"][0]["mlp"] = None
    d = _variant(LALEPEL["A"], tmp_path / "old", 970, change)
    ids = ids_of("A", 300, seed=23)
    r = Replayer(d, dtype, 384, max_requests=2)
    compare(collect(r, portions("p", ids, sizes=(130, 2, 61, 17, 3)))["p"], d, ids, dtype, "old token, portions")
    collect(r, whole("other", ids_of("A", 50, seed=5)))
    compare(collect(r, bulk_and_tail("t", ids, tail=60))["t"], d, ids, dtype, "old token, decoding")
    cfg, w = plain_model(str(d))
    assert np.abs(pl.forward_logits(w, cfg, ids)[-1] - pl.forward_logits(w, cfg, ids[150:])[-1]).max() > 0.05      # (the first half still counts at the end)


@pytest.mark.parametrize("dtype", DTYPES)
def test_layers_without_a_window_or_a_shared_expert(tmp_path, dtype):
    """No mask: every earlier key is seen (and pages are kept for good)."""
    from alofa_amd.replay import Replayer

    def change(cfg):
        for l in cfg["layers"]:
            if l["type"] == "latent_attention":
                del l["mixer"]["mask"]
            elif l["mlp"] is not None:
                l["mlp"].pop("shared", None)
    d = _variant(LALEPEL["A"], tmp_path / "open", 975, change)
    ids = ids_of("A", 150, seed=43)
    r = Replayer(d, dtype, 256, max_requests=2)
    compare(collect(r, portions("p", ids))["p"], d, ids, dtype, "no window, portions")
    compare(collect(r, bulk_and_tail("t", ids, tail=50))["t"], d, ids, dtype, "no window, decoding")


def test_which_kernels_serve_which_layer(replayers, monkeypatch):
    """In bfloat16 the latents are one key head of the engine's matrix-core kernels; heads of a size that no prefill kernel is built for take the
    window part's matrix-core kernel for portions; float32 and odd sizes go through the kernel that takes a wavefront per row and head."""
    from alofa_amd import ops
    calls = {}

    def counted(name):
        real = getattr(ops, name)

        def call(*a, **k):
            calls[name] = calls.get(name, 0) + 1
            return real(*a, **k)
        return call
    for name in ("attention_prefill", "attention_decode", "span_attention", "span_attention_mfma", "experts_up", "weighted_relu_squared", "chunked_recurrence", "linear_recurrence"):
        monkeypatch.setattr(ops, name, counted(name))

    def run(model, dtype, steps):
        calls.clear()
        collect(replayers(model, dtype), steps)
        return dict(calls)
    assert run("C", "bfloat16", whole("m", ids_of("C", 70))) == {"attention_prefill": 3, "experts_up": 3, "linear_recurrence": 1}
    assert run("C", "bfloat16", whole("m", ids_of("C", 100))) == {"attention_prefill": 3, "experts_up": 3, "chunked_recurrence": 1}      # (from 96 rows of one request on)
    assert run("C", "float32", whole("m", ids_of("C", 70))) == {"span_attention": 3, "weighted_relu_squared": 3, "linear_recurrence": 1}
    assert run("C", "bfloat16", [{"step": 0, "entries": [{"id": "m", "tokens": [1], "want": []}], "end": ["m"]}]) == {"attention_decode": 3, "experts_up": 3, "linear_recurrence": 1}
    # (D: heads of 80 channels take the window part's kernel; heads of 24 and 40 are widened to 48, and of 13 and 6 to 16)
    assert run("D", "bfloat16", whole("m", ids_of("D", 70))) == {"span_attention_mfma": 1, "attention_prefill": 2, "experts_up": 1}


def test_greedy_generation_through_the_engine(lalepel_dirs):
    """The engine's own loop and scheduler: prompts of unequal length, more than a batch holds at once."""
    from alofa_amd import Engine
    for name in ("A", "B", "C"):
        cfg, w = plain_model(str(lalepel_dirs[name]))
        prompts = [random_ids(300 + i, n, cfg["vocab"]) for i, n in enumerate((5, 23, 2, 41, 17, 9))]
        want = [pl.greedy(w, cfg, p, 8) for p in prompts]
        engine = Engine(lalepel_dirs[name], dtype="float32", max_tokens=64, max_batch=4, token_budget=48, max_chunk=16)
        assert engine.generate(prompts, max_new=8) == want, name
        engine.cache.check()
        if name == "B":      # (its logits lie close together: rounding alone moves many a greedy choice)
            continue
        got = Engine(lalepel_dirs[name], dtype="bfloat16", max_tokens=64, max_batch=4).generate(prompts, max_new=8)
        agree = sum(a == b for g, r in zip(got, want) for a, b in zip(g, r))
        assert agree >= 34, f"{name}: {agree}/48 greedy tokens agree with the plain model in bfloat16"


def test_decode_steps_replay_a_captured_graph(replayers, lalepel_dirs):
    """Every replay must move the state on and fill the next slot of the pages; other requests' eager steps lie between."""
    for name in ("A", "C", "D"):
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
        compare(got, lalepel_dirs[name], ids, "bfloat16", f"{name} graph decode")


def test_the_programs_take_the_design_by_its_config(lalepel_dirs, tmp_path):
    """bin/generate and bin/trace_run on a folder of this design."""
    import os
    import subprocess
    from conftest import ROOT
    d = lalepel_dirs["A"]
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
