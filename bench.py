"""Decode and prefill throughput of the engine at the layer sizes of the
Qwen2.5 family with random weights, on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch B] [--layers L] [--dtype bfloat16]
                    [--config 0.5b|7b|32b]

The default (0.5b) is the headline: a step is one decode step of the whole
engine loop (scheduler tick, the step function over the paged cache, greedy
choice, settle) with every request of the batch decoding one token; W untimed
steps, then exactly K timed ones. One JSON line is printed; ``value`` is decoded
tokens per second at the default batch of 8. Beside it:

  prefill    one 2,048-token prompt: tokens a second, and its flops / time / peak
  roofline   the decode step's bytes (every weight once + the live requests' cache) / time
  points     decode at batch 1 and 64, and near the end of the context window
  spread     median and min..max of the per-step time over interleaved repeats of every point
             (the reference's method: src/alofa/cli.mojo:212-245, :819-850)
  roofs      what this GPU gives in this process: a device copy of 1 GiB and a large bf16 matrix
             product (the reference wants measured roofs, never constants:
             src/alofa/verify/__init__.mojo:10-17); ``frac`` divides by the published peaks,
             ``frac_measured`` by these
  memory     device bytes of weights, cache pool and scratch

``--config 7b`` and ``--config 32b`` run the larger configurations' workloads
(a continuous batch of 64 requests with prompts of 128..2,048 tokens under
chunked prefill; 8 prompts of 16,384 tokens and decoding at batch 32 with a
context of 4,096) through the same engine and print their own line;
``--config 1.5b``, ``3b`` and ``14b`` run the continuous batch at those sizes.
``--sweep batch`` and ``--sweep context`` take any of the configurations.

``--design tugalix``, ``--design rerupel``, ``--design retotar``, ``--design ludelorn``, ``--design lalepel`` and ``--design nodopel`` measure another design beside Qwen2 (Retotar and Ludelorn: beside
Tugalix; Lalepel: beside Rerupel; Nodopel: beside both Rerupel and Qwen2) at equal sizes: prefill of one prompt and
decode steps at batch 1, 8 and 64, at a few widths (``--sizes``), a line per point and model."""
import argparse
import json
import statistics
import sys
import tempfile
import time
from pathlib import Path

ROOT = Path(__file__).resolve().parent
sys.path.insert(0, str(ROOT))

PEAK_HBM_GBS = 8000.0
PEAK_FLOPS = {"bfloat16": 2.5e15, "float32": 157.3e12}


def family(layers, hidden, heads, kv_heads, inter, vocab, tied, max_pos=32768):
    return {"architectures": ["Qwen2ForCausalLM"], "model_type": "qwen2", "num_hidden_layers": layers, "hidden_size": hidden,
            "num_attention_heads": heads, "num_key_value_heads": kv_heads, "intermediate_size": inter, "vocab_size": vocab,
            "rope_theta": 1000000.0, "rms_norm_eps": 1e-6, "tie_word_embeddings": tied, "use_sliding_window": False,
            "max_position_embeddings": max_pos}


CONFIGS = {
    "0.5b": family(24, 896, 14, 2, 4864, 151936, True),
    "1.5b": family(28, 1536, 12, 2, 8960, 151936, True),
    "3b": family(36, 2048, 16, 2, 11008, 151936, True),
    "7b": family(28, 3584, 28, 4, 18944, 152064, False),
    "14b": family(48, 5120, 40, 8, 13824, 152064, False),
    "32b": family(64, 5120, 40, 8, 27648, 152064, False, 40960),
}
QWEN25_05B = CONFIGS["0.5b"]
CONTEXT, PROMPT, BLOCK = 4096, 512, 16


def say(text):
    print(f"[bench] {text}", file=sys.stderr, flush=True)


def linear_params_per_layer(c):
    h, d = c["hidden_size"], c["hidden_size"] // c["num_attention_heads"]
    qd, kvd, i = c["num_attention_heads"] * d, c["num_key_value_heads"] * d, c["intermediate_size"]
    return h * (qd + 2 * kvd) + qd * h + 3 * h * i


def decode_bytes(c, ctx_lens, dtype_bytes=2):
    """Bytes one decode step has to read: every weight it uses once (layer
    matrices, biases, norms, the output matrix) and the cache of the live requests."""
    h, d, L = c["hidden_size"], c["hidden_size"] // c["num_attention_heads"], c["num_hidden_layers"]
    qd, kvd = c["num_attention_heads"] * d, c["num_key_value_heads"] * d
    per_layer = linear_params_per_layer(c) * dtype_bytes + (qd + 2 * kvd) * 4 + 2 * h * 4
    weights = L * per_layer + h * 4 + c["vocab_size"] * h * dtype_bytes
    cache = sum(ctx_lens) * 2 * kvd * dtype_bytes * L
    return weights + cache


def prefill_flops(c, T, wanted=1, start=0):
    """Flops of running T tokens of one request that stand at positions start..start+T-1."""
    h, d, L = c["hidden_size"], c["hidden_size"] // c["num_attention_heads"], c["num_hidden_layers"]
    linear = 2 * T * linear_params_per_layer(c) * L
    keys = T * start + T * (T + 1) // 2                               # (query, key) pairs under the causal bound
    attention = L * 4 * d * c["num_attention_heads"] * keys           # QK^T and PV
    return linear + attention + 2 * wanted * h * c["vocab_size"]


def sync():
    import torch
    torch.cuda.synchronize()


# ------------------------------------------------------------------ measured roofs

def measure_roofs():
    """What the GPU gives in this process: GB/s of a device-to-device copy of 1 GiB of bfloat16
    (bytes read + bytes written over time) and TFLOP/s of a large bfloat16 matrix product (the
    vendor library's: a yardstick, not part of the engine)."""
    import torch
    n = 1 << 29                                              # 2**29 bfloat16 = 1 GiB
    src = torch.empty(n, dtype=torch.bfloat16, device="cuda").normal_()
    dst = torch.empty_like(src)
    a = torch.randn(8192, 8192, dtype=torch.bfloat16, device="cuda")
    b = torch.randn(8192, 8192, dtype=torch.bfloat16, device="cuda")
    out = torch.empty(8192, 8192, dtype=torch.bfloat16, device="cuda")
    copy_s, gemm_s = [], []
    for i in range(6):
        sync()
        t0 = time.perf_counter()
        for _ in range(4):
            dst.copy_(src)
        sync()
        t1 = time.perf_counter()
        for _ in range(4):
            torch.matmul(a, b, out=out)
        sync()
        t2 = time.perf_counter()
        if i:                                                # the first round warms up
            copy_s.append((t1 - t0) / 4)
            gemm_s.append((t2 - t1) / 4)
    del src, dst, a, b, out
    torch.cuda.empty_cache()
    return {"hbm_copy_gbs": round(2 * n * 2 / min(copy_s) / 1e9, 1), "gemm_bf16_tflops": round(2 * 8192 ** 3 / min(gemm_s) / 1e12, 1),
            "how": "best of 5 rounds: copy of 1 GiB bf16 (read + write), 8192^3 bf16 product of the vendor library"}


# ------------------------------------------------------------------------ points

class DecodePoint:
    """Requests of one batch size kept decoding; ``run(n)`` times n more steps."""

    def __init__(self, model, cfg, dtype, batch, prompt, seed=0, context=CONTEXT):
        import numpy as np
        from alofa_amd import Engine
        rng = np.random.default_rng(seed)
        per_req = (context + BLOCK - 1) // BLOCK
        self.batch, self.cfg = batch, cfg
        self.eng = Engine(None, dtype=dtype, max_tokens=context, max_batch=batch, kv_blocks=per_req * batch + 64, block_size=BLOCK,
                          token_budget=max(2048, batch), max_chunk=512, watermark_permille=1000, model=model)
        core = self.eng.core
        for r in range(batch):
            core.submit(r + 1, [int(t) for t in rng.integers(0, cfg["vocab_size"], prompt)], context - prompt)
        while not (core.last_action and len(core.last_action.decode) == batch and not core.last_action.prefill):
            core.tick()

    def run(self, steps):
        """Seconds per step over ``steps`` decode steps, bracketed by synchronisation."""
        core = self.eng.core
        sync()
        t0 = time.perf_counter()
        for _ in range(steps):
            rows = core.tick()
            assert rows == self.batch, f"a timed step ran {rows} rows, not {self.batch}"
        sync()
        return (time.perf_counter() - t0) / steps

    def context_lengths(self):
        return [self.eng.cache.length(r + 1) for r in range(self.batch)]

    def close(self):
        import torch
        for r in range(self.batch):
            self.eng.core.cancel(r + 1)
        self.eng.core.tick()
        self.eng = None
        torch.cuda.empty_cache()


class PrefillPoint:
    """One prompt of T tokens run whole in one step; ``run()`` times it on fresh pages."""

    def __init__(self, model, cfg, dtype, T=2048, seed=1):
        import numpy as np
        from alofa_amd.cache.manager import CacheManager
        from alofa_amd.engine.step import StepFunction
        self.T, self.cfg, self.rng = T, cfg, np.random.default_rng(seed)
        m = model[1]
        self.cache = CacheManager(m.cache_needs(), m.state_needs(), (T + BLOCK - 1) // BLOCK + 4, BLOCK, max_requests=4,
                                  device=m.rt.device, dtype=m.rt.dtype)
        self.fn = StepFunction(m, self.cache, n_positions=max(T, 64))
        self.n = 0

    def run(self):
        from alofa_amd.engine.step import StepEntry
        ids = [int(t) for t in self.rng.integers(0, self.cfg["vocab_size"], self.T)]
        self.n += 1
        self.cache.admit(self.n)
        sync()
        t0 = time.perf_counter()
        self.fn.run([StepEntry(self.n, ids, [self.T - 1])])
        sync()
        dt = time.perf_counter() - t0
        self.cache.free(self.n)
        return dt


def spread(samples):
    return {"median_ms": round(statistics.median(samples) * 1e3, 4), "min_ms": round(min(samples) * 1e3, 4),
            "max_ms": round(max(samples) * 1e3, 4), "repeats": len(samples)}


def device_model(cfg, dtype, seed):
    """(config, model) with random weights drawn on the device: for sizes whose file would take minutes to write."""
    import torch
    from alofa_amd.config import config_from_dict
    from alofa_amd.model import Model, expected_tensors, runtime
    from alofa_amd.weights import random_tensors
    config = config_from_dict(cfg)
    spec = config.spec()
    rt = runtime(dtype)
    weights = random_tensors(expected_tensors(spec), seed, device=rt.device)
    model = Model(spec, weights, rt)
    del weights
    torch.cuda.empty_cache()
    return config, model


# ------------------------------------------------------------------- the headline

def headline(args):
    from alofa_amd.model import load_model
    from alofa_amd.weights import write_random_model
    cfg = dict(QWEN25_05B, num_hidden_layers=args.layers)
    dbytes = 2 if args.dtype == "bfloat16" else 4
    with tempfile.TemporaryDirectory() as d:
        write_random_model(cfg, d, seed=20260918)
        model = load_model(d, args.dtype)
    if args.only_prefill:
        p = PrefillPoint(model, cfg, args.dtype)
        p.run()
        pt = min(p.run() for _ in range(3))
        print(json.dumps({"prefill": {"value": round(2048 / pt, 1), "tokens": 2048, "ms": round(pt * 1e3, 3),
                                      "frac": round(prefill_flops(cfg, 2048) / pt / PEAK_FLOPS[args.dtype], 4)}}))
        return 0
    timed = args.steps + args.warmup + (0 if args.no_points else 5 * max(8, args.steps // 2))      # steps this batch's requests decode
    if not 1 <= args.prompt <= CONTEXT - timed - 1:
        print(f"--prompt must leave room for the decode steps within the context of {CONTEXT}")
        return 2
    roofs = None if args.no_points else measure_roofs()
    main_point = DecodePoint(model, cfg, args.dtype, args.batch, args.prompt)
    memory = main_point.eng.memory()
    say(f"device memory: weights {memory['weights'] / 2**20:.1f} MiB + cache pool {memory['cache_pool'] / 2**20:.1f} MiB (batch {args.batch} x {CONTEXT} tokens)"
        f" + scratch {memory['scratch'] / 2**20:.1f} MiB")
    main_point.run(args.warmup) if args.warmup else None
    ms = main_point.run(args.steps)                                    # exactly K timed steps after W untimed ones
    ctx_lens = main_point.context_lengths()
    memory = main_point.eng.memory()
    value = args.batch / ms
    achieved = decode_bytes(cfg, ctx_lens, dbytes) / ms / 1e9
    out = {
        "metric": "decode tok/s @ batch 8 (Qwen2.5-0.5B sizes); prefill tok/s @ 2,048 tok; decode @ batch 1/64 under points",
        "value": round(value, 1), "unit": "tok/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(ms * 1e3, 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "data": "synthetic (random weights N(0, 0.02), uniform random token ids)",
        "config": {"model": "Qwen2.5-0.5B sizes, random weights", "layers": args.layers, "layers_full": QWEN25_05B["num_hidden_layers"],
                   "hidden": 896, "heads": 14, "kv_heads": 2, "head_dim": 64, "intermediate": 4864, "vocab": 151936,
                   "global_batch": args.batch, "seq_len": CONTEXT, "prompt_len": args.prompt, "decode_context": int(sum(ctx_lens) / len(ctx_lens)),
                   "kv_block": BLOCK, "tied_embeddings": True, "parallelism": "single GPU"},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": PEAK_HBM_GBS, "unit": "GB/s",
                     "frac": round(achieved / PEAK_HBM_GBS, 4)},
        "memory": {k: int(v) for k, v in memory.items()},
    }
    if not args.no_points:
        T = 2048
        reps, n = 5, max(8, args.steps // 2)
        others = {1: DecodePoint(model, cfg, args.dtype, 1, PROMPT), 64: DecodePoint(model, cfg, args.dtype, 64, PROMPT)}
        prefill = PrefillPoint(model, cfg, args.dtype, T)
        points = {args.batch: main_point, **{b: p for b, p in others.items() if b != args.batch}}
        for p in others.values():
            p.run(max(4, args.warmup // 2))
        prefill.run()
        samples = {f"decode_b{b}": [] for b in points}
        samples["prefill"] = []
        for _ in range(reps):                                           # interleaved: every point once per round
            for b, p in points.items():
                samples[f"decode_b{b}"].append(p.run(n))
            samples["prefill"].append(prefill.run())
        pt = statistics.median(samples["prefill"])
        out["prefill"] = {"value": round(T / pt, 1), "tokens": T, "ms": round(pt * 1e3, 3),
                          "frac": round(prefill_flops(cfg, T) / pt / PEAK_FLOPS[args.dtype], 4)}
        out["points"] = {f"decode_b{b}": round(b / statistics.median(samples[f"decode_b{b}"]), 1) for b in (1, 64)}
        out["spread"] = {k: spread(v) for k, v in samples.items()}
        for p in others.values():
            p.close()
        main_point.close()
        # the same near the end of the context window (prompts of 3,840 tokens)
        for b in (8, 64):
            p = DecodePoint(model, cfg, args.dtype, b, CONTEXT - 256)
            p.run(max(4, args.warmup // 4))
            out["points"][f"decode_b{b}_ctx{CONTEXT - 256}"] = round(b / p.run(max(16, args.steps // 4)), 1)
            p.close()
        out["roofs"] = roofs
        out["roofline"]["frac_measured"] = round(achieved / roofs["hbm_copy_gbs"], 4)
        if args.dtype == "bfloat16":
            out["prefill"]["frac_measured"] = round(prefill_flops(cfg, T) / pt / (roofs["gemm_bf16_tflops"] * 1e12), 4)
    print(json.dumps(out))
    return 0


# --------------------------------------------------------- the larger configurations

def flat_config(name, cfg, layers, **more):
    d = cfg["hidden_size"] // cfg["num_attention_heads"]
    return {"model": f"Qwen2.5-{name.upper()} sizes, random weights", "layers": layers, "layers_full": CONFIGS[name]["num_hidden_layers"],
            "hidden": cfg["hidden_size"], "heads": cfg["num_attention_heads"], "kv_heads": cfg["num_key_value_heads"], "head_dim": d,
            "intermediate": cfg["intermediate_size"], "vocab": cfg["vocab_size"], "kv_block": BLOCK,
            "tied_embeddings": cfg["tie_word_embeddings"], "parallelism": "single GPU", **more}


def continuous_batch(args):
    """64 requests with prompts of uniform random length in [128, 2048] and 256 generated tokens
    each, all submitted at once, under chunked prefill with chunks of 512 (a budget of 2,048
    tokens a tick): the whole run through the engine loop, timed from the first tick to the last."""
    import numpy as np
    from alofa_amd import Engine
    name = args.config
    layers = args.layers or CONFIGS[name]["num_hidden_layers"]
    cfg = dict(CONFIGS[name], num_hidden_layers=layers)
    say(f"drawing {name} weights on the device ({layers} layers)")
    model = device_model(cfg, args.dtype, 20260918)
    n_req, new, context = 64, 256, 8192
    rng = np.random.default_rng(7)
    lens = [int(n) for n in rng.integers(128, 2049, n_req)]
    per_req = (max(lens) + new + BLOCK - 1) // BLOCK
    eng = Engine(None, dtype=args.dtype, max_tokens=context, max_batch=n_req, kv_blocks=per_req * n_req + 64, block_size=BLOCK,
                 token_budget=2048, max_chunk=512, watermark_permille=1000, model=model, report=say)
    core = eng.core

    def run():
        import torch
        base = (core.ticks + 1) * 1000
        for r, n in enumerate(lens):
            core.submit(base + r, [int(t) for t in rng.integers(0, cfg["vocab_size"], n)], new)
        # The ticks are timed on the device, by events recorded behind every tick's launches and read when the run
        # is over: waiting for a tick on the host would take away the head start the loop has on the device (it
        # prepares a tick while the one before runs), and with it a tenth of the throughput at these sizes.
        marks, kinds = [torch.cuda.Event(enable_timing=True)], []
        sync()
        marks[0].record()
        t0 = time.perf_counter()
        while core.has_work():
            core.tick()
            act = core.last_action
            kinds.append(("decode", 0) if len(act.decode) == n_req and not act.prefill else ("mixed", core.last_rows) if act.prefill else ("other", 0))
            marks.append(torch.cuda.Event(enable_timing=True))
            marks[-1].record()
        sync()
        dt = time.perf_counter() - t0
        spans = [marks[i].elapsed_time(marks[i + 1]) / 1e3 for i in range(len(kinds))]
        decode = [t for t, (k, _) in zip(spans, kinds) if k == "decode"]
        mixed = [(t, rows) for t, (k, rows) in zip(spans, kinds) if k == "mixed"]
        if mixed:
            say(f"{len(mixed)} ticks with prompt portions: {sum(t for t, _ in mixed) / len(mixed) * 1e3:.3f} ms and {sum(r for _, r in mixed) / len(mixed):.0f} rows a tick")
        for r in range(n_req):
            assert len(core.output(base + r)) == new
            core.release(base + r)
        return dt, len(kinds), sum(decode), len(decode)
    roofs = measure_roofs()
    say("warm-up run")
    run()
    runs = [run() for _ in range(3)]                      # three timed runs after the warm-up; the median one is reported
    dt, ticks, decode_s, decode_steps = sorted(runs, key=lambda r: r[0])[1]
    dbytes = 2 if args.dtype == "bfloat16" else 4
    mean_ctx = [n + new // 2 for n in lens]
    step_ms = decode_s / max(1, decode_steps) * 1e3
    achieved = decode_bytes(cfg, mean_ctx, dbytes) / (step_ms / 1e3) / 1e9 if decode_steps else None
    out = {"metric": f"generated tok/s, continuous batch of 64 requests (prompts U[128,2048], 256 new tokens, chunked prefill 512), Qwen2.5-{name.upper()} sizes",
           "value": round(n_req * new / dt, 1), "unit": "tok/s", "n_gpus": 1, "steps": ticks, "warmup": ticks, "ms_per_step": round(dt / ticks * 1e3, 4),
           "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
           "data": "synthetic (random weights N(0, 0.02) drawn on the device, uniform random token ids)",
           "config": flat_config(name, cfg, layers, global_batch=n_req, seq_len=context, prompt_tokens=sum(lens), new_tokens=new, max_chunk=512, token_budget=2048),
           "total_tok_s": round((sum(lens) + n_req * new) / dt, 1), "seconds": round(dt, 3),
           "roofline": {"bound": "hbm", "what": "the ticks in which all 64 requests decode and nothing is prefilled", "steps": decode_steps, "ms_per_step": round(step_ms, 4),
                        "achieved": round(achieved, 1) if achieved else None, "peak": PEAK_HBM_GBS, "unit": "GB/s"},
           "spread": {"seconds": {"median": round(dt, 3), "min": round(min(r[0] for r in runs), 3), "max": round(max(r[0] for r in runs), 3), "repeats": len(runs)},
                      "generated_tok_s": sorted(round(n_req * new / r[0], 1) for r in runs),
                      "decode_step": spread([r[2] / max(1, r[3]) for r in runs])},
           "roofs": roofs, "memory": {k: int(v) for k, v in eng.memory().items()}}
    if achieved:
        out["roofline"]["frac"] = round(achieved / PEAK_HBM_GBS, 4)
        out["roofline"]["frac_measured"] = round(achieved / roofs["hbm_copy_gbs"], 4)
    print(json.dumps(out))
    return 0


def long_prompts(args):
    """8 requests, each with a prompt of 16,384 tokens and 128 generated tokens (chunked prefill,
    chunks of 2,048 under a budget of 4,096 tokens a tick), then decoding at batch 32 with a
    context of 4,096 tokens, which reads the most cache per step."""
    import numpy as np
    from alofa_amd import Engine
    name = "32b"
    layers = args.layers or CONFIGS[name]["num_hidden_layers"]
    cfg = dict(CONFIGS[name], num_hidden_layers=layers)
    say(f"drawing {name} weights on the device ({layers} layers)")
    model = device_model(cfg, args.dtype, 20260918)
    dbytes = 2 if args.dtype == "bfloat16" else 4
    n_req, plen, new, context = 8, 16384, 128, 32768
    roofs = measure_roofs()
    rng = np.random.default_rng(8)
    per_req = (plen + new + BLOCK - 1) // BLOCK
    eng = Engine(None, dtype=args.dtype, max_tokens=context, max_batch=n_req, kv_blocks=per_req * n_req + 64, block_size=BLOCK,
                 token_budget=4096, max_chunk=2048, watermark_permille=1000, model=model, report=say)
    core = eng.core

    def run(base):
        """All eight prompts through the engine loop; the ticks that bring prompt portions are timed by themselves."""
        for r in range(n_req):
            core.submit(base + r, [int(t) for t in rng.integers(0, cfg["vocab_size"], plen)], new)
        sync()
        t0 = time.perf_counter()
        prefill_s, prefill_tokens, prefill_fl, ticks = 0.0, 0, 0.0, 0
        while core.has_work():
            t1 = time.perf_counter()
            core.tick()
            act = core.last_action
            if act.prefill:                     # ticks that bring prompt portions (later ones carry a few decoded tokens beside them)
                sync()
                prefill_s += time.perf_counter() - t1
                prefill_tokens += sum(e - s for _, s, e in act.prefill)
                prefill_fl += sum(prefill_flops(cfg, e - s, wanted=int(e == plen), start=s) for _, s, e in act.prefill)
            ticks += 1
            if ticks % 16 == 0:
                say(f"tick {ticks}: {prefill_tokens} prompt tokens so far")
        sync()
        dt = time.perf_counter() - t0
        for r in range(n_req):
            assert len(core.output(base + r)) == new
            core.release(base + r)
        return {"prefill_s": prefill_s, "tokens": prefill_tokens, "flops": prefill_fl, "ticks": ticks, "seconds": dt}
    passes = [run(1000), run(2000)]                           # two passes (the first also warms up); the faster one is reported
    best = min(passes, key=lambda p: p["prefill_s"])
    memory = eng.memory()
    del eng, core
    out = {"metric": "prefill tok/s over 8 prompts of 16,384 tokens (chunks of 2,048); decode tok/s @ batch 32, context 4,096 under points; Qwen2.5-32B sizes",
           "value": round(best["tokens"] / best["prefill_s"], 1), "unit": "tok/s", "n_gpus": 1, "steps": best["ticks"], "warmup": passes[0]["ticks"],
           "ms_per_step": round(best["seconds"] / best["ticks"] * 1e3, 3),
           "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
           "data": "synthetic (random weights N(0, 0.02) drawn on the device, uniform random token ids)",
           "config": flat_config(name, cfg, layers, global_batch=n_req, seq_len=context, prompt_len=plen, new_tokens=new, max_chunk=2048, token_budget=4096),
           "prefill": {"value": round(best["tokens"] / best["prefill_s"], 1), "tokens": best["tokens"], "ms": round(best["prefill_s"] * 1e3, 1),
                       "frac": round(best["flops"] / best["prefill_s"] / PEAK_FLOPS[args.dtype], 4)},
           "spread": {"prefill_tok_s": [round(p["tokens"] / p["prefill_s"], 1) for p in passes]},
           "seconds_whole_run": round(best["seconds"], 2), "generated_tok_s_whole_run": round(n_req * new / best["seconds"], 1), "memory": {k: int(v) for k, v in memory.items()}}
    if args.dtype == "bfloat16":
        out["prefill"]["frac_measured"] = round(best["flops"] / best["prefill_s"] / (roofs["gemm_bf16_tflops"] * 1e12), 4)
    p = DecodePoint(model, cfg, args.dtype, 32, 4096 - 128, context=4096 + 64)
    p.run(8)
    samples = [p.run(24) for _ in range(3)]
    ms = statistics.median(samples)
    ctx_lens = p.context_lengths()
    achieved = decode_bytes(cfg, ctx_lens, dbytes) / ms / 1e9
    out["points"] = {"decode_b32_ctx4096": round(32 / ms, 1)}
    out["spread"]["decode_b32_ctx4096"] = spread(samples)
    out["roofline"] = {"bound": "hbm", "what": "decode step at batch 32, context about 4,096", "ms_per_step": round(ms * 1e3, 4), "achieved": round(achieved, 1),
                       "peak": PEAK_HBM_GBS, "unit": "GB/s", "frac": round(achieved / PEAK_HBM_GBS, 4), "frac_measured": round(achieved / roofs["hbm_copy_gbs"], 4)}
    out["roofs"] = roofs
    p.close()
    print(json.dumps(out))
    return 0


def sweep(args):
    """Decode steps over batch sizes (at a context of about 550) or over contexts (batch 1, 8, 32): one line per
    point with ms per step, tokens a second and the bytes the step has to read / time. At the 0.5B sizes, or with
    --config 1.5b .. 32b at those (batches up to 64; --layers for fewer layers than the configuration has)."""
    name = args.config
    cfg = dict(CONFIGS[name], num_hidden_layers=args.layers or CONFIGS[name]["num_hidden_layers"])
    model = device_model(cfg, args.dtype, 20260918)
    dbytes = 2 if args.dtype == "bfloat16" else 4
    batches = (1, 2, 4, 8, 16, 17, 24, 32, 48, 64, 96, 128, 192, 256) if name == "0.5b" else (1, 2, 4, 8, 16, 17, 32, 64) if name in ("1.5b", "3b") else (1, 2, 4, 8, 16, 32, 64)
    if args.batches:
        batches = tuple(int(b) for b in args.batches.split(","))
    cases = ([(b, PROMPT) for b in batches] if args.sweep == "batch" else
             [(b, p) for p in (2048, 8192, 16384, 30000) for b in (1, 8, 32)])
    for batch, prompt in cases:
        pt = DecodePoint(model, cfg, args.dtype, batch, prompt, context=max(CONTEXT, prompt + 256))
        pt.run(8)
        s = pt.run(24)
        byts = decode_bytes(cfg, pt.context_lengths(), dbytes)
        print(json.dumps({"model": name, "layers": cfg["num_hidden_layers"], "batch": batch, "context": prompt, "ms_per_step": round(s * 1e3, 4), "tok_s": round(batch / s, 1),
                          "gb_s": round(byts / s / 1e9, 1), "frac_hbm": round(byts / s / 1e9 / PEAK_HBM_GBS, 4)}), flush=True)
        pt.close()
    return 0


# ------------------------------------------------------------------- another design beside the closest one

def tugalix_sizes(width, heads, dim, ff, layers, vocab=32000):
    """A Tugalix model of ``layers`` layers in the order parallel, retention, gated linear attention, retention, every one
    with a feed-forward, and the Qwen2 model of equal width, heads, layers and feed-forward weights beside it."""
    kv = max(1, heads // 4)
    rot = {"dims": dim, "base": 1000000.0}
    kinds = [("parallel", {"left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "rot": rot},
                           "right": {"heads": heads, "dim": dim, "rank": 64}, "left_scale": 1.0, "right_scale": 1.0}),
             ("retention", {"heads": heads, "dim": dim, "vdim": dim, "rot": rot, "decay": [1.0 - 2.0 ** (-5 - i % 8) for i in range(heads)]}),
             ("gla", {"heads": heads, "dim": dim, "vdim": dim, "tau": 16.0, "rank": 16}),
             ("retention", {"heads": heads, "dim": dim, "vdim": dim, "rot": rot, "decay": [1.0 - 2.0 ** (-5 - i % 8) for i in range(heads)]})]
    tug = {"architecture": "Tugalix", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "canon": {"taps": 4}, "logit_scale": 1.0,
           "layers": [{"type": kinds[i % 4][0], "mixer": kinds[i % 4][1], "mlp": {"kind": "dense", "ff": ff}} for i in range(layers)]}
    qwen = dict(family(layers, width, heads, kv, ff * 2 // 3 // 64 * 64, vocab, False), head_dim=dim)
    return tug, qwen


def rerupel_sizes(width, heads, dim, ff, layers, vocab=32000):
    """A Rerupel model of ``layers`` layers (the first with a dense feed-forward, the others with sixteen experts of which a
    token takes four, and one that every token takes; latents of twice a head's size; all layers but the first in a loop that
    is passed once), and the Qwen2 model of equal width, heads and layers whose feed-forward has as many channels as a
    token's five experts together."""
    expert = max(64, ff // 8 // 64 * 64)
    mixer = {"heads": heads, "dim": dim, "vdim": dim, "kv_rank": 2 * dim, "scale": dim ** -0.5}
    moe = {"kind": "moe", "router": {"experts": 16, "top": 4, "scale": 1.0}, "expert": {"ff": expert, "limit": 7.0}, "shared": {"ff": expert, "limit": 7.0}}
    rer = {"architecture": "Rerupel", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "residual_mult": 1.0, "logit_softcap": 30.0,
           "embedding": {"scale": 1.0, "bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}}, "loop": {"start": 1, "stop": layers, "times": 1},
           "layers": [{"type": "latent_attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if i == 0 else moe} for i in range(layers)]}
    qwen = dict(family(layers, width, heads, max(1, heads // 4), 5 * expert, vocab, False), head_dim=dim)
    return rer, qwen


def retotar_sizes(width, heads, dim, ff, layers, vocab=32000):
    """A Retotar model of ``layers`` layers in the order attention (a window of 1,024 keys), lightning, mlstm, attention that reads the
    first one's pages, every one with sixteen experts of which a token takes four (four identity experts beside them, four groups of which
    two are kept), and beside it the closest other design, Tugalix, at equal width, heads and layers, with a dense feed-forward of as many
    weights as a token's four experts."""
    kv = max(1, heads // 4)
    expert = max(64, ff // 8 // 64 * 64)
    rot = {"dims": dim // 2, "base": 10000.0, "scaling": {"factor": 4.0}}
    attention = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "rot": rot, "scale": 8.0 / dim, "mask": {"size": 1024}}
    moe = {"kind": "moe", "router": {"experts": 16, "top": 4, "identity": 4, "groups": {"count": 4, "keep": 2}}, "expert": {"ff": expert}}

    def mixer(i):
        k = i % 4
        if k == 1:
            return "lightning", {"heads": heads, "dim": dim, "vdim": dim, "decay": [1.0 - 2.0 ** (-5 - h % 8) for h in range(heads)]}
        if k == 2:
            return "mlstm", {"heads": heads, "dim": dim, "vdim": dim, "gate_cap": 15.0}
        return "attention", dict(attention, kv_from=i - 3) if k == 3 else dict(attention)
    ret = {"architecture": "Retotar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
           "layers": [{"type": mixer(i)[0], "mixer": mixer(i)[1], "mlp": moe} for i in range(layers)]}
    return ret, tugalix_sizes(width, heads, dim, 6 * expert, layers, vocab)[0]


def ludelorn_sizes(width, heads, dim, ff, layers, vocab=32000):
    """A Ludelorn model of ``layers`` layers in the order parallel (attention within 1,024 keys beside a state-space mixer of as many heads,
    state channels as a head has channels), attention within 512 keys with pooled blocks of 16 behind them, parallel, attention with a bias
    by distance and a sink within 512 keys, every one with a dense feed-forward, and beside it the closest other design, Tugalix (attention
    beside a recurrence, dense feed-forwards), at equal width, heads, layers and feed-forward."""
    kv = max(1, heads // 4)
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": 1024},
            "rot": {"dims": dim, "base": 250000.0, "scaling": {"factor": 4.0, "original": 4096, "fast": 16.0, "slow": 2.0}}}
    right = {"heads": heads, "vdim": dim, "state": dim, "groups": max(1, heads // 8), "conv": 4, "norm_groups": max(1, heads // 8)}
    kinds = [("parallel", {"left": left, "right": right}),
             ("attention", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": 512, "pool": 16}, "rot": {"dims": dim // 2, "base": 100000.0}}),
             ("parallel", {"left": left, "right": right}),
             ("attention_2", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": 8.0 / dim, "mask": {"size": 512}, "bias_max": 512.0, "bias_rows": 32})]
    lud = {"architecture": "Ludelorn", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
           "layers": [{"type": kinds[i % 4][0], "mixer": kinds[i % 4][1], "mlp": {"kind": "dense", "ff": ff}} for i in range(layers)]}
    return lud, tugalix_sizes(width, heads, dim, ff, layers, vocab)[0]


def lalepel_sizes(width, heads, dim, ff, layers, vocab=32000):
    """A Lalepel model of ``layers`` layers in the order latent attention (a window of 1,024 keys, latents that make one head of twice a head's size
    with the turned part of half a head's), retention, latent attention, latent attention, the first with a dense feed-forward, the others with
    sixteen experts of which a token takes four and one that every token takes, and beside it the closest other design, Rerupel (attention over
    latents, the same experts with a gate matrix), at equal width, heads, layers and feed-forward."""
    expert = max(64, ff // 8 // 64 * 64)
    latent = {"heads": heads, "dim": dim, "rot_dim": dim // 2, "vdim": dim, "q_rank": 3 * width // 8 // 64 * 64 or 64, "kv_rank": 3 * dim // 2, "scale": (1.5 * dim) ** -0.5,
              "rot": {"dims": dim // 2, "base": 250000.0, "scaling": {"factor": 4.0, "original": 4096, "fast": 16.0, "slow": 2.0}}, "mask": {"size": 1024}}
    retention = {"heads": heads, "dim": dim, "vdim": dim, "decay": [1.0 - 2.0 ** (-5 - h % 8) for h in range(heads)]}
    moe = {"kind": "moe", "router": {"experts": 16, "top": 4}, "expert": {"ff": expert}, "shared": {"ff": expert}}
    lal = {"architecture": "Lalepel", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
           "layers": [{"type": "retention" if i % 4 == 1 else "latent_attention", "mixer": retention if i % 4 == 1 else latent,
                       "mlp": {"kind": "dense", "ff": ff} if i == 0 else moe} for i in range(layers)]}
    return lal, rerupel_sizes(width, heads, dim, ff, layers, vocab)[0]


def nodopel_sizes(width, heads, dim, ff, layers, vocab=32000):
    """A Nodopel model of ``layers`` layers on four copies of the stream (heads of two maps of half a head's size over values of a head's size, a window of 1,024
    keys that keeps the first 64, capped scores; the first layer with a dense feed-forward, the others with sixteen experts and four identity experts of which a token takes four,
    and one that every token takes; all layers but the first in a loop that is passed once), beside it the closest other designs: Rerupel (the same experts, one latent
    key head) at equal width, heads, layers and feed-forward, and Qwen2 within the same window (grouped-query attention with biases at equal head counts and sizes) with as many
    feed-forward channels as a token's five experts."""
    expert = max(64, ff // 8 // 64 * 64)
    mixer = {"heads": heads, "kv_heads": max(1, heads // 4), "dim": dim // 2, "vdim": dim, "scale": (dim // 2) ** -0.5, "softcap": 50.0, "diff": 0.3, "mask": {"size": 1024, "keep_first": 64},
             "rot": {"dims": dim // 2, "base": 500000.0, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    moe = {"kind": "moe", "router": {"experts": 16, "top": 4, "identity": 4}, "expert": {"ff": expert}, "shared": {"ff": expert}}
    nod = {"architecture": "Nodopel", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "streams": 4, "loop": {"start": 1, "stop": layers, "times": 1},
           "layers": [{"type": "attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if i == 0 else moe} for i in range(layers)]}
    rer, qwen = rerupel_sizes(width, heads, dim, ff, layers, vocab)
    return nod, rer, dict(qwen, use_sliding_window=True, sliding_window=1024, max_window_layers=0)


DESIGN_MODELS = {"tugalix": tugalix_sizes, "rerupel": rerupel_sizes, "retotar": retotar_sizes, "ludelorn": ludelorn_sizes, "lalepel": lalepel_sizes, "nodopel": nodopel_sizes}
DESIGN_BESIDE = {"retotar": ("tugalix",), "ludelorn": ("tugalix",), "lalepel": ("rerupel",), "nodopel": ("rerupel", "qwen2")}      # the models a design is measured beside, where that is not Qwen2 alone
DESIGN_SIZES = {"256": (256, 4, 64, 1024, 4), "1k": (1024, 16, 64, 4096, 8), "2k": (2048, 16, 128, 8192, 8), "4k": (4096, 32, 128, 14336, 4)}
DESIGN_DEFAULT = ("1k", "2k", "4k")      # ("256": a small one, for a quick look)


def designs(args):
    """Prefill (one prompt of 2,048 tokens in one step) and decode steps (batch 1, 8 and 64 at a context of about 550) of
    another design beside Qwen2 at equal sizes, random weights: one line per point and model."""
    sizes = args.sizes.split(",") if args.sizes else list(DESIGN_DEFAULT)
    for size in sizes:
        if size not in DESIGN_SIZES:
            print(f"no such size: {size} (known: {','.join(DESIGN_SIZES)})")
            return 2
        for name, cfg in zip((args.design, *DESIGN_BESIDE.get(args.design, ("qwen2",))), DESIGN_MODELS[args.design](*DESIGN_SIZES[size])):
            if args.only and name != args.only:
                continue
            cfg = dict(cfg, vocab_size=cfg.get("vocab_size", cfg.get("vocab")))      # (the points draw their tokens by this key)
            model = device_model({k: v for k, v in cfg.items() if not (name != "qwen2" and k == "vocab_size")}, args.dtype, 20261126)
            weights = model[1].weight_bytes()
            if not args.no_prefill:
                pp = PrefillPoint(model, cfg, args.dtype, T=args.prompt_tokens)
                pp.run()
                pre = [pp.run() for _ in range(5)]
                print(json.dumps({"design": name, "size": size, "point": "prefill", "tokens": args.prompt_tokens, **spread(pre),
                                  "tok_s": round(args.prompt_tokens / statistics.median(pre), 1)}), flush=True)
                del pp
            for batch in (int(b) for b in (args.batches or "1,8,64").split(",") if int(b) > 0):      # (--batches 0: the prefill point alone)
                pt = DecodePoint(model, cfg, args.dtype, batch, PROMPT)
                pt.run(args.warmup)
                s = pt.run(args.steps)
                print(json.dumps({"design": name, "size": size, "point": "decode", "batch": batch, "context": PROMPT, "ms_per_step": round(s * 1e3, 4),
                                  "tok_s": round(batch / s, 1), "weights_gb_s": round(weights / s / 1e9, 1)}), flush=True)
                pt.close()
            del model
    return 0


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=128)
    ap.add_argument("--warmup", type=int, default=16)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--config", default="0.5b", choices=sorted(CONFIGS), help="layer sizes and workload (default: the headline)")
    ap.add_argument("--prompt", type=int, default=PROMPT, help="prompt length of the timed decode steps' requests (context = prompt + steps so far)")
    ap.add_argument("--layers", type=int, default=None, help="fewer layers than the configuration has, where memory or time needs it")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--no-points", action="store_true", help="skip the batch 1 / 64 points, the prefill, the repeats and the roofs")
    ap.add_argument("--only-prefill", action="store_true", help="run the 2,048-token prefill alone (for profiling) and print its line")
    ap.add_argument("--serve", action="store_true", help="the continuous batch of 64 requests (prompts of 128..2,048 tokens, 256 new tokens, chunks of 512) at the sizes of --config")
    ap.add_argument("--batches", default=None, help="with --sweep batch: these batch sizes only (comma-separated), e.g. to profile one point")
    ap.add_argument("--sweep", choices=["batch", "context"], default=None, help="decode steps over batch sizes or over contexts, a line per point (the sizes of --config)")
    ap.add_argument("--design", choices=sorted(DESIGN_MODELS), default=None, help="prefill and decode of this design beside the closest one at equal sizes (--sizes), a line per point")
    ap.add_argument("--sizes", default=None, help=f"with --design: which of {','.join(DESIGN_SIZES)} (comma-separated; default {','.join(DESIGN_DEFAULT)})")
    ap.add_argument("--only", choices=sorted(DESIGN_MODELS) + ["qwen2"], default=None, help="with --design: this model alone (for profiling)")
    ap.add_argument("--prompt-tokens", type=int, default=2048, help="with --design: tokens of the prefill point's prompt")
    ap.add_argument("--no-prefill", action="store_true", help="with --design: decode points only")
    args = ap.parse_args()
    if args.gpus != 1:
        print("bench.py measures one GPU only: this engine has no multi-GPU path (--gpus must be 1)")
        return 2

    from alofa_amd.csrc.build import load
    load()
    if args.design:
        return designs(args)
    if args.sweep:
        return sweep(args)
    if args.config in ("1.5b", "3b", "7b", "14b") or args.serve:
        return continuous_batch(args)
    if args.config == "32b":
        return long_prompts(args)
    args.layers = args.layers or QWEN25_05B["num_hidden_layers"]
    return headline(args)


if __name__ == "__main__":
    sys.exit(main())
