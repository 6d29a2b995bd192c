"""Decode and prefill throughput of the Llama-3.2-1B shape on one MI355X.

    python bench.py --gpus 1 --steps K --warmup W

A step is one decode step of the engine (schedule, run the model on one token
per sequence from the paged cache, sample, read the tokens back).  The default
run has the layer sizes of Llama-3.2-1B with seeded random weights, 8 sequences
and a context of 8192 tokens: each sequence's prompt is prefilled by the engine
so that the timed steps end at the context length.  One JSON line is printed:
``value`` is decoded tokens a second at batch 8 (from the mean step time, as the
reference reports it, tokasaurus/benchmarks/bench_model.py:318-324); ``prefill`` is one
2,048-token prompt (mean of 10); ``roofline`` prices the decode step against the bytes it
must read; ``points`` holds decode at batch 1 and 64; ``timing`` gives mean, median and
minimum of the timed iterations (the reference's timer, tokasaurus/utils.py:199-251);
``measured`` holds two ceilings taken in the same process, a device copy of 1 GiB and one
large bfloat16 product, and the fractions of them beside the fractions of the vendor's peaks.
"""

from __future__ import annotations

import argparse
import json
import sys
import time

HBM_PEAK_GBS = 8000.0  # MI355X HBM3E
PEAK_TFLOPS = {"bf16": 2500.0, "fp32": 157.3}  # dense MFMA peaks

LLAMA_1B = {
    "architectures": ["LlamaForCausalLM"],
    "model_type": "llama",
    "num_hidden_layers": 16,
    "hidden_size": 2048,
    "num_attention_heads": 32,
    "num_key_value_heads": 8,
    "intermediate_size": 8192,
    "vocab_size": 128256,
    "rope_theta": 500000.0,
    "rope_scaling": {"rope_type": "llama3", "factor": 32.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                     "original_max_position_embeddings": 8192},
    "rms_norm_eps": 1e-5,
    "tie_word_embeddings": True,
    "max_position_embeddings": 131072,
}
CONTEXT = 8192
PREFILL_TOKENS = 2048
PAGE_SIZE = 16


def say(msg: str) -> None:
    print(f"[bench] {msg}", file=sys.stderr, flush=True)


def parse() -> argparse.Namespace:
    p = argparse.ArgumentParser()
    p.add_argument("--gpus", type=int, default=1)
    p.add_argument("--steps", type=int, default=64)
    p.add_argument("--warmup", type=int, default=8)
    p.add_argument("--batch", type=int, default=8)
    p.add_argument("--context", type=int, default=CONTEXT)
    p.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    p.add_argument("--layers", type=int, default=None, help="run fewer layers than the model has (recorded in config)")
    p.add_argument("--points", default="1,64", help="other decode batch sizes to measure, comma separated ('' for none)")
    p.add_argument("--sweep", default="2048,5120",
                   help="further contexts at which every batch size is timed: with the context itself they cover the "
                        "workload's decode from a 2,048-token prompt to 8,192 tokens ('' for none)")
    p.add_argument("--large", default="256,1024",
                   help="large decode batches, timed at --large-context under --large-budget tokens a step, the "
                        "settings the reference serves this model with ('' for none)")
    p.add_argument("--large-context", type=int, default=1536)
    p.add_argument("--large-budget", type=int, default=32768)
    p.add_argument("--max-tokens-per-forward", type=int, default=8192)
    p.add_argument("--no-prefill", action="store_true")
    p.add_argument("--prefill-only", action="store_true", help="time only the prefill (for profiles); prints its record alone")
    p.add_argument("--prefill-tokens", type=int, default=PREFILL_TOKENS,
                   help="length of the prompt whose prefill is timed (the headline's is 2048; at most the context)")
    p.add_argument("--eager", action="store_true", help="no HIP graphs")
    p.add_argument("--shape", default="1b", choices=sorted(SHAPES), help="layer sizes (the default is the headline's)")
    p.add_argument("--workload", default=None, choices=sorted(WORKLOADS),
                   help="instead of the decode steps: a whole workload through Engine.generate (prints its own line)")
    p.add_argument("--scenario", default=None, choices=["chunked-prefill", "mixed-decode"],
                   help="instead of the decode steps, a case that shapes of one length do not show (prints its own line): "
                        "chunked-prefill: one prompt of --context tokens in portions of --portion tokens; "
                        "mixed-decode: decode steps of --batch - 1 requests of --short tokens beside one of --context tokens")
    p.add_argument("--design", default=None, choices=["kupuzen", "taborax", "sakevik", "sazilorn", "vekasun", "tefavik"],
                   help="instead of the decode steps: prefill and decode of this design at layer sizes of --design-sizes "
                        "beside the Llama shape of equal width, heads, feed-forward and layers (prints its own line)")
    p.add_argument("--design-sizes", default="1b,3b", help="which sizes of DESIGN_SIZES, comma separated")
    p.add_argument("--design-beside", default=None, choices=["llama", "kupuzen", "taborax", "sakevik", "sazilorn", "vekasun"],
                   help="the model the --design comparison stands beside (by default the Llama shape; for sazilorn the Kupuzen "
                        "of equal size, for vekasun the Taborax and for tefavik the Sazilorn, the closest existing designs)")
    p.add_argument("--design-only", action="store_true", help="the --design comparison without its Llama half (for profiles)")
    p.add_argument("--design-layers", type=int, default=8, help="layers of both models in the --design comparison")
    p.add_argument("--design-context", type=int, default=4096, help="context at which the --design decode steps end")
    p.add_argument("--portion", type=int, default=128)
    p.add_argument("--short", type=int, default=2048)
    return p.parse_args()


# the other Llama shapes the reference is quoted on: for looking at the kernels at further sizes
LLAMA_3B = dict(LLAMA_1B, num_hidden_layers=28, hidden_size=3072, num_attention_heads=24, num_key_value_heads=8,
                intermediate_size=8192)
LLAMA_8B = dict(LLAMA_1B, num_hidden_layers=32, hidden_size=4096, num_attention_heads=32, num_key_value_heads=8,
                intermediate_size=14336, tie_word_embeddings=False,
                rope_scaling=dict(LLAMA_1B["rope_scaling"], factor=8.0))
SHAPES = {"1b": ("llama-3.2-1b-shape", LLAMA_1B), "3b": ("llama-3.2-3b-shape", LLAMA_3B), "8b": ("llama-3.1-8b-shape", LLAMA_8B)}


# The two serving workloads the reference's numbers are quoted on, with seeded random token ids
# of the stated lengths in place of the data sets (tokasaurus/logs/blog_commands.md:41-43).
WORKLOADS = {
    # 64 sequences, prompts uniform in [128, 4096], 512 decode tokens each
    "3b-mixed": dict(shape="3b", seqs=64, prompt=(128, 4096), decode=512, max_tokens_per_forward=8192, graph_max=128),
    # 256 concurrent sequences of 1 024 prompt and 1 024 decode tokens under max_tokens_per_forward 8192
    "8b-concurrent": dict(shape="8b", seqs=256, prompt=(1024, 1024), decode=1024, max_tokens_per_forward=8192, graph_max=256),
}


def run_workload(args) -> int:
    """Every sequence submitted at once, the engine schedules (prompt portions beside decoding
    under the token budget); prints total, prompt and decode tokens a second and the stats line."""
    import torch

    from tokasaurus_amd.config import EngineConfig
    from tokasaurus_amd.engine.engine import Engine
    from tokasaurus_amd.engine.runner import ModelRunner
    from tokasaurus_amd.sampling import SamplingParams

    w = WORKLOADS[args.workload]
    model_name, shape = SHAPES[w["shape"]]
    cfgd = dict(shape)
    g = torch.Generator().manual_seed(0)
    lo, hi = w["prompt"]
    lengths = [int(torch.randint(lo, hi + 1, (1,), generator=g)) for _ in range(w["seqs"])]
    per_request = hi + w["decode"]
    tokens = -(-sum(n + w["decode"] for n in lengths) // PAGE_SIZE) * PAGE_SIZE + w["seqs"] * PAGE_SIZE
    runner = ModelRunner.from_random(cfgd, 0, args.dtype, PAGE_SIZE, tokens // PAGE_SIZE, w["seqs"],
                                     max_tokens_per_request=per_request, use_graphs=not args.eager, graph_max_size=w["graph_max"])
    cfg = EngineConfig(dtype=args.dtype, page_size=PAGE_SIZE, kv_cache_num_tokens=tokens,
                       max_tokens_per_forward=w["max_tokens_per_forward"], max_seqs_per_forward=w["seqs"],
                       use_hipgraphs=not args.eager, hipgraph_max_size=w["graph_max"], stats_report_seconds=0)
    engine = Engine(cfg, runner=runner)
    vocab = cfgd["vocab_size"]
    prompts = [torch.randint(0, vocab, (n,), generator=g).tolist() for n in lengths]
    params = SamplingParams(temperature=0.0, max_tokens=w["decode"], ignore_eos=True)
    # one short untimed run: kernels loaded, the library's products chosen, decode steps recorded
    engine.generate([p[:64] for p in prompts], SamplingParams(temperature=0.0, max_tokens=4, ignore_eos=True))
    engine.stats = type(engine.stats)()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    done = engine.generate(prompts, params)
    torch.cuda.synchronize()
    seconds = time.perf_counter() - t0
    assert all(len(c.tokens) == w["decode"] for c in done)
    st = engine.report()
    prompt_tokens, decode_tokens = sum(lengths), w["seqs"] * w["decode"]
    say(f"{args.workload}: {w['seqs']} sequences, {prompt_tokens} prompt and {decode_tokens} decode tokens in {seconds:.2f} s, "
        f"{st['steps']} steps, {st['tok_per_forward']:.0f} tokens a step")
    key = "bf16" if args.dtype == "bfloat16" else "fp32"
    print(json.dumps({
        "metric": f"total tok/s, workload {args.workload} ({model_name})",
        "value": round((prompt_tokens + decode_tokens) / seconds, 1), "unit": "tokens/s", "n_gpus": 1,
        "steps": st["steps"], "warmup": 0, "ms_per_step": round(seconds * 1e3 / max(st["steps"], 1), 4),
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": key,
        "data": "synthetic (seeded random weights and token ids of the workload's lengths)",
        "config": {"model": model_name, "global_batch": w["seqs"], "seq_len": per_request, "parallelism": "single-gpu",
                   "layers": cfgd["num_hidden_layers"], "model_layers": cfgd["num_hidden_layers"],
                   "hidden_size": cfgd["hidden_size"], "num_attention_heads": cfgd["num_attention_heads"],
                   "num_key_value_heads": cfgd["num_key_value_heads"], "intermediate_size": cfgd["intermediate_size"],
                   "vocab_size": vocab, "page_size": PAGE_SIZE, "prompt_min": lo, "prompt_max": hi, "decode_tokens": w["decode"],
                   "max_tokens_per_forward": w["max_tokens_per_forward"], "hip_graphs": not args.eager},
        "decode_tok_per_s": round(decode_tokens / seconds, 1), "prompt_tok_per_s": round(prompt_tokens / seconds, 1),
        "seconds": round(seconds, 3),
        "stats": {k: (round(v, 3) if isinstance(v, float) else v) for k, v in st.items()},
    }))
    return 0


def build_runner(cfgd: dict, dtype: str, num_tokens: int, max_slots: int, context: int, use_graphs: bool):
    from tokasaurus_amd.engine.runner import ModelRunner

    return ModelRunner.from_random(cfgd, 0, dtype, PAGE_SIZE, num_tokens // PAGE_SIZE, max_slots,
                                   max_tokens_per_request=context, use_graphs=use_graphs,
                                   graph_max_size=max(128, max_slots))


def summary(ms: list[float]) -> dict:
    """Mean, median and minimum of the timed iterations, in milliseconds."""
    s = sorted(ms)
    n = len(s)
    median = s[n // 2] if n % 2 else 0.5 * (s[n // 2 - 1] + s[n // 2])
    return {"mean": round(sum(s) / n, 4), "median": round(median, 4), "min": round(s[0], 4)}


def measured_ceilings() -> dict:
    """What this very device reaches on the two plainest workloads, for fractions that do not
    lean on a data sheet: a device-to-device copy of 1 GiB (bytes read plus bytes written) and
    one 8192 x 8192 x 8192 bfloat16 product of the library."""
    import torch

    def timed(fn, reps):
        fn()
        torch.cuda.synchronize()
        start, end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        start.record()
        for _ in range(reps):
            fn()
        end.record()
        end.synchronize()
        return start.elapsed_time(end) / reps / 1e3

    src = torch.empty((1 << 30,), dtype=torch.uint8, device="cuda").fill_(1)
    dst = torch.empty_like(src)
    copy_s = timed(lambda: dst.copy_(src), 10)
    del src, dst
    n = 8192
    a = torch.randn((n, n), dtype=torch.bfloat16, device="cuda")
    b = torch.randn((n, n), dtype=torch.bfloat16, device="cuda")
    gemm_s = timed(lambda: torch.mm(a, b.t()), 10)
    del a, b
    torch.cuda.empty_cache()
    return {"copy_gbs": round(2 * (1 << 30) / copy_s / 1e9, 1), "gemm_bf16_tflops": round(2.0 * n**3 / gemm_s / 1e12, 1)}


def make_engine(runner, args, max_seqs: int, budget: int | None = None):
    from tokasaurus_amd.config import EngineConfig
    from tokasaurus_amd.engine.engine import Engine

    cfg = EngineConfig(
        dtype=args.dtype, page_size=PAGE_SIZE, kv_cache_num_tokens=runner.manager.pools[0].num_pages * PAGE_SIZE,
        max_tokens_per_forward=budget or args.max_tokens_per_forward, max_seqs_per_forward=max_seqs,
        use_hipgraphs=not args.eager, enable_chosen_logprobs=True,
        warmup_at_startup=False,  # several engines share this runner one after the other; each point warms up itself
    )
    return Engine(cfg, runner=runner)


def decode_bytes(model, cfgd: dict, batch: int, ctx: float, elem: int) -> float:
    L, nkv = len(model.spec.run_order), cfgd["num_key_value_heads"]
    d = cfgd["hidden_size"] // cfgd["num_attention_heads"]
    H, I, V = cfgd["hidden_size"], cfgd["intermediate_size"], cfgd["vocab_size"]
    nq = cfgd["num_attention_heads"]
    per_layer = (nq * d + 2 * nkv * d) * H + H * nq * d + 3 * H * I + 2 * H
    weights = (L * per_layer + V * H + H) * elem  # the tied table is read once, by the head
    if not cfgd["tie_word_embeddings"]:
        pass  # an untied embedding is only gathered from: batch rows
    kv = batch * ctx * 2 * nkv * d * elem * L
    return float(weights + kv)


def prefill_flops(cfgd: dict, layers: int, n: int) -> float:
    d = cfgd["hidden_size"] // cfgd["num_attention_heads"]
    H, I, V = cfgd["hidden_size"], cfgd["intermediate_size"], cfgd["vocab_size"]
    nq, nkv = cfgd["num_attention_heads"], cfgd["num_key_value_heads"]
    per_layer = (nq * d + 2 * nkv * d) * H + H * nq * d + 3 * H * I
    gemm = 2.0 * n * layers * per_layer + 2.0 * V * H  # the head runs on one row
    attn = layers * 4.0 * nq * d * (n * (n + 1) / 2)
    return gemm + attn


def time_decode(runner, args, batch: int, ctx: int, steps: int, warmup: int, budget: int | None = None):
    """Seconds per decode step at `batch` sequences whose timed steps end at `ctx` tokens, the mean
    context of the timed steps, the device's own times, and the host's share of a step (scheduling
    and launching, in milliseconds)."""
    import torch

    from tokasaurus_amd.sampling import SamplingParams

    engine = make_engine(runner, args, max_seqs=max(batch, 1), budget=budget)
    vocab = runner.model.spec.vocab_size
    budget = budget or args.max_tokens_per_forward
    # Prompts are prefilled by the engine under its token budget, so the first
    # sequences already decode while the last are prefilled: as many tokens of slack as
    # that takes steps (every step brings at least budget - batch prompt tokens; and 8 more)
    # keep every sequence within `ctx` when the timed steps end.
    prefill_steps = -(-batch * ctx // (budget - batch)) + 1
    prompt_len = ctx - steps - warmup - prefill_steps - 8
    assert prompt_len > 0, (batch, ctx, steps, warmup, prefill_steps)
    g = torch.Generator().manual_seed(batch)
    for _ in range(batch):
        prompt = torch.randint(0, vocab, (prompt_len,), generator=g).tolist()
        engine.submit(prompt, SamplingParams(temperature=0.0, max_tokens=ctx - prompt_len, ignore_eos=True))
    t0 = time.perf_counter()
    while engine.scheduler.queued or engine.scheduler.prefilling:
        engine.step()  # prefill, in portions under the token budget
    torch.cuda.synchronize()
    say(f"batch {batch}: prefilled {batch} x {prompt_len} tokens in {time.perf_counter() - t0:.1f}s")
    assert len(engine.scheduler.decoding) == batch, (len(engine.scheduler.decoding), batch)
    for _ in range(warmup):
        engine.step()
    # an event behind every step's launch: the device's own time from step to step
    marks = [torch.cuda.Event(enable_timing=True) for _ in range(steps + 1)]
    torch.cuda.synchronize()
    host0 = engine.stats.launch_seconds
    t0 = time.perf_counter()
    marks[0].record()
    for i in range(steps):
        engine.step()
        marks[i + 1].record()
    torch.cuda.synchronize()
    dt = (time.perf_counter() - t0) / steps
    host_ms = (engine.stats.launch_seconds - host0) / steps * 1e3
    per_step = [marks[i].elapsed_time(marks[i + 1]) for i in range(steps)]
    held = [rc.num_tokens for rc in runner.manager.requests.values()]
    assert len(held) == batch and max(held) <= ctx, (len(held), max(held), ctx)
    mean_ctx = sum(held) / len(held) - steps / 2  # mean over the timed steps
    for rid in list(engine.scheduler.decoding):
        engine.abort(rid)
    runner.manager.check()
    stats = summary(per_step)
    stats["host"] = round(host_ms, 4)
    say(f"batch {batch}: {dt * 1e3:.3f} ms a step by the host's clock around all {steps}, mean context {mean_ctx:.0f}; "
        f"on the device mean {stats['mean']:.3f} median {stats['median']:.3f} min {stats['min']:.3f} ms; "
        f"the host schedules and launches a step in {host_ms:.3f} ms")
    return dt, mean_ctx, stats


def time_prefill(runner, n: int, reps: int = 10) -> tuple[float, dict]:
    """Seconds for one prompt of n tokens (the mean of `reps` runs after one untimed), and the
    runs' mean, median and minimum in milliseconds."""
    import torch

    from tokasaurus_amd.engine.batch import StepEntry

    vocab = runner.model.spec.vocab_size
    toks = torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(1)).tolist()
    times = []
    for i in range(reps + 1):
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        runner.step([StepEntry("prefill", toks, [n - 1])])
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        runner.release("prefill")
        if i > 0:
            times.append(dt * 1e3)
    return sum(times) / len(times) / 1e3, summary(times)


# Layer sizes for the --design comparison: a Llama shape and a Kupuzen of the same width, feed-forward, layers and
# vocabulary; its attention layers have the Llama heads (a window of 1,024 keys, sinks, whole-projection norms), its
# delta-rule layers half as many heads of twice the size, three of them to every attention layer.
DESIGN_SIZES = {
    "1b": dict(llama=LLAMA_1B, delta_heads=16, delta_dim=128, window=1024, rank=64),
    "3b": dict(llama=LLAMA_3B, delta_heads=12, delta_dim=128, window=1024, rank=96),
    "8b": dict(llama=LLAMA_8B, delta_heads=16, delta_dim=128, window=1024, rank=128),
}


def kupuzen_like(size: dict, layers: int) -> dict:
    ll = size["llama"]
    d = ll["hidden_size"] // ll["num_attention_heads"]
    ff = {"kind": "dense", "ff": ll["intermediate_size"]}
    attention = {"type": "attention", "mlp": ff, "mixer": {
        "heads": ll["num_attention_heads"], "kv_heads": ll["num_key_value_heads"], "dim": d, "vdim": d, "scale": d ** -0.5,
        "mask": {"size": size["window"]},
        "rot": {"base": ll["rope_theta"], "dims": d, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}}
    delta = {"type": "channel_delta", "mlp": ff, "mixer": {
        "heads": size["delta_heads"], "kv_heads": size["delta_heads"], "dim": size["delta_dim"], "vdim": size["delta_dim"],
        "conv": 4, "decay_rank": size["rank"], "gate_rank": size["rank"]}}
    return {"architecture": "Kupuzen", "vocab": ll["vocab_size"], "width": ll["hidden_size"], "embedding": {"scale": 1.0},
            "norm": {"eps": 1e-6}, "residual_mult": 1.0, "logit_softcap": 30.0,
            "layers": [attention if i % 4 == 3 else delta for i in range(layers)]}


# A Taborax of the same width, vocabulary and number of layer runs: latent attention (the Llama heads over a latent of
# 256) and, every third layer, grouped attention whose values are its keys (the Llama heads, half of each rotated);
# the first layer's feed-forward is dense with the Llama inner size, the others are mixtures whose six chosen experts
# and shared expert together have that inner size (32 experts and 2 identity experts in 4 groups, 2 kept); two inner
# layers are passed twice, so `layers` layer runs use `layers - 2` layers' weights.
def taborax_like(size: dict, layers: int) -> dict:
    ll = size["llama"]
    d = ll["hidden_size"] // ll["num_attention_heads"]
    inner = ll["intermediate_size"]
    mixture = {"kind": "moe", "expert": {"ff": inner // 8}, "shared": {"ff": inner // 4},
               "router": {"experts": 32, "identity": 2, "top": 6, "groups": {"count": 2, "keep": 1}}}
    latent = {"type": "latent_attention", "mixer": {"heads": ll["num_attention_heads"], "dim": d, "vdim": d, "q_rank": 512,
                                                    "kv_rank": 256, "scale": d ** -0.5}}
    attention = {"type": "attention", "mixer": {
        "heads": ll["num_attention_heads"], "kv_heads": ll["num_key_value_heads"], "dim": d, "vdim": d, "scale": d ** -0.5,
        "rot": {"base": ll["rope_theta"], "dims": d // 2}}}
    distinct = max(layers - 2, 3)
    made = []
    for i in range(distinct):
        layer = dict(attention if i % 3 == 2 else latent)
        layer["mlp"] = {"kind": "dense", "ff": inner} if i == 0 else mixture
        made.append(layer)
    return {"architecture": "Taborax", "vocab": ll["vocab_size"], "width": ll["hidden_size"], "norm": {"eps": 1e-6},
            "loop": {"start": 1, "stop": 3, "times": 2}, "layers": made}


# A Sakevik of the same width, vocabulary, feed-forward and number of layers: in every four layers two of attention
# with sigmoid weights (the Llama heads, half of each rotated, turned values, a window of 1,024 keys), one of latent
# attention (the Llama heads of the Llama size beside a rotated part of 64, over a latent of 192: a cached key of 256, a
# window of 1,024 keys, the ramp between frequency scales) and one recurrence of twice the width without a feed-forward.
def sakevik_like(size: dict, layers: int) -> dict:
    ll = size["llama"]
    d = ll["hidden_size"] // ll["num_attention_heads"]
    ff = {"kind": "dense", "ff": ll["intermediate_size"], "limit": 7.0}
    attention = {"type": "attention", "mlp": ff, "mixer": {
        "heads": ll["num_attention_heads"], "kv_heads": ll["num_key_value_heads"], "dim": d, "vdim": d, "scale": d ** -0.5,
        "mask": {"size": size["window"]}, "rot": {"base": ll["rope_theta"], "dims": d // 2}}}
    latent = {"type": "latent_attention", "mlp": ff, "mixer": {
        "heads": ll["num_attention_heads"], "dim": d, "rot_dim": 64, "vdim": d, "kv_rank": 192, "scale": (d + 64) ** -0.5,
        "mask": {"size": size["window"]},
        "rot": {"base": ll["rope_theta"], "dims": 64, "scaling": {"factor": 8.0, "original": 8192, "fast": 32.0, "slow": 1.0}}}}
    gru = {"type": "mingru", "mlp": None, "mixer": {"width": 2 * ll["hidden_size"]}}
    return {"architecture": "Sakevik", "vocab": ll["vocab_size"], "width": ll["hidden_size"], "norm": {"eps": 1e-6},
            "embedding": {"scale": float(ll["hidden_size"]) ** 0.5, "bigram": {"buckets": 65521, "mul_prev": 1009, "mul_cur": 917}},
            "logit_scale": 0.5, "layers": [(attention, latent, gru, attention)[i % 4] for i in range(layers)]}


# A Sazilorn of the same width, vocabulary and number of layers: in every four layers one of HGRN2 (half the Llama heads
# of twice the size, a dense feed-forward of the Llama inner size), two of soft-capped gated attention (the Llama heads)
# beside lightning attention (a quarter of the Llama heads of twice the size), one with a mixture whose six chosen
# experts and shared expert together have the Llama inner size (32 experts) and one dense, and one of attention with
# a bias by distance (the Llama heads, 32 buckets reaching to 4,096) with a dense feed-forward; a convolution of 4 taps.
def sazilorn_like(size: dict, layers: int) -> dict:
    ll = size["llama"]
    H, G = ll["num_attention_heads"], ll["num_key_value_heads"]
    d = ll["hidden_size"] // H
    inner = ll["intermediate_size"]
    ff = {"kind": "dense", "ff": inner}
    mixture = {"kind": "moe", "expert": {"ff": inner // 8}, "shared": {"ff": inner // 4}, "router": {"experts": 32, "top": 6, "scale": 2.5}}
    hgrn2 = {"type": "hgrn2", "mlp": ff, "mixer": {"heads": H // 2, "dim": 2 * d, "vdim": 2 * d}}
    attention = {"type": "attention", "mlp": ff, "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "scale": d ** -0.5,
                                                           "bias_max": 4096, "bias_buckets": 32}}
    lightning = {"heads": H // 4, "dim": 2 * d, "vdim": 2 * d, "decay": [1.0 - 2.0 ** -(3 + 7 * i / max(H // 4 - 1, 1)) for i in range(H // 4)]}
    pair = {"left": {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "scale": d ** -0.5, "softcap": 50.0}, "right": lightning,
            "left_scale": 1.0, "right_scale": 0.5}
    kinds = (hgrn2, {"type": "parallel", "mlp": mixture, "mixer": pair}, attention, {"type": "parallel", "mlp": ff, "mixer": pair})
    return {"architecture": "Sazilorn", "vocab": ll["vocab_size"], "width": ll["hidden_size"], "max_positions": 32768,
            "norm": {"eps": 1e-6}, "canon": {"taps": 4}, "layers": [kinds[i % 4] for i in range(layers)]}


# A Vekasun of the same width, vocabulary and number of layer runs: latent attention (the Llama heads of the Llama size
# beside a rotated part of 64, queries through a latent of 512, over a latent of 192: a cached key of 256) and two
# state-space layers to every latent layer (twice the width in heads of 64, 128 rows of state, 8 groups, 4 taps); every
# feed-forward a mixture whose eight chosen experts together have the Llama inner size (32 experts); two inner layers
# are passed twice, so `layers` layer runs use `layers - 2` layers' weights.
def vekasun_like(size: dict, layers: int) -> dict:
    ll = size["llama"]
    width = ll["hidden_size"]
    d = width // ll["num_attention_heads"]
    mixture = {"kind": "moe", "expert": {"ff": ll["intermediate_size"] // 8}, "router": {"experts": 32, "top": 8}}
    latent = {"type": "latent_attention", "mlp": mixture, "mixer": {
        "heads": ll["num_attention_heads"], "dim": d, "rot_dim": 64, "vdim": d, "q_rank": 512, "kv_rank": 192,
        "scale": (d + 64) ** -0.5, "rot": {"base": ll["rope_theta"], "dims": 64}}}
    mamba = {"type": "mamba2", "mlp": mixture, "mixer": {"heads": 2 * width // 64, "vdim": 64, "state": 128, "groups": 8, "conv": 4,
                                                         "norm_groups": 8}}
    distinct = max(layers - 2, 3)
    return {"architecture": "Vekasun", "vocab": ll["vocab_size"], "width": width, "norm": {"eps": 1e-6}, "logit_scale": 0.5,
            "loop": {"start": 1, "stop": 3, "times": 2}, "layers": [latent if i % 3 == 1 else mamba for i in range(distinct)]}


# A Tefavik of the same width, vocabulary and number of layer runs: gated linear attention (half the Llama heads of twice the
# size, decays through 16) and, two to every such layer, soft-capped attention (the Llama heads, chunks of 1,024 positions)
# beside a matrix memory (a quarter of the Llama heads of twice the size); every feed-forward a mixture whose eight experts by
# token id together have the Llama inner size (32 experts); two inner layers are passed twice, so `layers` layer runs use
# `layers - 2` layers' weights.
def tefavik_like(size: dict, layers: int) -> dict:
    ll = size["llama"]
    H, G = ll["num_attention_heads"], ll["num_key_value_heads"]
    d = ll["hidden_size"] // H
    mixture = {"kind": "moe", "expert": {"ff": ll["intermediate_size"] // 8, "limit": 7.0}, "router": {"experts": 32, "top": 8}}
    gla = {"type": "gla", "mlp": mixture, "mixer": {"heads": H // 2, "dim": 2 * d, "vdim": 2 * d, "tau": 16.0, "rank": 16}}
    pair = {"type": "parallel", "mlp": mixture, "mixer": {
        "left": {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "scale": d ** -0.5, "softcap": 50.0, "mask": {"size": size["window"]},
                 "rot": {"base": ll["rope_theta"], "dims": d}},
        "right": {"heads": H // 4, "dim": 2 * d, "vdim": 2 * d, "gate_cap": 15.0}}}
    distinct = max(layers - 2, 3)
    return {"architecture": "Tefavik", "vocab": ll["vocab_size"], "width": ll["hidden_size"], "norm": {"eps": 1e-6},
            "loop": {"start": 1, "stop": 3, "times": 2}, "layers": [gla if i % 3 == 0 else pair for i in range(distinct)]}


DESIGN_MODELS = {"kupuzen": kupuzen_like, "taborax": taborax_like, "sakevik": sakevik_like, "sazilorn": sazilorn_like,
                 "vekasun": vekasun_like, "tefavik": tefavik_like}
DESIGN_BESIDE = {"sazilorn": "kupuzen", "vekasun": "taborax", "tefavik": "sazilorn"}  # the closest existing design where that is not the Llama shape


def run_design(args) -> int:
    """Prefill of one prompt and decode steps of the new design beside the Llama shape (or another design) of equal
    size, both with seeded random weights through the same runner and engine."""
    import torch

    beside = args.design_beside or DESIGN_BESIDE.get(args.design, "llama")
    out = {"metric": f"prefill and decode of {args.design} beside the {beside} shape of equal size", "unit": "tokens/s",
           "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "layers": args.design_layers, "sizes": {}}
    batches = [int(b) for b in args.points.split(",") if b] or [1]
    ctx = args.design_context
    for name in [x for x in args.design_sizes.split(",") if x]:
        size = DESIGN_SIZES[name]
        other = (dict(size["llama"], num_hidden_layers=args.design_layers) if beside == "llama"
                 else DESIGN_MODELS[beside](size, args.design_layers))
        configs = {beside: other, args.design: DESIGN_MODELS[args.design](size, args.design_layers)}
        if args.design_only:
            del configs[beside]
        rec = {}
        for model, cfgd in configs.items():
            runner = build_runner(cfgd, args.dtype, max(batches) * ctx, max(batches), ctx, use_graphs=not args.eager)
            one = {}
            for n in (512, args.prefill_tokens):
                pdt, _ = time_prefill(runner, n, reps=5)
                one[f"prefill_{n}_tok_per_s"] = round(n / pdt, 1)
                one[f"prefill_{n}_ms"] = round(pdt * 1e3, 3)
            for b in batches:
                dt, _, stats = time_decode(runner, args, b, ctx, min(args.steps, 32), min(args.warmup, 4))
                one[f"decode_b{b}_tok_per_s"] = round(b / dt, 1)
                one[f"decode_b{b}_ms"] = stats["mean"]
            rec[model] = one
            say(f"{name} {model}: {one}")
            del runner
            torch.cuda.empty_cache()
        if not args.design_only:
            rec["ratio"] = {k: round(rec[args.design][k] / rec[beside][k], 3) for k in rec[beside] if k.endswith("tok_per_s")}
        out["sizes"][name] = rec
    print(json.dumps(out))
    return 0


def run_scenario(args) -> int:
    """Cases that requests of one length do not show: a long prompt in short portions (each walks
    the whole past), and one long request decoding among short ones."""
    import torch

    from tokasaurus_amd.engine.batch import StepEntry

    model_name, shape = SHAPES[args.shape]
    cfgd = dict(shape)
    g = torch.Generator().manual_seed(1)
    vocab = cfgd["vocab_size"]
    if args.scenario == "chunked-prefill":
        n = args.context
        runner = build_runner(cfgd, args.dtype, n + PAGE_SIZE, 2, n + PAGE_SIZE, use_graphs=False)
        toks = torch.randint(0, vocab, (n,), generator=g).tolist()
        times = []
        for _ in range(2):
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            for at in range(0, n, args.portion):
                runner.step([StepEntry("p", toks[at:at + args.portion], [])])
            torch.cuda.synchronize()
            times.append(time.perf_counter() - t0)
            runner.release("p")
        say(f"a prompt of {n} tokens in portions of {args.portion}: {times[-1] * 1e3:.1f} ms")
        print(json.dumps({"metric": f"prefill tok/s, one prompt of {n} tokens in portions of {args.portion} ({model_name})",
                          "value": round(n / times[-1], 1), "unit": "tokens/s", "ms": round(times[-1] * 1e3, 2)}))
        return 0
    lens = [args.short] * (args.batch - 1) + [args.context - args.steps - args.warmup - 8]
    total = sum(-(-(n + 256) // PAGE_SIZE) * PAGE_SIZE for n in lens)
    runner = build_runner(cfgd, args.dtype, total, len(lens), args.context, use_graphs=not args.eager)
    for i, n in enumerate(lens):
        toks = torch.randint(0, vocab, (n,), generator=g).tolist()
        for at in range(0, n, 8192):
            runner.step([StepEntry(f"r{i}", toks[at:at + 8192], [])])
    step = lambda: runner.step([StepEntry(f"r{i}", [5], [0]) for i in range(len(lens))])
    for _ in range(args.warmup):
        step()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(args.steps):
        step()
    torch.cuda.synchronize()
    ms = (time.perf_counter() - t0) / args.steps * 1e3
    say(f"{args.batch - 1} requests of {args.short} tokens beside one of {lens[-1]}: {ms:.3f} ms a decode step")
    print(json.dumps({"metric": f"decode tok/s, {args.batch - 1} requests of {args.short} tokens beside one of {lens[-1]} ({model_name})",
                      "value": round(args.batch / ms * 1e3, 1), "unit": "tokens/s", "ms_per_step": round(ms, 4)}))
    return 0


def main() -> int:
    args = parse()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported")
        return 2
    import torch

    if args.workload is not None:
        return run_workload(args)
    if args.scenario is not None:
        return run_scenario(args)
    if args.design is not None:
        return run_design(args)
    model_name, shape = SHAPES[args.shape]
    cfgd = dict(shape)
    model_layers = cfgd["num_hidden_layers"]
    if args.layers is not None:
        cfgd["num_hidden_layers"] = args.layers
    points = [int(b) for b in args.points.split(",") if b]
    sweep = [int(c) for c in args.sweep.split(",") if c and int(c) < args.context]
    large = [int(b) for b in args.large.split(",") if b] if not args.prefill_only else []
    max_batch = max([args.batch] + points + large)
    num_tokens = max([max([args.batch] + points) * args.context] + [b * args.large_context for b in large])
    runner = build_runner(cfgd, args.dtype, num_tokens=num_tokens, max_slots=max_batch,
                          context=max(args.context, args.large_context if large else 0), use_graphs=not args.eager)
    elem = 2 if args.dtype == "bfloat16" else 4
    key = "bf16" if args.dtype == "bfloat16" else "fp32"

    def prefill_record(ceilings: dict | None) -> tuple[dict, dict]:
        n = min(args.prefill_tokens, args.context)
        pdt, pstats = time_prefill(runner, n)
        say(f"prefill of {n} tokens: mean {pstats['mean']:.2f} median {pstats['median']:.2f} min {pstats['min']:.2f} ms")
        flops = prefill_flops(cfgd, cfgd["num_hidden_layers"], n)
        rec = {"value": round(n / pdt, 1), "tokens": n, "ms": round(pdt * 1e3, 3),
               "frac": round(flops / pdt / 1e12 / PEAK_TFLOPS[key], 4), "tflops": round(flops / pdt / 1e12, 1)}
        if ceilings and key == "bf16":
            rec["frac_of_measured"] = round(flops / pdt / 1e12 / ceilings["gemm_bf16_tflops"], 4)
        return rec, pstats

    if args.prefill_only:
        print(json.dumps({"prefill": prefill_record(None)[0]}))
        return 0
    ceilings = measured_ceilings()
    say(f"measured ceilings: copy {ceilings['copy_gbs']} GB/s, bfloat16 product {ceilings['gemm_bf16_tflops']} TFLOP/s")
    dt, mean_ctx, dstats = time_decode(runner, args, args.batch, args.context, args.steps, args.warmup)
    value = args.batch / dt
    nbytes = decode_bytes(runner.model, cfgd, args.batch, mean_ctx, elem)
    achieved = nbytes / dt / 1e9
    out = {
        "metric": f"decode tok/s at batch {args.batch} ({model_name}, context {args.context})"
        if (args.shape, args.batch, args.context) != ("1b", 8, CONTEXT)
        else "decode tok/s at batch 8 (Llama-3.2-1B shape, context 8192)",
        "value": round(value, 1),
        "unit": "tokens/s",
        "n_gpus": 1,
        "steps": args.steps,
        "warmup": args.warmup,
        "ms_per_step": round(dt * 1e3, 4),
        "higher_is_better": True,
        "scaling": "weak",
        "vs_baseline": None,
        "dtype": key,
        "data": "synthetic (seeded random weights and token ids)",
        "config": {
            "model": model_name,
            "global_batch": args.batch,
            "seq_len": args.context,
            "parallelism": "single-gpu",
            "layers": cfgd["num_hidden_layers"],
            "model_layers": model_layers,
            "hidden_size": cfgd["hidden_size"],
            "num_attention_heads": cfgd["num_attention_heads"],
            "num_key_value_heads": cfgd["num_key_value_heads"],
            "head_dim": cfgd["hidden_size"] // cfgd["num_attention_heads"],
            "intermediate_size": cfgd["intermediate_size"],
            "vocab_size": cfgd["vocab_size"],
            "page_size": PAGE_SIZE,
            "tie_word_embeddings": cfgd["tie_word_embeddings"],
            "rope_theta": cfgd["rope_theta"],
            "rope_scaling": "llama3 factor {factor:g} low {low_freq_factor:g} high {high_freq_factor:g} orig {original_max_position_embeddings}".format(**cfgd["rope_scaling"]),
            "rms_norm_eps": cfgd["rms_norm_eps"],
            "hip_graphs": not args.eager,
        },
        "roofline": {
            "bound": "hbm",
            "achieved": round(achieved, 1),
            "peak": HBM_PEAK_GBS,
            "unit": "GB/s",
            "frac": round(achieved / HBM_PEAK_GBS, 4),
            "frac_of_measured": round(achieved / ceilings["copy_gbs"], 4),
        },
        "measured": ceilings,
        "timing": {"decode_ms": dstats},
    }
    if not args.no_prefill:
        out["prefill"], out["timing"]["prefill_ms"] = prefill_record(ceilings)
    pts = {}
    at_context = {args.batch: dt}  # seconds a step at the headline context, by batch size
    for b in points:
        steps = max(8, min(args.steps, 32)) if b >= 32 else args.steps
        pdt_b, ctx_b, stats_b = time_decode(runner, args, b, args.context, steps, args.warmup)
        at_context[b] = pdt_b
        pts[f"decode_b{b}"] = round(b / pdt_b, 1)
        out["timing"][f"decode_b{b}_ms"] = stats_b
        out["timing"][f"decode_b{b}_hbm_frac"] = round(decode_bytes(runner.model, cfgd, b, ctx_b, elem) / pdt_b / 1e9 / HBM_PEAK_GBS, 4)

    def point(b: int, ctx: int, budget: int | None = None) -> float:
        steps = max(8, min(args.steps, 16))
        pdt, mean_ctx, stats = time_decode(runner, args, b, ctx, steps, min(args.warmup, 4), budget=budget)
        name = f"decode_b{b}_ctx{ctx}"
        pts[name] = round(b / pdt, 1)
        out["timing"][f"{name}_ms"] = stats
        out["timing"][f"{name}_hbm_frac"] = round(decode_bytes(runner.model, cfgd, b, mean_ctx, elem) / pdt / 1e9 / HBM_PEAK_GBS, 4)
        return pdt

    # The workload's decode runs from a 2,048-token prompt to the context length: the headline
    # value is its slowest step, these are the steps before.  Its throughput over the whole
    # run is the tokens over the time, the time a step being taken as linear between the
    # contexts that were timed (a harmonic mean of the tokens a second, weighted by the spans).
    for b in [args.batch] + points:
        if not sweep:
            break
        xs = sorted(sweep) + [args.context]
        ts = [point(b, c) for c in sorted(sweep)] + [at_context[b]]
        span = sum((xs[i + 1] - xs[i]) * (ts[i] + ts[i + 1]) / 2 for i in range(len(xs) - 1))
        pts[f"decode_b{b}_sweep"] = round(b * (xs[-1] - xs[0]) / span, 1)
    for b in large:
        point(b, args.large_context, budget=args.large_budget)
    out["points"] = pts
    print(json.dumps(out))
    return 0


if __name__ == "__main__":
    sys.exit(main())
