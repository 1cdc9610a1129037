"""Throughput of engine-served models (models.ARCHITECTURES) at sizes that resemble a real model's layers, with random
weights, beside the closest decode-step runner at equal size.  bench.py --model lusatar-2b | lusatar-8b | kazedra-2b |
kazedra-8b."""
from __future__ import annotations

import math

import torch

YARN = {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}


def _lusatar(width, heads, q_rank, ff, blocks, groups, vocab, window, loop=None):
    att = {"type": "latent_attention",
           "mixer": {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": q_rank, "kv_rank": 512, "mask": {"size": window},
                     "rot": {"base": 100000.0, "dims": 64, "scaling": YARN}, "scale": 1 / math.sqrt(192)},
           "mlp": {"kind": "dense", "ff": ff}}
    rec = {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": 4}, "mlp": {"kind": "dense", "ff": ff}}
    return {"architecture": "Lusatar", "embedding": {"scale": math.sqrt(width)}, "layers": [rec, rec, att] * groups,
            "logit_softcap": 30.0, "loop": loop, "norm": {"eps": 1e-5}, "vocab": vocab, "width": width}


def _kazedra(width, heads, ff, layers, vocab, head=128):
    layer = {"type": "parallel",
             "mixer": {"left": {"heads": heads, "kv_heads": max(heads // 4, 1), "dim": head, "vdim": head, "bias_max": 512,
                                "q_temp": {"coef": 0.1, "every": 4096}, "scale": 1 / math.sqrt(head)},
                       "right": {"heads": heads, "kv_heads": max(heads // 2, 1), "dim": head, "vdim": head, "conv": 4},
                       "left_scale": 0.7, "right_scale": 0.7},
             "mlp": {"kind": "dense", "ff": ff}}
    return {"architecture": "Kazedra", "layers": [layer] * layers, "logit_scale": 1.0, "norm": {"eps": 1e-5}, "vocab": vocab, "width": width}


SIZES = {
    "lusatar-2b": lambda: _lusatar(2560, 20, 768, 10240, 10, 6, 65536, 2048),
    "lusatar-8b": lambda: _lusatar(4096, 32, 1536, 16384, 16, 4, 131072, 4096, {"start": 3, "stop": 9, "times": 2}),
    "lusatar-tiny": lambda: _lusatar(256, 4, 128, 512, 2, 1, 512, 64),
    "kazedra-2b": lambda: _kazedra(2560, 20, 6912, 18, 65536),
    "kazedra-8b": lambda: _kazedra(4096, 32, 11008, 32, 131072),
    "kazedra-tiny": lambda: _kazedra(256, 4, 384, 2, 512, 64),
}


class RandomTensors(dict):
    """Random weights of a checkpoint's shapes, made on the device when they are asked for."""

    def __init__(self, shapes, device, seed=0):
        g = torch.Generator(device=device).manual_seed(seed)

        def make(name, shape):
            shape = [32 if n is None else n for n in shape]
            t = torch.randn(shape, device=device, generator=g)
            leaf = name.rsplit(".", 1)[-1]
            t = 1 + 0.1 * t if "norm" in leaf else t - 4.0 if leaf in ("lam", "A_log", "dt_bias") else t / math.sqrt(shape[-1])
            return t.to(torch.bfloat16)

        super().__init__({n: (lambda n=n, s=s: make(n, s)) for n, s in shapes.items()})


def build(name, device, max_context, dtype=torch.bfloat16):
    from .model_loader import Weights
    from .models import model_class

    cfg = SIZES[name]()
    cls = model_class(cfg)
    return cls(cfg, Weights(RandomTensors(cls.tensor_shapes(cfg), device), dtype, device), dtype, device, max_context)


def _event_ms(fn, n):
    fn()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(n):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / n


def _describe(model, rows: int, ctx: int):
    """What the report needs beside the model's weights: (layer runs, text, bytes of caches and states a decode step of
    `rows` sequences moves at `ctx` tokens, heads, feed-forward weights per layer as a gated width)."""
    cfg = model.config
    if cfg["architecture"] == "Lusatar":
        att = [r for r in model.runs if cfg["layers"][r.layer]["type"] == "latent_attention"]
        window = max(cfg["layers"][r.layer]["mixer"]["mask"]["size"] for r in att)
        return (len(model.runs), f"{len(model.runs)} layer runs ({len(att)} latent attention)", len(att) * rows * min(ctx, window) * 576 * 2,
                cfg["layers"][-1]["mixer"]["heads"], cfg["layers"][0]["mlp"]["ff"] * 2 // 3)
    n, c = len(model.layers), cfg["layers"][0]
    a, r = c["mixer"]["left"], c["mixer"]["right"]
    moved = n * rows * (ctx * (a["kv_heads"] * a["dim"] * 2 + 4) + 2 * r["heads"] * r["dim"] * r["vdim"] * 4)
    layer = model.layers[0].mixer.bytes() / 2 + 3 * model.width * c["mlp"]["ff"]
    attention = 2 * model.width * a["dim"] * (a["heads"] + a["kv_heads"])
    return (n, f"{n} layers of attention ({a['heads']} / {a['kv_heads']} heads) beside {r['heads']} delta-rule heads", moved, a["heads"],
            int((layer - attention) / (3 * model.width)))


def engine_workload(args, dev, world):
    """Decode: one step = one new token of every one of `batch` sequences of prefix + suffix tokens each, through the
    engine (host layout, graph replay, greedy pick).  Prefill: prompts of prefix + suffix tokens, eight at a time."""
    from .benchlib import aggregate, dist_helpers, timed_steps
    from .engine import Engine, Entry, SamplingParams, Sampler

    name = args.model.split("-")[0] + "-tiny" if args.tiny else args.model
    B, ctx = args.batch, args.prefix + args.suffix
    per_req = ctx + args.steps + args.warmup + 8
    model = build(name, dev, per_req)
    engine = Engine(model, B * per_req, B, use_graph=not args.no_graph)
    g = torch.Generator().manual_seed(0)
    prompts = torch.randint(0, model.vocab, (B, ctx), generator=g).tolist()
    seqs = [engine.open() for _ in range(B)]
    n = min(8, B)

    def prefill(lo):
        engine.step([Entry(seqs[i], prompts[i], [ctx - 1]) for i in range(lo, min(lo + n, B))])

    prefill(0)                                       # warm: kernels, library heuristics
    for i in range(n):
        engine.close(seqs[i])
        seqs[i] = engine.open()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for lo in range(0, B, n):
        prefill(lo)
    b.record()
    torch.cuda.synchronize()
    prefill_s = a.elapsed_time(b) / 1e3
    sampler, params = Sampler(dev), [SamplingParams()] * B
    last = [p[-1] for p in prompts]

    def step():
        last[:] = sampler(engine.step([Entry(s, [t], [0]) for s, t in zip(seqs, last)]), params)

    barrier, mx = dist_helpers(world, dev)
    elapsed = timed_steps(step, args.steps, max(args.warmup, 3), torch.cuda.synchronize, barrier, mx)
    graph = engine.graphs.get(B)
    replay_ms = _event_ms(graph.graph.replay, 10) if graph else None
    agg = aggregate(B, args.steps, world, elapsed)
    runs, text, moved, heads, gated_ff = _describe(model, B, ctx + args.warmup + args.steps // 2)
    uniq = model.weight_bytes() + moved
    step_s = (replay_ms or elapsed / args.steps * 1e3) / 1e3
    out = {
        "metric": f"decode tokens/s (whole job), {name} bf16 (random weights), batch {B}/GPU, {ctx}-token contexts",
        "value": round(agg["value"], 1), "unit": "tokens/s", "n_gpus": world, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(agg["ms_per_step"], 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16",
        "data": "synthetic",
        "config": {"model": name, "global_batch": B * world, "seq_len": ctx, "parallelism": f"replicas x{world}",
                   "workload": f"{text}, width {model.width}, vocab {model.vocab}",
                   "graph": graph is not None},
        "decode_graph_replay_ms": round(replay_ms, 4) if replay_ms else None,
        "decode_tokens_per_s_device": round(B / step_s, 1),
        "step_bytes_unique": int(uniq), "step_hbm_frac_of_8TBps": round(uniq / step_s / 8e12, 4),
        "prefill_tokens_per_s": round(B * ctx / prefill_s, 1), "prefill_batch_tokens": n * ctx,
    }
    flops = 2 * (model.weight_bytes() / 2 - model.head.N * model.head.K)
    out["prefill_product_tflops"] = round(flops * B * ctx / prefill_s / 1e12, 1)
    width, vocab = model.width, model.vocab
    del engine, model, graph, seqs
    torch.cuda.empty_cache()
    if not args.tiny:
        out["closest_model"] = llama_of_equal_size(args, dev, runs, width, heads, gated_ff, vocab, B, ctx)
    return out


def llama_of_equal_size(args, dev, layers, width, heads, ff, vocab, B, ctx):
    """The Llama runner's bf16 decode step and extend at the same width, layer count, weights per layer (ff: gated feed-forward that makes up for them), batch and
    context (contexts not shared)."""
    from . import ops
    from .decode_runner import LlamaConfig, LlamaDecoder
    from .mem_cache.memory_pool import MHATokenToKVPool
    from .prefill_runner import LlamaPrefill

    cfg = LlamaConfig(hidden=width, layers=layers, q_heads=heads, kv_heads=heads // 4, head_dim=128, inter=ff // 128 * 128,
                      vocab=vocab, quant="bf16")
    dec = LlamaDecoder(cfg, B, 1 + B * (ctx + 64), ctx + 64, device=dev)
    fused = dec.enable_fusion(True)
    dec.setup_shared_prefix_batch(ctx, 0, share=False)
    stream = torch.cuda.Stream(dev)
    with torch.cuda.stream(stream):
        dec.step()
        stream.synchronize()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph, stream=stream):
            dec.step()
        graph.replay()
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record(stream)
        for _ in range(10):
            graph.replay()
        b.record(stream)
        stream.synchronize()
    ms = a.elapsed_time(b) / 10
    uniq = dec.layer_weight_bytes() * layers + dec.lm_head.bytes() + layers * B * ctx * 2 * cfg.kv_heads * 128 * 2
    n = min(8, B)
    kv = MHATokenToKVPool(n * ctx, 1, torch.bfloat16, cfg.kv_heads, 128, layers, dev)
    pre = LlamaPrefill(dec, kv, n * ctx, use_graph=False)
    ids = torch.randint(0, vocab, (n * ctx,), device=dev)
    pos = torch.arange(ctx, device=dev).repeat(n)
    loc = torch.arange(1, n * ctx + 1, device=dev)
    qo = (torch.arange(n + 1, device=dev) * ctx).int()
    none = torch.zeros(n + 1, dtype=torch.int32, device=dev)
    ems = _event_ms(lambda: pre.extend(ids, pos, loc, qo, none, none[:1], ctx), 3)
    return {"model": f"Llama bf16, {layers} layers, width {width}, {heads} / {heads // 4} heads of 128, gated feed-forward of {cfg.inter}",
            "fused": bool(fused), "decode_graph_replay_ms": round(ms, 4), "decode_tokens_per_s_device": round(B / ms * 1e3, 1),
            "step_hbm_frac_of_8TBps": round(uniq / (ms / 1e3) / 8e12, 4), "prefill_tokens_per_s": round(n * ctx / ems * 1e3, 1),
            "prefill_product_tflops": round(dec.layer_weight_bytes() * layers * n * ctx / (ems / 1e3) / 1e12, 1)}
