"""Throughput of the hybrid decoders beside the closest dense decoder (Qwen2 layers) of equal size,
through the engine's own runner (scheduled batches, HIP sampler included): `python bench.py --hybrid`.

All models have random weights, the same width, heads, feed-forward weights (routed experts: of those that a token
runs), vocabulary and number of layer runs. Prints one JSON line: tokens/s of prompts (one long, eight short) and of decode steps at several
batch sizes. `--hybrid-model` and `--hybrid-phase` restrict it, e.g. under a profiler."""

from __future__ import annotations

import json
import time

SIZES = {  # layers that resemble a 2B and an 8B model's
    "2k": dict(width=2048, ff=6144, heads=16, window=1024, delta_heads=32, delta_kv=16, vocab=32768),
    "4k": dict(width=4096, ff=12288, heads=32, window=1024, delta_heads=64, delta_kv=32, vocab=32768),
}
MODELS = ("dovidra", "lipedra", "foduzen", "tativik", "qwen2")
RUNS = 6  # layer runs: latent, (delta, latent, delta) ... as below
PROMPTS = ((1, 8192), (8, 1024))
DECODES = ((1, 2048), (64, 2048), (256, 2048))


def hybrid_config(z):
    lat = {"type": "latent_attention", "mlp": {"kind": "dense", "ff": z["ff"]},
           "mixer": {"heads": z["heads"], "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 192 ** -0.5,
                     "mask": {"size": z["window"]},
                     "rot": {"base": 10000.0, "dims": 64,
                             "scaling": {"factor": 16.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}}
    dlt = {"type": "delta", "mlp": {"kind": "dense", "ff": z["ff"]},
           "mixer": {"heads": z["delta_heads"], "kv_heads": z["delta_kv"], "dim": 128, "vdim": 128, "conv": 4}}
    return {"architecture": "Dovidra", "layers": [lat, dlt, lat, dlt], "loop": {"start": 1, "stop": 3, "times": 2},
            "norm": {"eps": 1e-6}, "logit_softcap": 30.0, "vocab": z["vocab"], "width": z["width"]}


def parallel_config(z):
    """Differential attention whose two maps and values have the dense model's head and cache sizes; the last
    two layers share the keys and values of the one before them."""
    m = {"heads": z["heads"], "kv_heads": max(2, z["heads"] // 8), "dim": 64, "vdim": 128, "conv": 4, "diff": 0.5,
         "scale": 0.125, "rot": {"base": 10000.0, "dims": 32,
                                 "scaling": {"factor": 16.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    layers = [{"type": "attention", "mixer": dict(m, kv_from=RUNS - 3) if i >= RUNS - 2 else m,
               "mlp": {"kind": "dense", "ff": z["ff"], "limit": 7.0}} for i in range(RUNS)]
    return {"architecture": "Lipedra", "layers": layers, "norm": {"eps": 1e-6}, "embedding": {"scale": z["width"] ** 0.5},
            "vocab": z["vocab"], "width": z["width"]}


def normed_config(z):
    """Four layers of gated linear recurrence (as wide as the model, blocks of 128) and two of windowed attention with
    the dense model's heads beside a state space mixer (twice the width, heads of 64, state 128)."""
    rec = {"width": z["width"], "blocks": z["width"] // 128, "conv": 4}
    left = {"heads": z["heads"], "kv_heads": max(2, z["heads"] // 8), "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
            "mask": {"size": z["window"]}}
    right = {"heads": z["width"] // 32, "vdim": 64, "state": 128, "groups": 1, "conv": 4, "norm_groups": 1}
    layers = [{"type": "parallel", "mixer": {"left": left, "right": right}} if i % 3 == 2 else {"type": "rglru", "mixer": rec}
              for i in range(RUNS)]
    return {"architecture": "Foduzen", "layers": [dict(e, mlp={"kind": "dense", "ff": z["ff"] * 3 // 2}) for e in layers],
            "norm": {"eps": 1e-6}, "embedding": {"scale": z["width"] ** 0.5}, "vocab": z["vocab"], "width": z["width"]}


def routed_config(z):
    """Latent attention as in hybrid_config, its queries from a latent of 3/8 of the width, the second on the first's
    keys, and generalized delta layers as wide as the model, heads of 64; 64 experts, of which 8 run, out of 4 of 8
    groups."""
    m = {"heads": z["heads"], "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "q_rank": z["width"] * 3 // 8,
         "scale": 192 ** -0.5, "mask": {"size": z["window"]}, "rot": {"base": 10000.0, "dims": 64}}
    mlp = {"kind": "moe", "expert": {"ff": z["ff"] // 8}, "router": {"experts": 64, "top": 8, "groups": {"count": 8, "keep": 4}}}
    delta = {"type": "general_delta", "mlp": mlp, "mixer": {"heads": z["width"] // 64, "dim": 64, "decay_rank": 64}}
    layers = [delta if i % 2 else {"type": "latent_attention", "mixer": dict(m, kv_from=0) if i == 2 else m, "mlp": mlp}
              for i in range(RUNS)]
    return {"architecture": "Tativik", "layers": layers, "norm": {"eps": 1e-6, "groups": 4}, "residual_mult": 0.5,
            "vocab": z["vocab"], "width": z["width"]}


def dense_config(z):
    from transformers import Qwen2Config

    return Qwen2Config(vocab_size=z["vocab"], hidden_size=z["width"], intermediate_size=z["ff"], num_hidden_layers=RUNS,
                       num_attention_heads=z["heads"], num_key_value_heads=max(2, z["heads"] // 8),
                       max_position_embeddings=16384, tie_word_embeddings=False)


def build(kind, z, max_len):
    import torch

    from skyrl_amd.inference_engines.hybrid import HybridDecoder
    from skyrl_amd.inference_engines.model import PagedDecoder

    if kind != "qwen2":
        config = {"dovidra": hybrid_config, "lipedra": parallel_config, "foduzen": normed_config,
                  "tativik": routed_config}[kind](z)
        return HybridDecoder(config, "cuda:0", dtype=torch.bfloat16, seed=0, max_model_len=max_len)
    return PagedDecoder(dense_config(z), "cuda:0", seed=0, max_model_len=max_len)


def timed(fn, reps, warmup=2):
    import torch

    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    t = time.perf_counter()
    for _ in range(reps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t) / reps


def measure(kind, z, phases, prompts, decodes):
    import numpy as np
    import torch

    from skyrl_amd.inference_engines.engine import BLOCK_SIZE, ModelRunner, Request, RequestParams, ScheduledBatch

    max_len = max([L for _, L in prompts] + [c + BLOCK_SIZE for _, c in decodes])
    rows = max([n for n, _ in prompts] + [n for n, _ in decodes])
    blocks = max([n * (-(-L // BLOCK_SIZE)) for n, L in prompts] + [n * (-(-c // BLOCK_SIZE)) for n, c in decodes])
    model = build(kind, z, max_len)
    runner = ModelRunner(model, blocks, rows)
    rng = np.random.default_rng(0)
    greedy = RequestParams(temperature=0.0, max_tokens=1 << 19, ignore_eos=True)

    def requests(n, L):
        per = -(-L // BLOCK_SIZE)
        return [Request(rid=i, prompt=rng.integers(0, z["vocab"], L).tolist(), params=greedy, key=i,
                        blocks=list(range(i * per, (i + 1) * per)), row=i) for i in range(n)]

    def step(reqs, kind_, counts=None):
        return lambda: runner.execute(ScheduledBatch(kind_, reqs, np.zeros(len(reqs), dtype=np.int64),
                                                     [()] * len(reqs), counts))

    out = {"params": model.num_params()}
    with torch.no_grad():
        if "prefill" in phases:
            for n, L in prompts:
                reqs = requests(n, L)
                s = timed(step(reqs, "portions", [L] * n) if model.portions else step(reqs, "prefill"), 5)
                out[f"prefill_{n}x{L}"] = {"ms": round(s * 1e3, 3), "tokens_per_s": round(n * L / s)}
        if "decode" in phases:
            for n, c in decodes:
                reqs = requests(n, c)
                for r in reqs:
                    r.num_computed = c - 1
                s = timed(step(reqs, "decode", [1] * n), 30, warmup=5)
                out[f"decode_{n}@{c}"] = {"ms": round(s * 1e3, 3), "tokens_per_s": round(n / s)}
    runner.release_cache()
    model.release()
    del runner, model
    torch.cuda.empty_cache()
    return out


def run(args):
    phases = (args.hybrid_phase,) if args.hybrid_phase else ("prefill", "decode")
    kinds = (args.hybrid_model,) if args.hybrid_model else MODELS
    sizes = args.hybrid_size.split(",")
    prompts = [tuple(map(int, p.split("x"))) for p in args.hybrid_prompts.split(",")] if args.hybrid_prompts else PROMPTS
    decodes = [tuple(map(int, p.split("@"))) for p in args.hybrid_decodes.split(",")] if args.hybrid_decodes else DECODES
    res = {}
    for size in sizes:
        for kind in kinds:
            res.setdefault(size, {})[kind] = measure(kind, SIZES[size], phases, prompts, decodes)
            print(f"[bench] {size} {kind}: {json.dumps(res[size][kind])}", flush=True)
    print(json.dumps({"metric": "hybrid decoder throughput", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic",
                      "n_gpus": 1, "layer_runs": RUNS, "sizes": {s: SIZES[s] for s in sizes}, "results": res}))
