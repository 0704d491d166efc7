"""Helpers of the hybrid decoders' GPU tests: comparisons with the oracle, models, feeding, generation."""

import asyncio

import torch

from hybrid_cases import make_normed_weights, make_parallel_weights, make_sandwich_weights, make_weights
from oracle import hybrid_ref as ref
from skyrl_amd.inference_engines.engine import AMDInferenceEngine
from skyrl_amd.inference_engines.hybrid import HybridDecoder

DEV = torch.device("cuda:0")
DTYPES = [torch.float32, torch.bfloat16]


def weights_of(cfg, seed=0):
    return {"Lipedra": make_parallel_weights, "Foduzen": make_normed_weights, "Dovidra": make_weights,
            "Tativik": make_sandwich_weights}[cfg["architecture"]](cfg, seed)


def rms(x):
    return float(x.double().pow(2).mean().sqrt())


def close(got, want, dtype, f32=1e-4, bf16=2e-2):
    got, want = got.double().cpu(), want.double()
    err = rms(got - want) / max(rms(want), 1e-9)
    worst = float((got - want).abs().max()) / max(float(want.abs().max()), 1e-9)
    tol = f32 if dtype == torch.float32 else bf16
    assert err < tol and worst < 4 * tol, f"rms {err:.2e} worst {worst:.2e} tolerance {tol}"


def rnd(g, *shape, dtype=torch.float32, scale=1.0):
    return (torch.randn(shape, generator=g) * scale).to(dtype)


LIMIT = {torch.float32: 2e-5, torch.bfloat16: 4e-2}


def build(cfg, dtype, seed=0, max_len=512, w=None):
    w = weights_of(cfg, seed) if w is None else w
    m = HybridDecoder(cfg, DEV, dtype=dtype, seed=None, max_model_len=max_len)
    assert m.load_weights(w.items()) == len(w)
    return m, {k: v.double() for k, v in w.items()}


def tokens_of(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def feed(s, rid, toks, cuts):
    """All logits of a request fed in portions."""
    out, a = [], 0
    for n in cuts:
        out.append(s.step([{"id": rid, "tokens": toks[a:a + n], "want": list(range(n))}]))
        a += n
    assert a == len(toks)
    return torch.cat(out)


def model_close(got, want, dtype):
    err = (got.double() - want).pow(2).mean(-1).sqrt() / rms(want)
    assert float(err.max()) < LIMIT[dtype], f"worst {float(err.max()):.2e} at {int(err.argmax())}"


def greedy(w, cfg, prompt, n):
    out, margins = [], []
    for _ in range(n):
        lg, _ = ref.forward(prompt + out, w, cfg)
        top = lg[-1].topk(2)
        out.append(int(top.indices[0]))
        margins.append(float(top.values[0] - top.values[1]))
    return out, margins


def generate(m, prompts, num_blocks, max_prefill=64, graphs=True, **params):
    eng = AMDInferenceEngine(m, num_blocks=num_blocks, max_num_seqs=4, max_prefill_tokens=max_prefill, use_graphs=graphs)
    out = asyncio.run(eng.generate({"prompt_token_ids": prompts, "sampling_params": dict(params, logprobs=0)}))
    return out, eng
