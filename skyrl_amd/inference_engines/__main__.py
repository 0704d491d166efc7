"""Generate from a checkpoint folder on one GPU: python -m skyrl_amd.inference_engines --model DIR ...

Prompts are token ids (this engine takes ids; a checkpoint may come without a tokenizer), one prompt per
--prompt-ids, or one JSON list a line on standard input. Prints one JSON object per prompt."""

from __future__ import annotations

import argparse
import asyncio
import json
import sys
from typing import List, Optional


def parse(argv: Optional[List[str]] = None) -> argparse.Namespace:
    ap = argparse.ArgumentParser(prog="skyrl_amd.inference_engines", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    ap.add_argument("--prompt-ids", action="append", default=[], metavar="IDS", help="comma separated token ids; repeatable")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--max-model-len", type=int, default=None)
    ap.add_argument("--max-num-seqs", type=int, default=64)
    ap.add_argument("--max-prefill-tokens", type=int, default=8192, help="tokens of prompts and decodes in one step")
    ap.add_argument("--num-blocks", type=int, default=None, help="16-token cache blocks (default: half of the free memory)")
    ap.add_argument("--max-tokens", type=int, default=16)
    ap.add_argument("--temperature", type=float, default=1.0)
    ap.add_argument("--top-p", type=float, default=1.0)
    ap.add_argument("--top-k", type=int, default=-1)
    ap.add_argument("--min-p", type=float, default=0.0)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--stop-token-ids", default="", help="comma separated")
    ap.add_argument("--logprobs", action="store_true")
    return ap.parse_args(argv)


def main(argv: Optional[List[str]] = None) -> int:
    args = parse(argv)
    ids = lambda text: [int(t) for t in text.split(",") if t.strip()]  # noqa: E731
    prompts = [ids(p) for p in args.prompt_ids] or [json.loads(line) for line in sys.stdin if line.strip()]

    import torch

    from .engine import AMDInferenceEngine
    from .registry import load_decoder

    params = {"max_tokens": args.max_tokens, "temperature": args.temperature, "top_p": args.top_p, "top_k": args.top_k,
              "min_p": args.min_p, "seed": args.seed, "stop_token_ids": ids(args.stop_token_ids), "logprobs": 0}
    with torch.no_grad():
        model = load_decoder(args.model, "cuda:0", getattr(torch, args.dtype), max_model_len=args.max_model_len)
        engine = AMDInferenceEngine(model, num_blocks=args.num_blocks, max_num_seqs=args.max_num_seqs,
                                    max_prefill_tokens=args.max_prefill_tokens)
        out = asyncio.run(engine.generate({"prompt_token_ids": prompts, "sampling_params": params}))
    for i in range(len(prompts)):
        line = {"response_ids": out["response_ids"][i], "stop_reason": out["stop_reasons"][i]}
        if args.logprobs:
            line["logprobs"] = out["response_logprobs"][i]
        print(json.dumps(line))
    return 0


if __name__ == "__main__":
    sys.exit(main())
