"""Replay a trace of given tokens through the engine and write logits (the program is bin/trace_run).

Steps come on standard input, one JSON object a line:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
Each entry gives a request's next tokens and the places among them whose logits are asked for; `end`
lists the requests that are finished after the step. All entries of a step are one batch of
EngineCore.run_portions: the engine's own step, cache, state rows and kernels, without sampling. For a
step that asks for logits <out>/<step>.f32 holds them, f32 [wanted, vocab]; after every step a line
"done <step>" is printed."""

from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Callable, Dict, Iterable, Optional

from .engine import BLOCK_SIZE, EngineCore, ModelRunner, Request

MAX_LIVE = 4  # requests that hold a state row at a time


class TraceSession:
    """An engine over one model whose requests are fed by hand."""

    def __init__(self, model, max_tokens: int, max_live: int = MAX_LIVE, use_graphs: bool = True):
        blocks = max(1, -(-max_tokens // BLOCK_SIZE))
        self.core = EngineCore(ModelRunner(model, blocks, max_live, use_graphs=use_graphs, fused_lmhead="off"), blocks,
                               max_num_seqs=max_live, max_model_len=model.max_model_len, portions=model.portions)
        self.live: Dict[str, Request] = {}

    def step(self, entries: Iterable[dict], end: Iterable[str] = ()):
        """Run one step; returns the wanted logits (f32, on the host) or None."""
        work = []
        for e in entries:
            r = self.live.get(e["id"])
            if r is None:
                r = self.live[e["id"]] = self.core.open_request()
            work.append((r, e["tokens"], e.get("want") or []))
        logits = self.core.run_portions(work) if work else None
        out = None if logits is None else logits.float().cpu()
        for i in end:
            r = self.live.pop(i, None)
            if r is not None:
                self.core.close_request(r)
        return out


def main(argv: Optional[list] = None, prepare: Optional[Callable] = None) -> int:
    """prepare: called with the names of the kernel libraries that the model needs, before the GPU is used."""
    ap = argparse.ArgumentParser(prog="trace_run", description="replay token steps from stdin, write their logits")
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time")
    ap.add_argument("--no-graphs", action="store_true", help="run decode steps eagerly")
    args = ap.parse_args(argv)

    import torch

    from .registry import kernel_libraries, load_decoder, read_config

    if prepare is not None:
        prepare(kernel_libraries(read_config(args.model)))
    if not torch.cuda.is_available():
        print("trace_run needs a GPU", file=sys.stderr)
        return 1
    torch.backends.cuda.matmul.allow_tf32 = False
    with torch.no_grad():
        model = load_decoder(args.model, "cuda:0", getattr(torch, args.dtype),
                             max_model_len=-(-args.max_tokens // BLOCK_SIZE) * BLOCK_SIZE)
        session = TraceSession(model, args.max_tokens, use_graphs=not args.no_graphs)
        for line in sys.stdin:
            if not line.strip():
                continue
            s = json.loads(line)
            out = session.step(s.get("entries", []), s.get("end", []))
            if out is not None:
                path = os.path.join(args.out, f"{s['step']}.f32")
                with open(path + ".part", "wb") as f:
                    f.write(out.numpy().astype("<f4").tobytes())
                os.replace(path + ".part", path)
            print(f"done {s['step']}", flush=True)
    torch.cuda.synchronize()
    return 0
