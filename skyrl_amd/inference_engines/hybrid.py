"""Hybrid decoder: a list of layers, each with its own kind of mixer (paged attention or recurrent
state) and feed-forward, part of which may run several times with the same weights.

Dovidra is such a design: latent attention under a sliding window beside gated delta rule layers,
bias-free layer norms before each half, tanh-form GELU gates, a looped range of layers that adds one
learned vector per pass, and a tanh cap on the logits. Lipedra is another: differential attention, some
layers over an earlier layer's keys and values, beside clamped gates with biases in parallel layers (one
RMS norm, mixer and feed-forward in the same two matrix products), and a scaled embedding. Foduzen is a
third: gated linear recurrences, and layers of windowed attention beside a state space mixer, which read
the residual itself and whose outputs are normed (one number as the weight), xIELU feed-forwards, sinusoidal
position vectors. Tativik is a fourth: latent attention with low-rank queries, sinks and head gates, some layers over an
earlier layer's latents, and a generalized delta rule; routed experts; every sublayer stands between two norms in equal
parts and is gated before the second, and the embedding is normed. The model is what config.json lists; the mechanisms are mixers.py; `DESIGNS` holds what a
design fixes.

The residual stream is f32. One pass of the HIP norm kernel adds the previous sublayer's output and
(at the start of a loop pass) its vector, stores the stream and writes the next product's input; where
outputs are normed, one pass norms the sublayer's output (or joins and norms two), adds it, stores the
stream and writes the next product's input, at the end the final norm. Between two norms likewise: gate, norm, add,
store, norm.

HybridDecoder has PagedDecoder's interface (model.py), so the engine's scheduler, runner, sampler and
weight updates serve it unchanged; besides, it takes portions: a step may continue several prompts
and decode others at the same time (`forward_portions`).
"""

from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Any, Dict, Iterable, Iterator, List, Optional, Tuple

import torch
import torch.nn.functional as F

from . import kernels
from . import layer_kernels as lk
from .mixers import (EXPERT_FEEDFORWARDS, FEEDFORWARDS, MIXERS, PLAIN_FEEDFORWARDS, PROMPT_MIN, Gated, Products,
                     SideBySide, Weights)
from .model import StepInputs

DEFAULT_MAX_MODEL_LEN = 32768


@dataclass(frozen=True)
class Design:
    """What a design fixes for every model of it."""

    norm: str                # of layer_kernels.NORMS
    norm_base: float = 0.0   # added to the stored norm weights
    parallel: bool = False   # mixer and feed-forward read one norm and are added together
    mlp: Dict[str, Any] = field(default_factory=dict)  # feed-forward constants
    feedforwards: Dict[str, Any] = field(default_factory=lambda: FEEDFORWARDS)
    output_norms: bool = False  # sublayers read the residual, their outputs are normed
    scalar_norms: bool = False  # a norm's weight is one number
    sinusoid: Optional[float] = None  # base of the position vectors added to the embedding
    sandwich: bool = False   # sublayers between two norms in equal parts, gated before the second; normed embedding
    mixers: Dict[str, Dict[str, Any]] = field(default_factory=dict)  # mixer constants by type


DESIGNS = {
    "Dovidra": Design(norm="layer", mlp={"act": "gelu_tanh"}),
    "Lipedra": Design(norm="rms", norm_base=1.0, parallel=True, mlp={"act": "clamped", "alpha": 1.702, "bias": True}),
    "Foduzen": Design(norm="rms", output_norms=True, scalar_norms=True, sinusoid=10000.0, feedforwards=PLAIN_FEEDFORWARDS),
    "Tativik": Design(norm="rms", sandwich=True, feedforwards=EXPERT_FEEDFORWARDS,
                      mixers={"latent_attention": {"sink": True, "gate": True, "halves": True}}),
}


@dataclass
class LayerRun:
    layer: int
    step: Optional[int] = None  # the pass whose vector is added before this layer (first layer of a pass)


@dataclass
class HybridSpec:
    """What the engine reads of a model, and the layer order."""

    design: Design
    vocab_size: int
    hidden_size: int
    embed_scale: float
    norm_eps: float
    logit_softcap: Optional[float]
    layers: List[Dict[str, Any]]
    runs: List[LayerRun]
    loop_times: int
    max_position_embeddings: int
    eos_token_id: Optional[int] = None
    tie_word_embeddings: bool = False
    initializer_range: float = 0.02
    norm_groups: int = 1       # equal parts of a row that are normed apart (sandwich)
    residual_mult: float = 1.0  # of what a sublayer adds (sandwich)

    @property
    def num_layers(self) -> int:
        return len(self.runs)

    @classmethod
    def from_config(cls, cfg: Dict[str, Any]) -> "HybridSpec":
        layers, design = cfg["layers"], DESIGNS[cfg["architecture"]]
        for e in layers:
            if e["type"] not in MIXERS:
                raise ValueError(f"unknown layer type {e['type']!r} (known: {sorted(MIXERS)})")
            if e.get("mlp") and e["mlp"]["kind"] not in design.feedforwards:
                raise ValueError(f"unknown feed-forward {e['mlp']['kind']!r} (known: {sorted(design.feedforwards)})")
            if (e["type"] == "parallel") and not design.output_norms:
                raise ValueError("mixers side by side need a design that norms outputs")
        for i, e in enumerate(layers):
            j = e["mixer"].get("kv_from")
            if j is None:
                continue
            m, keys = layers[j]["mixer"] if 0 <= j < i else None, getattr(MIXERS[e["type"]], "shared_keys", None)
            if m is None or keys is None or layers[j]["type"] != e["type"] or m.get("kv_from") is not None \
                    or any(m.get(k) != e["mixer"].get(k) for k in keys):
                raise ValueError(f"layer {i}: kv_from {j} is no earlier layer with such keys and values of its own")
        n, loop = len(layers), cfg.get("loop")
        runs, times = [], 0
        if loop and (design.output_norms or design.sandwich):
            raise ValueError("this design has no looped layers")
        if loop:
            a, b, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
            if not 0 <= a <= b <= n or times < 0:
                raise ValueError(f"loop {loop} does not fit {n} layers")
            runs += [LayerRun(i) for i in range(a)]
            for t in range(times):
                runs += [LayerRun(i, t if i == a else None) for i in range(a, b)]
            runs += [LayerRun(i) for i in range(b, n)]
        else:
            runs = [LayerRun(i) for i in range(n)]
        eos = cfg.get("eos_token_id")
        return cls(design=design, vocab_size=int(cfg["vocab"]), hidden_size=int(cfg["width"]),
                   embed_scale=float((cfg.get("embedding") or {}).get("scale", 1.0)), norm_eps=float(cfg["norm"]["eps"]),
                   logit_softcap=float(cfg["logit_softcap"]) if cfg.get("logit_softcap") else None, layers=layers,
                   runs=runs, loop_times=times,
                   max_position_embeddings=int(cfg.get("max_position_embeddings") or DEFAULT_MAX_MODEL_LEN),
                   eos_token_id=None if eos is None else int(eos), norm_groups=int(cfg["norm"].get("groups") or 1),
                   residual_mult=float(cfg.get("residual_mult", 1.0)))


class HybridCache:
    """Cache or state of every layer run: a looped layer has one per pass. Paged runs share the
    sequences' block tables; recurrent state is indexed by the request's persistent batch row. A run that
    reads another layer's keys and values holds that layer's last run's."""

    def __init__(self, model: "HybridDecoder", num_blocks: int, num_rows: int):
        self.num_blocks, self.num_rows = num_blocks, num_rows
        self.runs, last = [], {}
        for r in model.spec.runs:
            mixer = model.layers[r.layer]["mixer"]
            source = () if mixer.kv_from is None else (last[mixer.kv_from],)
            last[r.layer] = mixer.make_state(num_blocks, num_rows, model.device, *source)
            self.runs.append(last[r.layer])


class HybridDecoder:
    """Weights + forward of a hybrid decoder over a HybridCache."""

    portions = True         # serves steps that mix prompt portions with decoded tokens
    def __init__(self, config: Dict[str, Any], device, dtype: torch.dtype = torch.bfloat16,
                 seed: Optional[int] = 0, max_model_len: Optional[int] = None):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("dtype must be bfloat16 or float32")
        self.config = config
        self.spec = HybridSpec.from_config(config)
        self.device, self.dtype = torch.device(device), dtype
        self.max_model_len = max_model_len or self.spec.max_position_embeddings
        self.workspace = kernels.DecodeWorkspace(self.device)          # decode steps: captured graphs hold it
        self.portion_workspace = kernels.DecodeWorkspace(self.device)  # eager portion steps: free to grow
        self._alloc(seed)

    # recurrent state cannot be shared by prefix
    @property
    def prefix_cacheable(self) -> bool:
        return all(MIXERS[e["type"]].prefix_cacheable(e["mixer"]) for e in self.spec.layers)

    # logits = hidden . lm_head^T: the sampler may run in that product's epilogue
    @property
    def plain_lm_head(self) -> bool:
        return self.spec.logit_softcap is None

    # a biased product of one row copies the bias first instead of adding it in the library's kernel
    @property
    def min_bucket(self) -> int:
        subs = [sub[1] for L in self.layers for sub in L["subs"]]
        return 2 if any(isinstance(sub, Products) and sub.biased for sub in subs) else 1

    # ---------------------------------------------------------------- weights
    def _alloc(self, seed: Optional[int]):
        s = self.spec
        w = Weights(self.device, self.dtype, seed, s.initializer_range)
        H = s.hidden_size
        d = s.design
        size = () if d.scalar_norms else (H,)
        norm = (lambda: w.zeros(*size)) if d.norm_base else (lambda: w.ones(*size))
        self.embed = w.matrix(s.vocab_size, H)
        self.layers: List[Dict[str, Any]] = []
        for e in s.layers:
            mixer = MIXERS[e["type"]](e["mixer"], H, s.norm_eps, self.max_model_len, w, **d.mixers.get(e["type"], {}))
            mlp = d.feedforwards[e["mlp"]["kind"]](e["mlp"], H, w, **d.mlp) if e.get("mlp") else None
            joined = hasattr(mixer, "inner")  # its products are Products'
            L = {"mixer": mixer, "mlp": mlp, "norm1": norm(), "norm2": None}
            if d.sandwich:
                L["subs"] = [(L["norm1"], Gated(mixer, H, w), norm())]
                if mlp is not None:
                    L["norm2"] = norm()
                    L["subs"].append((L["norm2"], Gated(mlp, H, w), norm()))
            elif d.parallel and mlp is not None:
                if not joined:
                    raise ValueError(f"{e['type']!r} layers cannot be parallel to a feed-forward")
                L["subs"] = [(L["norm1"], Products([mixer, mlp], H, w))]
            else:
                if isinstance(mixer, SideBySide):
                    sub = Products(mixer.parts, H, w, apart=True)
                else:
                    sub = Products([mixer], H, w) if joined else mixer
                L["subs"] = [(L["norm1"], sub)]
                if mlp is not None:
                    L["norm2"] = norm()
                    L["subs"].append((L["norm2"], Products([mlp], H, w)))
            self.layers.append(L)
        self.loop_step = w.matrix(s.loop_times, H) if s.loop_times else None
        self.norm = norm()
        self.embed_norm = norm() if d.sandwich else None
        if d.sandwich and H % s.norm_groups:
            raise ValueError("the width must be a multiple of norm.groups")
        self.turns = None  # revolutions per position of each pair of the position vector's columns
        if d.sinusoid:
            i = torch.arange((H + 1) // 2, dtype=torch.float64)
            self.turns = (d.sinusoid ** (-2.0 * i / H) / (2 * math.pi)).to(self.device)
        self.lm_head = w.matrix(s.vocab_size, H)

    def _param_views(self) -> Dict[str, torch.Tensor]:
        """Checkpoint name -> view into the (fused) storage."""
        out = {"embed": self.embed, "final.norm": self.norm, "head": self.lm_head}
        if self.loop_step is not None:
            out["loop.step"] = self.loop_step
        if self.embed_norm is not None:
            out["embed.norm"] = self.embed_norm
        for i, L in enumerate(self.layers):
            p = f"l{i}."
            out[p + "norm1"] = L["norm1"]
            for name, t in L["mixer"].params():
                out[p + "mix." + name] = t
            if L["norm2"] is not None:
                out[p + "norm2"] = L["norm2"]
            if L["mlp"] is not None:
                for name, t in L["mlp"].params():
                    out[p + "mlp." + name] = t
            if self.spec.design.sandwich:
                for k, (_, sub, after) in enumerate(L["subs"], 1):
                    out.update({f"{p}norm{k}b": after, f"{p}rg{k}": sub.weight, f"{p}rg{k}.b": sub.bias})
        return out

    def hf_named_tensors(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from self._param_views().items()

    def load_weights(self, named: Iterable[Tuple[str, torch.Tensor]]) -> int:
        """Copy named tensors into place (any subset; unknown names and wrong shapes raise)."""
        views = self._param_views()
        n = 0
        with torch.no_grad():
            for name, t in named:
                dst = views.get(name)
                if dst is None:
                    raise KeyError(f"unknown parameter {name!r}")
                if tuple(t.shape) != tuple(dst.shape):
                    raise ValueError(f"{name}: shape {tuple(t.shape)} != {tuple(dst.shape)}")
                dst.copy_(t, non_blocking=True)
                n += 1
            for L in self.layers:
                L["mixer"].refresh()
        return n

    def num_params(self) -> int:
        return sum(int(t.numel()) for t in self._param_views().values())

    def release(self):
        self.embed = self.lm_head = self.norm = self.loop_step = self.embed_norm = None
        self.layers = []

    # ---------------------------------------------------------------- cache and plans
    def make_cache(self, num_blocks: int, num_rows: int) -> HybridCache:
        return HybridCache(self, num_blocks, num_rows)

    def block_bytes(self) -> int:
        return max(1, sum(self.layers[r.layer]["mixer"].block_bytes() for r in self.spec.runs))

    def row_bytes(self) -> int:
        return sum(self.layers[r.layer]["mixer"].row_bytes() for r in self.spec.runs)

    def decode_split(self, nb: int) -> Tuple[int, Optional[int]]:
        """(max_ctx, nparts) of a captured decode step: each mixer splits by its own window."""
        return self.max_model_len, None

    def reserve(self, token_counts: Iterable[int]) -> None:
        """Size the merge workspace for these step sizes, so that a captured graph never sees it move."""
        need = 0
        for n in token_counts:
            for L in self.layers:
                need = max(need, L["mixer"].workspace_bytes(n, self.max_model_len))
        if need:
            self.workspace.get(need)

    @staticmethod
    def is_short(tokens: int) -> bool:
        """Whether a portion takes the per-token forms; the runner orders a step's short portions first."""
        return tokens < PROMPT_MIN

    def plan(self, seq_lens: List[int], starts: List[int], n_short: int):
        """Host plan of the prompt forms, tuples of numpy arrays and sizes by the mixers' keys (host_plans)."""
        plan, first = {}, sum(seq_lens[:n_short])
        for L in self.layers:
            if n_short == len(seq_lens) and not getattr(L["mixer"], "plans_short", False):
                continue  # the per-token forms need none
            for key, make in L["mixer"].host_plans(seq_lens, starts, n_short, first):
                if key not in plan:
                    plan[key] = make()
        return plan or None

    # ---------------------------------------------------------------- forward
    def _run_layers(self, inp: StepInputs, cache: HybridCache, want: Optional[torch.Tensor], trail=None):
        """Final-norm output of the wanted tokens (None: all). `trail` collects the residual after every
        layer run (inspection)."""
        s = self.spec
        if s.design.output_norms:
            return self._run_output_normed(inp, cache, want, trail)
        if s.design.sandwich:
            return self._run_sandwich(inp, cache, want, trail)
        norm = dict(eps=s.norm_eps, kind=s.design.norm, base=s.design.norm_base)
        h = lk.embed(inp.tokens, self.embed, s.embed_scale)
        x = torch.empty(h.shape, dtype=self.dtype, device=self.device)
        delta = None
        ws = self.workspace if inp.one_token else self.portion_workspace
        for r, state in zip(s.runs, cache.runs):
            step = None if r.step is None else self.loop_step[r.step]
            for weight, sub in self.layers[r.layer]["subs"]:
                lk.add_norm(delta, h, weight, step=step, out=x, **norm)
                delta, step = sub.forward(x, inp, state, ws), None
            if trail is not None:
                trail.append(h + delta.float())
        if want is None:
            return lk.add_norm(delta, h, self.norm, out=x, **norm)
        return lk.add_norm(None if delta is None else delta[want], h[want], self.norm, **norm)

    def _run_output_normed(self, inp: StepInputs, cache: HybridCache, want: Optional[torch.Tensor], trail=None):
        s = self.spec
        x = torch.empty((inp.tokens.shape[0], s.hidden_size), dtype=self.dtype, device=self.device)
        h = lk.embed(inp.tokens, self.embed, s.embed_scale, None if self.turns is None else inp.positions, self.turns, x)
        ws = self.workspace if inp.one_token else self.portion_workspace
        last = len(s.runs) - 1
        for i, (r, state) in enumerate(zip(s.runs, cache.runs)):
            L = self.layers[r.layer]
            for k, (weight, sub) in enumerate(L["subs"]):
                delta = sub.forward(x, inp, state, ws)
                join = {}
                if isinstance(delta, tuple):
                    join = {"pair": L["mixer"].out_norms, "share": L["mixer"].SHARE}
                if i == last and k == len(L["subs"]) - 1:
                    if trail is not None:
                        lk.norm_add(delta, (full := h.clone()), weight, s.norm_eps, **join)
                        trail.append(full)
                    if want is not None:
                        delta = tuple(t[want] for t in delta) if join else delta[want]
                        h, x = h[want], None
                    return lk.norm_add(delta, h, weight, s.norm_eps, final=self.norm, out=x, **join)
                lk.norm_add(delta, h, weight, s.norm_eps, out=x, **join)
            if trail is not None:
                trail.append(h.clone())
        raise ValueError("a model needs a layer")

    def _run_sandwich(self, inp: StepInputs, cache: HybridCache, want: Optional[torch.Tensor], trail=None):
        s = self.spec
        norm = dict(eps=s.norm_eps, groups=s.norm_groups)
        steps = [(state, *sub) for r, state in zip(s.runs, cache.runs) for sub in self.layers[r.layer]["subs"]]
        ends = {sum(len(self.layers[q.layer]["subs"]) for q in s.runs[:k + 1]) - 1 for k in range(len(s.runs))}
        before = [st[1] for st in steps] + [self.norm]  # the norm ahead of every sublayer, then the final one
        h = torch.empty((inp.tokens.shape[0], s.hidden_size), dtype=torch.float32, device=self.device)
        x = lk.gate_norm_add(self.embed, h, self.embed_norm, before[0], rows=inp.tokens, fresh=True, **norm)
        ws = self.workspace if inp.one_token else self.portion_workspace
        for k, (state, _, sub, after) in enumerate(steps):
            y, gate = sub.forward(x, inp, state, ws)
            args = dict(norm, mult=s.residual_mult, parts=sub.rows_per_token, gate_bias=sub.bias)
            last = k == len(steps) - 1
            if last and trail is not None:
                lk.gate_norm_add(y, (full := h.clone()), after, self.norm, gate=gate, **args)
                trail.append(full)
            if last and want is not None:
                y = y.view(-1, sub.rows_per_token, s.hidden_size)[want].view(-1, s.hidden_size)
                h, gate, x = h[want], gate[want], None
            x = lk.gate_norm_add(y, h, after, before[k + 1], gate=gate, out=x, **args)
            if trail is not None and k in ends and not last:
                trail.append(h.clone())
        return x

    def forward_decode(self, inp: StepInputs, cache: HybridCache) -> torch.Tensor:
        """One token per row: final hidden states [n, H]."""
        return self._run_layers(inp, cache, None)

    def forward_portions(self, inp: StepInputs, cache: HybridCache, trail=None) -> torch.Tensor:
        """A step of portions: final hidden states of the tokens `inp.want` lists."""
        return self._run_layers(inp, cache, inp.want, trail)

    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """f32 [n, V]."""
        return lk.softcap(F.linear(hidden, self.lm_head), self.spec.logit_softcap)
