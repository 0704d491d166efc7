"""Layer mechanisms of the hybrid decoders: latent attention, gated and generalized delta rules, differential
attention, gated linear recurrence, windowed attention beside a state space mixer, gated and plain MLPs, routed
experts.

A mechanism owns its weights (fused where one product serves several tensors), names them for
loading and saving, sizes and allocates its cache or state, and runs a step over it with the HIP
kernels of layer_kernels.py; matrix products are hipBLASLt through torch. Every size and constant is
a parameter; nothing here knows a particular model. `MIXERS` and `FEEDFORWARDS` map the type names of
a config.json to these classes.

A sublayer is `forward(x, inp, state, workspace)`. Most leave their input and output products to
`Products`, which runs one sublayer, a mixer and a feed-forward that read the same input side by side in
the same two products, or two mixers whose outputs are normed apart and joined (`SideBySide`). `Gated` puts the
logits of a gate on the sublayer's result beside it.

A step is a StepInputs (model.py): tokens of several sequences, each with its own first position. In
a portion step the first `n_short` sequences (single decoded tokens and short portions) come first;
the rest are prompts or long portions, which take the prompt forms of the kernels.
"""

from __future__ import annotations

import math
from typing import Any, Dict, Iterator, List, Optional, Tuple

import numpy as np
import torch
import torch.nn.functional as F

from . import kernels
from . import layer_kernels as lk

BLOCK_SIZE = kernels.BLOCK_SIZE
# From this many tokens on a portion takes the prompt forms (keys expanded once per key, chunked
# recurrence) instead of one query row or one recurrence step per token.
PROMPT_MIN = 32
ATTEND_WORKGROUPS = 256  # of the decode attention: one per CU (more split finer than they overlap)
PREFILL_TILE = 128  # queries per workgroup of the prompt attention


class Weights:
    """Allocates one layer's tensors on the model's device and dtype, randomly or zeroed."""

    def __init__(self, device, dtype, seed: Optional[int], std: float):
        self.device, self.dtype, self.std = torch.device(device), dtype, std
        self.gen = None
        if seed is not None:
            self.gen = torch.Generator(device=self.device)
            self.gen.manual_seed(seed)

        self.tables: Dict[Tuple, torch.Tensor] = {}

    def rotary(self, rot: Dict[str, Any], max_pos: int) -> torch.Tensor:
        """rotary_table on the device, one for all layers of equal rotation."""
        key = (repr(sorted(rot.items(), key=lambda kv: kv[0])), max_pos)
        if key not in self.tables:
            self.tables[key] = rotary_table(rot, max_pos).to(self.device)
        return self.tables[key]

    def matrix(self, *shape) -> torch.Tensor:
        t = torch.empty(shape, dtype=self.dtype, device=self.device)
        return t.zero_() if self.gen is None else t.normal_(0.0, self.std, generator=self.gen)

    def ones(self, *shape, dtype=None) -> torch.Tensor:
        return torch.ones(shape, dtype=dtype or self.dtype, device=self.device)

    def zeros(self, *shape, dtype=None) -> torch.Tensor:
        return torch.zeros(shape, dtype=dtype or self.dtype, device=self.device)


def split_rows(t: torch.Tensor, names_and_rows) -> Iterator[Tuple[str, torch.Tensor]]:
    """(name, view) of consecutive row ranges of a fused weight."""
    a = 0
    for name, n in names_and_rows:
        yield name, t[a:a + n]
        a += n


# ---------------------------------------------------------------- rotary positions
def rotary_table(rot: Dict[str, Any], max_pos: int) -> torch.Tensor:
    """f32 [max_pos, dims]: cos | sin halves, one entry per rotated pair. With `scaling` the
    frequencies are YaRN's blend of the interpolated and the original ones, and cos and sin carry its
    amplitude. Angles are formed in f64 and rounded once."""
    D, base = int(rot["dims"]), float(rot["base"])
    i = np.arange(D // 2, dtype=np.float64)
    f = base ** (-2.0 * i / D)
    amp = 1.0
    sc = rot.get("scaling")
    if sc:
        factor, original = float(sc["factor"]), float(sc["original"])

        def turns_dim(turns):  # the (fractional) dimension that makes `turns` turns over `original` positions
            return D * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))

        lo = max(math.floor(turns_dim(float(sc["fast"]))), 0)
        hi = min(math.ceil(turns_dim(float(sc["slow"]))), D - 1)
        ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
        f = f / factor * ramp + f * (1.0 - ramp)
        amp = 0.1 * math.log(factor) + 1.0
    a = np.arange(max_pos, dtype=np.float64)[:, None] * f[None]
    return torch.from_numpy(np.concatenate([np.cos(a) * amp, np.sin(a) * amp], 1).astype(np.float32))


# ---------------------------------------------------------------- portion plans (host)
def prompt_plan(seq_lens: List[int], starts: List[int], first_seq: int, first_token: int, window: Optional[int]):
    """Host plan of the prompt attention of sequences first_seq.. whose tokens begin at first_token of
    the step: (seg int32 [n, 4], tiles int32 [m, 8], packed rows, longest segment). A segment is the
    part of a sequence's cache its portion can see: from the window's reach before the portion's first
    token, on a block boundary, to its last token."""
    seg, tiles, rows, longest, tok = [], [], 0, 1, first_token
    for i in range(first_seq, len(seq_lens)):
        L, s = seq_lens[i], starts[i]
        lo = max(0, s - window + 1) // BLOCK_SIZE * BLOCK_SIZE if window else 0
        n = s + L - lo
        seg.append((i, lo, n, rows))
        for a in range(0, L, PREFILL_TILE):
            tiles.append((tok + a, min(PREFILL_TILE, L - a), s + a, rows, lo, 0, 0, 0))
        rows += (n + 63) // 64 * 64
        longest = max(longest, n)
        tok += L
    return (np.asarray(seg, dtype=np.int32).reshape(-1, 4), np.asarray(tiles, dtype=np.int32).reshape(-1, 8), rows,
            longest)


def chunk_plan(seq_lens: List[int], first_seq: int, first_token: int):
    """Host plan of the chunked recurrence of sequences first_seq..: (chunk int32 [n, 4], seq_chunks int32
    [sequences + 1])."""
    chunk, ends, tok = [], [0], first_token
    for i in range(first_seq, len(seq_lens)):
        for a in range(0, seq_lens[i], lk.CHUNK):
            chunk.append((tok + a, min(lk.CHUNK, seq_lens[i] - a), i, 0))
        ends.append(len(chunk))
        tok += seq_lens[i]
    return np.asarray(chunk, dtype=np.int32).reshape(-1, 4), np.asarray(ends, dtype=np.int32)


def tile_plan(seq_lens: List[int], starts: List[int], first_seq: int, first_token: int,
              window: Optional[int] = None) -> np.ndarray:
    """Query tiles int32 [m, 4] of causal attention of sequences first_seq..: first token, tokens, position
    of the first, sequence; the tiles with the most keys (in `window`) first."""
    tiles, tok = [], first_token
    for i in range(first_seq, len(seq_lens)):
        L, s = seq_lens[i], starts[i]
        tiles += [(tok + a, min(PREFILL_TILE, L - a), s + a, i) for a in range(0, L, PREFILL_TILE)]
        tok += L
    tiles.sort(key=lambda t: -(t[1] + min(t[2], window or t[2])))
    return np.asarray(tiles, dtype=np.int32).reshape(-1, 4)


def run_plan(seq_lens: List[int], starts: List[int], first_seq: int, first_token: int) -> np.ndarray:
    """Runs int32 [n, 2] (first token, tokens) of sequences first_seq.., cut where a position is a
    multiple of lk.RUN, so that a run's cache slots are consecutive."""
    runs, tok = [], first_token
    for i in range(first_seq, len(seq_lens)):
        L, s = seq_lens[i], starts[i]
        cuts = np.unique(np.concatenate([[0, L], np.arange(-s % lk.RUN, L, lk.RUN)]))
        runs.append(np.stack([tok + cuts[:-1], np.diff(cuts)], 1))
        tok += L
    return np.concatenate(runs).astype(np.int32)


# Workgroups of a prompt walk: what the CUs hold at once (four and three each).
LINEAR_WALK = 1024
STATE_WALK = 768
WALK_CHUNKS = 4  # chunks per run of the state space walk at least: a run's state is written and read once more


def chunk_runs(seq_lens: List[int], first_seq: int, first_token: int, per_run: int, total: int = LINEAR_WALK,
               least: int = 1):
    """Sequences first_seq.. as chunks, and their chunks in runs, at least `least` chunks long, so that about
    `total` workgroups walk them, per_run of them per run: (chunk int32 [n, 4], the fourth number the
    chunk's run, runs int32 [m, 4]: first chunk, chunks, sequence, 1 if the sequence has several runs + 2 if its
    last, seq_runs int32 [sequences + 1])."""
    chunk, ends = chunk_plan(seq_lens, first_seq, first_token)
    size = max(least, -(-len(chunk) * per_run // total))
    runs, seq_runs = [], [0]
    for i in range(len(ends) - 1):
        n = int(ends[i + 1] - ends[i])
        k = max(1, round(n / size))
        cuts = [int(ends[i]) + n * j // k for j in range(k + 1)]
        for j, (a, b) in enumerate(zip(cuts, cuts[1:])):
            chunk[a:b, 3] = len(runs)
            runs.append((a, b - a, first_seq + i, (k > 1) + 2 * (j == k - 1)))
        seq_runs.append(len(runs))
    return chunk, np.asarray(runs, dtype=np.int32).reshape(-1, 4), np.asarray(seq_runs, dtype=np.int32)


def walk_plan(seq_lens: List[int], first_seq: int, first_token: int, per_run: int):
    """Host plan of the state space prompt form of sequences first_seq..: (chunk, runs, pick int32 [k], chain int32
    [j, 2]) as skyrl_ssd_prompt takes them."""
    chunk, runs, seq_runs = chunk_runs(seq_lens, first_seq, first_token, per_run, STATE_WALK, WALK_CHUNKS)
    chain = [(a, b - a) for a, b in zip(seq_runs, seq_runs[1:]) if b - a > 1]
    pick = [r for r, kind in enumerate(runs[:, 3]) if kind == 1]
    return chunk, runs, np.asarray(pick, dtype=np.int32), np.asarray(chain, dtype=np.int32).reshape(-1, 2)


class Products:
    """The input and the output product of sublayers that read the same input and whose outputs are
    summed: the parts' input rows stacked and their output columns side by side, one product each. Parts
    start at multiples of 8 elements (16 bytes). A part has `in_rows`, `out_cols`, `in_bias`, `out_bias`,
    takes its views of the weights in `bind` and computes `inner(proj, out, ...)` between the products.
    With `apart` every part has an output product and a state of its own, and the outputs are a tuple. With
    `beside` that many more input rows, `w_beside`, follow the parts', and forward returns (output, their product)."""

    def __init__(self, parts: List[Any], width: int, w: Weights, apart: bool = False, beside: int = 0):
        self.parts, self.ranges, self.apart, self.beside = parts, [], apart, None
        a = c = 0
        for p in parts:
            self.ranges.append((a, c))
            a, c = a + (p.in_rows + 7) // 8 * 8, c + (p.out_cols + 7) // 8 * 8
        if beside:
            self.beside, a = (a, a + beside), a + (beside + 7) // 8 * 8
        self.w_in = w.matrix(a, width)
        if beside:
            self.w_beside = self.w_in[self.beside[0]:self.beside[1]]
        self.b_in = w.zeros(a) if any(p.in_bias for p in parts) else None
        if apart:
            self.outs = [(w.matrix(width, p.out_cols), w.zeros(width) if p.out_bias else None) for p in parts]
            for p, (a, _), (wo, bo) in zip(parts, self.ranges, self.outs):
                p.bind(self.w_in[a:a + p.in_rows], self.b_in[a:a + p.in_rows] if p.in_bias else None, wo, bo)
            return
        if sum(p.out_bias for p in parts) > 1:
            raise ValueError("one part at most may have an output bias")
        self.w_out = w.matrix(width, c)
        self.b_out = w.zeros(width) if any(p.out_bias for p in parts) else None
        self.padded = any(p.out_cols % 8 for p in parts)
        for p, (a, c) in zip(parts, self.ranges):
            p.bind(self.w_in[a:a + p.in_rows], self.b_in[a:a + p.in_rows] if p.in_bias else None,
                   self.w_out[:, c:c + p.out_cols], self.b_out if p.out_bias else None)

    @property
    def biased(self) -> bool:
        return self.b_in is not None or any(p.out_bias for p in self.parts)

    def forward(self, x: torch.Tensor, inp, state, workspace):
        proj = F.linear(x, self.w_in, self.b_in)
        if self.apart:
            outs = []
            for p, (a, _), (wo, bo), st in zip(self.parts, self.ranges, self.outs, state):
                o = torch.empty((x.shape[0], p.out_cols), dtype=x.dtype, device=x.device)
                p.inner(proj[:, a:a + p.in_rows], o, inp, st, workspace)
                outs.append(F.linear(o, wo, bo))
            return tuple(outs)
        make = torch.zeros if self.padded else torch.empty  # padding columns meet weights: they must be finite
        cat = make((x.shape[0], self.w_out.shape[1]), dtype=x.dtype, device=x.device)
        for p, (a, c) in zip(self.parts, self.ranges):
            p.inner(proj[:, a:a + p.in_rows], cat[:, c:c + p.out_cols], inp, state, workspace)
        y = F.linear(cat, self.w_out, self.b_out)
        return y if self.beside is None else (y, proj[:, self.beside[0]:self.beside[1]])


class Gated:
    """A sublayer and the logits of an elementwise gate on its result, both from the same input: forward returns (rows
    [n * rows_per_token, width] of which a token's are summed, logits [n, width]); the bias joins where the gate is
    applied (layer_kernels.gate_norm_add)."""

    def __init__(self, sub, width: int, w: Weights):
        self.bias = w.zeros(width, dtype=torch.float32)
        self.rows_per_token = getattr(sub, "rows_per_token", 1)
        if hasattr(sub, "inner"):
            self.sub = Products([sub], width, w, beside=width)
            self.weight = self.sub.w_beside
        else:
            self.sub, self.weight = sub, w.matrix(width, width)

    def forward(self, x: torch.Tensor, inp, state, workspace):
        if isinstance(self.sub, Products):
            return self.sub.forward(x, inp, state, workspace)
        return self.sub.forward(x, inp, state, workspace), F.linear(x, self.weight)


class LatentAttention:
    """Attention over low-rank latents shared by all heads, with a rotated key part beside them and
    an optional sliding window. Caches [blocks, 16, row]: per token the normed latent | the rotated key
    part. Queries come from the input or, with `q_rank`, from a normed latent of it. A design may add a learned sink to
    each head's softmax, a sigmoid gate to each head's output, and pair the rotated dimensions by halves instead of
    neighbours. A layer with `kv_from` reads the cache of that layer, with up-projections of its own."""

    libraries = ("latent",)  # of _ffi.LAYER_LIBS, beside the common one
    paged = True
    in_bias = out_bias = False
    shared_keys = ("kv_rank", "rot_dim", "rot")  # equal in a layer and the one whose cache it reads

    @staticmethod
    def prefix_cacheable(m: Dict[str, Any]) -> bool:
        """Whether a page's content depends on the tokens before it alone, with no state beside the pages."""
        return True

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights, sink: bool = False,
                 gate: bool = False, halves: bool = False):
        self.heads, self.dim, self.rot_dim = int(m["heads"]), int(m["dim"]), int(m["rot_dim"])
        self.vdim, self.rank, self.scale = int(m["vdim"]), int(m["kv_rank"]), float(m["scale"])
        self.q_rank = int(m["q_rank"]) if m.get("q_rank") else 0
        self.kv_from = None if m.get("kv_from") is None else int(m["kv_from"])
        mask = m.get("mask")
        self.window = int(mask["size"]) if mask and mask.get("size") else None
        if int(m["rot"]["dims"]) != self.rot_dim:
            raise ValueError("latent attention rotates exactly its rot_dim part: rot.dims must equal rot_dim")
        if self.rot_dim % 2:
            raise ValueError("rot_dim must be even")
        self.eps, self.dtype, self.halves = eps, w.dtype, halves
        self.cos_sin = w.rotary(m["rot"], max_pos)
        H, qd = self.heads, self.dim + self.rot_dim
        own = self.kv_from is None
        self.q_rows = self.q_rank or H * qd
        self.rows = (("dq" if self.q_rank else "q", self.q_rows),) + (
            (("dkv", self.rank + self.rot_dim),) if own else ()) + ((("g", H),) if gate else ())
        self.in_rows, self.out_cols = sum(n for _, n in self.rows), H * self.vdim
        self.gate_at = self.in_rows - H if gate else None
        self.dq_norm = w.ones(self.q_rank) if self.q_rank else None
        self.wuq = w.matrix(H * qd, self.q_rank) if self.q_rank else None
        self.dkv_norm = w.ones(self.rank) if own else None
        self.wuk = w.matrix(H * self.dim, self.rank)
        self.wuv = w.matrix(H * self.vdim, self.rank)
        self.wuv_t = w.zeros(H, self.rank, self.vdim)  # per head transposed: the decode form's right operand
        self.sinks = w.zeros(H, dtype=torch.float32) if sink else None
        self.refresh()

    def bind(self, w_in, b_in, w_out, b_out) -> None:
        self.w_in, self.wo = w_in, w_out

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from split_rows(self.w_in, self.rows)
        for name, t in (("dq.norm", self.dq_norm), ("uq", self.wuq), ("dkv.norm", self.dkv_norm), ("uk", self.wuk),
                        ("uv", self.wuv), ("sink", self.sinks), ("o", self.wo)):
            if t is not None:
                yield name, t

    def refresh(self) -> None:
        """Recompute derived tensors, in place, after the weights changed."""
        self.wuv_t.copy_(self.wuv.view(self.heads, self.vdim, self.rank).transpose(1, 2))

    # ---- cache
    def block_bytes(self) -> int:
        if self.kv_from is not None:
            return 0
        return BLOCK_SIZE * lk.latent_row(self.rank, self.rot_dim) * self.dtype.itemsize

    def row_bytes(self) -> int:
        return 0

    def make_state(self, num_blocks: int, num_rows: int, device, source=None) -> torch.Tensor:
        """source: the state of the layer whose latents this one reads."""
        if source is not None:
            return source
        return torch.zeros((num_blocks, BLOCK_SIZE, lk.latent_row(self.rank, self.rot_dim)), dtype=self.dtype,
                           device=device)

    # ---- plans
    def host_plans(self, seq_lens, starts, first_seq, first_token):
        yield self.window, lambda: prompt_plan(seq_lens, starts, first_seq, first_token, self.window)

    # ---- decode split
    def nparts(self, tokens: int, max_ctx: int) -> int:
        ctx = min(max_ctx, self.window + BLOCK_SIZE) if self.window else max_ctx
        return kernels.choose_nparts(tokens, (self.heads + 31) // 32, ctx, target_waves=ATTEND_WORKGROUPS)

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        from .. import _ffi

        n = self.nparts(tokens, max_ctx)
        return int(_ffi.query("skyrl_latent_attend_workspace_bytes", tokens, self.heads, self.rank, n)) if n > 1 else 0

    # ---- step
    def _attend_rows(self, q, gate, out, inp, a: int, b: int, cache, workspace):
        """Tokens [a, b) in the decode form."""
        H, D, R = self.heads, self.dim, self.rank
        n = b - a
        q3 = q[a:b].view(n, H, D + self.rot_dim)
        qa = torch.bmm(q3[:, :, :D].transpose(0, 1), self.wuk.view(H, D, R))
        o = lk.latent_attend(qa, q3[:, :, D:], cache, R, self.rot_dim, inp.block_tables, inp.bt_row[a:b],
                             inp.positions[a:b], self.scale, self.window, nparts=self.nparts(n, inp.max_ctx),
                             part_min=kernels.MIN_PARTITION, workspace=workspace, sinks=self.sinks,
                             gate=None if gate is None else gate[a:b])
        out[a:b].view(n, H, self.vdim).copy_(torch.bmm(o, self.wuv_t).transpose(0, 1))

    def inner(self, proj: torch.Tensor, out: torch.Tensor, inp, cache: torch.Tensor, workspace) -> None:
        H, T, qr = self.heads, proj.shape[0], self.q_rank
        where = (self.rot_dim, inp.positions, inp.slots, self.cos_sin, cache, self.eps)
        own = {} if self.kv_from is not None else {"rank": self.rank, "norm_weight": self.dkv_norm}
        first = {"q_norm": self.dq_norm} if qr else {"heads": H, "dim": self.dim}
        lk.latent_write(proj, *where, halves=self.halves, **first, **own)
        q = proj[:, :self.q_rows]
        if qr:
            q = F.linear(q, self.wuq)
            lk.latent_write(q, *where, heads=H, dim=self.dim, halves=self.halves)
        gate = None if self.gate_at is None else proj[:, self.gate_at:]
        prompt = inp.plan is not None and self.window in inp.plan and lk.prefill_fits(self.dim, self.rot_dim, self.vdim, self.dtype)
        ts = inp.short_tokens if prompt else T
        for a in range(0, ts, 32768):  # the decode form's grid limit
            self._attend_rows(q, gate, out, inp, a, min(ts, a + 32768), cache, workspace)
        if ts < T:
            seg, tiles, rows, longest = inp.plan[self.window]
            latent, k_rot = lk.latent_gather(cache, self.rank, self.rot_dim, inp.block_tables, seg, rows, longest)
            k = F.linear(latent, self.wuk)
            v_t = torch.mm(self.wuv, latent.t())
            lk.latent_prefill(q, k, k_rot, v_t, tiles, H, self.dim, self.rot_dim, self.vdim, self.scale, self.window,
                              out, sinks=self.sinks, gate=gate)


class GatedDelta:
    """Gated delta rule with short causal convolutions on q, k and v. State per row (a running
    request): the f32 matrix of every head and the convolutions' last inputs."""

    libraries = ("delta",)
    paged = False
    kv_from = None

    @staticmethod
    def prefix_cacheable(m: Dict[str, Any]) -> bool:
        return False

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights):
        self.heads, self.kv_heads = int(m["heads"]), int(m["kv_heads"])
        self.dim, self.vdim, self.taps = int(m["dim"]), int(m["vdim"]), int(m["conv"])
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.shape = lk.delta_shape(self.heads, self.kv_heads, self.dim, self.vdim, self.taps, eps)
        self.width, self.dtype = width, w.dtype
        self.wproj = w.matrix(lk.delta_width(self.shape), width)
        self.conv = w.matrix(lk.delta_channels(self.shape), self.taps)
        self.a_log = w.zeros(self.heads, dtype=torch.float32)
        self.dt_bias = w.zeros(self.heads, dtype=torch.float32)
        self.norm = w.ones(self.vdim)
        self.wo = w.matrix(width, self.heads * self.vdim)

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        qk, v = self.kv_heads * self.dim, self.heads * self.vdim
        yield from split_rows(self.wproj, (("q", qk), ("k", qk), ("v", v), ("g", v), ("b", self.heads),
                                           ("a", self.heads)))
        yield from split_rows(self.conv, (("q.conv", qk), ("k.conv", qk), ("v.conv", v)))
        yield "A_log", self.a_log
        yield "dt_bias", self.dt_bias
        yield "norm", self.norm
        yield "o", self.wo

    def refresh(self) -> None:
        pass

    # ---- state
    def block_bytes(self) -> int:
        return 0

    def row_bytes(self) -> int:
        return (4 * self.heads * self.dim * lk.delta_vpad(self.shape)
                + self.taps * lk.delta_channels(self.shape) * self.dtype.itemsize)

    def make_state(self, num_blocks: int, num_rows: int, device):
        return (torch.zeros((num_rows, self.heads, self.dim, lk.delta_vpad(self.shape)), dtype=torch.float32,
                            device=device),
                torch.zeros((num_rows, self.taps, lk.delta_channels(self.shape)), dtype=self.dtype, device=device))

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        return 0

    def host_plans(self, seq_lens, starts, first_seq, first_token):
        yield "chunks", lambda: chunk_plan(seq_lens, first_seq, first_token)

    # ---- step
    def forward(self, x: torch.Tensor, inp, state, workspace) -> torch.Tensor:
        S, ring = state
        proj = F.linear(x, self.wproj)
        out = torch.empty((x.shape[0], self.heads * self.vdim), dtype=self.dtype, device=x.device)
        args = (self.conv, self.a_log, self.dt_bias, self.norm)
        n = inp.rows.shape[0]
        prompt = inp.plan is not None and "chunks" in inp.plan and lk.delta_prompt_fits(self.shape)
        k = inp.n_short if prompt else n
        if k:
            lk.delta_scan(self.shape, proj, *args, inp.cu[:k + 1], inp.rows[:k], inp.positions, S, ring,
                          inp.one_token, out)
        if k < n:
            chunk, seq_chunks = inp.plan["chunks"]
            lk.delta_prompt(self.shape, proj, *args, inp.cu, inp.rows, inp.positions, S, ring, chunk, seq_chunks, k,
                            inp.short_tokens, out)
        if not inp.one_token:
            lk.conv_save(proj, lk.delta_channels(self.shape), inp.cu, inp.rows, inp.positions, ring)
        return F.linear(out, self.wo)


class GeneralDelta:
    """Generalized delta rule: a decay per head and key channel from a low-rank projection, a removal along the unit key
    at a rate of its own, output norm per head and elementwise gate. State per row (a running request): the f32 matrix
    of every head."""

    libraries = ("gdelta",)
    paged = False
    kv_from = None
    in_bias = out_bias = False

    @staticmethod
    def prefix_cacheable(m: Dict[str, Any]) -> bool:
        return False

    @staticmethod
    def complete(m: Dict[str, Any], shape_of) -> Dict[str, Any]:
        """The mixer's entry with the size that only a checkpoint's tensors give; shape_of: a tensor's shape by name."""
        return m if "decay_rank" in m or shape_of("w1") is None else dict(m, decay_rank=int(shape_of("w1")[0]))

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights):
        self.heads, self.dim = int(m["heads"]), int(m["dim"])
        if not m.get("decay_rank"):
            raise ValueError("the generalized delta rule needs decay_rank, from its entry or from a checkpoint's w1")
        self.rank = int(m["decay_rank"])
        self.shape = lk.gdelta_shape(self.heads, self.dim, eps)
        self.dtype = w.dtype
        HD = self.out_cols = self.heads * self.dim
        self.rows = tuple((n, HD) for n in "rkvga") + (("w1", self.rank),)
        self.in_rows = 5 * HD + self.rank
        self.w2 = w.matrix(HD, self.rank)
        self.w0, self.a_bias = w.zeros(HD, dtype=torch.float32), w.zeros(HD, dtype=torch.float32)
        self.norm = w.ones(HD)

    def bind(self, w_in, b_in, w_out, b_out) -> None:
        self.w_in, self.wo = w_in, w_out

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from split_rows(self.w_in, self.rows)
        yield from (("w2", self.w2), ("w0", self.w0), ("a.b", self.a_bias), ("norm", self.norm), ("o", self.wo))

    def refresh(self) -> None:
        pass

    # ---- state
    def block_bytes(self) -> int:
        return 0

    def row_bytes(self) -> int:
        return 4 * self.heads * self.dim * lk.gdelta_vpad(self.shape)

    def make_state(self, num_blocks: int, num_rows: int, device) -> torch.Tensor:
        return torch.zeros((num_rows, self.heads, self.dim, lk.gdelta_vpad(self.shape)), dtype=torch.float32, device=device)

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        return 0

    def host_plans(self, seq_lens, starts, first_seq, first_token):
        yield "chunks", lambda: chunk_plan(seq_lens, first_seq, first_token)

    # ---- step
    def inner(self, proj: torch.Tensor, out: torch.Tensor, inp, state: torch.Tensor, workspace) -> None:
        wl = F.linear(lk.tanh(proj[:, 5 * self.out_cols:]), self.w2)
        args = (proj, wl, self.w0, self.a_bias, self.norm)
        n = inp.rows.shape[0]
        prompt = inp.plan is not None and "chunks" in inp.plan
        k = inp.n_short if prompt else n
        if k:
            lk.gdelta_scan(self.shape, *args, inp.cu[:k + 1], inp.rows[:k], inp.positions, state, out)
        if k < n:
            lk.gdelta_prompt(self.shape, *args, inp.cu, inp.rows, inp.positions, state, *inp.plan["chunks"], k, out)


class DifferentialAttention:
    """Full causal attention in two softmax maps per head over the same values, their weighted difference
    normed per head and gated; short causal convolutions and partial interleaved rotation on its
    projections. Caches, per layer with keys of its own, K [blocks, kv_heads, 16, both maps] and V
    transposed [blocks, kv_heads, vdim, 16]; state per row: the convolutions' last inputs. A layer with
    `kv_from` reads the cache of that layer and has queries only."""

    libraries = ("diff",)
    paged = True
    shared_keys = ("kv_heads", "dim", "vdim")
    in_bias, out_bias = True, False

    @staticmethod
    def prefix_cacheable(m: Dict[str, Any]) -> bool:
        return int(m["conv"]) == 1

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights):
        self.heads, self.kv_heads = int(m["heads"]), int(m["kv_heads"])
        self.dim, self.vdim, self.taps, self.diff = int(m["dim"]), int(m["vdim"]), int(m["conv"]), float(m["diff"])
        self.kv_from = None if m.get("kv_from") is None else int(m["kv_from"])
        rot = m["rot"]
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if int(rot["dims"]) % 2 or int(rot["dims"]) > self.dim:
            raise ValueError("rot.dims must be even and at most dim")
        self.shape = lk.diff_shape(self.heads, self.kv_heads, self.dim, self.vdim, int(rot["dims"]), self.taps,
                                   self.kv_from is None, float(m["scale"]), self.diff, eps)
        self.dtype = w.dtype
        self.cos_sin = w.rotary(rot, max_pos)
        self.channels = lk.diff_channels(self.shape)
        self.in_rows, self.out_cols = self.channels + self.heads, self.heads * self.vdim
        self.conv = w.matrix(self.channels, self.taps)
        self.lq1, self.lk1, self.lq2, self.lk2 = (w.matrix(self.dim) for _ in range(4))
        self.conv_t = w.zeros(self.taps, self.channels, dtype=torch.float32)  # the kernels' form of conv
        self.lam = w.zeros(1, dtype=torch.float32)
        self.refresh()

    def bind(self, w_in, b_in, w_out, b_out) -> None:
        self.w_in, self.b_in, self.wo = w_in, b_in, w_out

    def _rows(self):
        qk, v = 2 * self.heads * self.dim, self.kv_heads * self.vdim
        own = self.kv_from is None
        return (("q", qk),) + ((("k", 2 * self.kv_heads * self.dim), ("v", v)) if own else ())

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from split_rows(self.w_in, self._rows() + (("g", self.heads),))
        yield from split_rows(self.b_in, [(n + ".b", r) for n, r in self._rows()])
        yield from split_rows(self.conv, [(n + ".conv", r) for n, r in self._rows()])
        yield from (("lq1", self.lq1), ("lk1", self.lk1), ("lq2", self.lq2), ("lk2", self.lk2), ("o", self.wo))

    def refresh(self) -> None:
        """Recompute derived tensors, in place, after the weights changed."""
        self.conv_t.copy_(self.conv.t())
        a, b = ((q.float() * k.float()).sum() for q, k in ((self.lq1, self.lk1), (self.lq2, self.lk2)))
        self.lam.copy_(torch.exp(a) - torch.exp(b) + self.diff)

    # ---- cache
    def block_bytes(self) -> int:
        if self.kv_from is not None:
            return 0
        return self.kv_heads * BLOCK_SIZE * sum(lk.diff_pads(self.shape)) * self.dtype.itemsize

    def row_bytes(self) -> int:
        return self.taps * self.channels * self.dtype.itemsize

    def make_state(self, num_blocks: int, num_rows: int, device, source=None):
        """source: the state of the layer whose keys and values this one reads."""
        ring = torch.zeros((num_rows, self.taps, self.channels), dtype=self.dtype, device=device)
        if source is not None:
            return source[0], source[1], ring
        kw, vp = lk.diff_pads(self.shape)
        zeros = lambda *tail: torch.zeros((num_blocks, self.kv_heads) + tail, dtype=self.dtype, device=device)  # noqa: E731
        return zeros(BLOCK_SIZE, kw), zeros(vp, BLOCK_SIZE), ring

    # ---- plans
    def host_plans(self, seq_lens, starts, first_seq, first_token):
        yield "tiles", lambda: (tile_plan(seq_lens, starts, first_seq, first_token),
                                run_plan(seq_lens, starts, first_seq, first_token))

    def nparts(self, tokens: int, max_ctx: int) -> int:
        groups = -(-(self.heads // self.kv_heads) // 8)  # a wave takes eight query heads of a key head
        return kernels.choose_nparts(tokens, self.kv_heads * groups, max_ctx)

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        return lk.diff_workspace_bytes(self.shape, tokens, self.nparts(tokens, max_ctx))

    # ---- step
    def inner(self, proj: torch.Tensor, out: torch.Tensor, inp, state, workspace) -> None:
        k_cache, v_cache, ring = state
        T = proj.shape[0]
        seqs = (inp.cu, inp.rows, inp.bt_row, inp.positions, inp.slots, self.cos_sin, ring, k_cache, v_cache)
        prompt = inp.plan is not None and "tiles" in inp.plan and lk.diff_mfma(self.shape, self.dtype)
        ts = inp.short_tokens if prompt else T
        runs = inp.plan["tiles"][1] if prompt and lk.diff_runs_fit(self.shape, proj) else None
        q = lk.diff_write(self.shape, proj, self.conv_t, *seqs, save_conv=inp.one_token,
                          count=T if runs is None else ts)
        if runs is not None:
            lk.diff_write(self.shape, proj, self.conv_t, *seqs, q=q, runs=runs)
        if not inp.one_token and self.taps > 1:
            lk.conv_save(proj, self.channels, inp.cu, inp.rows, inp.positions, ring)
        gate = proj[:, self.channels:]
        for a in range(0, ts, 32768):  # the decode form's grid limit
            b = min(ts, a + 32768)
            lk.diff_attend(self.shape, q[a:b], gate[a:b], k_cache, v_cache, inp.block_tables, inp.bt_row[a:b],
                           inp.positions[a:b], self.lam, out[a:b], nparts=self.nparts(b - a, inp.max_ctx),
                           part_min=kernels.MIN_PARTITION, workspace=workspace)
        if ts < T:
            lk.diff_prefill(self.shape, q, gate, k_cache, v_cache, inp.block_tables, inp.plan["tiles"][0], self.lam, out)


class ShortConv:
    """Weights of a biased causal convolution per channel, `conv` [channels, taps] and `conv.b`, and the
    transposed f32 filters that the kernels read."""

    def __init__(self, channels: int, taps: int, w: Weights):
        self.conv, self.bias = w.matrix(channels, taps), w.zeros(channels, dtype=torch.float32)
        self.conv_t = w.zeros(taps, channels, dtype=torch.float32)
        self.refresh()

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from (("conv", self.conv), ("conv.b", self.bias))

    def refresh(self) -> None:
        self.conv_t.copy_(self.conv.t())


class GatedLinearRecurrence:
    """Recurrent block of a real gated linear recurrence (RG-LRU): a gelu branch gates a branch of short
    convolution and recurrence, whose two gates are block-diagonal. State per row: the f32 channels and the
    convolution's last inputs."""

    libraries = ("rglru",)
    paged = False
    kv_from = None
    plans_short = True
    in_bias, out_bias = True, False
    RATE = 8.0  # log decay = -RATE r softplus(lam)

    @staticmethod
    def prefix_cacheable(m: Dict[str, Any]) -> bool:
        return False

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights):
        self.channels, self.blocks, self.taps = int(m["width"]), int(m["blocks"]), int(m["conv"])
        if self.channels % self.blocks:
            raise ValueError("the recurrence's width must be a multiple of blocks")
        C, n = self.channels, self.channels // self.blocks
        self.dtype = w.dtype
        self.in_rows, self.out_cols = 2 * C, C
        self.conv = ShortConv(C, self.taps, w)
        self.ra, self.ri = w.matrix(self.blocks, n, n), w.matrix(self.blocks, n, n)
        self.gate_b = w.zeros(2, C, dtype=torch.float32)
        self.lam = w.zeros(C, dtype=torch.float32)
        self.gate_w = w.zeros(self.blocks, 2, *lk.rglru_pads(C, self.blocks))  # the kernels' form of ra, ri
        self.rate = w.zeros(C, dtype=torch.float32)
        self.plan_key = ("runs", lk.rglru_workgroups(C, self.blocks))
        self.refresh()

    def bind(self, w_in, b_in, w_out, b_out) -> None:
        self.w_in, self.b_in, self.wo = w_in, b_in, w_out

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        C = self.channels
        yield from split_rows(self.w_in, (("y", C), ("x", C)))
        yield from split_rows(self.b_in, (("y.b", C), ("x.b", C)))
        yield from self.conv.params()
        for i, (name, t) in enumerate((("ra", self.ra), ("ri", self.ri))):
            yield name, t
            yield name + ".b", self.gate_b[i].view(self.blocks, -1)
        yield from (("lam", self.lam), ("o", self.wo))

    def refresh(self) -> None:
        """Recompute derived tensors, in place, after the weights changed."""
        self.conv.refresh()
        n = self.ra.shape[1]
        self.gate_w[:, 0, :n, :n].copy_(self.ra)
        self.gate_w[:, 1, :n, :n].copy_(self.ri)
        self.rate.copy_(-self.RATE * F.softplus(self.lam.double(), threshold=50.0))

    # ---- state
    def block_bytes(self) -> int:
        return 0

    def row_bytes(self) -> int:
        return self.channels * (4 + self.taps * self.dtype.itemsize)

    def make_state(self, num_blocks: int, num_rows: int, device):
        return (torch.zeros((num_rows, self.channels), dtype=torch.float32, device=device),
                torch.zeros((num_rows, self.taps, self.channels), dtype=self.dtype, device=device))

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        return 0

    def host_plans(self, seq_lens, starts, first_seq, first_token):
        yield self.plan_key, lambda: chunk_runs(seq_lens, 0, 0, self.plan_key[1])

    # ---- step
    def inner(self, proj: torch.Tensor, out: torch.Tensor, inp, state, workspace) -> None:
        S, ring = state
        C = self.channels
        gates = (self.gate_w, self.gate_b, self.rate)
        if inp.one_token:
            lk.rglru_step(proj, C, self.blocks, self.conv.conv_t, self.conv.bias, *gates, inp.rows, inp.positions, S,
                          ring, out)
            return
        chunk, runs, seq_runs = inp.plan[self.plan_key]
        u = torch.empty((proj.shape[0], C), dtype=self.dtype, device=proj.device)
        x, seqs = proj[:, C:], (inp.cu, inp.rows, inp.positions)
        lk.conv_chunk(x, self.conv.conv_t, self.conv.bias, False, chunk, *seqs, ring, ((1, C, C, u.unsqueeze(1), None),))
        lk.rglru_prompt(proj, C, self.blocks, u, *gates, chunk, runs, seq_runs, 0, *seqs, S, out)
        lk.conv_save(x, C, *seqs, ring)


class WindowAttention:
    """Grouped attention with RMS-normed queries and keys, no rotation, an optional sliding window and an
    elementwise output gate; biases on its projections but the gate's. Caches K [blocks, kv_heads, 16, dim] and V
    transposed [blocks, kv_heads, vdim, 16], sizes padded."""

    libraries = ("attn",)
    paged = True
    kv_from = None
    in_bias, out_bias = True, True

    @staticmethod
    def prefix_cacheable(m: Dict[str, Any]) -> bool:
        return True

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights):
        self.heads, self.kv_heads = int(m["heads"]), int(m["kv_heads"])
        self.dim, self.vdim = int(m["dim"]), int(m["vdim"])
        mask = m.get("mask")
        self.window = int(mask["size"]) if mask and mask.get("size") else None
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.shape = lk.attn_shape(self.heads, self.kv_heads, self.dim, self.vdim, self.window, float(m["scale"]), eps)
        self.dtype = w.dtype
        self.qkv = lk.attn_channels(self.shape)
        self.out_cols = self.heads * self.vdim
        self.in_rows = self.qkv + self.out_cols
        self.q_norm, self.k_norm = w.ones(self.dim), w.ones(self.dim)

    def bind(self, w_in, b_in, w_out, b_out) -> None:
        self.w_in, self.b_in, self.wo, self.bo = w_in, b_in, w_out, b_out

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        rows = (("q", self.heads * self.dim), ("k", self.kv_heads * self.dim), ("v", self.kv_heads * self.vdim))
        yield from split_rows(self.w_in, rows + (("g", self.out_cols),))
        yield from split_rows(self.b_in, [(n + ".b", r) for n, r in rows])
        yield from (("q.norm", self.q_norm), ("k.norm", self.k_norm), ("o", self.wo), ("o.b", self.bo))

    def refresh(self) -> None:
        pass

    # ---- cache
    def block_bytes(self) -> int:
        return self.kv_heads * BLOCK_SIZE * sum(lk.attn_pads(self.shape)) * self.dtype.itemsize

    def row_bytes(self) -> int:
        return 0

    def make_state(self, num_blocks: int, num_rows: int, device):
        dp, vp = lk.attn_pads(self.shape)
        zeros = lambda *tail: torch.zeros((num_blocks, self.kv_heads) + tail, dtype=self.dtype, device=device)  # noqa: E731
        return zeros(BLOCK_SIZE, dp), zeros(vp, BLOCK_SIZE)

    # ---- plans
    def host_plans(self, seq_lens, starts, first_seq, first_token):
        args = (seq_lens, starts, first_seq, first_token)
        yield ("tiles", self.window), lambda: (tile_plan(*args, self.window),)
        yield "runs", lambda: (run_plan(*args),)

    def nparts(self, tokens: int, max_ctx: int) -> int:
        ctx = min(max_ctx, self.window + BLOCK_SIZE) if self.window else max_ctx
        groups = -(-(self.heads // self.kv_heads) // 16)  # a wave takes 16 query heads of a key head
        return kernels.choose_nparts(tokens, self.kv_heads * groups, ctx)

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        return lk.attn_workspace_bytes(self.shape, tokens, self.nparts(tokens, max_ctx))

    # ---- step
    def inner(self, proj: torch.Tensor, out: torch.Tensor, inp, state, workspace) -> None:
        k_cache, v_cache = state
        T = proj.shape[0]
        key = ("tiles", self.window)
        prompt = inp.plan is not None and key in inp.plan and lk.attn_mfma(self.shape, self.dtype)
        ts = inp.short_tokens if prompt else T
        runs = inp.plan["runs"][0] if prompt and lk.attn_runs_fit(self.shape, proj) else None
        args = (self.q_norm, self.k_norm, inp.slots, k_cache, v_cache)
        q = lk.attn_write(self.shape, proj, *args, count=T if runs is None else ts)
        if runs is not None:
            lk.attn_write(self.shape, proj, *args, q=q, runs=runs)
        gate = proj[:, self.qkv:]
        for a in range(0, ts, 32768):  # the decode form's grid limit
            b = min(ts, a + 32768)
            lk.attn_attend(self.shape, q[a:b], gate[a:b], k_cache, v_cache, inp.block_tables, inp.bt_row[a:b],
                           inp.positions[a:b], out[a:b], nparts=self.nparts(b - a, inp.max_ctx),
                           part_min=kernels.MIN_PARTITION, workspace=workspace)
        if ts < T:
            lk.attn_prefill(self.shape, q, gate, k_cache, v_cache, inp.block_tables, inp.plan[key][0], out)


class StateSpace:
    """State space mixer with a scalar decay per head (Mamba-2): biased short convolutions, a gate before a
    norm in equal parts. State per row: the f32 matrix of every head and the convolutions' last inputs."""

    libraries = ("ssd",)
    paged = False
    kv_from = None
    in_bias, out_bias = False, False

    @staticmethod
    def prefix_cacheable(m: Dict[str, Any]) -> bool:
        return False

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights):
        self.heads, self.vdim, self.state = int(m["heads"]), int(m["vdim"]), int(m["state"])
        self.groups, self.taps, self.norm_groups = int(m["groups"]), int(m["conv"]), int(m["norm_groups"])
        self.width = self.heads * self.vdim
        if self.heads % self.groups or self.width % self.norm_groups:
            raise ValueError("heads must be a multiple of groups, heads * vdim of norm_groups")
        self.shape = lk.ssd_shape(self.heads, self.vdim, self.state, self.groups, self.taps)
        self.eps, self.dtype = eps, w.dtype
        self.channels = lk.ssd_channels(self.shape)
        self.in_rows, self.out_cols = lk.ssd_width(self.shape), self.width
        self.conv = ShortConv(self.channels, self.taps, w)
        self.a_log, self.dt_bias, self.skip = (w.zeros(self.heads, dtype=torch.float32) for _ in range(3))
        self.norm = w.ones(self.width)
        self.plan_key = ("walk", self.heads * lk.ssd_slices(self.shape))

    def bind(self, w_in, b_in, w_out, b_out) -> None:
        self.w_in, self.wo = w_in, w_out

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield "in", self.w_in
        yield from self.conv.params()
        yield from (("dt_bias", self.dt_bias), ("A_log", self.a_log), ("D", self.skip), ("norm", self.norm),
                    ("o", self.wo))

    def refresh(self) -> None:
        self.conv.refresh()

    # ---- state
    def block_bytes(self) -> int:
        return 0

    def row_bytes(self) -> int:
        return (4 * self.heads * self.state * lk.ssd_ppad(self.shape)
                + self.taps * self.channels * self.dtype.itemsize)

    def make_state(self, num_blocks: int, num_rows: int, device):
        return (torch.zeros((num_rows, self.heads, self.state, lk.ssd_ppad(self.shape)), dtype=torch.float32,
                            device=device),
                torch.zeros((num_rows, self.taps, self.channels), dtype=self.dtype, device=device))

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        return 0

    def host_plans(self, seq_lens, starts, first_seq, first_token):
        yield self.plan_key, lambda: walk_plan(seq_lens, first_seq, first_token, self.plan_key[1])

    # ---- step
    def inner(self, proj: torch.Tensor, out: torch.Tensor, inp, state, workspace) -> None:
        S, ring = state
        y = torch.empty((proj.shape[0], self.width), dtype=self.dtype, device=proj.device)
        args = (self.conv.conv_t, self.conv.bias, self.a_log, self.dt_bias, self.skip)
        n = inp.rows.shape[0]
        prompt = inp.plan is not None and self.plan_key in inp.plan and lk.ssd_prompt_fits(self.shape, self.dtype)
        k = inp.n_short if prompt else n
        if k:
            lk.ssd_scan(self.shape, proj, *args, inp.cu[:k + 1], inp.rows[:k], inp.positions, S, ring, inp.one_token, y)
        if k < n:
            lk.ssd_prompt(self.shape, proj, *args, inp.cu, inp.rows, inp.positions, S, ring, *inp.plan[self.plan_key], y)
        if not inp.one_token:
            lk.conv_save(proj[:, self.width:], self.channels, inp.cu, inp.rows, inp.positions, ring)
        lk.gated_norm(y, proj[:, :self.width], self.norm, self.norm_groups, self.eps, out)


class SideBySide:
    """Two mixers over the same input, one input product, each output normed over the model's width: the
    layer's output norm joins them, half the sum of both (layer_kernels.norm_add)."""

    LEFT, RIGHT, SHARE = WindowAttention, StateSpace, 0.5
    libraries = LEFT.libraries + RIGHT.libraries
    kv_from = None

    @classmethod
    def prefix_cacheable(cls, m: Dict[str, Any]) -> bool:
        return cls.LEFT.prefix_cacheable(m["left"]) and cls.RIGHT.prefix_cacheable(m["right"])

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights):
        self.parts = [c(m[side], width, eps, max_pos, w) for c, side in ((self.LEFT, "left"), (self.RIGHT, "right"))]
        self.out_norms = (w.ones(width), w.ones(width))
        self.paged = any(p.paged for p in self.parts)
        self.plans_short = any(getattr(p, "plans_short", False) for p in self.parts)

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        for side, part, norm in zip(("left.", "right."), self.parts, self.out_norms):
            for name, t in part.params():
                yield side + name, t
            yield side + "out", norm

    def refresh(self) -> None:
        for p in self.parts:
            p.refresh()

    def block_bytes(self) -> int:
        return sum(p.block_bytes() for p in self.parts)

    def row_bytes(self) -> int:
        return sum(p.row_bytes() for p in self.parts)

    def make_state(self, num_blocks: int, num_rows: int, device):
        return tuple(p.make_state(num_blocks, num_rows, device) for p in self.parts)

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        return max(p.workspace_bytes(tokens, max_ctx) for p in self.parts)

    def host_plans(self, *args):
        for p in self.parts:
            yield from p.host_plans(*args)


class GatedMLP:
    """down(gated product of gate x and up x), gate and up fused: `act` of layer_kernels.ACTIVATIONS, with
    m["limit"] for the clamped one; `bias`: on every projection."""

    def __init__(self, m: Dict[str, Any], width: int, w: Weights, act: str = "gelu_tanh", alpha: float = 1.0,
                 bias: bool = False):
        self.ff, self.act, self.alpha = int(m["ff"]), act, alpha
        self.limit = float(m["limit"]) if act == "clamped" else 0.0
        self.in_rows, self.out_cols = 2 * self.ff, self.ff
        self.in_bias = self.out_bias = bias

    def bind(self, w_in, b_in, w_out, b_out) -> None:
        self.wgu, self.bgu, self.wd, self.bd = w_in, b_in, w_out, b_out

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from split_rows(self.wgu, (("gate", self.ff), ("up", self.ff)))
        yield "down", self.wd
        if self.in_bias:
            yield from split_rows(self.bgu, (("gate.b", self.ff), ("up.b", self.ff)))
            yield "down.b", self.bd

    def inner(self, proj: torch.Tensor, out: torch.Tensor, inp, state, workspace) -> None:
        lk.gate_mul(proj, self.act, self.alpha, self.limit, out=out)


class PlainMLP:
    """down(xIELU(up x)); the activation's two learned numbers are `act`."""

    in_bias = out_bias = False

    def __init__(self, m: Dict[str, Any], width: int, w: Weights):
        self.in_rows = self.out_cols = int(m["ff"])
        self.act = w.zeros(2)

    def bind(self, w_in, b_in, w_out, b_out) -> None:
        self.wu, self.wd = w_in, w_out

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from (("up", self.wu), ("down", self.wd), ("act", self.act))

    def inner(self, proj: torch.Tensor, out: torch.Tensor, inp, state, workspace) -> None:
        lk.xielu(proj, self.act, out=out)


class RoutedExperts:
    """Of many small silu-gated feed-forwards each token runs `top`, weighted by the sigmoid of their router logits;
    they are chosen by those scores plus a learned correction, out of the best groups of neighbours. forward returns a
    token's `top` weighted rows one after another, to be summed."""

    libraries = ("moe",)
    in_bias = out_bias = False

    def __init__(self, m: Dict[str, Any], width: int, w: Weights):
        ro = m["router"]
        groups = ro.get("groups") or {"count": 1, "keep": 1}
        self.ff, self.experts, self.rows_per_token = int(m["expert"]["ff"]), int(ro["experts"]), int(ro["top"])
        self.shape = lk.moe_shape(width, self.ff, self.experts, self.rows_per_token, int(groups["count"]), int(groups["keep"]))
        self.router = w.matrix(self.experts, width)
        self.correction = w.zeros(self.experts, dtype=torch.float32)
        self.gate_up = w.matrix(self.experts, 2, self.ff, width)
        self.down = w.matrix(self.experts, width, self.ff)

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        for e in range(self.experts):
            yield from ((f"e{e}.gate", self.gate_up[e, 0]), (f"e{e}.up", self.gate_up[e, 1]), (f"e{e}.down", self.down[e]))
        yield from (("router", self.router), ("correction", self.correction))

    def forward(self, x: torch.Tensor, inp, state, workspace) -> torch.Tensor:
        idx, weight = lk.moe_route(self.shape, x, self.router, self.correction)
        return lk.moe_experts(self.shape, x, idx, weight, self.gate_up, self.down)


MIXERS = {"latent_attention": LatentAttention, "delta": GatedDelta, "general_delta": GeneralDelta,
          "attention": DifferentialAttention, "rglru": GatedLinearRecurrence, "parallel": SideBySide}
FEEDFORWARDS = {"dense": GatedMLP}
PLAIN_FEEDFORWARDS = {"dense": PlainMLP}
EXPERT_FEEDFORWARDS = {"moe": RoutedExperts}
