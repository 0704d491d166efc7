"""Layer mechanisms of the hybrid decoders: latent attention, gated delta rule, gated MLP.

A mechanism owns its weights (fused where one product serves several tensors), names them for
loading and saving, sizes and allocates its cache or state, and runs a step over it with the HIP
kernels of layer_kernels.py; matrix products are hipBLASLt through torch. Every size and constant is
a parameter; nothing here knows a particular model. `MIXERS` and `FEEDFORWARDS` map the type names of
a config.json to these classes.

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


class LatentAttention:
    """Attention over low-rank latents shared by all heads, with a rotated key part beside them and
    an optional sliding window. Caches [blocks, 16, row]: per token the normed latent | the rotated key
    part."""

    paged = True

    def __init__(self, m: Dict[str, Any], width: int, eps: float, max_pos: int, w: Weights):
        self.heads, self.dim, self.rot_dim = int(m["heads"]), int(m["dim"]), int(m["rot_dim"])
        self.vdim, self.rank, self.scale = int(m["vdim"]), int(m["kv_rank"]), float(m["scale"])
        mask = m.get("mask")
        self.window = int(mask["size"]) if mask and mask.get("size") else None
        if int(m["rot"]["dims"]) != self.rot_dim:
            raise ValueError("latent attention rotates exactly its rot_dim part: rot.dims must equal rot_dim")
        if self.rot_dim % 2:
            raise ValueError("rot_dim must be even")
        self.eps, self.width, self.dtype = eps, width, w.dtype
        self.cos_sin = rotary_table(m["rot"], max_pos).to(w.device)
        H, qd = self.heads, self.dim + self.rot_dim
        self.wproj = w.matrix(H * qd + self.rank + self.rot_dim, width)
        self.dkv_norm = w.ones(self.rank)
        self.wuk = w.matrix(H * self.dim, self.rank)
        self.wuv = w.matrix(H * self.vdim, self.rank)
        self.wuv_t = w.zeros(H, self.rank, self.vdim)  # per head transposed: the decode form's right operand
        self.wo = w.matrix(width, H * self.vdim)
        self.refresh()

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from split_rows(self.wproj, (("q", self.heads * (self.dim + self.rot_dim)),
                                           ("dkv", self.rank + self.rot_dim)))
        yield "dkv.norm", self.dkv_norm
        yield "uk", self.wuk
        yield "uv", self.wuv
        yield "o", self.wo

    def refresh(self) -> None:
        """Recompute derived tensors, in place, after the weights changed."""
        self.wuv_t.copy_(self.wuv.view(self.heads, self.vdim, self.rank).transpose(1, 2))

    # ---- cache
    def block_bytes(self) -> int:
        return BLOCK_SIZE * lk.latent_row(self.rank, self.rot_dim) * self.dtype.itemsize

    def row_bytes(self) -> int:
        return 0

    def make_state(self, num_blocks: int, num_rows: int, device) -> torch.Tensor:
        return torch.zeros((num_blocks, BLOCK_SIZE, lk.latent_row(self.rank, self.rot_dim)), dtype=self.dtype,
                           device=device)

    # ---- decode split
    def nparts(self, tokens: int, max_ctx: int) -> int:
        ctx = min(max_ctx, self.window + BLOCK_SIZE) if self.window else max_ctx
        return kernels.choose_nparts(tokens, (self.heads + 31) // 32, ctx, target_waves=ATTEND_WORKGROUPS)

    def workspace_bytes(self, tokens: int, max_ctx: int) -> int:
        from .. import _ffi

        n = self.nparts(tokens, max_ctx)
        return int(_ffi.query("skyrl_latent_attend_workspace_bytes", tokens, self.heads, self.rank, n)) if n > 1 else 0

    # ---- step
    def _attend_rows(self, q, out, inp, a: int, b: int, cache, workspace):
        """Tokens [a, b) in the decode form."""
        H, D, R = self.heads, self.dim, self.rank
        n = b - a
        q3 = q[a:b].view(n, H, D + self.rot_dim)
        qa = torch.bmm(q3[:, :, :D].transpose(0, 1), self.wuk.view(H, D, R))
        o = lk.latent_attend(qa, q3[:, :, D:], cache, R, self.rot_dim, inp.block_tables, inp.bt_row[a:b],
                             inp.positions[a:b], self.scale, self.window, nparts=self.nparts(n, inp.max_ctx),
                             part_min=kernels.MIN_PARTITION, workspace=workspace)
        out[a:b].view(n, H, self.vdim).copy_(torch.bmm(o, self.wuv_t).transpose(0, 1))

    def forward(self, x: torch.Tensor, inp, cache: torch.Tensor, workspace) -> torch.Tensor:
        H, T = self.heads, x.shape[0]
        proj = F.linear(x, self.wproj)
        lk.latent_write(proj, H, self.dim, self.rot_dim, self.rank, self.dkv_norm, self.eps, inp.positions, inp.slots,
                        self.cos_sin, cache)
        qw = H * (self.dim + self.rot_dim)
        out = torch.empty((T, H * self.vdim), dtype=self.dtype, device=x.device)
        prompt = inp.plan is not None and lk.prefill_fits(self.dim, self.rot_dim, self.vdim, self.dtype)
        ts = inp.short_tokens if prompt else T
        q = proj[:, :qw]
        for a in range(0, ts, 32768):  # the decode form's grid limit
            self._attend_rows(q, out, inp, a, min(ts, a + 32768), cache, workspace)
        if ts < T:
            seg, tiles, rows, longest = inp.plan[self.window]
            latent, k_rot = lk.latent_gather(cache, self.rank, self.rot_dim, inp.block_tables, seg, rows, longest)
            k = F.linear(latent, self.wuk)
            v_t = torch.mm(self.wuv, latent.t())
            lk.latent_prefill(q, k, k_rot, v_t, tiles, H, self.dim, self.rot_dim, self.vdim, self.scale, self.window,
                              out)
        return F.linear(out, self.wo)


class GatedDelta:
    """Gated delta rule with short causal convolutions on q, k and v. State per row (a running
    request): the f32 matrix of every head and the convolutions' last inputs."""

    paged = False
    window = None

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

    # ---- step
    def forward(self, x: torch.Tensor, inp, state, workspace) -> torch.Tensor:
        S, ring = state
        proj = F.linear(x, self.wproj)
        out = torch.empty((x.shape[0], self.heads * self.vdim), dtype=self.dtype, device=x.device)
        args = (self.conv, self.a_log, self.dt_bias, self.norm)
        n = inp.rows.shape[0]
        k = inp.n_short if inp.plan is not None and lk.delta_prompt_fits(self.shape) else n
        if k:
            lk.delta_scan(self.shape, proj, *args, inp.cu[:k + 1], inp.rows[:k], inp.positions, S, ring,
                          inp.one_token, out)
        if k < n:
            chunk, seq_chunks = inp.plan["chunks"]
            lk.delta_prompt(self.shape, proj, *args, inp.cu, inp.rows, inp.positions, S, ring, chunk, seq_chunks, k,
                            inp.short_tokens, out)
        if not inp.one_token:
            lk.delta_save(self.shape, proj, inp.cu, inp.rows, inp.positions, ring)
        return F.linear(out, self.wo)


class GatedMLP:
    """down(act(gate x) * up x), gate and up fused."""

    def __init__(self, m: Dict[str, Any], width: int, w: Weights, act: str = "gelu_tanh"):
        self.ff, self.act = int(m["ff"]), act
        self.wgu = w.matrix(2 * self.ff, width)
        self.wd = w.matrix(width, self.ff)

    def params(self) -> Iterator[Tuple[str, torch.Tensor]]:
        yield from split_rows(self.wgu, (("gate", self.ff), ("up", self.ff)))
        yield "down", self.wd

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return F.linear(lk.gate_mul(F.linear(x, self.wgu), self.act), self.wd)


MIXERS = {"latent_attention": LatentAttention, "delta": GatedDelta}
FEEDFORWARDS = {"dense": GatedMLP}
