"""Host launchers of the hybrid decoders' layer kernels (include/skyrl_layers.h).

Shapes, dtypes and strides are checked here before every launch, as in kernels.py; there is no CPU
fallback."""

from __future__ import annotations

import ctypes
from typing import Optional

import torch

from .. import _ffi
from ..ops import _ptr, _require_gpu, _stream

NORMS = {"layer": 0, "rms": 1}
ACTIVATIONS = {"silu": 0, "gelu_tanh": 1, "clamped": 2}
_DTYPES = {torch.bfloat16: _ffi.BF16, torch.float32: _ffi.F32}


def _code(t: torch.Tensor) -> int:
    code = _DTYPES.get(t.dtype)
    if code is None:
        raise TypeError(f"activations must be bfloat16 or float32, got {t.dtype}")
    return code


def _check(t: Optional[torch.Tensor], name: str, dtype, shape=None, contiguous: bool = True):
    if t is None:
        return
    if t.dtype != dtype:
        raise TypeError(f"{name} must be {dtype}, got {t.dtype}")
    if shape is not None and tuple(t.shape) != tuple(shape):
        raise ValueError(f"{name} must be {tuple(shape)}, got {tuple(t.shape)}")
    if contiguous and not t.is_contiguous():
        raise ValueError(f"{name} must be contiguous")


def _check_view(t: torch.Tensor, name: str, dtype, shape):
    """Any row stride, unit column stride."""
    if t.dtype != dtype or tuple(t.shape) != tuple(shape) or (t.shape[1] > 1 and t.stride(1) != 1):
        raise ValueError(f"{name} must be {dtype} {tuple(shape)} with unit column stride")


def embed(tokens: torch.Tensor, table: torch.Tensor, scale: float, positions: Optional[torch.Tensor] = None,
          turns: Optional[torch.Tensor] = None, x: Optional[torch.Tensor] = None) -> torch.Tensor:
    """f32 rows of the embedding table times scale, plus, with `turns` f64 [(H + 1) // 2], each position's sine
    and cosine vector; `x`: filled with the same in the table's type."""
    dev = _require_gpu(tokens, table, positions, turns, x)
    n, H = tokens.shape[0], table.shape[1]
    _check(tokens, "tokens", torch.int64, (n,))
    _check(table, "table", table.dtype)
    if (positions is None) != (turns is None):
        raise ValueError("positions and turns go together")
    _check(positions, "positions", torch.int64, (n,))
    _check(turns, "turns", torch.float64, ((H + 1) // 2,))
    _check(x, "x", table.dtype, (n, H))
    out = torch.empty((n, H), dtype=torch.float32, device=dev)
    _ffi.call("skyrl_embed", _ptr(tokens), _ptr(table), n, H, float(scale), _ptr(positions), _ptr(turns), _ptr(out),
              _ptr(x), _code(table), _stream(dev))
    return out


def add_norm(delta: Optional[torch.Tensor], hidden: torch.Tensor, weight: torch.Tensor, eps: float,
             kind: str = "layer", step: Optional[torch.Tensor] = None,
             out: Optional[torch.Tensor] = None, base: float = 0.0) -> torch.Tensor:
    """hidden (f32, in place) += delta and += step (one vector for every row), then the norm, times
    base + weight (base 1: the weight is stored as its distance from 1)."""
    dev = _require_gpu(hidden, weight, delta, step, out)
    n, H = hidden.shape
    _check(hidden, "hidden", torch.float32)
    _check(weight, "weight", weight.dtype, (H,))
    _check(delta, "delta", weight.dtype, (n, H))
    _check(step, "step", weight.dtype, (H,))
    if out is None:
        out = torch.empty((n, H), dtype=weight.dtype, device=dev)
    _check(out, "out", weight.dtype, (n, H))
    _ffi.call("skyrl_add_norm", _ptr(delta), _ptr(hidden), _ptr(step), _ptr(weight), float(base), n, H, float(eps),
              NORMS[kind], _ptr(out), _code(weight), _stream(dev))
    return out


def norm_add(delta, hidden: torch.Tensor, weight: torch.Tensor, eps: float, pair=None, share: float = 0.5,
             final: Optional[torch.Tensor] = None, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """hidden (f32, in place) += rms(delta) * weight. With `pair` = (wa, wb) `delta` is two outputs (a, b), joined
    to share (rms(a) wa + rms(b) wb) first. Returns hidden in the weight's type, or rms(hidden) * final. A weight
    is one number (a 0-d tensor) or a vector."""
    a, b = delta if pair is not None else (delta, None)
    wa, wb = pair if pair is not None else (None, None)
    dev = _require_gpu(a, b, wa, wb, hidden, weight, final, out)
    n, H = hidden.shape
    _check(hidden, "hidden", torch.float32)
    for t, name in ((a, "delta"), (b, "second delta")):
        _check(t, name, weight.dtype, (n, H))
    for t, name in ((wa, "first pair weight"), (wb, "second pair weight")):
        _check(t, name, weight.dtype, (H,))
    for t, name in ((weight, "weight"), (final, "final weight")):
        if t is not None and tuple(t.shape) not in ((), (H,)):
            raise ValueError(f"{name} must be one number or [{H}]")
        _check(t, name, weight.dtype)
    if out is None:
        out = torch.empty((n, H), dtype=weight.dtype, device=dev)
    _check(out, "out", weight.dtype, (n, H))
    _ffi.call("skyrl_norm_add", _ptr(a), _ptr(wa), _ptr(b), _ptr(wb), float(share), _ptr(hidden), _ptr(weight),
              weight.numel(), _ptr(final), 0 if final is None else final.numel(), n, H, float(eps), _ptr(out),
              _code(weight), _stream(dev))
    return out


def gate_norm_add(a: torch.Tensor, hidden: torch.Tensor, weight: torch.Tensor, next_weight: torch.Tensor, eps: float,
                  groups: int = 1, mult: float = 1.0, parts: int = 1, gate: Optional[torch.Tensor] = None,
                  gate_bias: Optional[torch.Tensor] = None, rows: Optional[torch.Tensor] = None, fresh: bool = False,
                  out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """hidden (f32 [n, H], in place; fresh: from 0) += mult norm(y) weight, y the sum of `parts` consecutive rows of a,
    times sigmoid(gate + gate_bias) with a gate; returns norm(hidden) next_weight. A norm is an RMS norm in `groups`
    equal parts of the row. `rows` int64 [n]: which rows of a (parts 1)."""
    dev = _require_gpu(a, hidden, weight, next_weight, gate, gate_bias, rows, out)
    n, H = hidden.shape
    _check(hidden, "hidden", torch.float32)
    if a.dim() != 2 or a.shape[1] != H or (rows is None and a.shape[0] != n * parts) or (rows is not None and parts != 1):
        raise ValueError(f"a must be [{n} * parts, {H}], with rows [any, {H}] and one part")
    _check(a, "a", weight.dtype)
    _check(weight, "weight", weight.dtype, (H,))
    _check(next_weight, "next_weight", weight.dtype, (H,))
    _check(rows, "rows", torch.int64, (n,))
    if (gate is None) != (gate_bias is None):
        raise ValueError("gate and gate_bias go together")
    if gate is not None:
        _check_view(gate, "gate", weight.dtype, (n, H))
        _check(gate_bias, "gate_bias", torch.float32, (H,))
    if out is None:
        out = torch.empty((n, H), dtype=weight.dtype, device=dev)
    _check(out, "out", weight.dtype, (n, H))
    _ffi.call("skyrl_gate_norm_add", _ptr(a), _ptr(rows), parts, _ptr(gate), 0 if gate is None else max(gate.stride(0), H),
              _ptr(gate_bias), _ptr(weight), groups, float(eps), float(mult), _ptr(hidden), int(fresh), _ptr(next_weight), n, H,
              _ptr(out), _code(weight), _stream(dev))
    return out


def tanh(x: torch.Tensor) -> torch.Tensor:
    """tanh of x [n, I] (a column range), contiguous."""
    dev = _require_gpu(x)
    n, I = x.shape
    _check_view(x, "x", x.dtype, (n, I))
    out = torch.empty((n, I), dtype=x.dtype, device=dev)
    _ffi.call("skyrl_tanh", _ptr(x), max(x.stride(0), I), n, I, _ptr(out), _code(x), _stream(dev))
    return out


def xielu(x: torch.Tensor, pq: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """xIELU of x [n, I] with the learned pair pq; both may be column ranges."""
    dev = _require_gpu(x, pq, out)
    n, I = x.shape
    _check_view(x, "x", x.dtype, (n, I))
    _check(pq, "pq", x.dtype, (2,))
    if out is None:
        out = torch.empty((n, I), dtype=x.dtype, device=dev)
    _check_view(out, "out", x.dtype, (n, I))
    _ffi.call("skyrl_xielu", _ptr(x), x.stride(0), n, I, _ptr(pq), _ptr(out), out.stride(0), _code(x), _stream(dev))
    return out


def gate_mul(gate_up: torch.Tensor, act: str, alpha: float = 1.0, limit: float = 0.0,
             out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The gated product of the fused [n, 2I] projection (skyrl_gate_mul); both may be column ranges."""
    dev = _require_gpu(gate_up, out)
    n, I2 = gate_up.shape
    _check_view(gate_up, "gate_up", gate_up.dtype, (n, I2))
    if out is None:
        out = torch.empty((n, I2 // 2), dtype=gate_up.dtype, device=dev)
    _check_view(out, "out", gate_up.dtype, (n, I2 // 2))
    _ffi.call("skyrl_gate_mul", _ptr(gate_up), gate_up.stride(0), n, I2 // 2, ACTIVATIONS[act], float(alpha),
              float(limit), _ptr(out), out.stride(0), _code(gate_up), _stream(dev))
    return out


def conv_save(x: torch.Tensor, channels: int, cu, rows, positions, ring: torch.Tensor) -> None:
    """Store the last inputs of each sequence's short convolutions, columns [0, channels) of x."""
    dev = _require_gpu(x, cu, rows, positions, ring)
    T, n = x.shape[0], rows.shape[0]
    if x.dim() != 2 or x.shape[1] < channels or x.stride(1) != 1:
        raise ValueError(f"x must be [T, >= {channels}] with unit column stride")
    _check(cu, "cu", torch.int32, (n + 1,))
    _check(rows, "rows", torch.int32, (n,))
    _check(positions, "positions", torch.int64, (T,))
    if ring.dim() != 3 or ring.shape[2] != channels:
        raise ValueError("ring must be [rows, taps, channels]")
    _check(ring, "ring", x.dtype)
    _ffi.call("skyrl_conv_save", _ptr(x), x.stride(0), channels, ring.shape[1], _ptr(cu), _ptr(rows), _ptr(positions),
              n, _ptr(ring), _code(x), _stream(dev))


def softcap(x: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    """f32 cap * tanh(x / cap); a plain f32 copy without a cap."""
    dev = _require_gpu(x)
    _check(x, "x", x.dtype)
    out = torch.empty(x.shape, dtype=torch.float32, device=dev)
    _ffi.call("skyrl_softcap", _ptr(x), _ptr(out), x.numel(), float(cap or 0.0), _code(x), _stream(dev))
    return out


# ---------------------------------------------------------------- latent attention
def latent_row(rank: int, rot_dim: int) -> int:
    """Elements of one cached token: latent | rotated key part | padding to a multiple of 32."""
    return (rank + rot_dim + 31) // 32 * 32


def _check_cache(cache: torch.Tensor, rank: int, rot_dim: int, dtype):
    if cache.dim() != 3 or cache.shape[1] != 16 or cache.shape[2] != latent_row(rank, rot_dim):
        raise ValueError("cache must be [blocks, 16, latent_row(rank, rot_dim)]")
    _check(cache, "cache", dtype)


def _check_table(block_tables, bt_row, positions, T):
    if block_tables.dtype != torch.int32 or block_tables.dim() != 2 or block_tables.stride(1) != 1:
        raise ValueError("block_tables must be int32 [n, blocks] with unit column stride")
    _check(bt_row, "bt_row", torch.int32, (T,))
    _check(positions, "positions", torch.int64, (T,))


def _check_rotation(positions, cos_sin, rot_dim, T):
    _check(positions, "positions", torch.int64, (T,))
    if cos_sin.dim() != 2 or cos_sin.shape[1] != rot_dim:
        raise ValueError("cos_sin must be [max_pos, rot_dim]")
    _check(cos_sin, "cos_sin", torch.float32)


def latent_write(proj, rot_dim, positions, slots, cos_sin, cache, eps, heads: int = 0, dim: int = 0, q_norm=None,
                 rank: int = 0, norm_weight=None, halves: bool = False) -> None:
    """Rows of ``proj`` in place, each part optional: with `heads` the rotated parts of the queries at the row's start
    are turned, with `q_norm` [q_rank] the query latent there is normed; with `rank` the key latent and its rotated part
    that follow are normed, turned and written into the cache."""
    dev = _require_gpu(proj, q_norm, norm_weight, positions, slots, cos_sin, cache)
    T = proj.shape[0]
    q_rank = 0 if q_norm is None else q_norm.shape[0]
    at = q_rank or heads * (dim + rot_dim)
    width = at + (rank + rot_dim if rank else 0)
    if (heads and q_rank) or proj.dim() != 2 or proj.shape[1] < width or proj.stride(1) != 1:
        raise ValueError(f"proj must be [T, >= {width}] with unit column stride, queries or their latent first")
    _check_rotation(positions, cos_sin, rot_dim, T)
    _check(q_norm, "q_norm", proj.dtype, (q_rank,))
    if rank:
        _check(norm_weight, "norm_weight", proj.dtype, (rank,))
        _check(slots, "slots", torch.int64, (T,))
        _check_cache(cache, rank, rot_dim, proj.dtype)
    _ffi.call("skyrl_latent_write", _ptr(proj), proj.stride(0), T, heads, dim, rot_dim, int(halves), q_rank, _ptr(q_norm),
              rank, at, _ptr(norm_weight), float(eps), _ptr(positions), _ptr(slots), _ptr(cos_sin), _ptr(cache),
              cache.shape[2] if rank else 0, _code(proj), _stream(dev))


def _check_end(sinks, gate, heads, T, dtype):
    _check(sinks, "sinks", torch.float32, (heads,))
    if gate is not None:
        _check_view(gate, "gate", dtype, (T, heads))
    return 0 if gate is None else max(gate.stride(0), heads)


def latent_attend(qa, q_rot, cache, rank, rot_dim, block_tables, bt_row, positions, scale, window, nparts=1,
                  part_min=64, workspace=None, sinks=None, gate=None) -> torch.Tensor:
    """Latent-space attention, one query row per token. qa [heads, T, rank]; q_rot [T, heads, rot_dim]
    (any token and head stride); returns [heads, T, rank]. sinks f32 [heads]: exp(sink) joins the denominators; gate
    [T, heads]: outputs times its sigmoid."""
    dev = _require_gpu(qa, q_rot, cache, block_tables, bt_row, positions, sinks, gate)
    heads, T, R = qa.shape
    _check(qa, "qa", cache.dtype, (heads, T, rank))
    if q_rot.dtype != qa.dtype or tuple(q_rot.shape) != (T, heads, rot_dim) or (rot_dim > 1 and q_rot.stride(2) != 1):
        raise ValueError("q_rot must be [T, heads, rot_dim] with unit last stride")
    _check_cache(cache, rank, rot_dim, qa.dtype)
    _check_table(block_tables, bt_row, positions, T)
    gate_stride = _check_end(sinks, gate, heads, T, qa.dtype)
    out = torch.empty_like(qa)
    ws = None
    if nparts > 1 and mfma_attend(rank, rot_dim, qa.dtype):
        need = _ffi.query("skyrl_latent_attend_workspace_bytes", T, heads, rank, nparts)
        ws = workspace.get(need) if workspace is not None else torch.empty(need, dtype=torch.uint8, device=dev)
    else:
        nparts = 1
    _ffi.call("skyrl_latent_attend", _ptr(qa), _ptr(q_rot), q_rot.stride(0), q_rot.stride(1), _ptr(cache),
              cache.shape[2], _ptr(block_tables), block_tables.stride(0), _ptr(bt_row), _ptr(positions), T, heads,
              rank, rot_dim, float(scale), int(window or 0), part_min, nparts, _ptr(sinks), _ptr(gate), gate_stride,
              _ptr(out), _ptr(ws), _code(qa), _stream(dev))
    return out


def mfma_attend(rank: int, rot_dim: int, dtype) -> bool:
    return bool(_ffi.query("skyrl_latent_attend_mfma", rank, rot_dim, latent_row(rank, rot_dim), _DTYPES[dtype]))


def latent_gather(cache, rank, rot_dim, block_tables, seg, nrows: int, max_count: int):
    """Packed (latent [nrows, rank], k_rot [nrows, rot_dim]) of the segments ``seg`` int32 [n, 4]: block-table
    row, first position, count, first packed row. nrows covers every segment rounded up to 64."""
    dev = _require_gpu(cache, block_tables, seg)
    _check_cache(cache, rank, rot_dim, cache.dtype)
    _check(seg, "seg", torch.int32, (seg.shape[0], 4))
    latent = torch.empty((nrows, rank), dtype=cache.dtype, device=dev)
    k_rot = torch.empty((nrows, rot_dim), dtype=cache.dtype, device=dev)
    _ffi.call("skyrl_latent_gather", _ptr(cache), cache.shape[2], _ptr(block_tables), block_tables.stride(0),
              _ptr(seg), seg.shape[0], max_count, rank, rot_dim, _ptr(latent), _ptr(k_rot), _code(cache),
              _stream(dev))
    return latent, k_rot


def latent_prefill(q, k_nope, k_rot, v_t, tiles, heads, dim, rot_dim, vdim, scale, window, out, sinks=None,
                   gate=None) -> torch.Tensor:
    """Windowed attention of prompt tiles over packed keys. q [T, >= heads * (dim + rot_dim)]; k_nope
    [rows, heads * dim]; k_rot [rows, rot_dim]; v_t [heads * vdim, rows]; out [T, heads * vdim]; sinks and gate as in
    latent_attend."""
    dev = _require_gpu(q, k_nope, k_rot, v_t, tiles, out, sinks, gate)
    rows = k_nope.shape[0]
    for t, name in ((q, "q"), (k_nope, "k_nope"), (k_rot, "k_rot"), (v_t, "v_t"), (out, "out")):
        if t.dtype != torch.bfloat16 or t.dim() != 2 or t.stride(1) != 1:
            raise ValueError(f"{name} must be bf16, 2-D, with unit column stride")
    if q.shape[1] < heads * (dim + rot_dim) or k_nope.shape[1] != heads * dim or out.shape[1] != heads * vdim \
            or out.shape[0] != q.shape[0]:
        raise ValueError("latent_prefill: q / k_nope / out widths do not match the heads")
    _check(k_rot, "k_rot", torch.bfloat16, (rows, rot_dim))
    if v_t.shape != (heads * vdim, rows) or rows % 64:
        raise ValueError("v_t must be [heads * vdim, rows] with rows a multiple of 64")
    _check(tiles, "tiles", torch.int32, (tiles.shape[0], 8))
    gate_stride = _check_end(sinks, gate, heads, q.shape[0], q.dtype)
    _ffi.call("skyrl_latent_prefill", _ptr(q), q.stride(0), _ptr(k_nope), k_nope.stride(0), _ptr(k_rot), _ptr(v_t),
              v_t.stride(0), _ptr(tiles), tiles.shape[0], heads, dim, rot_dim, vdim, float(scale), int(window or 0),
              _ptr(sinks), _ptr(gate), gate_stride, _ptr(out), out.stride(0), _stream(dev))
    return out


def prefill_fits(dim: int, rot_dim: int, vdim: int, dtype) -> bool:
    return dtype == torch.bfloat16 and 0 < dim and dim + rot_dim <= 256 and vdim <= 256


# ---------------------------------------------------------------- gated delta rule
def delta_shape(heads, kv_heads, dim, vdim, taps, eps) -> _ffi.DeltaShape:
    return _ffi.DeltaShape(heads, kv_heads, dim, vdim, taps, eps)


def delta_channels(sh) -> int:
    """Channels of the short convolutions: q | k | v."""
    return 2 * sh.kv_heads * sh.dim + sh.heads * sh.vdim


def delta_width(sh) -> int:
    """Columns of the fused projection: q | k | v | output gate | beta | decay."""
    return delta_channels(sh) + sh.heads * sh.vdim + 2 * sh.heads


def delta_vpad(sh) -> int:
    return (sh.vdim + 3) // 4 * 4


def _check_delta(sh, proj, cu, rows, positions, conv_state, state=None):
    T = proj.shape[0]
    if proj.dim() != 2 or proj.shape[1] != delta_width(sh) or proj.stride(1) != 1:
        raise ValueError(f"proj must be [T, {delta_width(sh)}] with unit column stride")
    n = rows.shape[0]
    _check(rows, "rows", torch.int32, (n,))
    _check(cu, "cu", torch.int32, (n + 1,))
    _check(positions, "positions", torch.int64, (T,))
    if conv_state.dim() != 3 or tuple(conv_state.shape[1:]) != (sh.taps, delta_channels(sh)):
        raise ValueError("conv_state must be [rows, taps, channels]")
    _check(conv_state, "conv_state", proj.dtype)
    if state is not None:
        _check(state, "state", torch.float32, (conv_state.shape[0], sh.heads, sh.dim, delta_vpad(sh)))
    return n


def _check_delta_weights(sh, dtype, conv_w, a_log, dt_bias, norm_w=None):
    _check(conv_w, "conv_w", dtype, (delta_channels(sh), sh.taps))
    _check(a_log, "a_log", torch.float32, (sh.heads,))
    _check(dt_bias, "dt_bias", torch.float32, (sh.heads,))
    _check(norm_w, "norm_w", dtype, (sh.vdim,))


def delta_scan(sh, proj, conv_w, a_log, dt_bias, norm_w, cu, rows, positions, state, conv_state, save_conv,
               out) -> torch.Tensor:
    """Token by token over each sequence's tokens [cu[s], cu[s + 1]); state and (save_conv: one token per
    sequence) convolution inputs updated in place."""
    dev = _require_gpu(proj, conv_w, a_log, dt_bias, norm_w, cu, rows, positions, state, conv_state, out)
    n = _check_delta(sh, proj, cu, rows, positions, conv_state, state)
    _check_delta_weights(sh, proj.dtype, conv_w, a_log, dt_bias, norm_w)
    if out.dtype != proj.dtype or out.shape != (proj.shape[0], sh.heads * sh.vdim) or out.stride(1) != 1:
        raise ValueError("out must be [T, heads * vdim]")
    _ffi.call("skyrl_delta_scan", ctypes.byref(sh), _ptr(proj), proj.stride(0), _ptr(conv_w), _ptr(a_log),
              _ptr(dt_bias), _ptr(norm_w), _ptr(cu), _ptr(rows), _ptr(positions), n, _ptr(state), _ptr(conv_state),
              int(save_conv), _ptr(out), out.stride(0), _code(proj), _stream(dev))
    return out


CHUNK = 64  # tokens per chunk of the prompt form


def delta_prompt_fits(sh) -> bool:
    return sh.dim <= 256


def delta_prompt(sh, proj, conv_w, a_log, dt_bias, norm_w, cu, rows, positions, state, conv_state, chunk, seq_chunks,
                 first_seq: int, first_token: int, out) -> torch.Tensor:
    """Chunked form over the sequences from first_seq on, whose tokens are [first_token, T): chunk int32
    [n, 4] and seq_chunks int32 [sequences + 1] (mixers.chunk_plan). `state` is updated in place; the
    convolution inputs are conv_save's."""
    dev = _require_gpu(proj, conv_w, a_log, dt_bias, norm_w, cu, rows, positions, state, conv_state, chunk,
                       seq_chunks, out)
    n = _check_delta(sh, proj, cu, rows, positions, conv_state, state)
    _check_delta_weights(sh, proj.dtype, conv_w, a_log, dt_bias, norm_w)
    T, nc, nseq = proj.shape[0], chunk.shape[0], n - first_seq
    _check(chunk, "chunk", torch.int32, (nc, 4))
    _check(seq_chunks, "seq_chunks", torch.int32, (nseq + 1,))
    if out.dtype != proj.dtype or out.shape != (T, sh.heads * sh.vdim) or out.stride(1) != 1:
        raise ValueError("out must be [T, heads * vdim]")
    d16, v16 = (sh.dim + 15) // 16 * 16, (sh.vdim + 15) // 16 * 16
    f32 = lambda *shape: torch.empty(shape, dtype=torch.float32, device=dev)  # noqa: E731
    qk, v = f32(T, 2, sh.kv_heads, d16), f32(T, sh.heads, sh.vdim)
    lg, beta = f32(T, sh.heads), f32(T, sh.heads)
    kt = f32(nc, sh.kv_heads, d16, CHUNK)
    W, U = f32(nc, sh.heads, CHUNK, d16), f32(nc, sh.heads, v16, CHUNK)
    P, G = f32(nc, sh.heads, CHUNK, CHUNK), f32(nc, sh.heads, CHUNK)
    o, st, ref = f32(T, sh.heads, sh.vdim), _stream(dev), ctypes.byref(sh)
    _ffi.call("skyrl_delta_conv", ref, _ptr(proj), proj.stride(0), _ptr(conv_w), _ptr(a_log), _ptr(dt_bias),
              _ptr(chunk), nc, _ptr(cu), _ptr(rows), _ptr(positions), _ptr(conv_state), _ptr(qk), _ptr(kt), _ptr(v), _ptr(lg),
              _ptr(beta), _code(proj), st)
    _ffi.call("skyrl_delta_chunk", ref, _ptr(chunk), nc, _ptr(qk), _ptr(v), _ptr(lg), _ptr(beta), _ptr(W), _ptr(U),
              _ptr(P), _ptr(G), st)
    _ffi.call("skyrl_delta_chain", ref, _ptr(chunk), _ptr(seq_chunks), first_seq, nseq, _ptr(cu), _ptr(rows),
              _ptr(positions), _ptr(qk), _ptr(kt), _ptr(W), _ptr(U), _ptr(P), _ptr(G), _ptr(state), _ptr(o), st)
    _ffi.call("skyrl_delta_out", ref, _ptr(o), _ptr(proj), proj.stride(0), _ptr(norm_w), first_token, T, _ptr(out),
              out.stride(0), _code(proj), st)
    return out


# ---------------------------------------------------------------- differential attention
RUN = 8  # tokens per thread of the prompt's write


def diff_shape(heads, kv_heads, dim, vdim, rot_dims, taps, kv, scale, diff, eps) -> _ffi.DiffShape:
    """kv: the projection has keys and values (False: the layer reads another's)."""
    return _ffi.DiffShape(heads, kv_heads, dim, vdim, rot_dims, taps, int(kv), scale, diff, eps)


def diff_channels(sh) -> int:
    """Channels of the short convolutions: q | k | v."""
    return 2 * sh.heads * sh.dim + (sh.kv_heads * (2 * sh.dim + sh.vdim) if sh.kv else 0)


def diff_pads(sh):
    """(columns of a cached key or padded query row, rows of a cached value tile)."""
    return (sh.dim + 15) // 16 * 32, (sh.vdim + 15) // 16 * 16


def diff_mfma(sh, dtype) -> bool:
    """Whether the matrix kernels (split decode, prompt form) take the shape."""
    return bool(_ffi.query("skyrl_diff_mfma", ctypes.byref(sh), _DTYPES[dtype]))


def diff_runs_fit(sh, proj) -> bool:
    return (proj.dtype == torch.bfloat16 and sh.dim % 8 == 0 and sh.vdim % 8 == 0 and sh.taps <= 8
            and proj.stride(0) % 8 == 0 and proj.data_ptr() % 16 == 0)


def _check_diff_cache(sh, k_cache, v_cache, dtype):
    kw, vp = diff_pads(sh)
    _check(k_cache, "k_cache", dtype, (k_cache.shape[0], sh.kv_heads, 16, kw))
    _check(v_cache, "v_cache", dtype, (k_cache.shape[0], sh.kv_heads, vp, 16))


def diff_write(sh, proj, conv_t, cu, rows, bt_row, positions, slots, cos_sin, ring, k_cache, v_cache,
               save_conv: bool = False, q=None, first: int = 0, count: Optional[int] = None, runs=None) -> torch.Tensor:
    """Convolution, rotation, queries out [T, heads, padded], keys and values into the cache, for tokens
    [first, first + count) or, with `runs` int32 [n, 2] (mixers.run_plan), for those. conv_t f32 [taps,
    channels]; a given `q` is filled in place."""
    dev = _require_gpu(proj, conv_t, cu, rows, bt_row, positions, slots, cos_sin, ring, k_cache, v_cache, runs, q)
    T, n, ch = proj.shape[0], rows.shape[0], diff_channels(sh)
    if proj.dim() != 2 or proj.shape[1] < ch or proj.stride(1) != 1:
        raise ValueError(f"proj must be [T, >= {ch}] with unit column stride")
    _check(conv_t, "conv_t", torch.float32, (sh.taps, ch))
    _check(cu, "cu", torch.int32, (n + 1,))
    _check(rows, "rows", torch.int32, (n,))
    _check(bt_row, "bt_row", torch.int32, (T,))
    _check(positions, "positions", torch.int64, (T,))
    _check(slots, "slots", torch.int64, (T,))
    if cos_sin.dim() != 2 or cos_sin.shape[1] != sh.rot_dims:
        raise ValueError("cos_sin must be [max_pos, rot_dims]")
    _check(cos_sin, "cos_sin", torch.float32)
    _check(ring, "ring", proj.dtype, (ring.shape[0], sh.taps, ch))
    _check_diff_cache(sh, k_cache, v_cache, proj.dtype)
    kw = diff_pads(sh)[0]
    if q is None:
        make = torch.empty if kw == 2 * sh.dim else torch.zeros  # the padding must be zero
        q = make((T, sh.heads, kw), dtype=proj.dtype, device=dev)
    _check(q, "q", proj.dtype, (T, sh.heads, kw))
    ref, st = ctypes.byref(sh), _stream(dev)
    args = (ref, _ptr(proj), proj.stride(0), _ptr(conv_t), _ptr(cu), _ptr(rows), _ptr(bt_row), _ptr(positions),
            _ptr(slots), _ptr(cos_sin), _ptr(ring))
    if runs is not None:
        _check(runs, "runs", torch.int32, (runs.shape[0], 2))
        for a in range(0, runs.shape[0], 65535):  # the grid's limit
            part = runs[a:a + 65535]
            _ffi.call("skyrl_diff_write_runs", *args, _ptr(part), part.shape[0], _ptr(q), _ptr(k_cache), _ptr(v_cache),
                      st)
        return q
    count = T - first if count is None else count
    if not 0 <= first <= first + count <= T:
        raise ValueError("diff_write: token range outside the step")
    _ffi.call("skyrl_diff_write", *args, int(save_conv), first, count, _ptr(q), _ptr(k_cache), _ptr(v_cache),
              _code(proj), st)
    return q


def diff_workspace_bytes(sh, tokens: int, nparts: int) -> int:
    return int(_ffi.query("skyrl_diff_attend_workspace_bytes", ctypes.byref(sh), tokens, nparts))


def _check_diff_io(sh, q, gate, lam, out):
    T = q.shape[0]
    _check(q, "q", q.dtype, (T, sh.heads, diff_pads(sh)[0]))
    _check_view(gate, "gate", q.dtype, (T, sh.heads))
    _check(lam, "lambda", torch.float32, (1,))
    _check_view(out, "out", q.dtype, (T, sh.heads * sh.vdim))


def diff_attend(sh, q, gate, k_cache, v_cache, block_tables, bt_row, positions, lam, out, nparts: int = 1,
                part_min: int = 64, workspace=None) -> torch.Tensor:
    """One query row per token over its sequence's pages; gate [T, heads] before its sigmoid."""
    dev = _require_gpu(q, gate, k_cache, v_cache, block_tables, bt_row, positions, lam, out)
    T = q.shape[0]
    _check_diff_io(sh, q, gate, lam, out)
    _check_diff_cache(sh, k_cache, v_cache, q.dtype)
    _check_table(block_tables, bt_row, positions, T)
    ws = None
    if nparts > 1 and diff_mfma(sh, q.dtype):
        need = diff_workspace_bytes(sh, T, nparts)
        ws = workspace.get(need) if workspace is not None else torch.empty(need, dtype=torch.uint8, device=dev)
    else:
        nparts = 1
    _ffi.call("skyrl_diff_attend", ctypes.byref(sh), _ptr(q), _ptr(gate), gate.stride(0), _ptr(k_cache), _ptr(v_cache),
              _ptr(block_tables), block_tables.stride(0), _ptr(bt_row), _ptr(positions), T, _ptr(lam), part_min, nparts,
              _ptr(out), out.stride(0), _ptr(ws), _code(q), _stream(dev))
    return out


def diff_prefill(sh, q, gate, k_cache, v_cache, block_tables, tiles, lam, out) -> torch.Tensor:
    """Prompt tiles int32 [n, 4] (mixers.tile_plan) over their sequences' pages, which already hold the
    portion's own keys and values."""
    dev = _require_gpu(q, gate, k_cache, v_cache, block_tables, tiles, lam, out)
    _check_diff_io(sh, q, gate, lam, out)
    _check_diff_cache(sh, k_cache, v_cache, torch.bfloat16)
    if block_tables.dtype != torch.int32 or block_tables.dim() != 2 or block_tables.stride(1) != 1:
        raise ValueError("block_tables must be int32 [n, blocks] with unit column stride")
    _check(tiles, "tiles", torch.int32, (tiles.shape[0], 4))
    _ffi.call("skyrl_diff_prefill", ctypes.byref(sh), _ptr(q), _ptr(gate), gate.stride(0), _ptr(k_cache),
              _ptr(v_cache), _ptr(block_tables), block_tables.stride(0), _ptr(tiles), tiles.shape[0], _ptr(lam),
              _ptr(out), out.stride(0), _stream(dev))
    return out


# ---------------------------------------------------------------- short convolutions of prompts
def _check_steps(cu, rows, positions, T: Optional[int] = None):
    n = rows.shape[0]
    _check(rows, "rows", torch.int32, (n,))
    _check(cu, "cu", torch.int32, (n + 1,))
    _check(positions, "positions", torch.int64, (positions.shape[0] if T is None else T,))
    return n


def conv_chunk(x: torch.Tensor, conv_t: torch.Tensor, bias: Optional[torch.Tensor], silu: bool, chunk, cu, rows,
               positions, ring, sections) -> None:
    """Convolution, bias and activation of x's first columns at the tokens of `chunk` int32 [n, 4]
    (mixers.chunk_plan). sections: (units, size, padded, rows or None, cols or None) over consecutive channels,
    rows [T, units, padded], cols [chunks, units, padded, CHUNK] in x's type."""
    dev = _require_gpu(x, conv_t, bias, chunk, cu, rows, positions, ring)
    taps, ch = conv_t.shape
    T, nc = x.shape[0], chunk.shape[0]
    if x.dim() != 2 or x.shape[1] < ch or (ch > 1 and x.stride(1) != 1):
        raise ValueError(f"x must be [T, >= {ch}] with unit column stride")
    _check(conv_t, "conv_t", torch.float32)
    _check(bias, "bias", torch.float32, (ch,))
    _check(chunk, "chunk", torch.int32, (nc, 4))
    _check_steps(cu, rows, positions, T)
    _check(ring, "ring", x.dtype, (ring.shape[0], taps, ch))
    sec = (_ffi.ConvSection * len(sections))()
    for i, (units, size, padded, by_row, by_col) in enumerate(sections):
        _check(by_row, "rows of a section", x.dtype, (T, units, padded))
        _check(by_col, "cols of a section", x.dtype, (nc, units, padded, CHUNK))
        sec[i] = _ffi.ConvSection(units, size, padded, *(None if t is None else t.data_ptr() for t in (by_row, by_col)))
    for a in range(0, nc, 65535):  # the grid's limit
        n = min(65535, nc - a)
        part = (_ffi.ConvSection * len(sections))()
        for i, s in enumerate(sec):
            cols = sections[i][4]
            part[i] = _ffi.ConvSection(s.units, s.size, s.padded, s.rows, None if cols is None else cols[a:].data_ptr())
        _ffi.call("skyrl_conv_chunk", _ptr(x), x.stride(0), ch, taps, _ptr(conv_t), _ptr(bias), int(silu),
                  _ptr(chunk[a:a + n]), n, _ptr(cu), _ptr(rows), _ptr(positions), _ptr(ring), part, len(sections),
                  _code(x), _stream(dev))


# ---------------------------------------------------------------- gated linear recurrence
def rglru_pads(width: int, blocks: int):
    """(padded outputs, padded inputs) of a block's gate matrices."""
    size = width // blocks
    return (size + 15) // 16 * 16, (size + 31) // 32 * 32


def _check_rglru(proj, width, blocks, gate_w, gate_b, rate, state, out):
    T = proj.shape[0]
    if proj.dim() != 2 or proj.shape[1] < 2 * width or proj.stride(1) != 1:
        raise ValueError(f"proj must be [T, >= {2 * width}] with unit column stride")
    _check(gate_w, "gate_w", proj.dtype, (blocks, 2) + rglru_pads(width, blocks))
    _check(gate_b, "gate_b", torch.float32, (2, width))
    _check(rate, "rate", torch.float32, (width,))
    _check(state, "state", torch.float32, (state.shape[0], width))
    _check_view(out, "out", proj.dtype, (T, width))


def rglru_step(proj, width: int, blocks: int, conv_t, conv_b, gate_w, gate_b, rate, rows, positions, state, ring,
               out) -> None:
    """One token per sequence: state and ring updated in place."""
    dev = _require_gpu(proj, conv_t, conv_b, gate_w, gate_b, rate, rows, positions, state, ring, out)
    n, taps = proj.shape[0], conv_t.shape[0]
    _check_rglru(proj, width, blocks, gate_w, gate_b, rate, state, out)
    _check(conv_t, "conv_t", torch.float32, (taps, width))
    _check(conv_b, "conv_b", torch.float32, (width,))
    _check(rows, "rows", torch.int32, (n,))
    _check(positions, "positions", torch.int64, (n,))
    _check(ring, "ring", proj.dtype, (state.shape[0], taps, width))
    _ffi.call("skyrl_rglru_step", _ptr(proj), proj.stride(0), width, blocks, taps, _ptr(conv_t), _ptr(conv_b),
              _ptr(gate_w), _ptr(gate_b), _ptr(rate), _ptr(rows), _ptr(positions), n, _ptr(state), _ptr(ring), _ptr(out),
              out.stride(0), _code(proj), _stream(dev))


def rglru_workgroups(width: int, blocks: int) -> int:
    """Workgroups per run of chunks of the prompt form: 64 columns of a block each."""
    return blocks * ((rglru_pads(width, blocks)[0] + 63) // 64)


def rglru_prompt(proj, width: int, blocks: int, u, gate_w, gate_b, rate, chunk, runs, seq_runs, seq0: int, cu, rows,
                 positions, state, out) -> None:
    """Tokens of the chunks, of the sequences from seq0 on (mixers.chunk_runs); u [T, width] is
    conv_chunk's."""
    dev = _require_gpu(proj, u, gate_w, gate_b, rate, chunk, runs, seq_runs, cu, rows, positions, state, out)
    T, nc, nr = proj.shape[0], chunk.shape[0], runs.shape[0]
    _check_rglru(proj, width, blocks, gate_w, gate_b, rate, state, out)
    n = _check_steps(cu, rows, positions, T) - seq0
    _check(u, "u", proj.dtype, (T, width))
    _check(chunk, "chunk", torch.int32, (nc, 4))
    _check(runs, "runs", torch.int32, (nr, 4))
    _check(seq_runs, "seq_runs", torch.int32, (n + 1,))
    h, a = (torch.empty((T, width), dtype=torch.float32, device=dev) for _ in range(2))
    s_in = torch.empty((nr, width), dtype=torch.float32, device=dev)
    _ffi.call("skyrl_rglru_prompt", _ptr(proj), proj.stride(0), width, blocks, _ptr(u), _ptr(gate_w), _ptr(gate_b),
              _ptr(rate), _ptr(chunk), nc, _ptr(runs), nr, _ptr(seq_runs), seq0, n, _ptr(cu), _ptr(rows), _ptr(positions), _ptr(state),
              _ptr(h), _ptr(a), _ptr(s_in), _ptr(out), out.stride(0), _code(proj), _stream(dev))


# ---------------------------------------------------------------- windowed attention with an output gate
def attn_shape(heads, kv_heads, dim, vdim, window, scale, eps) -> _ffi.AttnShape:
    return _ffi.AttnShape(heads, kv_heads, dim, vdim, int(window or 0), scale, eps)


def attn_channels(sh) -> int:
    """Columns of the projection: q | k | v."""
    return (sh.heads + sh.kv_heads) * sh.dim + sh.kv_heads * sh.vdim


def attn_pads(sh):
    """(columns of a cached key or padded query row, rows of a cached value tile)."""
    return (sh.dim + 31) // 32 * 32, (sh.vdim + 15) // 16 * 16


def attn_mfma(sh, dtype) -> bool:
    """Whether the matrix kernels (split decode, prompt form) take the shape."""
    return bool(_ffi.query("skyrl_attn_mfma", ctypes.byref(sh), _DTYPES[dtype]))


def attn_runs_fit(sh, proj) -> bool:
    return (proj.dtype == torch.bfloat16 and sh.dim % 8 == 0 and sh.dim <= 512 and sh.vdim % 8 == 0
            and proj.stride(0) % 8 == 0 and proj.data_ptr() % 16 == 0)


def _check_attn_cache(sh, k_cache, v_cache, dtype):
    dp, vp = attn_pads(sh)
    _check(k_cache, "k_cache", dtype, (k_cache.shape[0], sh.kv_heads, 16, dp))
    _check(v_cache, "v_cache", dtype, (k_cache.shape[0], sh.kv_heads, vp, 16))


def attn_write(sh, proj, q_norm, k_norm, slots, k_cache, v_cache, q=None, count: Optional[int] = None,
               runs=None) -> torch.Tensor:
    """Normed queries out [T, heads, padded], normed keys and values into the cache, for the first `count` tokens
    or, with `runs` int32 [n, 2] (mixers.run_plan), for those. A given `q` is filled in place."""
    dev = _require_gpu(proj, q_norm, k_norm, slots, k_cache, v_cache, q, runs)
    T, dp = proj.shape[0], attn_pads(sh)[0]
    if proj.dim() != 2 or proj.shape[1] < attn_channels(sh) or proj.stride(1) != 1:
        raise ValueError(f"proj must be [T, >= {attn_channels(sh)}] with unit column stride")
    _check(q_norm, "q_norm", proj.dtype, (sh.dim,))
    _check(k_norm, "k_norm", proj.dtype, (sh.dim,))
    _check(slots, "slots", torch.int64, (T,))
    _check_attn_cache(sh, k_cache, v_cache, proj.dtype)
    if q is None:
        make = torch.empty if dp == sh.dim else torch.zeros  # the padding must be zero
        q = make((T, sh.heads, dp), dtype=proj.dtype, device=dev)
    _check(q, "q", proj.dtype, (T, sh.heads, dp))
    if runs is not None:
        _check(runs, "runs", torch.int32, (runs.shape[0], 2))
        n = runs.shape[0]
    else:
        n = T if count is None else count
        if not 0 <= n <= T:
            raise ValueError("attn_write: token range outside the step")
    _ffi.call("skyrl_attn_write", ctypes.byref(sh), _ptr(proj), proj.stride(0), _ptr(q_norm), _ptr(k_norm), _ptr(slots),
              _ptr(runs), 0, n, _ptr(q), _ptr(k_cache), _ptr(v_cache), _code(proj), _stream(dev))
    return q


def attn_workspace_bytes(sh, tokens: int, nparts: int) -> int:
    return int(_ffi.query("skyrl_attn_attend_workspace_bytes", ctypes.byref(sh), tokens, nparts))


def _check_attn_io(sh, q, gate, out):
    T = q.shape[0]
    _check(q, "q", q.dtype, (T, sh.heads, attn_pads(sh)[0]))
    _check_view(gate, "gate", q.dtype, (T, sh.heads * sh.vdim))
    _check_view(out, "out", q.dtype, (T, sh.heads * sh.vdim))


def attn_attend(sh, q, gate, k_cache, v_cache, block_tables, bt_row, positions, out, nparts: int = 1,
                part_min: int = 64, workspace=None) -> torch.Tensor:
    """One query row per token over its window's pages; gate [T, heads * vdim] before its sigmoid."""
    dev = _require_gpu(q, gate, k_cache, v_cache, block_tables, bt_row, positions, out)
    T = q.shape[0]
    _check_attn_io(sh, q, gate, out)
    _check_attn_cache(sh, k_cache, v_cache, q.dtype)
    _check_table(block_tables, bt_row, positions, T)
    ws = None
    if nparts > 1 and attn_mfma(sh, q.dtype):
        need = attn_workspace_bytes(sh, T, nparts)
        ws = workspace.get(need) if workspace is not None else torch.empty(need, dtype=torch.uint8, device=dev)
    else:
        nparts = 1
    _ffi.call("skyrl_attn_attend", ctypes.byref(sh), _ptr(q), _ptr(gate), gate.stride(0), _ptr(k_cache), _ptr(v_cache),
              _ptr(block_tables), block_tables.stride(0), _ptr(bt_row), _ptr(positions), T, part_min, nparts, _ptr(out),
              out.stride(0), _ptr(ws), _code(q), _stream(dev))
    return out


def attn_prefill(sh, q, gate, k_cache, v_cache, block_tables, tiles, out) -> torch.Tensor:
    """Prompt tiles int32 [n, 4] (mixers.tile_plan) over their sequences' pages, which already hold the
    portion's own keys and values."""
    dev = _require_gpu(q, gate, k_cache, v_cache, block_tables, tiles, out)
    _check_attn_io(sh, q, gate, out)
    _check_attn_cache(sh, k_cache, v_cache, torch.bfloat16)
    if block_tables.dtype != torch.int32 or block_tables.dim() != 2 or block_tables.stride(1) != 1:
        raise ValueError("block_tables must be int32 [n, blocks] with unit column stride")
    _check(tiles, "tiles", torch.int32, (tiles.shape[0], 4))
    _ffi.call("skyrl_attn_prefill", ctypes.byref(sh), _ptr(q), _ptr(gate), gate.stride(0), _ptr(k_cache),
              _ptr(v_cache), _ptr(block_tables), block_tables.stride(0), _ptr(tiles), tiles.shape[0], _ptr(out),
              out.stride(0), _stream(dev))
    return out


# ---------------------------------------------------------------- state space mixer
def ssd_shape(heads, vdim, state, groups, taps) -> _ffi.SSDShape:
    return _ffi.SSDShape(heads, vdim, state, groups, taps)


def ssd_channels(sh) -> int:
    """Channels of the short convolution: x | B | C."""
    return sh.heads * sh.vdim + 2 * sh.groups * sh.state


def ssd_width(sh) -> int:
    """Columns of the projection: z | x | B | C | dt."""
    return sh.heads * sh.vdim + ssd_channels(sh) + sh.heads


def ssd_ppad(sh) -> int:
    return (sh.vdim + 3) // 4 * 4


def ssd_prompt_fits(sh, dtype) -> bool:
    return dtype == torch.bfloat16 and sh.state <= 256


def ssd_slices(sh) -> int:
    """Workgroups per head of the prompt form: 64 value columns each."""
    return (sh.vdim + 63) // 64


def _check_ssd(sh, proj, conv_t, conv_b, a_log, dt_bias, skip, state, ring, y):
    T, ch = proj.shape[0], ssd_channels(sh)
    if proj.dim() != 2 or proj.shape[1] < ssd_width(sh) or proj.stride(1) != 1:
        raise ValueError(f"proj must be [T, >= {ssd_width(sh)}] with unit column stride")
    _check(conv_t, "conv_t", torch.float32, (sh.taps, ch))
    _check(conv_b, "conv_b", torch.float32, (ch,))
    for t, name in ((a_log, "a_log"), (dt_bias, "dt_bias"), (skip, "skip")):
        _check(t, name, torch.float32, (sh.heads,))
    _check(state, "state", torch.float32, (state.shape[0], sh.heads, sh.state, ssd_ppad(sh)))
    _check(ring, "ring", proj.dtype, (state.shape[0], sh.taps, ch))
    _check_view(y, "y", proj.dtype, (T, sh.heads * sh.vdim))


def ssd_scan(sh, proj, conv_t, conv_b, a_log, dt_bias, skip, cu, rows, positions, state, ring, save_conv, y) -> None:
    """Token by token over each sequence's tokens [cu[s], cu[s + 1]) into y [T, heads * vdim], before the gated
    norm; state and (save_conv: one token per sequence) convolution inputs updated in place."""
    dev = _require_gpu(proj, conv_t, conv_b, a_log, dt_bias, skip, cu, rows, positions, state, ring, y)
    _check_ssd(sh, proj, conv_t, conv_b, a_log, dt_bias, skip, state, ring, y)
    n = _check_steps(cu, rows, positions, proj.shape[0])
    _ffi.call("skyrl_ssd_scan", ctypes.byref(sh), _ptr(proj), proj.stride(0), _ptr(conv_t), _ptr(conv_b), _ptr(a_log),
              _ptr(dt_bias), _ptr(skip), _ptr(cu), _ptr(rows), _ptr(positions), n, _ptr(state), _ptr(ring),
              int(save_conv), _ptr(y), y.stride(0), _code(proj), _stream(dev))


def ssd_prompt(sh, proj, conv_t, conv_b, a_log, dt_bias, skip, cu, rows, positions, state, ring, chunk, super_, pick,
               chain, y) -> None:
    """Chunked form over the chunks int32 [n, 4] and runs of chunks (mixers.walk_plan); `state` is updated in
    place, the convolution inputs are conv_save's."""
    dev = _require_gpu(proj, conv_t, conv_b, a_log, dt_bias, skip, cu, rows, positions, state, ring, chunk, super_, pick,
                       chain, y)
    _check_ssd(sh, proj, conv_t, conv_b, a_log, dt_bias, skip, state, ring, y)
    T, nc, ns = proj.shape[0], chunk.shape[0], super_.shape[0]
    _check(super_, "super", torch.int32, (ns, 4))
    _check(pick, "pick", torch.int32, (pick.shape[0],))
    _check(chain, "chain", torch.int32, (chain.shape[0], 2))
    H, P, N, G = sh.heads, sh.vdim, sh.state, sh.groups
    vp, np_, inner = (P + 15) // 16 * 16, (N + 31) // 32 * 32, H * P
    make = torch.empty if (vp, np_) == (P, N) else torch.zeros  # padding meets the other operand: zero
    xt, bt = (make(s, dtype=proj.dtype, device=dev) for s in ((nc, H, vp, CHUNK), (nc, G, np_, CHUNK)))
    brow, crow = (make((T, G, np_), dtype=proj.dtype, device=dev) for _ in range(2))
    conv_chunk(proj[:, inner:], conv_t, conv_b, True, chunk, cu, rows, positions, ring,
               ((H, P, vp, None, xt), (G, N, np_, brow, bt), (G, N, np_, crow, None)))
    multi = pick.shape[0] > 0
    runs = torch.empty((ns if multi else 1, H, np_, vp), dtype=torch.float32, device=dev)
    scores = torch.empty((nc, G, 10, 256), dtype=torch.float32, device=dev)
    gtot = torch.empty((ns if multi else 1, H), dtype=torch.float32, device=dev)
    dt = proj[:, inner + ssd_channels(sh):]
    _ffi.call("skyrl_ssd_prompt", ctypes.byref(sh), _ptr(xt), _ptr(bt), _ptr(brow), _ptr(crow), _ptr(dt), dt.stride(0),
              _ptr(a_log), _ptr(dt_bias), _ptr(skip), _ptr(chunk), nc, _ptr(super_), ns, _ptr(pick), pick.shape[0],
              _ptr(chain), chain.shape[0], _ptr(cu), _ptr(rows), _ptr(positions), _ptr(state), _ptr(scores), _ptr(runs),
              _ptr(gtot), _ptr(y), y.stride(0), _stream(dev))


def gated_norm(y: torch.Tensor, z: torch.Tensor, weight: torch.Tensor, groups: int, eps: float,
               out: torch.Tensor) -> torch.Tensor:
    """rms over each of `groups` equal parts of y silu(z), times weight; y, z and out may be column ranges."""
    dev = _require_gpu(y, z, weight, out)
    n, W = y.shape
    for t, name in ((y, "y"), (z, "z"), (out, "out")):
        _check_view(t, name, weight.dtype, (n, W))
    _check(weight, "weight", weight.dtype, (W,))
    _ffi.call("skyrl_gated_norm", _ptr(y), y.stride(0), _ptr(z), z.stride(0), _ptr(weight), n, W, groups, float(eps),
              _ptr(out), out.stride(0), _code(weight), _stream(dev))
    return out


# ---------------------------------------------------------------- generalized delta rule
def gdelta_shape(heads, dim, eps) -> _ffi.GeneralDeltaShape:
    if not 0 < dim <= 256:
        raise ValueError("the generalized delta rule takes a dim of at most 256")
    return _ffi.GeneralDeltaShape(heads, dim, eps)


def gdelta_vpad(sh) -> int:
    return (sh.dim + 3) // 4 * 4


def _check_gdelta(sh, proj, wl, w0, a_bias, norm_w, cu, rows, positions, state, out):
    T, n, HD = proj.shape[0], rows.shape[0], sh.heads * sh.dim
    if proj.dim() != 2 or proj.shape[1] < 5 * HD or proj.stride(1) != 1:
        raise ValueError(f"proj must be [T, >= {5 * HD}] with unit column stride")
    _check_view(wl, "wl", proj.dtype, (T, HD))
    _check(w0, "w0", torch.float32, (HD,))
    _check(a_bias, "a_bias", torch.float32, (HD,))
    _check(norm_w, "norm_w", proj.dtype, (HD,))
    _check(rows, "rows", torch.int32, (n,))
    _check(cu, "cu", torch.int32, (n + 1,))
    _check(positions, "positions", torch.int64, (T,))
    _check(state, "state", torch.float32, (state.shape[0], sh.heads, sh.dim, gdelta_vpad(sh)))
    _check_view(out, "out", proj.dtype, (T, HD))
    return n


def gdelta_scan(sh, proj, wl, w0, a_bias, norm_w, cu, rows, positions, state, out) -> torch.Tensor:
    """Token by token over each sequence's tokens [cu[s], cu[s + 1]); state updated in place. proj [T, >= 5 heads dim]:
    r | k | v | output gate | removal rate; wl [T, heads dim] the decay logits."""
    dev = _require_gpu(proj, wl, w0, a_bias, norm_w, cu, rows, positions, state, out)
    n = rows.shape[0]
    if cu.shape[0] != n + 1:
        raise ValueError("cu must be [sequences + 1]")
    _check_gdelta(sh, proj, wl, w0, a_bias, norm_w, cu, rows, positions, state, out)
    _ffi.call("skyrl_gdelta_scan", ctypes.byref(sh), _ptr(proj), proj.stride(0), _ptr(wl), wl.stride(0), _ptr(w0),
              _ptr(a_bias), _ptr(norm_w), _ptr(cu), _ptr(rows), _ptr(positions), n, _ptr(state), _ptr(out), out.stride(0),
              _code(proj), _stream(dev))
    return out


def gdelta_prompt(sh, proj, wl, w0, a_bias, norm_w, cu, rows, positions, state, chunk, seq_chunks, first_seq: int,
                  out) -> torch.Tensor:
    """Chunked form over the sequences from first_seq on: chunk int32 [n, 4] and seq_chunks int32 [sequences + 1]
    (mixers.chunk_plan). `state` is updated in place."""
    dev = _require_gpu(proj, wl, w0, a_bias, norm_w, cu, rows, positions, state, chunk, seq_chunks, out)
    n = _check_gdelta(sh, proj, wl, w0, a_bias, norm_w, cu, rows, positions, state, out)
    nc, nseq, HD = chunk.shape[0], n - first_seq, sh.heads * sh.dim
    _check(chunk, "chunk", torch.int32, (nc, 4))
    _check(seq_chunks, "seq_chunks", torch.int32, (nseq + 1,))
    d16 = (sh.dim + 15) // 16 * 16
    f32 = lambda *tail: torch.empty((nc, sh.heads) + tail, dtype=torch.float32, device=dev)  # noqa: E731
    M, N, S, R, O = f32(d16, d16), f32(d16, d16), f32(d16, d16), f32(CHUNK, d16), f32(CHUNK, d16)
    st, ref = _stream(dev), ctypes.byref(sh)
    _ffi.call("skyrl_gdelta_chunk", ref, _ptr(proj), proj.stride(0), _ptr(wl), wl.stride(0), _ptr(w0), _ptr(a_bias),
              _ptr(chunk), nc, _ptr(M), _ptr(N), _ptr(R), _ptr(O), _code(proj), st)
    _ffi.call("skyrl_gdelta_chain", ref, _ptr(chunk), _ptr(seq_chunks), first_seq, nseq, _ptr(cu), _ptr(rows),
              _ptr(positions), _ptr(M), _ptr(N), _ptr(state), _ptr(S), st)
    gate = proj[:, 3 * HD:4 * HD]
    _ffi.call("skyrl_gdelta_out", ref, _ptr(chunk), nc, _ptr(R), _ptr(O), _ptr(S), _ptr(gate), proj.stride(0), _ptr(norm_w),
              _ptr(out), out.stride(0), _code(proj), st)
    return out


# ---------------------------------------------------------------- routed experts
def moe_shape(width, ff, experts, top, groups=1, keep=1) -> _ffi.MoeShape:
    if not 0 < experts <= 1024 or groups <= 0 or experts % groups:
        raise ValueError("experts must be at most 1024 and a multiple of groups")
    if not 0 < keep <= groups or not 0 < top <= experts // groups * keep:
        raise ValueError("keep must be in [1, groups] and top at most the experts of the kept groups")
    return _ffi.MoeShape(width, ff, experts, top, groups, keep)


def moe_route(sh, x, router, correction):
    """(experts int32 [n, top], their scores f32 [n, top]) of every row of x."""
    dev = _require_gpu(x, router, correction)
    n = x.shape[0]
    _check(x, "x", x.dtype, (n, sh.width))
    _check(router, "router", x.dtype, (sh.experts, sh.width))
    _check(correction, "correction", torch.float32, (sh.experts,))
    idx = torch.empty((n, sh.top), dtype=torch.int32, device=dev)
    weight = torch.empty((n, sh.top), dtype=torch.float32, device=dev)
    _ffi.call("skyrl_moe_route", ctypes.byref(sh), _ptr(x), n, _ptr(router), _ptr(correction), _ptr(idx), _ptr(weight),
              _code(x), _stream(dev))
    return idx, weight


def moe_tile(sh, n: int) -> int:
    """Rows per tile of the experts' products for n tokens."""
    mean = n * sh.top / sh.experts
    return 256 if mean >= 112 else 128 if mean >= 48 else 64 if mean >= 12 else 16


def moe_sort(sh, idx, tm: int):
    """(order int32 [tiles, tm], tile_expert int32 [tiles + 1]): the (token, expert) pairs by expert; the last entry is
    the number of tiles in use."""
    dev = _require_gpu(idx)
    _check(idx, "idx", torch.int32, (idx.shape[0], sh.top))
    pairs = idx.numel()
    tiles = int(_ffi.query("skyrl_moe_tiles", sh.experts, pairs, tm))
    order = torch.empty((tiles, tm), dtype=torch.int32, device=dev)
    tile_expert = torch.empty((tiles + 1,), dtype=torch.int32, device=dev)
    scratch = int(_ffi.query("skyrl_moe_counts", sh.experts, pairs))
    counts = torch.empty((scratch,), dtype=torch.int32, device=dev) if scratch else None
    _ffi.call("skyrl_moe_sort", _ptr(idx), pairs, sh.experts, tm, tiles, _ptr(counts), _ptr(order), _ptr(tile_expert), _stream(dev))
    return order, tile_expert


def moe_experts(sh, x, idx, weight, gate_up, down, tm: Optional[int] = None) -> torch.Tensor:
    """Rows [n * top, width]: every pair's expert output times its weight. gate_up [experts, 2, ff, width], down
    [experts, width, ff]."""
    dev = _require_gpu(x, idx, weight, gate_up, down)
    n = x.shape[0]
    _check(x, "x", x.dtype, (n, sh.width))
    _check(idx, "idx", torch.int32, (n, sh.top))
    _check(weight, "weight", torch.float32, (n, sh.top))
    _check(gate_up, "gate_up", x.dtype, (sh.experts, 2, sh.ff, sh.width))
    _check(down, "down", x.dtype, (sh.experts, sh.width, sh.ff))
    tm = tm or moe_tile(sh, n)
    out = torch.empty((n * sh.top, sh.width), dtype=x.dtype, device=dev)
    if n == 0:
        return out
    order, tile_expert = moe_sort(sh, idx, tm)
    tiles = order.shape[0]
    act = torch.empty((tiles * tm, sh.ff), dtype=x.dtype, device=dev)
    ref, st = ctypes.byref(sh), _stream(dev)
    _ffi.call("skyrl_moe_gate_up", ref, _ptr(x), _ptr(gate_up), _ptr(order), _ptr(tile_expert), tm, tiles, _ptr(act),
              _code(x), st)
    _ffi.call("skyrl_moe_down", ref, _ptr(act), _ptr(down), _ptr(order), _ptr(tile_expert), tm, tiles, _ptr(weight),
              _ptr(out), _code(x), st)
    return out
