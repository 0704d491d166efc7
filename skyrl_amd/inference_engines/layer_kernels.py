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


def embed(tokens: torch.Tensor, table: torch.Tensor, scale: float) -> torch.Tensor:
    """f32 rows of the embedding table times scale."""
    dev = _require_gpu(tokens, table)
    n, H = tokens.shape[0], table.shape[1]
    _check(tokens, "tokens", torch.int64, (n,))
    _check(table, "table", table.dtype)
    out = torch.empty((n, H), dtype=torch.float32, device=dev)
    _ffi.call("skyrl_embed", _ptr(tokens), _ptr(table), n, H, float(scale), _ptr(out), _code(table), _stream(dev))
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


def latent_write(proj, heads, dim, rot_dim, rank, norm_weight, eps, positions, slots, cos_sin, cache) -> None:
    """Rotate the q parts of ``proj`` in place; write the normed latent and the rotated key part."""
    dev = _require_gpu(proj, norm_weight, positions, slots, cos_sin, cache)
    T = proj.shape[0]
    width = heads * (dim + rot_dim) + rank + rot_dim
    if proj.dim() != 2 or proj.shape[1] != width or proj.stride(1) != 1:
        raise ValueError(f"proj must be [T, {width}] with unit column stride")
    _check(norm_weight, "norm_weight", proj.dtype, (rank,))
    _check(positions, "positions", torch.int64, (T,))
    _check(slots, "slots", torch.int64, (T,))
    if cos_sin.dim() != 2 or cos_sin.shape[1] != rot_dim:
        raise ValueError("cos_sin must be [max_pos, rot_dim]")
    _check(cos_sin, "cos_sin", torch.float32)
    _check_cache(cache, rank, rot_dim, proj.dtype)
    _ffi.call("skyrl_latent_write", _ptr(proj), proj.stride(0), T, heads, dim, rot_dim, rank, _ptr(norm_weight),
              float(eps), _ptr(positions), _ptr(slots), _ptr(cos_sin), _ptr(cache), cache.shape[2], _code(proj),
              _stream(dev))


def latent_attend(qa, q_rot, cache, rank, rot_dim, block_tables, bt_row, positions, scale, window, nparts=1,
                  part_min=64, workspace=None) -> torch.Tensor:
    """Latent-space attention, one query row per token. qa [heads, T, rank]; q_rot [T, heads, rot_dim]
    (any token and head stride); returns [heads, T, rank]."""
    dev = _require_gpu(qa, q_rot, cache, block_tables, bt_row, positions)
    heads, T, R = qa.shape
    _check(qa, "qa", cache.dtype, (heads, T, rank))
    if q_rot.dtype != qa.dtype or tuple(q_rot.shape) != (T, heads, rot_dim) or (rot_dim > 1 and q_rot.stride(2) != 1):
        raise ValueError("q_rot must be [T, heads, rot_dim] with unit last stride")
    _check_cache(cache, rank, rot_dim, qa.dtype)
    _check_table(block_tables, bt_row, positions, T)
    out = torch.empty_like(qa)
    ws = None
    if nparts > 1 and mfma_attend(rank, rot_dim, qa.dtype):
        need = _ffi.query("skyrl_latent_attend_workspace_bytes", T, heads, rank, nparts)
        ws = workspace.get(need) if workspace is not None else torch.empty(need, dtype=torch.uint8, device=dev)
    else:
        nparts = 1
    _ffi.call("skyrl_latent_attend", _ptr(qa), _ptr(q_rot), q_rot.stride(0), q_rot.stride(1), _ptr(cache),
              cache.shape[2], _ptr(block_tables), block_tables.stride(0), _ptr(bt_row), _ptr(positions), T, heads,
              rank, rot_dim, float(scale), int(window or 0), part_min, nparts, _ptr(out), _ptr(ws), _code(qa),
              _stream(dev))
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


def latent_prefill(q, k_nope, k_rot, v_t, tiles, heads, dim, rot_dim, vdim, scale, window, out) -> torch.Tensor:
    """Windowed attention of prompt tiles over packed keys. q [T, >= heads * (dim + rot_dim)]; k_nope
    [rows, heads * dim]; k_rot [rows, rot_dim]; v_t [heads * vdim, rows]; out [T, heads * vdim]."""
    dev = _require_gpu(q, k_nope, k_rot, v_t, tiles, out)
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
    _ffi.call("skyrl_latent_prefill", _ptr(q), q.stride(0), _ptr(k_nope), k_nope.stride(0), _ptr(k_rot), _ptr(v_t),
              v_t.stride(0), _ptr(tiles), tiles.shape[0], heads, dim, rot_dim, vdim, float(scale), int(window or 0),
              _ptr(out), out.stride(0), _stream(dev))
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
