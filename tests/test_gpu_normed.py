"""Gated linear recurrences, windowed attention beside a state space mixer, output norms and xIELU (Foduzen) on
the GPU: every kernel alone, then the model through the engine's own steps, against the plain restatement in
oracle/hybrid_ref.py. Tolerances as in test_gpu_hybrid.py."""

import asyncio
import io
import json
import math

import numpy as np
import pytest
import torch

from hybrid_cases import NORMED, attend, make_normed_weights, normed_config, rglru, side, ssd
from hybrid_gpu import DEV, DTYPES, build, close, feed, generate, greedy, model_close, rms, rnd, tokens_of
from oracle import hybrid_ref as ref
from skyrl_amd.inference_engines import layer_kernels as lk
from skyrl_amd.inference_engines import mixers
from skyrl_amd.inference_engines.engine import AMDInferenceEngine
from skyrl_amd.inference_engines.trace import TraceSession

pytestmark = pytest.mark.gpu
BS = mixers.BLOCK_SIZE
BF16 = torch.bfloat16
dev = lambda t: None if t is None else t.to(DEV)  # noqa: E731


# ---------------------------------------------------------------- embedding, norms, activation
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [72, 1, 515, 130])
def test_embed_with_position_vectors(H, dtype):
    g = torch.Generator().manual_seed(H)
    table, tok = rnd(g, 31, H, dtype=dtype), torch.tensor([3, 0, 30, 3, 17, 5])
    pos = torch.tensor([0, 1, 2, 77, 8191, 262143])
    turns = 500.0 ** (-2.0 * torch.arange((H + 1) // 2, dtype=torch.float64) / H) / (2 * math.pi)
    x = torch.empty((6, H), dtype=dtype, device=DEV)
    h = lk.embed(dev(tok), dev(table), 2.3, dev(pos), dev(turns), x)
    want = table[tok].double() * 2.3 + ref.sinusoid(pos, H, 500.0)
    assert float((h.double().cpu() - want).abs().max()) < 3e-6 * max(1, float(want.abs().max()))
    close(x, want, dtype, f32=1e-6, bf16=4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [72, 1, 515, 2056, 4100, 8192])
def test_norm_add(H, dtype):
    """One output or two, one number or a vector as the weight, with and without the final norm."""
    g = torch.Generator().manual_seed(H)
    vec = lambda: rnd(g, H, dtype=dtype, scale=0.5) + 1  # noqa: E731
    eps, share = 3e-3, 0.37
    for k, (pair, weight, final) in enumerate(((False, rnd(g, dtype=dtype), None), (True, rnd(g, dtype=dtype), None),
                                               (False, vec(), rnd(g, dtype=dtype)), (True, vec(), vec()))):
        a, b, h = (rnd(g, 5, H, scale=s) for s in (3.0, 0.2, 2.0))
        a, b, wa, wb = a.to(dtype), b.to(dtype), vec(), vec()
        a[3] = 0
        m = a.double() if not pair else share * (ref.rms_norm(a.double(), wa.double(), eps) + ref.rms_norm(b.double(), wb.double(), eps))
        want = h.double() + ref.rms_norm(m, weight.double(), eps)
        hd = dev(h)
        out = lk.norm_add((dev(a), dev(b)) if pair else dev(a), hd, dev(weight), eps, final=dev(final),
                          **({"pair": (dev(wa), dev(wb)), "share": share} if pair else {}))
        close(hd, want, torch.float32, f32=2e-6)
        close(out, want if final is None else ref.rms_norm(want, final.double(), eps), dtype, f32=1e-5, bf16=4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff,pad", [(100, 0), (33, 3), (64, 8)])
def test_xielu_in_column_ranges(ff, pad, dtype):
    g = torch.Generator().manual_seed(ff)
    wide = rnd(g, 9, ff + 2 * pad, dtype=dtype, scale=3.0)
    wide[0, :pad + 5] = 0
    pq = torch.tensor([0.7, -1.3]).to(dtype)
    out = torch.full((9, ff + 2 * pad), 7.0, dtype=dtype, device=DEV)
    lk.xielu(dev(wide)[:, pad:pad + ff], dev(pq), out=out[:, pad:pad + ff])
    close(out[:, pad:pad + ff], ref.xielu(wide[:, pad:pad + ff].double(), *pq.double()), dtype, f32=1e-5, bf16=4e-3)
    assert bool((out[:, :pad] == 7).all()) and bool((out[:, pad + ff:] == 7).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,groups,pad", [(72, 1, 0), (60, 4, 3), (4096, 8, 8), (8200, 1, 0), (6144, 3, 0), (9, 9, 1)])
def test_gated_norm(width, groups, pad, dtype):
    g = torch.Generator().manual_seed(width)
    y, z, w = (rnd(g, *s, dtype=dtype, scale=k) for s, k in (((7, width), 0.1), ((7, width + 2 * pad), 2.0), ((width,), 1.0)))
    out = torch.full((7, width + 2 * pad), 7.0, dtype=dtype, device=DEV)
    lk.gated_norm(dev(y), dev(z)[:, pad:pad + width], dev(w), groups, 1e-3, out[:, pad:pad + width])
    want = ref.grouped_gated_norm(y.double(), z[:, pad:pad + width].double(), w.double(), groups, 1e-3)
    close(out[:, pad:pad + width], want, dtype, f32=1e-5, bf16=5e-3)
    assert bool((out[:, :pad] == 7).all()) and bool((out[:, pad + width:] == 7).all())


# ---------------------------------------------------------------- sequences cut into steps
CUTS = [  # steps of two sequences (61 and 150 tokens): tokens of each, 0: not in the step
    [(1, 2), (2, 33), (1, 1), (0, 1), (40, 3), (3, 71), (14, 39)],
    [(61, 150)], [(0, 150), (61, 0)], [(2, 64), (31, 65), (28, 21)]]


class Steps:
    """Feeds two sequences' rows in steps; state rows start full of other values, an idle row is in the batch of
    one-token steps."""

    lens, rows = (61, 150), (2, 0)

    def __init__(self, inputs, dtype):
        self.u, self.dtype, self.out = inputs, dtype, [[], []]

    def run(self, cuts, step):
        """step(x, cu, rows, positions, lens, starts) -> outputs of the step's tokens."""
        at = [0, 0]
        for c in cuts:
            parts = [(i, n) for i, n in enumerate(c) if n]
            one = all(n == 1 for _, n in parts)
            lens, starts, rows = [n for _, n in parts], [at[i] for i, _ in parts], [self.rows[i] for i, _ in parts]
            x = [self.u[i][at[i]:at[i] + n] for i, n in parts]
            if one:  # an idle row in front
                lens, starts, rows, x = [1] + lens, [0] + starts, [-1] + rows, [self.u[0][:1]] + x
            pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)])
            cu = torch.tensor([0] + lens).cumsum(0).int()
            out = step(dev(torch.cat(x)), dev(cu), dev(torch.tensor(rows, dtype=torch.int32)), dev(pos), lens, starts)
            for (i, n), t in zip(parts, out.split(lens)[1 if one else 0:]):
                self.out[i].append(t)
                at[i] += n
        assert tuple(at) == self.lens
        return [torch.cat(o) for o in self.out]


def plan_of(fn, *args):
    return [torch.from_numpy(a).to(DEV) for a in fn(*args)]


# ---------------------------------------------------------------- short convolution of prompts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", CUTS[1:])
@pytest.mark.parametrize("units,taps,silu", [(((2, 24, 24), (1, 16, 32), (3, 8, 8)), 4, True), (((3, 20, 32), (2, 7, 9)), 3, False),
                                             (((1, 72, 72),), 8, False), (((5, 8, 16), (1, 40, 48)), 11, True),
                                             (((1, 50, 50),), 1, True), (((1, 264, 264),), 2, False)])
def test_conv_chunk(units, taps, silu, cuts, dtype):
    ch = sum(u * s for u, s, _ in units)
    g = torch.Generator().manual_seed(ch)
    conv, bias = rnd(g, ch, taps, dtype=dtype), rnd(g, ch)
    seqs = Steps([rnd(g, n, ch + 8, dtype=dtype) for n in Steps.lens], dtype)
    ring = torch.full((3, taps, ch), 9.0, dtype=dtype, device=DEV)

    def step(x, cu, rows, pos, lens, starts):
        chunk, _ = plan_of(mixers.chunk_plan, lens, 0, 0)
        T, nc = len(x), len(chunk)
        make = lambda *s: torch.full(s, 5.0, dtype=dtype, device=DEV)  # noqa: E731
        sec = [(u, s, p, make(T, u, p), make(nc, u, p, lk.CHUNK)) for u, s, p in units]
        lk.conv_chunk(x, dev(conv.t().float().contiguous()), dev(bias), silu, chunk, cu, rows, pos, ring, sec)
        lk.conv_save(x, ch, cu, rows, pos, ring)
        for u, s, p, r, c in sec:
            assert bool((r[..., s:] == 5).all()) and bool((c[:, :, s:] == 5).all())
            t = 0
            for i, (first, n, *_) in enumerate(chunk.tolist()):  # the tiles are the rows transposed, zero past the end
                assert first == t and torch.equal(c[i, :, :s, :n].permute(2, 0, 1), r[t:t + n, :, :s])
                assert not bool(c[i, :, :s, n:].any())
                t += n
        return torch.cat([r[..., :s].reshape(T, -1) for _, s, _, r, _ in sec], 1)

    got = seqs.run(cuts, step)
    for o, u in zip(got, seqs.u):
        y = ref.short_conv(u[:, :ch].double(), conv.double()) + bias.double()
        close(o, ref.silu(y) if silu else y, dtype, f32=1e-5, bf16=4e-3)
    assert bool((ring[1] == 9).all())


# ---------------------------------------------------------------- gated linear recurrence
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("C,blocks,taps", [(256, 2, 4), (60, 3, 3), (96, 1, 1), (320, 1, 4), (136, 17, 9), (7, 7, 2)])
@pytest.mark.parametrize("per_run", [1, 1024])
def test_rglru(C, blocks, taps, per_run, cuts, dtype):
    """A run of chunks per chunk, and one per sequence. Decays from 1 - 1e-6 to almost nothing, so that a lost or stale state shows."""
    g = torch.Generator().manual_seed(C)
    n = C // blocks
    m = mixers.GatedLinearRecurrence({"width": C, "blocks": blocks, "conv": taps}, 1, 0.0, 8, mixers.Weights(DEV, dtype, None, 0.0))
    w = {"conv": rnd(g, C, taps), "conv.b": rnd(g, C), "lam": rnd(g, C, scale=4.0) - 4, "ra": rnd(g, blocks, n, n, scale=2 / n ** 0.5),
         "ri": rnd(g, blocks, n, n, scale=2 / n ** 0.5), "ra.b": rnd(g, blocks, n), "ri.b": rnd(g, blocks, n)}
    w = {k: t.to(dtype) for k, t in w.items()}
    m.bind(torch.zeros(2 * C, 1, device=DEV), torch.zeros(2 * C, device=DEV), None, None)
    for name, t in m.params():
        if name in w:
            t.copy_(w[name])
    m.refresh()
    S, ring = m.make_state(0, 3, DEV)
    S.fill_(50.0)
    ring.fill_(9.0)
    seqs = Steps([rnd(g, k, 2 * C + 8, dtype=dtype) for k in Steps.lens], dtype)

    def step(x, cu, rows, pos, lens, starts):
        class inp:
            pass

        inp.cu, inp.rows, inp.positions, inp.one_token = cu, rows, pos, all(k == 1 for k in lens)
        inp.plan = {m.plan_key: plan_of(mixers.chunk_runs, lens, 0, 0, per_run)}
        out = torch.full((len(x), C + 3), 7.0, dtype=dtype, device=DEV)
        m.inner(x, out[:, :C], inp, (S, ring), None)
        assert bool((out[:, C:] == 7).all())
        return out[:, :C]

    got = seqs.run(cuts, step)
    w = {k: t.double() for k, t in w.items()}
    for o, x, row in zip(got, seqs.u, seqs.rows):
        x = x.double()
        u = ref.short_conv(x[:, C:2 * C], w["conv"]) + w["conv.b"]
        st = ref.gated_linear_recurrence(u, ref.block_gates(u, w, "ra"), ref.block_gates(u, w, "ri"), w["lam"])
        close(o, st * ref.gelu_tanh(x[:, :C]), dtype, f32=2e-5)
        close(S[row], st[-1], dtype, f32=2e-5)
    assert bool((S[1] == 50).all()) and bool((ring[1] == 9).all())


# ---------------------------------------------------------------- windowed attention
def paged_kv(g, lens, G, D, V, dtype, spare=3):
    """Keys and values over shuffled blocks; slots past a sequence's end hold NaN, padding zeros."""
    dp, vp = lk.attn_pads(lk.attn_shape(G, G, D, V, 0, 1.0, 1e-6))
    need = [-(-n // BS) for n in lens]
    nb = sum(need) + spare
    perm = torch.randperm(nb, generator=g)
    kc, vc = torch.full((nb, G, BS, dp), math.nan), torch.full((nb, G, vp, BS), math.nan)
    tables = torch.zeros(len(lens), max(need), dtype=torch.int32)
    K, V_, used = [], [], 0
    for i, n in enumerate(lens):
        blocks = perm[used:used + need[i]]
        used += need[i]
        tables[i, :need[i]] = blocks.int()
        k, v = rnd(g, n, G, D, dtype=dtype), rnd(g, n, G, V, dtype=dtype)
        flat = torch.full((need[i] * BS, G, dp), math.nan)
        flat[:n] = 0
        flat[:n, :, :D] = k.float()
        kc[blocks] = flat.view(need[i], BS, G, dp).transpose(1, 2)
        flat = torch.full((need[i] * BS, G, vp), math.nan)
        flat[:n] = 0
        flat[:n, :, :V] = v.float()
        vc[blocks] = flat.view(need[i], BS, G, vp).permute(0, 2, 3, 1)
        K.append(k)
        V_.append(v)
    return kc.to(dtype).to(DEV), vc.to(dtype).to(DEV), tables.to(DEV), K, V_


def pad_q(q, dtype):
    T, H, D = q.shape
    out = torch.zeros(T, H, (D + 31) // 32 * 32, dtype=dtype)
    out[..., :D] = q
    return out.to(DEV)


def standing_out(q, K, p, window, turn):
    """Points the query at a key: its own, the one before, just inside the window, just outside it, the first, a
    page's border."""
    lo = max(0, p - window + 1) if window else 0
    j = (p, max(0, p - 1), lo, max(0, lo - 1), 0, p // BS * BS, min(p, lo + 1))[turn % 7]
    return 0.6 * K[j].float() + 0.3 * q.float()


def window_oracle(q, K, V, positions, sh):
    """q [n, H, D] at `positions` over one sequence's K [m, G, D], V [m, G, V]."""
    g = torch.arange(sh.heads) // (sh.heads // sh.kv_heads)
    s = torch.einsum("ihd,jhd->hij", q.double(), K[:, g].double()) * sh.scale
    j, i = torch.arange(len(K))[None], torch.as_tensor(positions)[:, None]
    see = (j <= i) & ((i - j < sh.window) if sh.window else (j >= 0))
    return torch.einsum("hij,jhv->ihv", torch.softmax(s.masked_fill(~see, -math.inf), -1), V[:, g].double()).reshape(len(q), -1)


ATTEND = [  # heads, kv_heads, dim, vdim, window
    (4, 2, 20, 28, 37), (6, 3, 32, 64, 16), (16, 2, 64, 128, 100), (20, 1, 16, 40, None), (3, 3, 100, 72, 1), (4, 1, 128, 256, 64),
    (9, 1, 48, 200, 17), (2, 1, 30, 150, 2), (2, 2, 144, 300, 50), (12, 4, 61, 5, 333), (2, 1, 256, 160, 65), (3, 1, 64, 64, 15),
    (2, 1, 290, 32, 40)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,window", ATTEND)
def test_attend(heads, kv_heads, dim, vdim, window, dtype):
    """Contexts around page and window edges, unsplit and split; per head one key stands out."""
    g = torch.Generator().manual_seed(dim + heads)
    w = window or 0
    pos = sorted({0, 1, 2, 14, 15, 16, 17, 63, 64, 65, 200, 333, 700} | {max(0, w + d) for d in (-2, -1, 0, 1, 15)})
    kc, vc, tables, K, V = paged_kv(g, [p + 1 for p in pos], kv_heads, dim, vdim, dtype)
    T, W = len(pos), heads * vdim
    sh = lk.attn_shape(heads, kv_heads, dim, vdim, window, 2.0 / math.sqrt(dim), 3e-5)
    q, gate = rnd(g, T, heads, dim), rnd(g, T, W + 3, dtype=dtype, scale=2.0)
    for i, p in enumerate(pos):
        for h in range(heads):
            q[i, h] = standing_out(q[i, h], K[i][:, h // (heads // kv_heads)], p, window, h + i)
    q = q.to(dtype)
    want = torch.cat([window_oracle(q[i:i + 1], K[i], V[i], [p], sh) for i, p in enumerate(pos)])
    want = want * torch.sigmoid(gate[:, 3:].double())
    iota = torch.arange(T, dtype=torch.int32, device=DEV)
    for nparts, part_min in ((1, 64), (3, 16), (40, 64)):
        out = torch.full((T, W + 9), 7.0, dtype=dtype, device=DEV)
        lk.attn_attend(sh, pad_q(q, dtype), dev(gate)[:, 3:], kc, vc, tables, iota, torch.tensor(pos, device=DEV),
                       out[:, 4:4 + W], nparts=nparts, part_min=part_min)
        close(out[:, 4:4 + W], want, dtype)
        assert bool((out[:, :4] == 7).all()) and bool((out[:, 4 + W:] == 7).all())


PREFILL = [  # heads, kv_heads, dim, vdim, window, [(start, tokens)]
    (4, 2, 20, 28, 37, [(0, 70), (5, 33)]), (6, 3, 32, 64, 16, [(0, 130), (300, 64), (79, 40)]),
    (8, 1, 64, 128, 128, [(0, 300), (1100, 129)]), (16, 2, 64, 120, None, [(0, 128), (1, 32), (200, 40)]),
    (3, 1, 16, 40, 1, [(17, 200)]), (2, 1, 100, 72, 63, [(64, 128), (63, 65)]), (2, 2, 128, 256, 40, [(3, 135)]),
    (2, 1, 48, 200, 65, [(0, 64), (0, 65)]), (3, 3, 30, 150, 2, [(15, 50)]), (2, 1, 96, 16, 200, [(250, 48), (1000, 200)]),
    (2, 1, 240, 136, 70, [(100, 90)]), (8, 8, 128, 128, 96, [(31, 150)])]


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,window,segs", PREFILL)
def test_prefill(heads, kv_heads, dim, vdim, window, segs):
    g = torch.Generator().manual_seed(dim + vdim)
    kc, vc, tables, K, V = paged_kv(g, [3] + [s + n for s, n in segs], kv_heads, dim, vdim, BF16)
    lens, starts = [3] + [n for _, n in segs], [0] + [s for s, _ in segs]
    T, W = sum(lens), heads * vdim
    sh = lk.attn_shape(heads, kv_heads, dim, vdim, window, 2.0 / math.sqrt(dim), 1e-5)
    q, gate = rnd(g, T, heads, dim), rnd(g, T, W, dtype=BF16, scale=2.0)
    tok = 3
    for i, (s, n) in enumerate(segs, 1):
        for t in range(n):
            for h in range(heads):
                q[tok + t, h] = standing_out(q[tok + t, h], K[i][:, h // (heads // kv_heads)], s + t, window, t + h)
        tok += n
    q = q.to(BF16)
    tiles = torch.from_numpy(mixers.tile_plan(lens, starts, 1, 3, window)).to(DEV)
    out = torch.zeros(T, W + 5, dtype=BF16, device=DEV)
    lk.attn_prefill(sh, pad_q(q, BF16), dev(gate), kc, vc, tables, tiles, out[:, :W])
    assert not bool(out[:3].any()) and not bool(out[:, W:].any())
    tok = 3
    for i, (s, n) in enumerate(segs, 1):
        want = window_oracle(q[tok:tok + n], K[i], V[i], range(s, s + n), sh) * torch.sigmoid(gate[tok:tok + n].double())
        close(out[tok:tok + n, :W], want, BF16)
        tok += n


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 20, 28), (6, 3, 24, 16), (2, 1, 64, 128), (3, 1, 11, 7), (16, 16, 128, 64),
                                                     (1, 1, 200, 264)])
def test_attn_write(heads, kv_heads, dim, vdim, dtype):
    """Token by token, in portions and in runs: queries, keys and values where they belong and nowhere else."""
    g = torch.Generator().manual_seed(dim)
    sh, eps = lk.attn_shape(heads, kv_heads, dim, vdim, 5, 1.0, 2e-2), 2e-2
    ch, (dp, vp) = lk.attn_channels(sh), lk.attn_pads(sh)
    lens = (61, 90)
    u = [rnd(g, n, ch + 8, dtype=dtype) for n in lens]
    qn, kn = (rnd(g, dim, dtype=dtype) for _ in range(2))
    need = [-(-n // BS) for n in lens]
    perm = torch.randperm(sum(need) + 2, generator=g)
    blocks = perm[:sum(need)].split(need)
    kc = torch.full((len(perm), kv_heads, BS, dp), 5.0, dtype=dtype, device=DEV)
    vc = torch.full((len(perm), kv_heads, vp, BS), 5.0, dtype=dtype, device=DEV)
    at, qs = [0, 0], [[], []]
    runs_fit = dtype == BF16 and dim % 8 == 0 and vdim % 8 == 0
    for c in ((1, 2), (2, 33), (1, 1), (40, 3), (17, 51)):
        x = dev(torch.cat([u[i][at[i]:at[i] + n] for i, n in enumerate(c)] + [u[0][:1]]))
        pos = [torch.arange(at[i], at[i] + n) for i, n in enumerate(c)]
        slots = dev(torch.cat([blocks[i][p // BS] * BS + p % BS for i, p in enumerate(pos)] + [torch.tensor([-1])]))
        args = (sh, x, dev(qn), dev(kn), slots, kc, vc)
        if runs_fit and min(c) > 2:
            q = lk.attn_write(*args, count=0)
            runs = mixers.run_plan(list(c), at, 0, 0)
            lk.attn_write(*args, q=q, runs=torch.from_numpy(runs).to(DEV))
        else:
            q = lk.attn_write(*args)
        for i, n in enumerate(c):
            qs[i].append(q[(0, c[0])[i]:][:n])
            at[i] += n
    assert tuple(at) == lens
    for i, n in enumerate(lens):
        x = u[i].double()
        got = torch.cat(qs[i])
        close(got[..., :dim], ref.rms_norm(x[:, :heads * dim].view(n, heads, dim), qn.double(), eps), dtype, f32=1e-5, bf16=4e-3)
        assert not bool(got[..., dim:].any())
        a = heads * dim
        key = kc[blocks[i]].transpose(1, 2).reshape(-1, kv_heads, dp)
        val = vc[blocks[i]].permute(0, 3, 1, 2).reshape(-1, kv_heads, vp)
        close(key[:n, :, :dim], ref.rms_norm(x[:, a:a + kv_heads * dim].view(n, kv_heads, dim), kn.double(), eps), dtype, f32=1e-5, bf16=4e-3)
        assert torch.equal(val[:n, :, :vdim].cpu().double(), x[:, a + kv_heads * dim:ch].view(n, kv_heads, vdim))
        for t, real in ((key, dim), (val, vdim)):  # padding and slots past the end are not touched
            assert bool((t[n:] == 5).all()) and bool((t[..., real:] == 5).all())
    assert bool((kc[perm[sum(need):]] == 5).all()) and bool((vc[perm[sum(need):]] == 5).all())


# ---------------------------------------------------------------- state space mixer
SSD = [  # heads, vdim, state, groups, taps
    (4, 64, 128, 2, 4), (3, 20, 18, 1, 5), (6, 72, 40, 3, 7), (2, 24, 160, 1, 1), (5, 7, 9, 5, 3), (2, 150, 64, 1, 2), (1, 64, 256, 1, 4)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("heads,vdim,state,groups,taps", SSD)
def test_ssd(heads, vdim, state, groups, taps, cuts, dtype, monkeypatch):
    """Decays from none over hundreds of tokens to all within one; long portions in one and in several runs of chunks."""
    monkeypatch.setattr(mixers, "WALK_CHUNKS", 1)
    g = torch.Generator().manual_seed(state + heads)
    sh = lk.ssd_shape(heads, vdim, state, groups, taps)
    inner, ch = heads * vdim, lk.ssd_channels(sh)
    conv, bias = rnd(g, ch, taps, dtype=dtype), rnd(g, ch, scale=0.3)
    a_log, dtb, skip = torch.linspace(-7, 2.5, heads), rnd(g, heads), rnd(g, heads)
    S = torch.full((3, heads, state, lk.ssd_ppad(sh)), 50.0, device=DEV)
    ring = torch.full((3, taps, ch), 9.0, dtype=dtype, device=DEV)
    seqs = Steps([rnd(g, n, lk.ssd_width(sh) + 4, dtype=dtype) for n in Steps.lens], dtype)
    w = (dev(conv.t().float().contiguous()), dev(bias), dev(a_log), dev(dtb), dev(skip))

    def step(x, cu, rows, pos, lens, starts):
        y = torch.full((len(x), inner + 4), 7.0, dtype=dtype, device=DEV)
        one = all(n == 1 for n in lens)
        order = [n for n in lens if n < mixers.PROMPT_MIN]
        k = len(order) if lk.ssd_prompt_fits(sh, dtype) and lens[:len(order)] == order else len(lens)  # short ones first
        if k:
            lk.ssd_scan(sh, x, *w, cu[:k + 1].contiguous(), rows[:k].contiguous(), pos, S, ring, one, y[:, :inner])
        if k < len(lens):
            lk.ssd_prompt(sh, x, *w, cu, rows, pos, S, ring, *plan_of(mixers.walk_plan, lens, k, sum(lens[:k]), 512), y[:, :inner])
        if not one:
            lk.conv_save(x[:, inner:], ch, cu, rows, pos, ring)
        assert bool((y[:, inner:] == 7).all())
        return y[:, :inner]

    got = seqs.run(cuts, step)
    for o, x, row in zip(got, seqs.u, seqs.rows):
        x, T = x.double(), len(x)
        c = ref.silu(ref.short_conv(x[:, inner:inner + ch], conv.double()) + bias.double())
        group = torch.arange(heads) // (heads // groups)
        B, C = (c[:, a:a + groups * state].view(T, groups, state)[:, group] for a in (inner, inner + groups * state))
        dt = ref.softplus(x[:, inner + ch:inner + ch + heads] + dtb.double())
        y, st = ref.state_space_recurrence(c[:, :inner].view(T, heads, vdim), B, C, dt, a_log.double(), skip.double())
        for h in range(heads):  # heads differ in size
            close(o.view(T, heads, vdim)[:, h], y[:, h], dtype, f32=2e-5)
            close(S[row, h, :, :vdim], st[h], dtype, f32=2e-5)
    assert bool((S[1] == 50).all()) and bool((ring[1] == 9).all())


def test_prompt_walk_is_exact_beyond_bf16():
    """State and decays stay f32 in the matrix products: with inputs that bf16 holds exactly, the chunked form
    agrees with the recurrence to f32 rounding before its one rounding of the output."""
    H, P, N, T = 2, 64, 128, 320
    sh = lk.ssd_shape(H, P, N, 1, 1)
    inner, ch = H * P, lk.ssd_channels(sh)
    g = torch.Generator().manual_seed(5)
    x = rnd(g, T, lk.ssd_width(sh), dtype=BF16)
    w = [torch.full((1, ch), 1.0), torch.zeros(ch), torch.tensor([-5.0, -3.0]), torch.zeros(H), torch.ones(H)]
    cu, rows, pos = torch.tensor([0, T], dtype=torch.int32), torch.zeros(1, dtype=torch.int32), torch.arange(T)
    S = torch.zeros(1, H, N, P, device=DEV)
    ring = torch.zeros(1, 1, ch, dtype=BF16, device=DEV)
    y = torch.empty(T, inner, dtype=BF16, device=DEV)
    lk.ssd_prompt(sh, dev(x), *map(dev, w), dev(cu), dev(rows), dev(pos), S, ring,
                  *plan_of(mixers.walk_plan, [T], 0, 0, 512), y)
    c = ref.silu(x[:, inner:inner + ch].float()).to(BF16).double()
    B, C = (c[:, a:a + N].view(T, 1, N).expand(T, H, N) for a in (inner, inner + N))
    dt = ref.softplus(x[:, inner + ch:].double())
    want, st = ref.state_space_recurrence(c[:, :inner].view(T, H, P), B, C, dt, w[2].double(), w[4].double())
    assert rms(S[0].double().cpu() - st) < 2e-4 * rms(st)  # the convolution's rounding may differ by one bf16 step here and there
    close(y.view(T, H, P), want, BF16, bf16=4e-3)


# ---------------------------------------------------------------- the model through the engine's steps
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(NORMED))
def test_model_whole_portions_and_decode(name, dtype):
    cfg = NORMED[name]
    m, w = build(cfg, dtype)
    toks = tokens_of(cfg, 150, 1)
    want, _ = ref.forward(toks, w, cfg)
    s = TraceSession(m, 512)
    for i, cuts in enumerate(([150], [2] * 10 + [130], [1] * 150, [33, 31, 32, 1, 1, 2, 16, 17, 1, 16], [3, 64, 60, 23])):
        model_close(feed(s, f"r{i}", toks, cuts), want, dtype)
        s.step([], [f"r{i}"])  # the next request takes its pages and state row
    assert s.core.allocator.num_free == s.core.allocator.num_blocks and len(s.core._free_rows) == 4


@pytest.mark.parametrize("name", sorted(NORMED))
def test_residual_after_every_layer(name):
    cfg = NORMED[name]
    m, w = build(cfg, torch.float32)
    toks = tokens_of(cfg, 60, 3)
    logits, trail = ref.forward(toks, w, cfg)
    s = TraceSession(m, 64, use_graphs=False)
    r = s.core.open_request()
    r.prompt, r.blocks = list(toks), s.core.allocator.allocate(4)
    got = []
    inp = s.core.runner._portion_inputs(s.core._batch_of([(r, 60)]), [(0, 59), (0, 3)])
    hidden = m.forward_portions(inp, s.core.runner.cache, got)
    assert len(got) == len(trail) == len(cfg["layers"])
    for a, b in zip(got, trail):
        close(a, b, torch.float32, f32=1e-5)
    close(m.logits(hidden), logits[[59, 3]], torch.float32, f32=2e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("graphs", [True, False])
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_mixed_batches_equal_each_request_alone(name, graphs, dtype):
    """Requests of unequal lengths, some decoding while others are in their prompts, some left out of
    steps, ended and replaced by others on the same pages and rows."""
    cfg = NORMED[name]
    m, w = build(cfg, dtype)
    lens = {"a": 120, "b": 49, "c": 1, "d": 90, "e": 70, "f": 33}
    toks = {k: tokens_of(cfg, n, i) for i, (k, n) in enumerate(lens.items())}
    want = {k: ref.forward(t, w, cfg)[0] for k, t in toks.items()}
    s = TraceSession(m, 128 + 64 + 128 + 128, use_graphs=graphs)
    at, got = {k: 0 for k in lens}, {k: [] for k in lens}
    plan = [{"a": 40, "b": 1, "c": 1}, {"a": 1, "b": 2}, {"d": 35, "b": 40}, {"a": 1, "b": 1, "d": 1}, {"a": 1, "d": 1},
            {"e": 2, "a": 70, "d": 2}, {"b": 1, "a": 1, "d": 1, "e": 1}, {"b": 1, "d": 1}, {"b": 3, "a": 5, "e": 33},
            {"a": 1, "d": 48}, {"f": 32, "e": 32, "d": 1}, {"e": 1, "f": 1}, {"e": 1}]
    for st in plan:
        ents = [{"id": k, "tokens": toks[k][at[k]:at[k] + n], "want": list(range(n))} for k, n in st.items()]
        for k, n in st.items():
            at[k] += n
        out = s.step(ents, [k for k in st if at[k] == lens[k]])
        for k, n in st.items():
            got[k].append(out[:n])
            out = out[n:]
    for k in lens:
        t = torch.cat(got[k])
        assert len(t) == at[k] > 0
        model_close(t, want[k][:len(t)], dtype)


def window_case(size):
    """One layer whose attention alone is heard (the other mixer's output norm is zero). The queries of tokens
    21 .. 40 are the keys of tokens 1 .. 20; such pairs stand size - 1 (inside) and size (outside) tokens apart."""
    cfg = normed_config([side(attend(heads=2, kv_heads=1, dim=32, vdim=32, window=size, scale=0.9), ssd())], width=64, no_mlp=(0,),
                        scale=30.0)
    w = make_normed_weights(cfg, 5)
    g = torch.Generator().manual_seed(1)
    common = torch.randn(32, 64, generator=g) * 0.3
    w["l0.mix.left.k"] = common.to(BF16)
    w["l0.mix.left.q"] = torch.cat([common.roll(32, 1)] * 2).to(BF16)
    w["embed"][21:41] = w["embed"][1:21].roll(32, 1)
    w["l0.mix.right.out"] *= 0
    w["l0.norm1"] = torch.tensor(60.0).to(BF16)  # the layer is louder than the embedding
    for n in ("q", "k"):
        w[f"l0.mix.left.{n}.norm"] = torch.ones(32).to(BF16)
        w[f"l0.mix.left.{n}.b"] *= 0
    toks = torch.randint(41, cfg["vocab"], (300,), generator=g).tolist()
    found, taken = ([], []), set()
    for k, i in enumerate(range(size + 1, 300, 5)):
        j = i - (size - 1) - k % 2
        if taken.isdisjoint((i, j)):
            taken |= {i, j}
            toks[i], toks[j] = 21 + k % 20, 1 + k % 20
            found[k % 2].append(i)
    return cfg, w, toks, *found


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [2, 16, 33, 64, 100])
def test_window_edges_in_prompts_and_decoding(size, dtype):
    cfg, w, toks, inside, outside = window_case(size)
    wd = {k: v.double() for k, v in w.items()}
    want, _ = ref.forward(toks, wd, cfg)

    def with_window(n):
        left = dict(cfg["layers"][0]["mixer"]["left"], mask={"size": n})
        other = dict(cfg, layers=[dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], left=left))])
        return (ref.forward(toks, wd, other)[0] - want).pow(2).mean(-1).sqrt() / rms(want)

    if size > 2:  # a window one token off would show
        assert float(with_window(size - 1)[inside].mean()) > 0.1 and float(with_window(size + 1)[outside].mean()) > 0.1
    m, _ = build(cfg, dtype)
    m.load_weights(w.items())
    s = TraceSession(m, 320)
    for i, cuts in enumerate(([300], [101] + [1] * 199, [37] * 8 + [4], [2] * 150)):
        model_close(feed(s, f"w{i}", toks, cuts), want, dtype)
        s.step([], [f"w{i}"])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["rglru", "ssd"])
def test_long_decoding_with_far_memory(kind, dtype):
    """States that hardly decay: the first tokens are heard hundreds of tokens later, through decode steps and portions."""
    layer = rglru(width=64, blocks=2, conv=2) if kind == "rglru" else side(attend(window=4), ssd(heads=2, vdim=32, state=32, conv=2, norm_groups=2))
    cfg = normed_config([layer], width=64, no_mlp=(0,))
    w = make_normed_weights(cfg, 5)
    if kind == "rglru":
        w["l0.mix.lam"][:] = -9.0
    else:
        w["l0.mix.right.A_log"][:] = -6.0
        w["l0.mix.left.out"] *= 0
    w["l0.norm1"] = torch.tensor(15.0).to(BF16)
    toks = tokens_of(cfg, 620, 8)
    wd = {k: v.double() for k, v in w.items()}
    want, _ = ref.forward(toks, wd, cfg)
    changed, _ = ref.forward([(t + 1) % cfg["vocab"] for t in toks[:200]] + toks[200:], wd, cfg)
    assert float((changed[560:] - want[560:]).pow(2).mean().sqrt()) > 0.03 * rms(want)
    m, _ = build(cfg, dtype, max_len=640)
    m.load_weights(w.items())
    s = TraceSession(m, 640)
    model_close(feed(s, "x", toks, [101] + [1] * 519), want, dtype)
    s.step([], ["x"])
    model_close(feed(s, "y", toks, [37] * 16 + [28]), want, dtype)


def test_cut_does_not_change_bf16_logits_beyond_rounding():
    """The same prompt in portions on both sides of the short-portion limit, token by token and whole."""
    cfg = NORMED["wide"]
    m, _ = build(cfg, BF16)
    toks = tokens_of(cfg, 96, 12)
    outs = []
    for cuts in ([96], [32, 64], [31, 33, 32], [16] * 6, [1] * 96):
        s = TraceSession(m, 128)
        outs.append(feed(s, "x", toks, cuts))
    for o in outs[1:]:
        model_close(o, outs[0].double(), BF16)


@pytest.mark.parametrize("rows", [3, 40])
def test_graph_replays_at_larger_layers(rows):
    """Captured decode steps with products of a real model's size, every replay against the eager step."""
    cfg = normed_config([rglru(width=1024, blocks=8, conv=4),
                         side(attend(heads=8, kv_heads=2, dim=64, vdim=128, window=40),
                              ssd(heads=16, vdim=64, state=128, groups=2, conv=4, norm_groups=2))],
                        width=1024, ff=2048, vocab=4096)
    m, _ = build(cfg, BF16)
    prompts = [tokens_of(cfg, 10 + i % 7, i) for i in range(rows)]
    ids = [f"r{i}" for i in range(rows)]
    sessions = [TraceSession(m, 64 * rows, max_live=rows, use_graphs=g) for g in (True, False)]
    for s in sessions:
        s.step([{"id": k, "tokens": p, "want": []} for k, p in zip(ids, prompts)])
    for t in range(6):
        step = [{"id": k, "tokens": [(31 * t + 7 * i) % cfg["vocab"]], "want": [0]} for i, k in enumerate(ids)]
        a, b = (s.step(step) for s in sessions)
        model_close(a, b.double(), BF16)
        torch.cuda.synchronize()


# ---------------------------------------------------------------- generation
def test_greedy_generation_through_the_scheduler():
    """Six prompts on four rows, prompts cut by the step budget: f32 tokens equal the oracle's argmax
    chain, logprobs its log softmax; a cache too small for all preempts and recomputes."""
    cfg = NORMED["odd"]
    m, w = build(cfg, torch.float32)
    prompts = [tokens_of(cfg, n, 20 + n) for n in (1, 5, 40, 90, 17, 33)]
    expect = [greedy(w, cfg, p, 12) for p in prompts]
    assert min(min(mg) for _, mg in expect) > 1e-4
    for blocks in (200, 12):
        out, eng = generate(m, prompts, blocks, temperature=0.0, max_tokens=12, ignore_eos=True)
        assert out["response_ids"] == [e for e, _ in expect]
        assert eng.core.allocator.num_free == blocks
        assert (eng.core.num_preemptions > 0) == (blocks == 12)
        lg, _ = ref.forward(prompts[3] + expect[3][0], w, cfg)
        lp = torch.log_softmax(lg, -1)
        for i, t in enumerate(expect[3][0]):
            assert abs(out["response_logprobs"][3][i] - float(lp[89 + i, t])) < 1e-3


def test_bf16_generation_alone_and_in_a_batch():
    """Greedy bf16 tokens alone and in a batch agree up to the first near-tie; the head's product may run in
    the sampler's kernel."""
    cfg = NORMED["wide"]
    m, w = build(cfg, BF16)
    prompts = [tokens_of(cfg, n, 40 + n) for n in (3, 50, 70)]
    batch, eng = generate(m, prompts, 100, temperature=0.0, max_tokens=30, ignore_eos=True)
    assert eng.runner.fused_steps > 0
    for i, p in enumerate(prompts):
        alone, _ = generate(m, [p], 100, max_prefill=4096, graphs=False, temperature=0.0, max_tokens=30, ignore_eos=True)
        a, b = alone["response_ids"][0], batch["response_ids"][i]
        k = next((j for j in range(30) if a[j] != b[j]), None)
        if k is not None:
            lg, _ = ref.forward(p + a[:k], w, cfg)
            assert float(lg[-1, a[k]] - lg[-1, b[k]]) < 0.3


def test_weight_update_sleep_and_wake():
    """Updated weights reach every derived tensor and captured graph; sleep drops cache and state."""
    cfg = NORMED["odd"]
    m, _ = build(cfg, torch.float32)
    w2 = make_normed_weights(cfg, 77)
    p = [tokens_of(cfg, 25, 1)]
    eng = AMDInferenceEngine(m, num_blocks=50, max_num_seqs=2)
    req = {"prompt_token_ids": p, "sampling_params": {"temperature": 0.0, "max_tokens": 8, "ignore_eos": True}}

    async def run():
        first = await eng.generate(req)
        await eng.update_named_weights({"names": list(w2), "tensors": [t.to(DEV) for t in w2.values()]})
        second = await eng.generate(req)
        await eng.sleep(level=1)
        await eng.wake_up()
        third = await eng.generate(req)
        return first["response_ids"], second["response_ids"], third["response_ids"]

    a, b, c = asyncio.run(run())
    want, _ = greedy({k: v.double() for k, v in w2.items()}, cfg, p[0], 8)
    assert a != b and b == c == [want]


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_program_and_command_line(tmp_path, dtype, capsys, monkeypatch):
    """A checkpoint folder through the trace replay program and the generation command line."""
    from safetensors.torch import save_file

    from skyrl_amd.inference_engines import __main__ as cli
    from skyrl_amd.inference_engines import trace

    cfg = NORMED["odd"]
    w = make_normed_weights(cfg, 4)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    toks = tokens_of(cfg, 45, 6)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:40], "want": [39]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[40:42], "want": []},
                                     {"id": "b", "tokens": toks[:1], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[42:], "want": [2, 0]}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps)) + "\n"))
    assert trace.main(["--model", str(tmp_path), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "128"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1", "done 2"]
    want, _ = ref.forward(toks, {k: v.double() for k, v in w.items()}, cfg)
    for step, rows in ((0, [39]), (1, [0]), (2, [44, 42])):
        got = np.fromfile(str(tmp_path / f"{step}.f32"), dtype="<f4").reshape(len(rows), cfg["vocab"])
        model_close(torch.from_numpy(got), want[rows], getattr(torch, dtype))
    assert cli.main(["--model", str(tmp_path), "--dtype", dtype, "--prompt-ids", ",".join(map(str, toks)), "--temperature",
                     "0", "--max-tokens", "3", "--num-blocks", "20", "--max-model-len", "256"]) == 0
    ids = json.loads(capsys.readouterr().out.strip().splitlines()[-1])["response_ids"]
    assert len(ids) == 3 and float(want[44].max() - want[44, ids[0]]) < (1e-3 if dtype == "float32" else 0.3)
