"""Differential attention and parallel layers (Lipedra) on the GPU: every kernel alone, then the model
through the engine's own steps, against the plain restatement in oracle/hybrid_ref.py. Tolerances as in
test_gpu_hybrid.py."""

import asyncio
import io
import json
import math

import numpy as np
import pytest
import torch

from hybrid_cases import PARALLEL, diff_attention, make_parallel_weights, parallel_config
from hybrid_gpu import DEV, DTYPES, build, close, feed, generate, greedy, model_close, rms, rnd, tokens_of
from oracle import hybrid_ref as ref
from skyrl_amd.inference_engines import layer_kernels as lk
from skyrl_amd.inference_engines import mixers
from skyrl_amd.inference_engines.engine import AMDInferenceEngine
from skyrl_amd.inference_engines.trace import TraceSession

pytestmark = pytest.mark.gpu
BS = mixers.BLOCK_SIZE
BF16 = torch.bfloat16


# ---------------------------------------------------------------- embedding, norm about one, clamped gate
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [72, 1, 515])
def test_embed_and_norm_about_one(H, dtype):
    g = torch.Generator().manual_seed(H)
    table, tok = rnd(g, 31, H, dtype=dtype), torch.tensor([3, 0, 30, 3, 17])
    x = lk.embed(tok.to(DEV), table.to(DEV), 3.7)
    assert x.dtype == torch.float32
    close(x, table[tok].double() * 3.7, torch.float32, f32=1e-6)
    w, d = rnd(g, H, dtype=dtype, scale=0.3), rnd(g, 5, H, dtype=dtype)
    want_h = table[tok].double() * 3.7 + d.double()
    out = lk.add_norm(d.to(DEV), x, w.to(DEV), 2e-3, kind="rms", base=1.0)
    close(x, want_h, torch.float32, f32=1e-6)
    close(out, ref.rms_norm_about_one(want_h, w.double(), 2e-3), dtype, f32=1e-5, bf16=4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff,pad", [(100, 0), (33, 3), (64, 8)])
def test_clamped_gate_in_column_ranges(ff, pad, dtype):
    """Values on both sides of every clamp; input and output are ranges of wider rows."""
    g = torch.Generator().manual_seed(ff)
    wide = rnd(g, 9, 2 * ff + 2 * pad, dtype=dtype, scale=2.0)
    x = wide[:, pad:pad + 2 * ff]
    out = torch.full((9, ff + 2 * pad), 7.0, dtype=dtype, device=DEV)
    lk.gate_mul(wide.to(DEV)[:, pad:pad + 2 * ff], "clamped", 1.702, 1.1, out=out[:, pad:pad + ff])
    w = {"gate": torch.eye(2 * ff).double()[:ff], "up": torch.eye(2 * ff).double()[ff:], "down": torch.eye(ff).double(),
         "gate.b": torch.zeros(ff).double(), "up.b": torch.zeros(ff).double(), "down.b": torch.zeros(ff).double()}
    close(out[:, pad:pad + ff], ref.clamped_ff(x.double(), w, "", 1.1), dtype, f32=1e-5, bf16=4e-3)
    assert bool((out[:, :pad] == 7).all()) and bool((out[:, pad + ff:] == 7).all())


# ---------------------------------------------------------------- convolution, rotation, cache write
ROT = {"base": 90.0, "dims": 0, "scaling": {"factor": 3.0, "original": 50, "fast": 5.0, "slow": 0.3}}
WRITE = [  # heads, kv_heads, dim, vdim, rot_dims, taps, own keys
    (4, 2, 20, 28, 8, 3, True), (6, 3, 24, 16, 24, 4, True), (2, 1, 64, 128, 32, 4, True), (3, 1, 11, 7, 10, 2, True),
    (4, 4, 16, 40, 6, 1, True), (2, 2, 40, 24, 2, 8, True), (2, 1, 8, 8, 4, 12, True), (5, 1, 24, 64, 10, 3, False)]


class WriteCase:
    """Sequences whose steps are cut in different ways; rows and cache start full of other values."""

    def __init__(self, shape, dtype, lens, seed=0):
        H, G, D, V, rd, taps, kv = shape
        self.sh = lk.diff_shape(H, G, D, V, rd, taps, kv, 1.0, 0.5, 1e-6)
        g = torch.Generator().manual_seed(seed + D)
        self.ch, self.dtype, self.rot = lk.diff_channels(self.sh), dtype, dict(ROT, dims=rd)
        self.pad = 5 if D % 8 else 8  # further columns of the projection
        self.u = [rnd(g, n, self.ch + self.pad, dtype=dtype) for n in lens]
        conv = rnd(g, self.ch, taps, dtype=dtype)
        self.want = [self.oracle(u[:, :self.ch].double(), conv.double()) for u in self.u]
        self.conv_t = conv.t().float().contiguous().to(DEV)
        self.table = mixers.rotary_table(self.rot, 256).to(DEV)
        self.kw, self.vp = lk.diff_pads(self.sh)
        self.ring = torch.full((4, taps, self.ch), 9.0, dtype=dtype, device=DEV)
        need = [-(-n // BS) for n in lens]
        perm = torch.randperm(sum(need) + 2, generator=g)
        self.blocks = perm[:sum(need)].split(need)
        self.kc = torch.full((len(perm), G, BS, self.kw), 5.0, dtype=dtype, device=DEV)
        self.vc = torch.full((len(perm), G, self.vp, BS), 5.0, dtype=dtype, device=DEV)
        self.spare = perm[sum(need):]
        self.q = [[] for _ in lens]

    def oracle(self, u, conv):
        sh, T = self.sh, len(u)
        y = ref.short_conv(u, conv)
        nq, nk = 2 * sh.heads * sh.dim, 2 * sh.kv_heads * sh.dim
        q = ref.rotate_maps(y[:, :nq].view(T, -1, 2, sh.dim), self.rot)
        if not sh.kv:
            return q, None, None
        return q, ref.rotate_maps(y[:, nq:nq + nk].view(T, -1, 2, sh.dim), self.rot), y[:, nq + nk:].view(T, -1, sh.vdim)

    def step(self, parts, n_short=None):
        """parts: [(sequence or -1, row, start, tokens)]; sequences from n_short on take the run form."""
        lens = [n for *_, n in parts]
        u = torch.cat([self.u[max(i, 0)][s:s + n] for i, _, s, n in parts]).to(DEV)
        cu = torch.tensor([0] + lens).cumsum(0).int().to(DEV)
        rows = torch.tensor([r for _, r, *_ in parts], dtype=torch.int32, device=DEV)
        seq = torch.arange(len(parts), dtype=torch.int32).repeat_interleave(torch.tensor(lens)).to(DEV)
        pos = torch.cat([torch.arange(s, s + n) for *_, s, n in parts])
        slots = torch.cat([torch.full((n,), -1) if i < 0 else self.blocks[i][torch.arange(s, s + n) // BS] * BS
                           + torch.arange(s, s + n) % BS for i, _, s, n in parts])
        pos, slots = pos.to(DEV), slots.to(DEV)
        args = (self.sh, u, self.conv_t, cu, rows, seq, pos, slots, self.table, self.ring, self.kc, self.vc)
        one = all(n == 1 for n in lens)
        k = len(parts) if n_short is None else n_short
        first = sum(lens[:k])
        q = lk.diff_write(*args, save_conv=one, count=first)
        if k < len(parts):
            runs = torch.from_numpy(mixers.run_plan(lens, [s for *_, s, _ in parts], k, first)).to(DEV)
            lk.diff_write(*args, q=q, runs=runs)
        if not one:
            lk.conv_save(u, self.ch, cu, rows, pos, self.ring)
        for (i, *_), t in zip(parts, q.split(lens)):
            if i >= 0:
                self.q[i].append(t)

    def check(self):
        sh, dp = self.sh, self.kw // 2
        for i, (q, k, v) in enumerate(self.want):
            got = torch.cat(self.q[i]).view(len(q), sh.heads, 2, dp)
            close(got[..., :sh.dim], q, self.dtype, f32=1e-5, bf16=4e-3)
            assert not bool(got[..., sh.dim:].any())
            if not sh.kv:
                continue
            b, n = self.blocks[i], len(q)
            key = self.kc[b].transpose(1, 2).reshape(-1, sh.kv_heads, 2, dp)
            val = self.vc[b].permute(0, 3, 1, 2).reshape(-1, sh.kv_heads, self.vp)
            close(key[:n, :, :, :sh.dim], k, self.dtype, f32=1e-5, bf16=4e-3)
            close(val[:n, :, :sh.vdim], v, self.dtype, f32=1e-5, bf16=4e-3)
            for t, real in ((key, sh.dim), (val, sh.vdim)):  # padding and slots past the end are not touched
                assert bool((t[n:] == 5).all()) and bool((t[..., real:] == 5).all())
        assert bool((self.kc[self.spare] == 5).all()) and bool((self.vc[self.spare] == 5).all())
        if not sh.kv:
            assert bool((self.kc == 5).all()) and bool((self.vc == 5).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", WRITE)
def test_diff_write(shape, dtype):
    c = WriteCase(shape, dtype, (61, 90))
    runs = dtype == BF16 and shape[2] % 8 == 0 and shape[3] % 8 == 0 and shape[5] <= 8
    a = b = 0
    for na, nb, k in ((1, 2, None), (2, 33, 1), (1, 1, None), (1, 1, None), (40, 3, None), (3, 37, 1), (13, 13, 0)):
        parts = [(0, 2, a, na), (1, 0, b, nb)]
        c.step(parts + ([(-1, -1, 0, 1)] if na == nb == 1 else []), k if runs else None)
        a, b = a + na, b + nb
    assert (a, b) == (61, 90)
    c.check()
    assert bool((c.ring[1] == 9).all()) and bool((c.ring[3] == 9).all())


def test_runs_are_cut_at_block_halves():
    runs = mixers.run_plan([2, 40, 9], [100, 5, 16], 1, 2)
    pos = {2 + i: 5 + i for i in range(40)} | {42 + i: 16 + i for i in range(9)}
    covered = []
    for t, n in runs.tolist():
        assert 1 <= n <= 8 and pos[t] // 8 == pos[t + n - 1] // 8 and pos[t + n - 1] - pos[t] == n - 1
        covered += range(t, t + n)
    assert covered == list(range(2, 51))


# ---------------------------------------------------------------- attention
def paged_kv(g, lens, G, D, V, dtype, spare=3):
    """Keys and values over shuffled blocks; slots past a sequence's end hold NaN, padding zeros."""
    sh = lk.diff_shape(G, G, D, V, 0, 1, True, 1.0, 0.5, 1e-6)
    kw, vp = lk.diff_pads(sh)
    need = [-(-n // BS) for n in lens]
    nb = sum(need) + spare
    perm = torch.randperm(nb, generator=g)
    kc, vc = torch.full((nb, G, BS, kw), math.nan), torch.full((nb, G, vp, BS), math.nan)
    tables = torch.zeros(len(lens), max(need), dtype=torch.int32)
    K, V_, used = [], [], 0
    for i, n in enumerate(lens):
        blocks = perm[used:used + need[i]]
        used += need[i]
        tables[i, :need[i]] = blocks.int()
        k, v = rnd(g, n, G, 2, D, dtype=dtype), rnd(g, n, G, V, dtype=dtype)
        flat = torch.full((need[i] * BS, G, 2, kw // 2), math.nan)
        flat[:n] = 0
        flat[:n, ..., :D] = k.float()
        kc[blocks] = flat.view(need[i], BS, G, kw).transpose(1, 2)
        flat = torch.full((need[i] * BS, G, vp), math.nan)
        flat[:n] = 0
        flat[:n, :, :V] = v.float()
        vc[blocks] = flat.view(need[i], BS, G, vp).permute(0, 2, 3, 1)
        K.append(k)
        V_.append(v)
    return kc.to(dtype).to(DEV), vc.to(dtype).to(DEV), tables.to(DEV), K, V_


def diff_oracle(q, K, V, gate, lam, sh):
    """q [H, 2, D] against the keys [n, G, 2, D] it sees."""
    out = []
    for h in range(sh.heads):
        g = h // (sh.heads // sh.kv_heads)
        a = [torch.softmax(K[:, g, m].double() @ q[h, m].double() * sh.scale, 0) @ V[:, g].double() for m in range(2)]
        out.append(ref.differential_combine(a[0], a[1], lam, sh.diff, sh.eps) * torch.sigmoid(gate[h].double()))
    return torch.stack(out)


def pad_q(q, dtype):
    T, H, _, D = q.shape
    out = torch.zeros(T, H, 2, (D + 15) // 16 * 16, dtype=dtype)
    out[..., :D] = q
    return out.view(T, H, -1).to(DEV)


ATTEND = [  # heads, kv_heads, dim, vdim
    (4, 2, 20, 28), (6, 3, 32, 64), (16, 2, 64, 128), (20, 1, 16, 40), (3, 3, 100, 72), (4, 1, 128, 256), (9, 1, 48, 200),
    (2, 1, 30, 150), (2, 2, 144, 300), (12, 4, 61, 5)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", ATTEND)
def test_diff_attend(heads, kv_heads, dim, vdim, dtype):
    """Contexts around block edges, unsplit and split; per head and map one key, near or far, stands out."""
    g = torch.Generator().manual_seed(dim + heads)
    pos = [0, 1, 2, 14, 15, 16, 17, 63, 64, 65, 200, 333, 700]
    kc, vc, tables, K, V = paged_kv(g, [p + 1 for p in pos], kv_heads, dim, vdim, dtype)
    T = len(pos)
    sh = lk.diff_shape(heads, kv_heads, dim, vdim, 0, 1, True, 1.0 / math.sqrt(dim), 0.35, 3e-5)
    q, gate = rnd(g, T, heads, 2, dim, dtype=dtype), rnd(g, T, heads + 3, dtype=dtype, scale=2.0)
    for i, p in enumerate(pos):
        for h in range(heads):
            for m in range(2):  # the two maps pick different keys
                j = ((0, p, p // 2, max(0, p - 1), min(p, 1), p // 3)[(h + 3 * m + i) % 6])
                q[i, h, m] = (K[i][j, h // (heads // kv_heads), m].float() * 0.6 + 0.3 * q[i, h, m].float()).to(dtype)
    lam = 0.83
    want = torch.stack([diff_oracle(q[i], K[i], V[i], gate[i, 3:], lam, sh) for i in range(T)]).reshape(T, -1)
    iota = torch.arange(T, dtype=torch.int32, device=DEV)
    for nparts, part_min in ((1, 64), (3, 16), (40, 64)):
        out = torch.full((T, heads * vdim + 9), 7.0, dtype=dtype, device=DEV)
        lk.diff_attend(sh, pad_q(q, dtype), gate.to(DEV)[:, 3:], kc, vc, tables, iota, torch.tensor(pos, device=DEV),
                       torch.tensor([lam], device=DEV), out[:, 4:4 + heads * vdim], nparts=nparts, part_min=part_min)
        close(out[:, 4:4 + heads * vdim], want, dtype)
        assert bool((out[:, :4] == 7).all()) and bool((out[:, 4 + heads * vdim:] == 7).all())


PREFILL = [  # heads, kv_heads, dim, vdim, [(start, tokens)]
    (4, 2, 20, 28, [(0, 70), (5, 33)]), (6, 3, 32, 64, [(0, 130), (300, 64), (79, 40)]),
    (8, 1, 64, 128, [(0, 300), (1100, 129)]), (16, 2, 64, 120, [(0, 128), (1, 32)]), (3, 1, 16, 40, [(17, 200)]),
    (2, 1, 100, 72, [(64, 128), (63, 65)]), (2, 2, 128, 256, [(3, 135)]), (2, 1, 48, 200, [(0, 64), (0, 65)]),
    (3, 3, 30, 150, [(15, 50)]), (2, 1, 96, 16, [(250, 48)])]


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,segs", PREFILL)
def test_diff_prefill(heads, kv_heads, dim, vdim, segs):
    g = torch.Generator().manual_seed(dim + vdim)
    kc, vc, tables, K, V = paged_kv(g, [3] + [s + n for s, n in segs], kv_heads, dim, vdim, BF16)
    lens, starts = [3] + [n for _, n in segs], [0] + [s for s, _ in segs]
    T = sum(lens)
    sh = lk.diff_shape(heads, kv_heads, dim, vdim, 0, 1, True, 1.0 / math.sqrt(dim), 0.6, 1e-5)
    q, gate = rnd(g, T, heads, 2, dim, dtype=BF16), rnd(g, T, heads, dtype=BF16, scale=2.0)
    want, tok, lam = torch.zeros(T, heads * vdim, dtype=torch.float64), 3, -0.4
    for i, (s, n) in enumerate(segs, 1):
        for t in range(n):
            p = s + t
            for h in range(heads):
                for m in range(2):
                    j = (0, p, max(0, p - 1), p // 2, max(0, p - 64), p // 64 * 64)[(t + h + 3 * m) % 6]
                    q[tok + t, h, m] = (K[i][j, h // (heads // kv_heads), m].float() * 0.6
                                        + 0.3 * q[tok + t, h, m].float()).to(BF16)
        k, v = (x[:, torch.arange(heads) // (heads // kv_heads)].double() for x in (K[i], V[i]))
        see = torch.arange(s + n)[None] <= torch.arange(s, s + n)[:, None]
        a = []
        for m in range(2):
            sc = torch.einsum("ihd,jhd->hij", q[tok:tok + n, :, m].double(), k[:, :, m]) * sh.scale
            a.append(torch.einsum("hij,jhv->ihv", torch.softmax(sc.masked_fill(~see, -math.inf), -1), v))
        o = ref.differential_combine(a[0], a[1], lam, sh.diff, sh.eps)
        want[tok:tok + n] = (o * torch.sigmoid(gate[tok:tok + n].double())[:, :, None]).reshape(n, -1)
        tok += n
    tiles = torch.from_numpy(mixers.tile_plan(lens, starts, 1, 3)).to(DEV)
    out = torch.zeros(T, heads * vdim + 5, dtype=BF16, device=DEV)
    lk.diff_prefill(sh, pad_q(q, BF16), gate.to(DEV), kc, vc, tables, tiles, torch.tensor([lam], device=DEV),
                    out[:, :heads * vdim])
    assert not bool(out[:3].any()) and not bool(out[:, heads * vdim:].any())
    tok = 3
    for _, n in segs:
        close(out[tok:tok + n, :heads * vdim], want[tok:tok + n], BF16)
        tok += n


# ---------------------------------------------------------------- the model through the engine's steps
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(PARALLEL))
def test_model_whole_portions_and_decode(name, dtype):
    cfg = PARALLEL[name]
    m, w = build(cfg, dtype)
    toks = tokens_of(cfg, 150, 1)
    want, _ = ref.forward(toks, w, cfg)
    s = TraceSession(m, 512)
    for i, cuts in enumerate(([150], [2] * 10 + [130], [1] * 150, [33, 31, 32, 1, 1, 2, 16, 17, 1, 16], [3, 64, 60, 23])):
        model_close(feed(s, f"r{i}", toks, cuts), want, dtype)
        s.step([], [f"r{i}"])  # the next request takes its pages and state row
    assert s.core.allocator.num_free == s.core.allocator.num_blocks and len(s.core._free_rows) == 4


@pytest.mark.parametrize("name", sorted(PARALLEL))
def test_residual_after_every_layer(name):
    cfg = PARALLEL[name]
    m, w = build(cfg, torch.float32)
    toks = tokens_of(cfg, 60, 3)
    _, trail = ref.forward(toks, w, cfg)
    s = TraceSession(m, 64, use_graphs=False)
    r = s.core.open_request()
    r.prompt, r.blocks = list(toks), s.core.allocator.allocate(4)
    got = []
    m.forward_portions(s.core.runner._portion_inputs(s.core._batch_of([(r, 60)]), [(0, 59)]), s.core.runner.cache, got)
    assert len(got) == len(trail) == len(cfg["layers"])
    for a, b in zip(got, trail):
        close(a, b, torch.float32, f32=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("graphs", [True, False])
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_mixed_batches_equal_each_request_alone(name, graphs, dtype):
    """Requests of unequal lengths, some decoding while others are in their prompts, some left out of
    steps, ended and replaced by others on the same pages and rows."""
    cfg = PARALLEL[name]
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


def far_case():
    """One attention layer in which the queries of tokens 7, 8 and 9 are the keys of tokens 1, 2 and 3, which
    stand at the start only: their embeddings and the two projections differ by a swap of the width's halves."""
    cfg = parallel_config([diff_attention(heads=2, kv_heads=1, dim=32, vdim=32, rot_dims=4, conv=2, scale=0.9,
                                          scaling=False, base=1e9)], width=64, no_mlp=(0,))
    w = make_parallel_weights(cfg, 5)
    g = torch.Generator().manual_seed(1)
    common = torch.randn(32, 64, generator=g) * 0.3
    w["l0.mix.k"] = torch.cat([common] * 2).to(BF16)
    w["l0.mix.q"] = torch.cat([common.roll(32, 1)] * 4).to(BF16)
    w["embed"][7:10] = w["embed"][1:4].roll(32, 1)
    w["l0.norm1"] *= 0
    w["l0.mix.lq1"] *= 0  # lambda = diff: equal maps do not cancel
    w["l0.mix.lq2"] *= 0
    for n in ("q", "k"):
        w[f"l0.mix.{n}.conv"] = torch.tensor([0.0, 1.0]).expand(len(w[f"l0.mix.{n}.b"]), 2).to(BF16).contiguous()
        w[f"l0.mix.{n}.b"] *= 0
    toks = [1, 2, 3] + torch.randint(10, cfg["vocab"], (700,), generator=g).tolist()
    far = list(range(40, 703, 53))
    for i in far:
        toks[i] = 7 + i % 3
    return cfg, w, toks, far


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_and_far_keys(dtype):
    """A long context decoded token by token and in portions, with queries that look for the first tokens."""
    cfg, w, toks, far = far_case()
    wd = {k: v.double() for k, v in w.items()}
    want, _ = ref.forward(toks, wd, cfg)
    changed, _ = ref.forward([4, 5, 6] + toks[3:], wd, cfg)
    assert float((changed[far] - want[far]).abs().mean()) > 0.1 * rms(want)  # the far keys matter
    m, _ = build(cfg, dtype, max_len=1024)
    m.load_weights(w.items())
    s = TraceSession(m, 1024)
    model_close(feed(s, "x", toks, [101] + [1] * 602), want, dtype)
    s.step([], ["x"])
    model_close(feed(s, "y", toks, [37] * 19), want, dtype)


def test_cut_does_not_change_bf16_logits_beyond_rounding():
    """The same prompt in portions on both sides of the short-portion limit, token by token and whole."""
    cfg = PARALLEL["wide"]
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
    cfg = parallel_config([diff_attention(heads=8, kv_heads=2, dim=64, vdim=128, rot_dims=32, conv=4),
                           diff_attention(heads=8, kv_heads=2, dim=64, vdim=128, rot_dims=32, conv=4, kv_from=0)],
                          width=1024, ff=(2048, 2.0), vocab=4096)
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
    cfg = PARALLEL["odd"]
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
    cfg = PARALLEL["wide"]
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
    cfg = PARALLEL["odd"]
    m, _ = build(cfg, torch.float32)
    w2 = make_parallel_weights(cfg, 77)
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

    cfg = PARALLEL["odd"]
    w = make_parallel_weights(cfg, 4)
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
