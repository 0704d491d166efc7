"""Hybrid decoder (latent attention, gated delta rule) on the GPU: every layer kernel alone, then
the model through the engine's own steps, against the plain restatement in oracle/hybrid_ref.py.

Tolerances: f32 kernels differ from the f64 oracle by summation order (1e-4 relative to the values'
scale); bf16 ones by one rounding of inputs and weights each (2e-2). Model logits are compared by
the root mean square of the difference over that of the reference."""

import asyncio
import math

import pytest
import torch

from hybrid_cases import CONFIGS, config, delta, latent, make_weights
from oracle import hybrid_ref as ref
from hybrid_gpu import DEV, DTYPES, build, close, feed, generate, greedy, model_close, rnd, tokens_of
from skyrl_amd.inference_engines import layer_kernels as lk
from skyrl_amd.inference_engines import mixers
from skyrl_amd.inference_engines.engine import AMDInferenceEngine
from skyrl_amd.inference_engines.trace import TraceSession

pytestmark = pytest.mark.gpu
BS = mixers.BLOCK_SIZE


# ---------------------------------------------------------------- norms, gates, cap
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,H", [(3, 72), (2, 2048), (5, 1001), (2, 5001), (2, 8192), (1, 6)])
def test_add_norm(n, H, dtype):
    g = torch.Generator().manual_seed(H)
    for kind in ("layer", "rms"):
        for with_delta, with_step in ((True, True), (True, False), (False, True), (False, False)):
            h = rnd(g, n, H, scale=3.0) + 2.0
            d, s, w = rnd(g, n, H, dtype=dtype), rnd(g, H, dtype=dtype), rnd(g, H, dtype=dtype)
            want_h = h.double() + (d.double() if with_delta else 0) + (s.double() if with_step else 0)
            want = (ref.layer_norm if kind == "layer" else ref.rms_norm)(want_h, w.double(), 1e-3)
            hd = h.to(DEV)
            out = lk.add_norm(d.to(DEV) if with_delta else None, hd, w.to(DEV), 1e-3, kind=kind,
                              step=s.to(DEV) if with_step else None)
            close(hd, want_h, torch.float32, f32=1e-6)
            close(out, want, dtype, f32=1e-5, bf16=4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("I", [100, 1, 513])
def test_gate_mul_and_softcap(I, dtype):
    g = torch.Generator().manual_seed(I)
    x = rnd(g, 7, 2 * I, dtype=dtype, scale=2.0)
    a, b = x[:, :I].double(), x[:, I:].double()
    close(lk.gate_mul(x.to(DEV), "gelu_tanh"), ref.gelu_tanh(a) * b, dtype, bf16=4e-3)
    close(lk.gate_mul(x.to(DEV), "silu"), ref.silu(a) * b, dtype, bf16=4e-3)
    close(lk.softcap(x.to(DEV), 2.5), 2.5 * torch.tanh(x.double() / 2.5), torch.float32, f32=1e-5)
    assert torch.equal(lk.softcap(x.to(DEV), None).cpu(), x.float())


# ---------------------------------------------------------------- latent attention
def paged_latents(g, lens, rank, rot, dtype, spare=3):
    """Per sequence latents and key parts scattered over shuffled blocks full of other values."""
    row = lk.latent_row(rank, rot)
    need = [-(-n // BS) for n in lens]
    nb = sum(need) + spare
    perm = torch.randperm(nb, generator=g)
    cache = torch.zeros(nb, BS, row)
    cache[:, :, :rank + rot] = torch.randn(nb, BS, rank + rot, generator=g)
    cache = cache.to(dtype)
    tables = torch.zeros(len(lens), max(need), dtype=torch.int32)
    dense, used = [], 0
    for i, n in enumerate(lens):
        blocks = perm[used:used + need[i]]
        used += need[i]
        tables[i, :need[i]] = blocks.int()
        dense.append(cache[blocks].reshape(-1, row)[:n, :rank + rot])
    return cache, tables, dense


ATTEND = [  # heads, rank, rot, window
    (3, 40, 12, 37), (16, 80, 24, 72), (5, 33, 6, 1), (17, 128, 32, None), (4, 256, 64, 65), (16, 512, 64, 130),
    (20, 512, 128, None), (2, 24, 2, 16), (2, 700, 20, 33)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,rank,rot,window", ATTEND)
def test_latent_attend(heads, rank, rot, window, dtype):
    """Positions around every page and window edge, unsplit and split, with one key per (token, head)
    made to stand out: the farthest the window keeps, or the nearest it drops."""
    g = torch.Generator().manual_seed(rank + heads)
    W = window or 10 ** 9
    pos = sorted({0, 1, 15, 16, 17, 31, 200, 333} | {p for p in (W - 2, W - 1, W, W + 1, W + 16) if 0 <= p < 400})
    cache, tables, dense = paged_latents(g, [p + 1 for p in pos], rank, rot, dtype)
    T = len(pos)
    q = rnd(g, T, heads, rank + rot, dtype=dtype)
    for i, p in enumerate(pos):  # head h: query along the key `d` back
        for h in range(heads):
            d = (min(W - 1, p), min(W, p), 0, min(W + 1, p))[h % 4]
            q[i, h] = (dense[i][p - d].float() * 0.5 + 0.3 * q[i, h].float()).to(dtype)
    scale = 1.0 / math.sqrt(rank + rot)
    want = torch.zeros(heads, T, rank, dtype=torch.float64)
    for i, p in enumerate(pos):
        lo = max(0, p - W + 1)
        K = dense[i][lo:p + 1].double()
        s = torch.softmax(q[i].double() @ K.T * scale, -1)
        want[:, i] = s @ K[:, :rank]
    qd = q.to(DEV)
    qa = qd[:, :, :rank].transpose(0, 1).contiguous()
    iota = torch.arange(T, dtype=torch.int32, device=DEV)
    for nparts, part_min in ((1, 64), (3, 16), (40, 64)):
        out = lk.latent_attend(qa, qd[:, :, rank:], cache.to(DEV), rank, rot, tables.to(DEV), iota,
                               torch.tensor(pos, device=DEV), scale, window, nparts=nparts, part_min=part_min)
        close(out, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,rot,rank", [(3, 20, 12, 40), (16, 128, 64, 512), (1, 7, 2, 9)])
def test_latent_write(heads, dim, rot, rank, dtype):
    g = torch.Generator().manual_seed(dim)
    T = 9
    proj = rnd(g, T, heads * (dim + rot) + rank + rot, dtype=dtype)
    w = rnd(g, rank, dtype=dtype)
    r = {"base": 300.0, "dims": rot, "scaling": {"factor": 2.5, "original": 40, "fast": 4.0, "slow": 0.3}}
    pos = torch.tensor([0, 1, 2, 77, 15, 16, 40, 41, 99])
    slots = torch.tensor([3, 40, 17, -1, 16, 15, 0, 63, 31])
    cache = torch.full((4, BS, lk.latent_row(rank, rot)), 7.0).to(dtype).to(DEV)
    pd = proj.to(DEV)
    lk.latent_write(pd, rot, pos.to(DEV), slots.to(DEV), mixers.rotary_table(r, 100).to(DEV), cache, 1e-4, heads=heads,
                    dim=dim, rank=rank, norm_weight=w.to(DEV))
    p = proj.double()
    q = p[:, :heads * (dim + rot)].view(T, heads, dim + rot)
    q = torch.cat([q[..., :dim], ref.rotate_pairs(q[..., dim:], pos, r)], -1)
    close(pd[:, :heads * (dim + rot)], q.reshape(T, -1), dtype, bf16=4e-3)
    lat = heads * (dim + rot)
    row = torch.cat([ref.rms_norm(p[:, lat:lat + rank], w.double(), 1e-4),
                     ref.rotate_pairs(p[:, lat + rank:], pos, r)], -1)
    got = cache.view(-1, cache.shape[2])
    keep = slots >= 0
    close(got[slots[keep].to(DEV)][:, :rank + rot], row[keep], dtype, bf16=4e-3)
    touched = torch.zeros(64, dtype=torch.bool)
    touched[slots[keep]] = True
    assert bool((got[~touched.to(DEV)] == 7.0).all()) and bool((got[:, rank + rot:] == 7.0).all())


PREFILL = [  # heads, dim, rot, vdim, rank, window, [(start, tokens)]
    (3, 20, 12, 28, 40, 37, [(0, 70), (5, 33)]),
    (6, 40, 24, 72, 48, 80, [(0, 130), (300, 64), (79, 40)]),
    (2, 128, 64, 128, 512, 100, [(0, 300), (1000, 129)]),
    (2, 64, 64, 64, 96, None, [(17, 200)]),
    (1, 130, 62, 140, 50, 1, [(3, 35)]),
    (2, 200, 56, 250, 64, 64, [(64, 128), (63, 65)]),
]


@pytest.mark.parametrize("heads,dim,rot,vdim,rank,window,segs", PREFILL)
def test_latent_prefill(heads, dim, rot, vdim, rank, window, segs):
    """Prompt form over paged latents: gather, the two up-projections, the windowed kernel."""
    g = torch.Generator().manual_seed(dim + vdim)
    dtype, W = torch.bfloat16, window or 10 ** 9
    cache, tables, dense = paged_latents(g, [s + n for s, n in segs], rank, rot, dtype)
    lens, starts = [n for _, n in segs], [s for s, _ in segs]
    short = 3  # tokens of other sequences ahead of these in the step
    T = short + sum(lens)
    wuk = rnd(g, heads * dim, rank, dtype=dtype, scale=1 / math.sqrt(rank))
    wuv = rnd(g, heads * vdim, rank, dtype=dtype, scale=1 / math.sqrt(rank))
    q = rnd(g, T, heads * (dim + rot), dtype=dtype)
    scale = 1.5 / math.sqrt(dim + rot)
    keys, vals, tok = [], [], short
    for i, (s, n) in enumerate(segs):
        c, kr = dense[i][:, :rank].double(), dense[i][:, rank:].double()
        k = (c @ wuk.double().T).view(-1, heads, dim)
        keys.append(torch.cat([k, kr[:, None].expand(-1, heads, rot)], -1))
        vals.append((c @ wuv.double().T).view(-1, heads, vdim))
        for t in range(n):  # the edge keys stand out for some queries
            p = s + t
            d = (0, min(W - 1, p), min(W, p))[t % 3]
            q[tok + t] = (q[tok + t].float() * 0.5 + 0.7 * keys[i][p - d].reshape(-1).float()).to(dtype)
        tok += n
    seg, tiles, rows, longest = mixers.prompt_plan(lens, starts, 0, short, window)
    lat, k_rot = lk.latent_gather(cache.to(DEV), rank, rot, tables.to(DEV), torch.from_numpy(seg).to(DEV), rows, longest)
    out = torch.zeros(T, heads * vdim, dtype=dtype, device=DEV)
    qd, wuk, wuv = q.to(DEV), wuk.to(DEV), wuv.to(DEV)
    lk.latent_prefill(qd, torch.nn.functional.linear(lat, wuk), k_rot, torch.mm(wuv, lat.t()),
                      torch.from_numpy(tiles).to(DEV), heads, dim, rot, vdim, scale, window, out)
    tok = short
    assert not bool(out[:short].any())
    for i, (s, n) in enumerate(segs):
        qi = q[tok:tok + n].double().view(n, heads, dim + rot)
        sc = torch.einsum("ihd,jhd->hij", qi, keys[i]) * scale
        d = (s + torch.arange(n))[:, None] - torch.arange(s + n)[None]
        sc = sc.masked_fill((d < 0) | (d >= W), float("-inf"))
        want = torch.einsum("hij,jhv->ihv", torch.softmax(sc, -1), vals[i]).reshape(n, -1)
        close(out[tok:tok + n], want, dtype)
        tok += n


# ---------------------------------------------------------------- gated delta rule
DELTA = [  # heads, kv_heads, dim, vdim, taps
    (4, 2, 24, 36, 3), (3, 1, 64, 48, 3), (2, 2, 128, 128, 4), (3, 3, 18, 10, 1), (2, 1, 200, 130, 9), (1, 1, 16, 200, 2),
    (2, 2, 5, 3, 8)]


class DeltaCase:
    def __init__(self, heads, kv_heads, dim, vdim, taps, dtype, seed=0, rows=5):
        g = torch.Generator().manual_seed(seed + dim)
        self.sh = lk.delta_shape(heads, kv_heads, dim, vdim, taps, 2e-5)
        self.dtype, self.g = dtype, g
        self.conv = rnd(g, lk.delta_channels(self.sh), taps, dtype=dtype)
        self.a_log = rnd(g, heads) - 2.0
        self.dt_bias = rnd(g, heads)
        self.norm = rnd(g, vdim, dtype=dtype) + 1
        self.dev = [t.to(DEV) for t in (self.conv, self.a_log, self.dt_bias, self.norm)]
        self.S = torch.full((rows, heads, dim, lk.delta_vpad(self.sh)), 3.0, device=DEV)  # left by another request
        self.S[..., vdim:] = 0
        self.ring = torch.full((rows, taps, lk.delta_channels(self.sh)), 5.0, device=DEV).to(dtype)

    def inputs(self, n):
        return rnd(self.g, n, lk.delta_width(self.sh), dtype=self.dtype)

    def oracle(self, proj):
        sh, p = self.sh, proj.double()
        H, K, D, V = sh.heads, sh.kv_heads, sh.dim, sh.vdim
        ch = lk.delta_channels(sh)
        x = ref.silu(ref.short_conv(p[:, :ch], self.conv.double()))
        grp = torch.tensor([h // (H // K) for h in range(H)])
        q = (ref.unit(x[:, :K * D].view(-1, K, D)) * D ** -0.5)[:, grp]
        k = ref.unit(x[:, K * D:2 * K * D].view(-1, K, D))[:, grp]
        v = x[:, 2 * K * D:].view(-1, H, V)
        w = {"b": torch.eye(H).double(), "a": torch.eye(H).double(), "A_log": self.a_log.double(),
             "dt_bias": self.dt_bias.double()}
        beta, _ = ref.delta_gates(p[:, ch + H * V:ch + H * V + H], w, "")
        _, g = ref.delta_gates(p[:, ch + H * V + H:], w, "")
        o, S = ref.delta_recurrence(q, k, v, beta, g)
        return ref.rms_norm(o, self.norm.double(), sh.eps).reshape(len(p), -1) * ref.silu(p[:, ch:ch + H * V]), S

    def step(self, parts, first_prompt=None):
        """parts: [(row, start, proj)]; sequences from first_prompt on take the chunked form."""
        lens = [len(p) for _, _, p in parts]
        cu = torch.tensor([0] + lens).cumsum(0).int().to(DEV)
        rows = torch.tensor([r for r, _, _ in parts], dtype=torch.int32, device=DEV)
        pos = torch.cat([torch.arange(s, s + n) for (_, s, _), n in zip(parts, lens)]).to(DEV)
        proj = torch.cat([p for _, _, p in parts]).to(DEV)
        out = torch.zeros(len(proj), self.sh.heads * self.sh.vdim, dtype=self.dtype, device=DEV)
        k = len(parts) if first_prompt is None else first_prompt
        one = all(n == 1 for n in lens) and k == len(parts)
        if k:
            lk.delta_scan(self.sh, proj, *self.dev, cu[:k + 1], rows[:k], pos, self.S, self.ring, one, out)
        if k < len(parts):
            first = sum(lens[:k])
            chunk, ends = (torch.from_numpy(a).to(DEV) for a in mixers.chunk_plan(lens, k, first))
            lk.delta_prompt(self.sh, proj, *self.dev, cu, rows, pos, self.S, self.ring, chunk, ends, k, first, out)
        if not one:
            lk.conv_save(proj, lk.delta_channels(self.sh), cu, rows, pos, self.ring)
        return out.split(lens)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", DELTA)
def test_delta_forms_against_the_recurrence(shape, dtype):
    """Two sequences cut differently (token by token, short scans, chunked portions, both forms in one
    step), rows that another request left full, and an idle row."""
    c = DeltaCase(*shape, dtype)
    n = 150
    a, b = c.inputs(n), c.inputs(n)
    (wa, Sa), (wb, Sb) = c.oracle(a), c.oracle(b)
    before = c.S[2].clone(), c.ring[2].clone()
    outa, outb = [], []
    ia = ib = 0
    for na, nb, prompt in ((1, 2, None), (2, 64, 1), (1, 1, None), (70, 5, None), (1, 37, 1), (75, 41, 0)):
        oa, ob, _ = c.step([(3, ia, a[ia:ia + na]), (1, ib, b[ib:ib + nb]), (-1, 0, c.inputs(1))], prompt) \
            if prompt is None else c.step([(3, ia, a[ia:ia + na]), (1, ib, b[ib:ib + nb])], prompt) + (None,)
        outa.append(oa)
        outb.append(ob)
        ia, ib = ia + na, ib + nb
    assert ia == n and ib == n
    close(torch.cat(outa), wa, dtype)
    close(torch.cat(outb), wb, dtype)
    close(c.S[3][..., :c.sh.vdim], Sa, torch.float32, f32=1e-4)
    close(c.S[1][..., :c.sh.vdim], Sb, torch.float32, f32=1e-4)
    assert torch.equal(before[0], c.S[2]) and torch.equal(before[1], c.ring[2])


@pytest.mark.parametrize("shape", DELTA[:3])
def test_delta_long_decode_keeps_its_state(shape):
    c = DeltaCase(*shape, torch.float32, seed=9)
    x = c.inputs(200)
    want, S = c.oracle(x)
    got = torch.cat([c.step([(0, t, x[t:t + 1])])[0] for t in range(200)])
    close(got, want, torch.float32)
    close(c.S[0][..., :c.sh.vdim], S, torch.float32)


def test_delta_recalls_one_far_write():
    """A key written once, long ago, with slow decay: the same key must read it back in every form."""
    c = DeltaCase(1, 1, 32, 16, 1, torch.float32)
    c.a_log[:] = -9.0
    c.dev[1].copy_(c.a_log)
    x = c.inputs(400) * 0.1
    ch = lk.delta_channels(c.sh)
    x[:, ch + 16] = -6.0  # beta near 0 ...
    x[7, ch + 16] = 6.0   # ... but for one token
    x[399, :32] = x[7, 32:64] * 50.0
    x[7, 64:80] *= 50.0
    want, _ = c.oracle(x)
    close(c.step([(0, 0, x)], 0)[0][399:], want[399:], torch.float32)
    c.step([(1, 0, x[:300])], 0)
    c.step([(1, 300, x[300:398])])
    c.step([(1, 398, x[398:399])])
    close(c.step([(1, 399, x[399:])])[0], want[399:], torch.float32)


# ---------------------------------------------------------------- the model through the engine's steps
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_model_whole_portions_and_decode(name, dtype):
    cfg = CONFIGS[name]
    m, w = build(cfg, dtype)
    toks = tokens_of(cfg, 150, 1)
    want, _ = ref.forward(toks, w, cfg)
    s = TraceSession(m, 512)
    for i, cuts in enumerate(([150], [2] * 10 + [130], [1] * 150, [33, 31, 32, 1, 1, 2, 16, 17, 1, 16], [3, 64, 60, 23])):
        model_close(feed(s, f"r{i}", toks, cuts), want, dtype)
        s.step([], [f"r{i}"])  # the next request takes its pages and state row
    assert s.core.allocator.num_free == s.core.allocator.num_blocks and len(s.core._free_rows) == 4


def test_residual_after_every_layer_run():
    cfg = CONFIGS["odd"]
    m, w = build(cfg, torch.float32)
    toks = tokens_of(cfg, 60, 3)
    _, trail = ref.forward(toks, w, cfg)
    s = TraceSession(m, 64, use_graphs=False)
    r = s.core.open_request()
    r.prompt, r.blocks = list(toks), s.core.allocator.allocate(4)
    got = []
    m.forward_portions(s.core.runner._portion_inputs(s.core._batch_of([(r, 60)]), [(0, 59)]), s.core.runner.cache, got)
    assert len(got) == len(trail) == 2 + 3 * 2
    for a, b in zip(got, trail):
        close(a, b, torch.float32, f32=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("graphs", [True, False])
def test_mixed_batches_equal_each_request_alone(graphs, dtype):
    """Requests of unequal lengths, some decoding while others are in their prompts, some left out of
    steps, ended and replaced by others on the same pages and rows."""
    cfg = CONFIGS["odd"]
    m, w = build(cfg, dtype)
    lens = {"a": 120, "b": 49, "c": 1, "d": 90, "e": 70, "f": 33}
    toks = {k: tokens_of(cfg, n, i) for i, (k, n) in enumerate(lens.items())}
    want = {k: ref.forward(t, w, cfg)[0] for k, t in toks.items()}
    s = TraceSession(m, 128 + 64 + 128 + 128, use_graphs=graphs)
    at = {k: 0 for k in lens}  # "e" stays unfinished
    got = {k: [] for k in lens}
    plan = [{"a": 40, "b": 1, "c": 1}, {"a": 1, "b": 2}, {"d": 35, "b": 40}, {"a": 1, "b": 1, "d": 1}, {"a": 1, "d": 1},
            {"e": 2, "a": 70, "d": 2}, {"b": 1, "a": 1, "d": 1, "e": 1}, {"b": 1, "d": 1}, {"b": 3, "a": 5, "e": 33},
            {"a": 1, "d": 48}, {"f": 32, "e": 32, "d": 1}, {"e": 1, "f": 1}, {"e": 1}]
    for st in plan:
        ents = [{"id": k, "tokens": toks[k][at[k]:at[k] + n], "want": list(range(n))} for k, n in st.items()]
        for k, n in st.items():
            at[k] += n
        ended = [k for k in st if at[k] == lens[k]]
        out = s.step(ents, ended)
        for k, n in st.items():
            got[k].append(out[:n])
            out = out[n:]
    for k in lens:
        t = torch.cat(got[k])
        model_close(t, want[k][:len(t)], dtype)
    assert sum(len(torch.cat(v)) for v in got.values()) == sum(at.values())


def test_graph_replays_match_eager_steps():
    """Captured decode steps, replayed with eager portion steps and host work between them."""
    cfg = CONFIGS["once"]
    m, _ = build(cfg, torch.bfloat16)
    toks, other = tokens_of(cfg, 60, 5), tokens_of(cfg, 200, 6)
    outs = []
    for graphs in (True, False):
        s = TraceSession(m, 512, use_graphs=graphs)
        rows = [s.step([{"id": "x", "tokens": toks[:20], "want": []}])]
        for i in range(20, 60):
            if i % 5 == 0:
                s.step([{"id": "y", "tokens": other[i:i + 4], "want": [0]}])
                torch.cuda.synchronize()
            rows.append(s.step([{"id": "x", "tokens": toks[i:i + 1], "want": [0]}]))
        outs.append(torch.cat(rows[1:]))
    model_close(outs[0], outs[1].double(), torch.bfloat16)


@pytest.mark.parametrize("rows", [3, 40])
def test_graph_replays_at_larger_layers(rows):
    """The same with library products of a real model's size in the captured step: every replay against
    the eager step on its own cache and state."""
    cfg = config([latent(heads=8, dim=128, rot_dim=64, vdim=128, kv_rank=512, window=40),
                  delta(heads=8, kv_heads=4, dim=128, vdim=128, conv=4)], width=1024, ff=2048, vocab=4096)
    m, _ = build(cfg, torch.bfloat16)
    prompts = [tokens_of(cfg, 10 + i % 7, i) for i in range(rows)]
    ids = [f"r{i}" for i in range(rows)]
    sessions = [TraceSession(m, 64 * rows, max_live=rows, use_graphs=g) for g in (True, False)]
    for s in sessions:
        s.step([{"id": k, "tokens": p, "want": []} for k, p in zip(ids, prompts)])
    for t in range(6):
        step = [{"id": k, "tokens": [(31 * t + 7 * i) % cfg["vocab"]], "want": [0]} for i, k in enumerate(ids)]
        a, b = (s.step(step) for s in sessions)
        model_close(a, b.double(), torch.bfloat16)
        torch.cuda.synchronize()


def test_no_garbage_collection_inside_a_capture():
    """A discarded engine's graphs must not be destroyed while another engine captures: with a collection
    due at every allocation, none runs inside a capture."""
    import gc

    cfg = CONFIGS["plain"]
    m, _ = build(cfg, torch.bfloat16)
    prompts = [tokens_of(cfg, 5, 1)]
    old = generate(m, prompts, 40, temperature=0.0, max_tokens=3, ignore_eos=True)[1]
    old.cycle = old  # only the collector frees it
    del old
    phases, threshold = [], gc.get_threshold()
    note = lambda phase, info: phases.append(torch.cuda.is_current_stream_capturing())  # noqa: E731
    gc.callbacks.append(note)
    gc.set_threshold(1, 1, 1)
    try:
        out, eng = generate(m, prompts, 40, temperature=0.0, max_tokens=3, ignore_eos=True)
    finally:
        gc.set_threshold(*threshold)
        gc.callbacks.remove(note)
    assert len(eng.runner._graphs) > 0 and len(out["response_ids"][0]) == 3
    assert phases and not any(phases) and gc.isenabled()


def test_steps_without_wanted_logits_keep_their_inputs():
    """Decode steps that fetch nothing run ahead of the host: their staged inputs must not be overwritten."""
    cfg = CONFIGS["plain"]
    m, w = build(cfg, torch.float32)
    toks = tokens_of(cfg, 120, 8)
    want, _ = ref.forward(toks, w, cfg)
    s = TraceSession(m, 128)
    out = None
    for i, t in enumerate(toks):
        out = s.step([{"id": "x", "tokens": [t], "want": [0] if i == 119 else []}])
    model_close(out, want[119:], torch.float32)


# ---------------------------------------------------------------- generation
def test_greedy_generation_through_the_scheduler():
    """Six prompts on four rows, prompts cut by the step budget: f32 tokens equal the oracle's argmax
    chain, logprobs its log softmax; a cache too small for all preempts and recomputes."""
    cfg = CONFIGS["odd"]
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
    assert eng.core.stats["portions_steps"] > 0 and eng.core.stats["decode_steps"] > 0


def test_bf16_generation_is_independent_of_the_batch():
    """Greedy bf16 tokens alone and in a batch agree up to the first near-tie."""
    cfg = CONFIGS["once"]
    m, w = build(cfg, torch.bfloat16)
    prompts = [tokens_of(cfg, n, 40 + n) for n in (3, 50, 70)]
    batch, _ = generate(m, prompts, 100, temperature=0.0, max_tokens=30, ignore_eos=True)
    for i, p in enumerate(prompts):
        alone, _ = generate(m, [p], 100, max_prefill=4096, graphs=False, temperature=0.0, max_tokens=30, ignore_eos=True)
        a, b = alone["response_ids"][0], batch["response_ids"][i]
        k = next((j for j in range(30) if a[j] != b[j]), None)
        if k is not None:
            lg, _ = ref.forward(p + a[:k], w, cfg)
            assert float(lg[-1, a[k]] - lg[-1, b[k]]) < 0.3


def test_sampling_parameters_and_seeds():
    cfg = CONFIGS["recurrent"]
    m, _ = build(cfg, torch.bfloat16)
    p = [tokens_of(cfg, 20, 3)]
    kw = dict(temperature=1.0, top_p=0.9, top_k=20, max_tokens=16, seed=11, repetition_penalty=1.2, min_tokens=4)
    a, _ = generate(m, p, 50, **kw)
    b, _ = generate(m, p, 50, **kw)
    c, _ = generate(m, p, 50, **dict(kw, seed=12))
    assert a["response_ids"] == b["response_ids"] != c["response_ids"]
    d, _ = generate(m, p, 50, temperature=0.0, max_tokens=5, stop_token_ids=list(range(cfg["vocab"])))
    assert d["stop_reasons"] == ["stop"] and len(d["response_ids"][0]) == 1


def test_weight_update_sleep_and_wake():
    """Updated weights reach every derived tensor and captured graph; sleep drops cache and state."""
    cfg = CONFIGS["odd"]
    m, _ = build(cfg, torch.float32)
    w2 = make_weights(cfg, 77)
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


def test_larger_layers_bf16():
    """Real-sized heads (rank 512, 128 + 64, delta 128 x 128) through both forms."""
    cfg = config([latent(heads=4, dim=128, rot_dim=64, vdim=128, kv_rank=512, window=80),
                  delta(heads=4, kv_heads=2, dim=128, vdim=128, conv=4)], width=256, ff=512, loop=(0, 2, 2))
    m, w = build(cfg, torch.bfloat16)
    toks = tokens_of(cfg, 200, 2)
    want, _ = ref.forward(toks, w, cfg)
    s = TraceSession(m, 512)
    for i, cuts in enumerate(([200], [100, 20, 40] + [1] * 40)):
        model_close(feed(s, f"r{i}", toks, cuts), want, torch.bfloat16)


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_program_and_command_line(tmp_path, dtype, capsys, monkeypatch):
    """A checkpoint folder through the trace replay program (steps on stdin, logits as files) and through
    the generation command line: the same greedy tokens."""
    import io
    import json

    import numpy as np
    from safetensors.torch import save_file

    from skyrl_amd.inference_engines import __main__ as cli
    from skyrl_amd.inference_engines import trace

    cfg = CONFIGS["odd"]
    w = make_weights(cfg, 4)
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
