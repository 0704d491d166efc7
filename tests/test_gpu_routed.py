"""Sublayers between two grouped norms, low-rank queries, sinks and head gates, the generalized delta rule and routed
experts (Tativik) on the GPU: every kernel alone, then the model through the engine's own steps, against the plain
restatement in oracle/hybrid_ref.py. Tolerances as in test_gpu_hybrid.py."""

import asyncio
import io
import json
import math

import numpy as np
import pytest
import torch

from hybrid_cases import SANDWICH, general, low_rank, make_sandwich_weights, routed, sandwich_config
from hybrid_gpu import DEV, DTYPES, build, close, feed, generate, greedy, model_close, rms, rnd, tokens_of
from oracle import hybrid_ref as ref
from skyrl_amd.inference_engines import layer_kernels as lk
from skyrl_amd.inference_engines import mixers
from skyrl_amd.inference_engines.engine import AMDInferenceEngine
from skyrl_amd.inference_engines.trace import TraceSession
from test_gpu_hybrid import paged_latents

pytestmark = pytest.mark.gpu
BS = mixers.BLOCK_SIZE
BF16 = torch.bfloat16
dev = lambda t: None if t is None else t.to(DEV)  # noqa: E731


# ---------------------------------------------------------------- norms, tanh
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,groups", [(72, 3), (70, 5), (1, 1), (515, 1), (2048, 4), (2056, 257), (4100, 41), (8192, 8), (8190, 9), (64, 64)])
def test_gate_norm_add(H, groups, dtype):
    """One row and a sum of rows, with and without gate and gathering, from a residual and from none."""
    g = torch.Generator().manual_seed(H + groups)
    n, eps = 5, 3e-3
    for k, (parts, gated, gather, pad) in enumerate(((1, True, False, 0), (3, True, False, 8), (8, False, False, 0), (1, False, True, 0),
                                                     (1, True, False, 3))):
        a = rnd(g, 9 if gather else n * parts, H, dtype=dtype)
        if not gather:
            a[2 * parts:3 * parts] = 0
        rows = torch.tensor([3, 8, 0, 3, 1]) if gather else None
        z = rnd(g, n, H + pad, dtype=dtype, scale=2.0)[:, pad:] if gated else None
        zb = rnd(g, H) if gated else None
        w, wn, h = (rnd(g, H, dtype=dtype, scale=0.5) + 1, rnd(g, H, dtype=dtype, scale=0.5) + 1, rnd(g, n, H, scale=2.0))
        y = a[rows].double() if gather else a.double().view(n, parts, H).sum(1)
        if gated:
            y = y * torch.sigmoid(z.double() + zb.double())
        want = (0 if gather else h.double()) + 0.37 * ref.grouped_rms_norm(y, w.double(), groups, eps)
        hd = dev(h)
        if gated:
            z = dev(torch.cat([torch.zeros(n, pad, dtype=dtype), z], 1))[:, pad:]
        out = lk.gate_norm_add(dev(a), hd, dev(w), dev(wn), eps, groups=groups, mult=0.37, parts=parts, gate=z, gate_bias=dev(zb),
                               rows=dev(rows), fresh=gather)
        close(hd, want, torch.float32, f32=4e-6)
        close(out, ref.grouped_rms_norm(want, wn.double(), groups, eps), dtype, f32=4e-6, bf16=4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("I,pad", [(64, 8), (5, 0), (33, 3)])
def test_tanh_of_a_column_range(I, pad, dtype):
    x = rnd(torch.Generator().manual_seed(I), 7, I + pad, dtype=dtype, scale=2.0)
    close(lk.tanh(dev(x)[:, pad:]), torch.tanh(x[:, pad:].double()), dtype, f32=1e-6, bf16=4e-3)


# ---------------------------------------------------------------- latent attention: low-rank queries, sinks, gates
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,rot,rank,q_rank", [(3, 20, 12, 40, 30), (16, 64, 32, 256, 384), (1, 7, 2, 9, 5)])
def test_latent_write_by_halves_with_a_query_latent(heads, dim, rot, rank, q_rank, dtype):
    g = torch.Generator().manual_seed(dim)
    T, r = 9, {"base": 300.0, "dims": rot}
    pos = torch.tensor([0, 1, 2, 77, 15, 16, 40, 41, 99])
    slots = torch.tensor([3, 40, 17, -1, 16, 15, 0, 63, 31])
    proj = rnd(g, T, q_rank + rank + rot + 5, dtype=dtype)
    wq, w = rnd(g, q_rank, dtype=dtype), rnd(g, rank, dtype=dtype)
    table = mixers.rotary_table(r, 100).to(DEV)
    cache = torch.full((4, BS, lk.latent_row(rank, rot)), 7.0).to(dtype).to(DEV)
    pd = proj.to(DEV)
    lk.latent_write(pd, rot, dev(pos), dev(slots), table, cache, 1e-4, q_norm=dev(wq), rank=rank, norm_weight=dev(w), halves=True)
    p = proj.double()
    close(pd[:, :q_rank], ref.rms_norm(p[:, :q_rank], wq.double(), 1e-4), dtype, f32=1e-6, bf16=4e-3)
    assert torch.equal(pd[:, q_rank:].cpu(), proj[:, q_rank:])
    row = torch.cat([ref.rms_norm(p[:, q_rank:q_rank + rank], w.double(), 1e-4),
                     ref.rotate_halves(p[:, q_rank + rank:q_rank + rank + rot], pos, r)], -1)
    got, keep = cache.view(-1, cache.shape[2]), slots >= 0
    close(got[slots[keep].to(DEV)][:, :rank + rot], row[keep], dtype, bf16=4e-3)
    touched = torch.zeros(64, dtype=torch.bool)
    touched[slots[keep]] = True
    assert bool((got[~touched.to(DEV)] == 7.0).all()) and bool((got[:, rank + rot:] == 7.0).all())
    before = cache.clone()
    q = rnd(g, T, heads * (dim + rot), dtype=dtype)
    qd = dev(q)
    lk.latent_write(qd, rot, dev(pos), dev(slots), table, cache, 1e-4, heads=heads, dim=dim, halves=True)
    q3 = q.double().view(T, heads, dim + rot)
    want = torch.cat([q3[..., :dim], ref.rotate_halves(q3[..., dim:], pos, r)], -1)
    close(qd, want.reshape(T, -1), dtype, bf16=4e-3)
    lk.latent_write(pd, rot, dev(pos), dev(slots), table, cache, 1e-4, q_norm=dev(wq), halves=True)  # another layer's keys
    assert torch.equal(cache, before)


SINKS = torch.tensor([-30.0, 0.0, 2.5, 9.0, 60.0])  # from unheard to all there is


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,rank,rot,window", [(5, 40, 12, 37), (20, 80, 24, 72), (5, 33, 6, 1), (16, 512, 64, 130), (7, 512, 128, None), (5, 700, 20, 33)])
def test_attend_with_sinks_and_gates(heads, rank, rot, window, dtype):
    """Unsplit and split decode, the farthest key in the window and the nearest outside standing out."""
    g = torch.Generator().manual_seed(rank + heads)
    W = window or 10 ** 9
    pos = sorted({0, 1, 15, 16, 17, 31, 200, 333} | {p for p in (W - 2, W - 1, W, W + 1, W + 16) if 0 <= p < 400})
    cache, tables, dense = paged_latents(g, [p + 1 for p in pos], rank, rot, dtype)
    T, scale = len(pos), 1.0 / math.sqrt(rank + rot)
    q, gate, sinks = rnd(g, T, heads, rank + rot, dtype=dtype), rnd(g, T, heads + 3, dtype=dtype, scale=2.0), SINKS.repeat(9)[:heads]
    for i, p in enumerate(pos):
        for h in range(heads):
            d = (min(W - 1, p), min(W, p), 0)[h % 3]
            q[i, h] = (dense[i][p - d].float() * 0.5 + 0.3 * q[i, h].float()).to(dtype)
    want = torch.zeros(heads, T, rank, dtype=torch.float64)
    for i, p in enumerate(pos):
        K = dense[i][max(0, p - W + 1):p + 1].double()
        s = torch.cat([q[i].double() @ K.T * scale, sinks.double()[:, None]], 1)
        want[:, i] = torch.softmax(s, -1)[:, :-1] @ K[:, :rank]
    gated = want * torch.sigmoid(gate[:, 3:].double()).T[:, :, None]
    qd = dev(q)
    qa = qd[:, :, :rank].transpose(0, 1).contiguous()
    iota = torch.arange(T, dtype=torch.int32, device=DEV)
    for nparts, part_min in ((1, 64), (3, 16), (40, 64)):
        for gt, expect in ((None, want), (dev(gate)[:, 3:], gated)):
            out = lk.latent_attend(qa, qd[:, :, rank:], dev(cache), rank, rot, dev(tables), iota, torch.tensor(pos, device=DEV), scale,
                                   window, nparts=nparts, part_min=part_min, sinks=dev(sinks), gate=gt)
            for h in range(heads):  # head by head: their sizes differ by the sinks
                if float(sinks[h]) < 50:
                    close(out[h], expect[h], dtype)
                else:
                    assert float(out[h].abs().max()) < 1e-12


@pytest.mark.parametrize("heads,dim,rot,vdim,rank,window,segs", [
    (5, 20, 12, 28, 40, 37, [(0, 70), (5, 33)]), (6, 40, 24, 72, 48, 80, [(0, 130), (300, 64), (79, 40)]),
    (5, 128, 64, 128, 512, 100, [(0, 300), (1000, 129)]), (4, 130, 62, 140, 50, 1, [(3, 35)])])
def test_prefill_with_sinks_and_gates(heads, dim, rot, vdim, rank, window, segs):
    g = torch.Generator().manual_seed(dim + vdim)
    cache, tables, dense = paged_latents(g, [s + n for s, n in segs], rank, rot, BF16)
    lens, starts, short = [n for _, n in segs], [s for s, _ in segs], 3
    T = short + sum(lens)
    wuk, wuv = (rnd(g, heads * d, rank, dtype=BF16, scale=1 / math.sqrt(rank)) for d in (dim, vdim))
    q, gate, sinks = rnd(g, T, heads * (dim + rot), dtype=BF16), rnd(g, T, heads, dtype=BF16, scale=2.0), SINKS.repeat(2)[:heads]
    scale = 1.5 / math.sqrt(dim + rot)
    seg, tiles, rows, longest = mixers.prompt_plan(lens, starts, 0, short, window)
    lat, k_rot = lk.latent_gather(dev(cache), rank, rot, dev(tables), dev(torch.from_numpy(seg)), rows, longest)
    out = torch.zeros(T, heads * vdim, dtype=BF16, device=DEV)
    lk.latent_prefill(dev(q), torch.nn.functional.linear(lat, dev(wuk)), k_rot, torch.mm(dev(wuv), lat.t()), dev(torch.from_numpy(tiles)),
                      heads, dim, rot, vdim, scale, window, out, sinks=dev(sinks), gate=dev(gate))
    tok = short
    assert not bool(out[:short].any())
    for i, (s, n) in enumerate(segs):
        c, kr = dense[i][:, :rank].double(), dense[i][:, rank:].double()
        k = torch.cat([(c @ wuk.double().T).view(-1, heads, dim), kr[:, None].expand(-1, heads, rot)], -1)
        v = (c @ wuv.double().T).view(-1, heads, vdim)
        qi = torch.zeros(s + n, heads, dim + rot, dtype=torch.float64)
        qi[s:] = q[tok:tok + n].double().view(n, heads, -1)
        want = ref.sink_attention(qi, k, v, scale, window, sinks.double())[s:] * torch.sigmoid(gate[tok:tok + n].double())[:, :, None]
        got = out[tok:tok + n].view(n, heads, vdim)
        for h in range(heads):
            if float(sinks[h]) < 50:
                close(got[:, h], want[:, h], BF16)
            else:
                assert float(got[:, h].abs().max()) < 1e-12
        tok += n


# ---------------------------------------------------------------- generalized delta rule
class Rule:
    """Two sequences through the kernels in portions; state rows start full of other values."""

    lens, rows = (61, 150), (2, 0)

    def __init__(self, heads, dim, dtype, seed=0, lens=None):
        g = torch.Generator().manual_seed(seed)
        self.dtype, self.HD, self.lens = dtype, heads * dim, lens or self.lens
        self.sh = lk.gdelta_shape(heads, dim, 1e-4)
        self.proj = [rnd(g, n, 5 * self.HD + 3, dtype=dtype) for n in self.lens]
        self.wl = [rnd(g, n, self.HD, dtype=dtype) for n in self.lens]
        self.w0 = rnd(g, self.HD, scale=2.5) - 3.0
        self.ab, self.norm = rnd(g, self.HD), (rnd(g, self.HD, scale=0.3) + 1).to(dtype)
        self.state = rnd(g, 4, heads, dim, lk.gdelta_vpad(self.sh), scale=5.0).to(DEV)

    def oracle(self, i):
        H, D, HD = self.sh.heads, self.sh.dim, self.HD
        p = self.proj[i].double()
        r, k, v, gate, al = (p[:, j * HD:(j + 1) * HD].reshape(-1, H, D) for j in range(5))
        decay = torch.exp(-math.exp(-0.5) * torch.sigmoid(self.wl[i].double() + self.w0.double())).view(-1, H, D)
        a = torch.sigmoid(al + self.ab.double().view(H, D))
        o, S = ref.general_delta_recurrence(r, k, v, decay, a)
        return (ref.rms(o, self.sh.eps) * self.norm.double().view(H, D) * torch.sigmoid(gate)).reshape(-1, HD), S

    def run(self, cuts, prompt=True):
        """cuts: per step, the tokens of both sequences. Steps of 32 and more go through the chunks."""
        at, outs = [0, 0], [[], []]
        for c in cuts:
            parts = sorted(((i, n) for i, n in enumerate(c) if n), key=lambda x: not (prompt is False or x[1] < 32))
            lens, starts = [n for _, n in parts], [at[i] for i, _ in parts]
            k = len(lens) if not prompt else sum(n < 32 for n in lens)
            x, wl = (dev(torch.cat([t[i][at[i]:at[i] + n] for i, n in parts])) for t in (self.proj, self.wl))
            pos = dev(torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)]))
            cu = dev(torch.tensor([0] + lens).cumsum(0).int())
            rows = dev(torch.tensor([self.rows[i] for i, _ in parts], dtype=torch.int32))
            out = torch.zeros(len(x), self.HD, dtype=self.dtype, device=DEV)
            args = (self.sh, x, wl, dev(self.w0), dev(self.ab), dev(self.norm))
            if k:
                lk.gdelta_scan(*args, cu[:k + 1].contiguous(), rows[:k].contiguous(), pos, self.state, out)
            if k < len(lens):
                plan = mixers.chunk_plan(lens, k, sum(lens[:k]))
                lk.gdelta_prompt(*args, cu, rows, pos, self.state, *(dev(torch.from_numpy(t)) for t in plan), k, out)
            for (i, n), t in zip(parts, out.split(lens)):
                outs[i].append(t)
                at[i] += n
        assert tuple(at) == self.lens
        return [torch.cat(o) for o in outs]

    def check(self, outs):
        H, D = self.sh.heads, self.sh.dim
        for i, o in enumerate(outs):
            want, S = self.oracle(i)
            close(o, want, self.dtype, f32=2e-5)
            close(self.state[self.rows[i], :, :, :D], S, torch.float32, f32=2e-5)


CUTS = [[(61, 150)], [(1, 1)] * 61 + [(0, 1)] * 89, [(32, 2), (2, 64), (27, 33), (0, 51)], [(5, 31), (56, 119)], [(60, 149), (1, 1)]]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("heads,dim", [(2, 64), (3, 20), (1, 7), (2, 16), (5, 32), (1, 60), (2, 128), (1, 72), (2, 200), (1, 256), (2, 1)])
def test_general_delta_forms(heads, dim, cuts, dtype):
    r = Rule(heads, dim, dtype, seed=dim)
    other = r.state[[1, 3]].clone()
    r.check(r.run(cuts))
    assert torch.equal(r.state[[1, 3]], other)  # rows of other requests are left alone


@pytest.mark.parametrize("dim", [32, 64, 100])
def test_general_delta_fast_decay_and_strong_removal(dim):
    """The largest decays there are (64 of them span e^-39) and removal rates near 1, in chunks."""
    r = Rule(2, dim, torch.float32, seed=5)
    r.w0, r.ab = r.w0 + 12.0, r.ab + 4.0
    r.check(r.run([(61, 150)]))


def test_general_delta_long_and_far():
    """One loud write, heard 700 tokens later through chunks, short portions and single steps."""
    n, D = 760, 32
    r = Rule(1, D, torch.float32, seed=3, lens=(n, n))
    r.w0 = torch.full((D,), -9.0)
    r.ab = torch.full((D,), -4.0)
    for p in r.proj:
        p[:, D:3 * D] *= 0.1
        p[5, D:2 * D] = 3.0 * torch.eye(D)[7]
        p[5, 2 * D:3 * D] *= 60
        p[700:, :D] = torch.eye(D)[7] * 2.0
    cuts = [(200, 2), (31, 300), (33, 0), (1, 1)] + [(1, 1)] * 200 + [(295, 257)]
    assert sum(c[0] for c in cuts) == sum(c[1] for c in cuts) == n
    r.check(r.run(cuts))
    quiet = Rule(1, D, torch.float32, seed=3, lens=(n, n))
    quiet.w0, quiet.ab, quiet.proj = r.w0, r.ab, [p.clone() for p in r.proj]
    quiet.proj[0][5, 2 * D:3 * D] = 0
    assert rms(quiet.oracle(0)[0][700:] - r.oracle(0)[0][700:]) > 0.3 * rms(r.oracle(0)[0][700:])


def test_idle_rows_are_skipped():
    r = Rule(2, 20, BF16)
    before = r.state.clone()
    x, wl = dev(r.proj[0][:2].contiguous()), dev(r.wl[0][:2].contiguous())
    out = torch.full((2, r.HD), 7.0, dtype=BF16, device=DEV)
    lk.gdelta_scan(r.sh, x, wl, dev(r.w0), dev(r.ab), dev(r.norm), torch.tensor([0, 1, 2], dtype=torch.int32, device=DEV),
                   torch.tensor([-1, 1], dtype=torch.int32, device=DEV), torch.zeros(2, dtype=torch.int64, device=DEV), r.state, out)
    assert bool((out[0] == 7).all()) and torch.equal(r.state[[0, 2, 3]], before[[0, 2, 3]]) and not torch.equal(r.state[1], before[1])


# ---------------------------------------------------------------- routed experts
def close_calls(choice, top, groups, keep):
    """Whether a token's choice hangs on less than 1e-5."""
    T, E = choice.shape
    per = E // groups
    best = choice.view(T, groups, per).topk(min(2, per), -1).values.sum(-1).sort(-1, descending=True).values
    near = (best[:, keep - 1] - best[:, keep]) < 1e-5 if keep < groups else torch.zeros(T, dtype=torch.bool)
    kept = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, choice.view(T, groups, per).topk(min(2, per), -1).values.sum(-1).topk(keep, -1).indices, True)
    flat = choice.masked_fill(~kept.repeat_interleave(per, 1), -9.0).sort(-1, descending=True).values[:, :top + 1]
    return near | ((flat[:, :-1] - flat[:, 1:]) < 1e-5).any(-1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,experts,top,groups,keep", [(72, 10, 3, 1, 1), (128, 64, 8, 8, 4), (70, 12, 2, 4, 3), (2048, 32, 4, 4, 1),
                                                           (96, 256, 8, 8, 3), (64, 100, 5, 10, 2), (512, 128, 70, 2, 2), (264, 600, 9, 6, 5), (40, 6, 4, 6, 4), (33, 1, 1, 1, 1)])
def test_route(width, experts, top, groups, keep, dtype):
    """Negative and positive choice scores, groups whose best expert alone would win."""
    g = torch.Generator().manual_seed(experts)
    sh = lk.moe_shape(width, 8, experts, top, groups, keep)
    for n, mean in ((37, -1.5), (1, 0.0), (16, 0.4)):
        x, router = rnd(g, n, width, dtype=dtype), rnd(g, experts, width, dtype=dtype, scale=1.5 / math.sqrt(width))
        corr = rnd(g, experts, scale=0.4) + mean
        corr[::max(1, experts // groups)] += 0.5
        scores = torch.sigmoid(x.double() @ router.double().T)
        idx, weight = ref.route(scores, corr.double(), top, groups, keep)
        got, gw = lk.moe_route(sh, dev(x), dev(router), dev(corr))
        ok = ~close_calls(scores + corr.double(), top, groups, keep)
        assert int(ok.sum()) >= n * 0.6
        assert torch.equal(got.cpu().long()[ok], idx[ok])
        torch.testing.assert_close(gw.cpu().double(), scores.gather(1, got.cpu().long()), rtol=2e-5, atol=2e-6)


def test_group_scores_are_sums_of_two():
    """The group of the single best expert loses to one with two good ones."""
    choice = torch.tensor([[0.9, 0.1, 0.1, 0.6, 0.7, 0.2, 0.5, 0.55]])
    sh = lk.moe_shape(8, 8, 8, 2, 2, 1)
    z = torch.logit(choice.clamp(1e-4, 1 - 1e-4)).float()
    idx, w = lk.moe_route(sh, dev(torch.ones(1, 8)), dev((z.T / 8).expand(8, 8).contiguous()), torch.zeros(8, device=DEV))
    assert idx.tolist() == [[0, 3]] and abs(float(w[0, 0]) - 0.9) < 1e-5  # 0.9 + 0.6 beats 0.7 + 0.55
    z[0, 3] = -4.0
    idx, _ = lk.moe_route(sh, dev(torch.ones(1, 8)), dev((z.T / 8).expand(8, 8).contiguous()), torch.zeros(8, device=DEV))
    assert idx.tolist() == [[4, 7]]  # 0.9 + 0.1 loses to 0.7 + 0.55
    # corrected scores below zero still beat those of the other groups
    idx, w = lk.moe_route(sh, dev(torch.ones(1, 8)), dev((z.T / 8).expand(8, 8).contiguous()), torch.full((8,), -3.0, device=DEV))
    assert idx.tolist() == [[4, 7]] and abs(float(w[0, 0]) - 0.7) < 1e-5


@pytest.mark.parametrize("pairs,experts,tm", [(1, 1, 16), (37, 5, 16), (1000, 64, 64), (4096, 600, 128), (20000, 16, 128), (9, 1024, 16), (70001, 130, 256), (4097, 3, 16)])
def test_sort_lists_every_pair_once(pairs, experts, tm):
    g = torch.Generator().manual_seed(pairs)
    sh = lk.moe_shape(8, 8, experts, 1)
    idx = (torch.rand(pairs, 1, generator=g) ** 2 * experts).int().clamp(max=experts - 1)  # uneven, some without any
    order, tile_expert = (t.cpu() for t in lk.moe_sort(sh, dev(idx), tm))
    used = tile_expert[:-1] >= 0
    assert int(tile_expert[-1]) == int(used.sum()) == sum(-(-int(c) // tm) for c in idx.flatten().bincount()) and not bool(used[int(used.sum()):].any())
    listed = order[used]
    for e, row in zip(tile_expert[:-1][used].tolist(), listed):
        assert bool((idx.flatten()[row[row >= 0].long()] == e).all())
    assert sorted(listed[listed >= 0].tolist()) == list(range(pairs))


EXPERTS = [  # width, ff, experts, top, tokens
    (72, 28, 10, 3, 37), (128, 64, 16, 2, 300), (70, 19, 6, 2, 5), (256, 200, 8, 8, 40), (136, 72, 4, 1, 1), (512, 96, 3, 2, 400), (64, 8, 40, 4, 16)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff,experts,top,n", EXPERTS)
def test_experts(width, ff, experts, top, n, dtype):
    """Every tile size, uneven loads, experts without tokens."""
    g = torch.Generator().manual_seed(width + ff)
    sh = lk.moe_shape(width, ff, experts, top)
    x = rnd(g, n, width, dtype=dtype)
    wgu, wd = rnd(g, experts, 2, ff, width, dtype=dtype, scale=1.5 / math.sqrt(width)), rnd(g, experts, width, ff, dtype=dtype, scale=1 / math.sqrt(ff))
    bias = 3.0 * torch.rand(experts, generator=g) ** 3
    idx = (torch.rand(n, experts, generator=g) + bias).topk(top, -1).indices.int()
    weight = torch.rand(n, top, generator=g) + 0.2
    X, G, D = x.double(), wgu.double(), wd.double()
    want = torch.stack([weight[t, i].double() * (D[e] @ (ref.silu(G[e, 0] @ X[t]) * (G[e, 1] @ X[t])))
                        for t in range(n) for i, e in enumerate(idx[t].tolist())])
    for tm in (None, 16, 64, 128, 256):
        close(lk.moe_experts(sh, dev(x), dev(idx), dev(weight), dev(wgu), dev(wd), tm=tm), want, dtype, f32=5e-6, bf16=8e-3)


@pytest.mark.parametrize("width,ff,experts,top,n", [(2048, 768, 32, 8, 1500), (1024, 512, 64, 4, 300), (4096, 320, 8, 2, 90)])
def test_tile_sizes_agree_bit_for_bit(width, ff, experts, top, n):
    """A row's sums are formed in the same order whatever its tile: products of a real layer's size, over and over."""
    g = torch.Generator(device=DEV).manual_seed(width)
    sh = lk.moe_shape(width, ff, experts, top)
    mk = lambda *s, scale=1.0: (torch.randn(s, generator=g, device=DEV) * scale).to(BF16)  # noqa: E731
    x, wgu, wd = mk(n, width), mk(experts, 2, ff, width, scale=0.03), mk(experts, width, ff, scale=0.03)
    idx, weight = lk.moe_route(sh, x, mk(experts, width, scale=0.03), torch.zeros(experts, device=DEV))
    outs = [lk.moe_experts(sh, x, idx, weight, wgu, wd, tm=tm) for _ in range(4) for tm in (16, 64, 128, 256)]
    rows = torch.randint(0, n * top, (8,), generator=torch.Generator().manual_seed(1))
    for r in rows.tolist():
        t, e = r // top, int(idx[r // top, r % top])
        h = x[t].double().cpu()
        a = ref.silu(wgu[e, 0].double().cpu() @ h) * (wgu[e, 1].double().cpu() @ h)
        close(outs[0][r], float(weight[t, r % top]) * (wd[e].double().cpu() @ a), BF16, bf16=8e-3)
    assert all(torch.equal(outs[0], o) for o in outs[1:])


# ---------------------------------------------------------------- the model through the engine's steps
def shaped(cfg, dtype, seed=0, max_len=512):
    """f32: routing by the tokens; bf16: a choice that rounding does not change."""
    return build(cfg, dtype, max_len=max_len, w=make_sandwich_weights(cfg, seed, steady=dtype == BF16))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(SANDWICH))
def test_model_whole_portions_and_decode(name, dtype):
    cfg = SANDWICH[name]
    m, w = shaped(cfg, dtype)
    toks = tokens_of(cfg, 150, 1)
    want, _ = ref.forward(toks, w, cfg)
    s = TraceSession(m, 512)
    for i, cuts in enumerate(([150], [2] * 10 + [130], [1] * 150, [33, 31, 32, 1, 1, 2, 16, 17, 1, 16], [3, 64, 60, 23])):
        model_close(feed(s, f"r{i}", toks, cuts), want, dtype)
        s.step([], [f"r{i}"])  # the next request takes its pages and state row
    assert s.core.allocator.num_free == s.core.allocator.num_blocks and len(s.core._free_rows) == 4


@pytest.mark.parametrize("name", sorted(SANDWICH))
def test_residual_after_every_layer(name):
    cfg = SANDWICH[name]
    m, w = shaped(cfg, torch.float32)
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
    cfg = SANDWICH[name]
    m, w = shaped(cfg, dtype)
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


def window_case(size, shared):
    """Attention layers alone, loud (their output norm's weight). The query of tokens 21 .. 40 is the key of tokens 1 ..
    20: the latent query is the latent key's mirror, unrotated; such pairs stand size - 1 (inside) and size (outside)
    tokens apart. With `shared` the window is that of a layer on the first one's latents."""
    W = 64
    one = low_rank(heads=2, dim=32, rot_dim=4, vdim=32, kv_rank=32, q_rank=32, window=7 if shared else size, scale=0.6)
    layers = [one] + ([low_rank(heads=2, dim=32, rot_dim=4, vdim=32, kv_rank=32, q_rank=32, window=size, scale=0.6, kv_from=0)] if shared else [])
    cfg = sandwich_config(layers, [None] * len(layers), width=W, groups=1, mult=1.0)
    w = make_sandwich_weights(cfg, 5)
    g = torch.Generator().manual_seed(1)
    common = torch.randn(32, W, generator=g) / 8
    w["l0.mix.dkv"][:32] = common.to(BF16)
    w["embed"][21:41] = w["embed"][1:21].roll(32, 1)
    ones = {"embed.norm", "l0.norm1", "l0.mix.dkv.norm"}
    loud = len(layers) - 1
    for i in range(len(layers)):
        p = f"l{i}."
        w[p + "mix.dq"] = common.roll(32, 1).to(BF16)
        w[p + "mix.uq"] = torch.cat([torch.cat([torch.eye(32), torch.zeros(4, 32)])] * 2).to(BF16)
        w[p + "mix.uk"] = torch.cat([torch.eye(32)] * 2).to(BF16)
        ones |= {p + "mix.dq.norm", p + "norm1"}
        w[p + "norm1b"] = torch.full((W,), 3.0 if i == loud else 0.0).to(BF16)
    for n in ones:
        w[n] = torch.ones_like(w[n])
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
@pytest.mark.parametrize("shared", [False, True])
@pytest.mark.parametrize("size", [2, 16, 33, 64, 100])
def test_window_edges_in_prompts_and_decoding(size, shared, dtype):
    cfg, w, toks, inside, outside = window_case(size, shared)
    wd = {k: v.double() for k, v in w.items()}
    want, _ = ref.forward(toks, wd, cfg)

    def with_window(n):
        e = cfg["layers"][-1]
        other = dict(cfg, layers=cfg["layers"][:-1] + [dict(e, mixer=dict(e["mixer"], mask={"size": n}))])
        return (ref.forward(toks, wd, other)[0] - want).pow(2).mean(-1).sqrt() / rms(want)

    if size > 2:  # a window one token off would show
        assert float(with_window(size - 1)[inside].mean()) > 0.1 and float(with_window(size + 1)[outside].mean()) > 0.1
    m, _ = build(cfg, dtype, w=w)
    s = TraceSession(m, 320)
    for i, cuts in enumerate(([300], [101] + [1] * 199, [37] * 8 + [4], [2] * 150)):
        model_close(feed(s, f"w{i}", toks, cuts), want, dtype)
        s.step([], [f"w{i}"])


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_with_far_memory(dtype):
    """States that hardly decay: the first tokens are heard hundreds of tokens later, through decode steps and portions."""
    cfg = sandwich_config([general(heads=2, dim=64)], [None], width=64, groups=2, mult=1.0)
    w = make_sandwich_weights(cfg, 5)
    w["l0.mix.w0"][:] = -9.0
    w["l0.mix.a.b"][:] = -5.0
    w["l0.norm1b"] *= 3
    toks = tokens_of(cfg, 620, 8)
    wd = {k: v.double() for k, v in w.items()}
    want, _ = ref.forward(toks, wd, cfg)
    changed, _ = ref.forward([(t + 1) % cfg["vocab"] for t in toks[:200]] + toks[200:], wd, cfg)
    assert float((changed[560:] - want[560:]).pow(2).mean().sqrt()) > 0.03 * rms(want)
    m, _ = build(cfg, dtype, max_len=640, w=w)
    s = TraceSession(m, 640)
    model_close(feed(s, "x", toks, [101] + [1] * 519), want, dtype)
    s.step([], ["x"])
    model_close(feed(s, "y", toks, [37] * 16 + [28]), want, dtype)


@pytest.mark.parametrize("what", ["sink", "g", "rg1", "a.b", "correction", "kv_from", "groups", "residual_mult"])
def test_every_part_is_heard(what):
    """A wrong sink, gate, rate, correction, cache or constant moves the oracle by far more than the tolerance."""
    cfg = SANDWICH["odd"]
    w = {k: v.double() for k, v in make_sandwich_weights(cfg, 0, steady=False).items()}
    toks = tokens_of(cfg, 60, 1)
    want, _ = ref.forward(toks, w, cfg)
    other, changed = dict(w), json.loads(json.dumps(cfg))
    for k in w:
        if k.endswith("." + what):
            other[k] = torch.zeros_like(w[k])
    if what == "kv_from":
        changed["layers"][2]["mixer"].pop("kv_from")
        other["l2.mix.dkv"], other["l2.mix.dkv.norm"] = w["l0.mix.dkv"], w["l0.mix.dkv.norm"]
    if what == "groups":
        changed["norm"]["groups"] = 1
    if what == "residual_mult":
        changed["residual_mult"] = 1.0
    assert rms(ref.forward(toks, other, changed)[0] - want) > 0.02 * rms(want)
    m, _ = build(cfg, torch.float32, w=make_sandwich_weights(cfg, 0, steady=False))
    model_close(feed(TraceSession(m, 64), "x", toks, [40, 20]), want, torch.float32)


def test_cut_does_not_change_bf16_logits_beyond_rounding():
    """The same prompt in portions on both sides of the short-portion limit, token by token and whole."""
    cfg = SANDWICH["wide"]
    m, _ = shaped(cfg, BF16)
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
    cfg = sandwich_config([general(heads=16, dim=64, decay_rank=64),
                           low_rank(heads=8, dim=128, rot_dim=64, vdim=128, kv_rank=256, q_rank=384, window=40)],
                          [routed(ff=256, experts=32, top=4, groups=(8, 4)), routed(ff=512, experts=16, top=2)], width=1024, groups=4, vocab=4096)
    m, _ = shaped(cfg, BF16)
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
    cfg = SANDWICH["odd"]
    m, w = shaped(cfg, torch.float32)
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
    cfg = SANDWICH["wide"]
    m, w = shaped(cfg, BF16)
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
    cfg = SANDWICH["odd"]
    m, _ = shaped(cfg, torch.float32)
    w2 = make_sandwich_weights(cfg, 77, steady=False)
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
    """A checkpoint folder, whose config leaves the decay's rank to a tensor's shape, through the trace replay program
    and the generation command line."""
    from safetensors.torch import save_file

    from skyrl_amd.inference_engines import __main__ as cli
    from skyrl_amd.inference_engines import trace

    cfg = json.loads(json.dumps(SANDWICH["odd"]))
    w = make_sandwich_weights(cfg, 4)
    for e in cfg["layers"]:
        e["mixer"].pop("decay_rank", None)
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
