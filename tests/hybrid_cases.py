"""Small hybrid-decoder configurations and weights for the tests, made from a seed."""

import math

import torch


def latent(heads=3, dim=20, rot_dim=12, vdim=28, kv_rank=40, window=37, scale=None, base=5000.0, scaling=True):
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 0.5}
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": rot,
         "scale": scale or 1.3 / math.sqrt(dim + rot_dim)}
    if window:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m}


def delta(heads=4, kv_heads=2, dim=24, vdim=36, conv=3):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def config(layers, width=72, vocab=211, ff=100, loop=None, softcap=9.0, eps=3e-5, no_mlp=()):
    layers = [dict(e, mlp=None if i in no_mlp else {"kind": "dense", "ff": ff}) for i, e in enumerate(layers)]
    cfg = {"architecture": "Dovidra", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    if softcap:
        cfg["logit_softcap"] = softcap
    return cfg


CONFIGS = {
    # odd sizes, two windows, a loop over both kinds
    "odd": config([delta(), latent(), latent(heads=5, dim=18, rot_dim=6, vdim=11, kv_rank=33, window=16),
                   delta(heads=3, kv_heads=3, dim=18, vdim=10, conv=5)], loop=(1, 3, 3)),
    # no loop, no cap, layers without a feed-forward, no window, no rotary scaling
    "plain": config([latent(window=None, scaling=False), delta(heads=2, kv_heads=1, dim=64, vdim=64, conv=4),
                     latent(window=1)], width=128, softcap=None, no_mlp=(0, 2)),
    # loop from the first to the last layer, once; shapes the matrix kernels take exactly
    "once": config([latent(heads=16, dim=32, rot_dim=32, vdim=32, kv_rank=96, window=50),
                    delta(heads=4, kv_heads=4, dim=32, vdim=48, conv=1)], width=96, ff=64, loop=(0, 2, 1)),
    # only recurrent layers, wide convolution
    "recurrent": config([delta(heads=6, kv_heads=3, dim=16, vdim=16, conv=9), delta(conv=2)], width=64,
                        loop=(1, 2, 2), no_mlp=(1,)),
}


def make_weights(cfg, seed=0):
    """bf16 tensors by checkpoint name. Decays span short and long memory, norms and gates are not 1."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    w = {}

    def mat(name, rows, cols, gain=1.0):
        w[name] = torch.randn(rows, cols, generator=g) * gain / math.sqrt(cols)

    def vec(name, n, mean=1.0, std=0.2):
        w[name] = mean + std * torch.randn(n, generator=g)

    w["embed"] = torch.randn(cfg["vocab"], W, generator=g)
    if cfg.get("loop"):
        w["loop.step"] = torch.randn(cfg["loop"]["times"], W, generator=g)
    for i, e in enumerate(cfg["layers"]):
        p, m = f"l{i}.", e["mixer"]
        vec(p + "norm1", W)
        q = p + "mix."
        if e["type"] == "latent_attention":
            H, C = m["heads"], m["kv_rank"]
            mat(q + "q", H * (m["dim"] + m["rot_dim"]), W, 2.0)
            mat(q + "dkv", C + m["rot_dim"], W, 1.5)
            vec(q + "dkv.norm", C)
            mat(q + "uk", H * m["dim"], C)
            mat(q + "uv", H * m["vdim"], C)
            mat(q + "o", W, H * m["vdim"])
        else:
            H, K = m["heads"], m["kv_heads"]
            for n, rows in (("q", K * m["dim"]), ("k", K * m["dim"]), ("v", H * m["vdim"])):
                mat(q + n, rows, W)
                w[q + n + ".conv"] = torch.randn(rows, m["conv"], generator=g) / math.sqrt(m["conv"])
            mat(q + "b", H, W)
            mat(q + "a", H, W)
            vec(q + "A_log", H, -2.0, 1.5)
            vec(q + "dt_bias", H, 0.0, 1.0)
            vec(q + "norm", m["vdim"])
            mat(q + "g", H * m["vdim"], W)
            mat(q + "o", W, H * m["vdim"], 1.5)
        if e.get("mlp"):
            vec(p + "norm2", W)
            mat(p + "mlp.gate", e["mlp"]["ff"], W)
            mat(p + "mlp.up", e["mlp"]["ff"], W)
            mat(p + "mlp.down", W, e["mlp"]["ff"])
    vec("final.norm", W)
    mat("head", cfg["vocab"], W, 3.0)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


# ---------------------------------------------------------------- parallel layers of differential attention
def diff_attention(heads=4, kv_heads=2, dim=20, vdim=28, conv=3, rot_dims=8, diff=0.35, scale=None, base=700.0,
                   scaling=True, kv_from=None):
    rot = {"base": base, "dims": rot_dims}
    if scaling:
        rot["scaling"] = {"factor": 5.0, "original": 48, "fast": 6.0, "slow": 0.4}
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "diff": diff, "rot": rot,
         "scale": scale or 1.4 / math.sqrt(dim)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def parallel_config(layers, width=72, vocab=203, ff=(100, 1.3), scale=2.7, eps=4e-5, no_mlp=()):
    layers = [dict(e, mlp=None if i in no_mlp else {"kind": "dense", "ff": ff[0] + 4 * i, "limit": ff[1] + 0.2 * i})
              for i, e in enumerate(layers)]
    return {"architecture": "Lipedra", "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "vocab": vocab, "width": width}


PARALLEL = {
    # sizes no vector width divides, two layers on one cache with other constants than its owner, no feed-forward
    "odd": parallel_config([diff_attention(), diff_attention(heads=6, kv_heads=3, dim=22, vdim=11, conv=5, rot_dims=22),
                            diff_attention(heads=6, kv_heads=3, dim=22, vdim=11, conv=2, rot_dims=22, kv_from=1, diff=0.7,
                                           scale=0.5),
                            diff_attention(heads=4, kv_heads=2, kv_from=0, conv=4)], no_mlp=(2,)),
    # exact matrix-kernel shapes, many query heads per key head (more than one group), no scaling
    "wide": parallel_config([diff_attention(heads=20, kv_heads=1, dim=32, vdim=64, rot_dims=16, scaling=False, conv=4),
                             diff_attention(heads=2, kv_heads=2, dim=64, vdim=128, rot_dims=64, conv=1),
                             diff_attention(heads=20, kv_heads=1, dim=32, vdim=64, rot_dims=16, scaling=False, kv_from=0,
                                            conv=4)], width=128, ff=(96, 0.7)),
    # padded shapes of the matrix kernels: both maps in one step, values beyond one tile count, many taps
    "padded": parallel_config([diff_attention(heads=3, kv_heads=1, dim=48, vdim=24, rot_dims=2, conv=8),
                               diff_attention(heads=8, kv_heads=4, dim=16, vdim=136, rot_dims=6, conv=11),
                               diff_attention(heads=2, kv_heads=1, dim=104, vdim=200, rot_dims=40, conv=6)], width=56,
                              ff=(68, 2.5), scale=0.6),
}


def make_parallel_weights(cfg, seed=0):
    """bf16 tensors by checkpoint name: biases, norm offsets and gates far from trivial, feed-forward
    projections that reach the clamp."""
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def rand(name, *shape, gain=1.0):
        w[name] = torch.randn(*shape, generator=g) * gain

    def proj(name, rows, cols, gain=1.0, bias=True):
        rand(name, rows, cols, gain=gain / math.sqrt(cols))
        if bias:
            rand(name + ".b", rows, gain=0.3)

    rand("embed", cfg["vocab"], W)
    for i, e in enumerate(cfg["layers"]):
        p, m = f"l{i}.", e["mixer"]
        q = p + "mix."
        rand(p + "norm1", W, gain=0.3)
        rows = [("q", 2 * m["heads"] * m["dim"])]
        if m.get("kv_from") is None:
            rows += [("k", 2 * m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])]
        for n, r in rows:
            proj(q + n, r, W, 1.3)
            rand(q + n + ".conv", r, m["conv"], gain=1 / math.sqrt(m["conv"]))
        for n in ("lq1", "lk1", "lq2", "lk2"):
            rand(q + n, m["dim"], gain=0.25)
        proj(q + "g", m["heads"], W, 1.5, bias=False)
        proj(q + "o", W, m["heads"] * m["vdim"], 1.5, bias=False)
        if e.get("mlp"):
            ff = e["mlp"]["ff"]
            proj(p + "mlp.gate", ff, W, 1.5)
            proj(p + "mlp.up", ff, W, 1.5)
            proj(p + "mlp.down", W, ff)
    rand("final.norm", W, gain=0.3)
    proj("head", cfg["vocab"], W, 3.0, bias=False)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


# ---------------------------------------------------------------- output-normed recurrent and side-by-side layers
def rglru(width=60, blocks=3, conv=3):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def attend(heads=4, kv_heads=2, dim=20, vdim=28, window=37, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or 1.6 / math.sqrt(dim)}
    if window:
        m["mask"] = {"size": window}
    return m


def ssd(heads=3, vdim=20, state=18, groups=1, conv=5, norm_groups=2):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def side(left=None, right=None):
    return {"type": "parallel", "mixer": {"left": left or attend(), "right": right or ssd()}}


def normed_config(layers, width=72, vocab=199, ff=100, scale=3.3, eps=2e-5, no_mlp=()):
    layers = [dict(e, mlp=None if i in no_mlp else {"kind": "dense", "ff": ff + 4 * i}) for i, e in enumerate(layers)]
    return {"architecture": "Foduzen", "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "vocab": vocab, "width": width}


NORMED = {
    # sizes no vector width divides, an odd state, one tap, no feed-forward in two layers
    "odd": normed_config([rglru(), side(), rglru(width=50, blocks=2, conv=1), side(attend(heads=3, kv_heads=3, dim=17, vdim=9, window=16),
                          ssd(heads=4, vdim=14, state=11, groups=2, conv=2, norm_groups=2))], width=70, no_mlp=(1, 2)),
    # shapes the matrix kernels take exactly, one key head, window 1 tile and a half, groups shared by heads
    "wide": normed_config([side(attend(heads=16, kv_heads=1, dim=64, vdim=128, window=96),
                                ssd(heads=4, vdim=64, state=128, groups=2, conv=4, norm_groups=1)),
                           rglru(width=256, blocks=2, conv=4), rglru(width=128, blocks=8, conv=4)], width=128, ff=96),
    # padded shapes: many query heads, values of more than one slice, nine taps, no window
    "padded": normed_config([rglru(width=96, blocks=6, conv=9),
                             side(attend(heads=20, kv_heads=1, dim=40, vdim=24, window=None),
                                  ssd(heads=6, vdim=72, state=40, groups=3, conv=7, norm_groups=2)),
                             side(attend(heads=2, kv_heads=2, dim=136, vdim=152, window=3),
                                  ssd(heads=2, vdim=24, state=160, groups=1, conv=1, norm_groups=2))], width=88, ff=60,
                            scale=0.8, no_mlp=(0,)),
}


def make_normed_weights(cfg, seed=0):
    """bf16 tensors by checkpoint name: decays from short to long memory, norms, gates and biases far from trivial."""
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def rand(name, *shape, gain=1.0, mean=0.0):
        w[name] = mean + torch.randn(*shape, generator=g) * gain

    def mat(name, rows, cols, gain=1.0, bias=False):
        rand(name, rows, cols, gain=gain / math.sqrt(cols))
        if bias:
            rand(name + ".b", rows, gain=0.4)

    def conv(q, channels, taps):
        rand(q + "conv", channels, taps, gain=1 / math.sqrt(taps))
        rand(q + "conv.b", channels, gain=0.3)

    def number(name):
        w[name] = (1 + 0.4 * torch.randn((), generator=g))

    rand("embed", cfg["vocab"], W)
    for i, e in enumerate(cfg["layers"]):
        p, m = f"l{i}.", e["mixer"]
        q = p + "mix."
        number(p + "norm1")
        if e["type"] == "rglru":
            C, b = m["width"], m["blocks"]
            mat(q + "y", C, W, 1.3 / cfg["embedding"]["scale"] ** 0.5, bias=True)
            mat(q + "x", C, W, 1.3 / cfg["embedding"]["scale"] ** 0.5, bias=True)
            conv(q, C, m["conv"])
            for n in ("ra", "ri"):
                rand(q + n, b, C // b, C // b, gain=1.5 / math.sqrt(C // b))
                rand(q + n + ".b", b, C // b, gain=0.7)
            rand(q + "lam", C, gain=3.0, mean=-4.0)
            mat(q + "o", W, C)
        else:
            a, s, l, r = m["left"], m["right"], q + "left.", q + "right."
            mat(l + "q", a["heads"] * a["dim"], W, bias=True)
            mat(l + "k", a["kv_heads"] * a["dim"], W, bias=True)
            mat(l + "v", a["kv_heads"] * a["vdim"], W, bias=True)
            rand(l + "q.norm", a["dim"], gain=0.3, mean=1.0)
            rand(l + "k.norm", a["dim"], gain=0.3, mean=1.0)
            mat(l + "g", a["heads"] * a["vdim"], W)
            mat(l + "o", W, a["heads"] * a["vdim"], bias=True)
            inner, ch = s["heads"] * s["vdim"], s["heads"] * s["vdim"] + 2 * s["groups"] * s["state"]
            mat(r + "in", inner + ch + s["heads"], W, 0.8)
            conv(r, ch, s["conv"])
            rand(r + "dt_bias", s["heads"], gain=1.0, mean=-1.5)
            rand(r + "A_log", s["heads"], gain=1.5, mean=-1.0)
            rand(r + "D", s["heads"])
            rand(r + "norm", inner, gain=0.3, mean=1.0)
            mat(r + "o", W, inner)
            rand(q + "left.out", W, gain=0.3, mean=1.0)
            rand(q + "right.out", W, gain=0.3, mean=1.0)
        if e.get("mlp"):
            ff = e["mlp"]["ff"]
            number(p + "norm2")
            mat(p + "mlp.up", ff, W, 0.8)
            mat(p + "mlp.down", W, ff)
            rand(p + "mlp.act", 2, gain=0.8)
    number("final.norm")
    mat("head", cfg["vocab"], W, 3.0)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


# ---------------------------------------------------------------- sublayers between two norms, routed experts
def low_rank(heads=3, dim=20, rot_dim=12, vdim=28, kv_rank=40, q_rank=30, window=37, scale=None, base=5000.0, kv_from=None):
    e = latent(heads, dim, rot_dim, vdim, kv_rank, window, scale, base, scaling=False)
    e["mixer"]["q_rank"] = q_rank
    if kv_from is not None:
        e["mixer"]["kv_from"] = kv_from
    return e


def general(heads=3, dim=20, decay_rank=6):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim, "decay_rank": decay_rank}}


def routed(ff=28, experts=10, top=3, groups=None):
    ro = {"experts": experts, "top": top}
    if groups:
        ro["groups"] = dict(zip(("count", "keep"), groups))
    return {"kind": "moe", "expert": {"ff": ff}, "router": ro}


def sandwich_config(layers, mlps, width=72, vocab=193, groups=3, eps=2e-5, mult=0.7):
    layers = [dict(e, mlp=f) for e, f in zip(layers, mlps)]
    return {"architecture": "Tativik", "layers": layers, "norm": {"eps": eps, "groups": groups}, "residual_mult": mult,
            "vocab": vocab, "width": width}


SANDWICH = {
    # sizes no vector width divides; a layer on another's latents with its own heads, sizes, window and scale; one layer
    # without a feed-forward; groups of two experts, of one, none
    "odd": sandwich_config([low_rank(heads=3, dim=10, rot_dim=6, vdim=7, kv_rank=19, q_rank=13, window=21), general(heads=3, dim=18, decay_rank=5),
                            low_rank(heads=5, dim=17, rot_dim=6, vdim=9, kv_rank=19, q_rank=11, window=None, kv_from=0), general(heads=2, dim=21)],
                           [routed(ff=19, experts=6, top=2, groups=(3, 2)), None, routed(ff=22, experts=7, top=1),
                            routed(ff=9, experts=5, top=3, groups=(5, 4))], width=70, groups=5, mult=0.4),
    # shapes the matrix kernels take, one group, one kept group, the head gates and sinks of 16 heads
    "wide": sandwich_config([general(heads=2, dim=64, decay_rank=16),
                             low_rank(heads=16, dim=32, rot_dim=32, vdim=64, kv_rank=96, q_rank=64, window=50),
                             low_rank(heads=8, dim=64, rot_dim=32, vdim=32, kv_rank=96, q_rank=40, window=50, kv_from=1)],
                            [routed(ff=64, experts=32, top=4, groups=(8, 3)), routed(ff=48, experts=16, top=2, groups=(4, 1)),
                             routed(ff=64, experts=16, top=8)], width=128, groups=1, mult=1.0),
    # more than one slab of channels, a state of many columns, one token's window, shared latents twice over
    "padded": sandwich_config([low_rank(heads=20, dim=24, rot_dim=8, vdim=40, kv_rank=136, q_rank=24, window=3), general(heads=2, dim=72),
                               low_rank(heads=2, dim=130, rot_dim=8, vdim=24, kv_rank=136, q_rank=50, window=64, kv_from=0),
                               general(heads=1, dim=136, decay_rank=40),
                               low_rank(heads=4, dim=8, rot_dim=8, vdim=16, kv_rank=136, q_rank=88, window=1, kv_from=0)],
                              [routed(ff=40, experts=12, top=4, groups=(2, 1)), routed(ff=24, experts=9, top=9), None, None, routed()],
                              width=88, groups=2, mult=0.35),
}


def make_sandwich_weights(cfg, seed=0, steady=True):
    """bf16 tensors by checkpoint name: decays from short to long memory, sinks and gates far from trivial. `steady`:
    the corrections alone decide which experts run, so that rounding does not change the choice."""
    g = torch.Generator().manual_seed(seed)
    W, w = cfg["width"], {}

    def rand(name, *shape, gain=1.0, mean=0.0):
        w[name] = mean + torch.randn(*shape, generator=g) * gain

    def mat(name, rows, cols, gain=1.0):
        rand(name, rows, cols, gain=gain / math.sqrt(cols))

    rand("embed", cfg["vocab"], W)
    for n in ("embed.norm", "final.norm"):
        rand(n, W, gain=0.3, mean=1.0)
    for i, e in enumerate(cfg["layers"]):
        p, m = f"l{i}.", e["mixer"]
        q = p + "mix."
        H = m["heads"]
        if e["type"] == "general_delta":
            HD = H * m["dim"]
            for n in "rkvga":
                mat(q + n, HD, W, 1.2)
            mat(q + "w1", m["decay_rank"], W, 1.2)
            mat(q + "w2", HD, m["decay_rank"], 1.5)
            rand(q + "w0", HD, gain=2.5, mean=-3.5)
            rand(q + "a.b", HD, gain=1.5)
            rand(q + "norm", HD, gain=0.3, mean=1.0)
            mat(q + "o", W, HD, 1.5)
        else:
            C, R = m["kv_rank"], m["rot_dim"]
            mat(q + "dq", m["q_rank"], W)
            rand(q + "dq.norm", m["q_rank"], gain=0.3, mean=1.0)
            mat(q + "uq", H * (m["dim"] + R), m["q_rank"], 1.6)
            if m.get("kv_from") is None:
                mat(q + "dkv", C + R, W, 1.5)
                rand(q + "dkv.norm", C, gain=0.3, mean=1.0)
            mat(q + "uk", H * m["dim"], C)
            mat(q + "uv", H * m["vdim"], C)
            rand(q + "sink", H, gain=1.5, mean=0.5)
            mat(q + "g", H, W, 1.5)
            mat(q + "o", W, H * m["vdim"], 1.5)
        subs = [1]
        if e.get("mlp"):
            subs.append(2)
            ro, ff, f = e["mlp"]["router"], e["mlp"]["expert"]["ff"], p + "mlp."
            for k in range(ro["experts"]):
                mat(f"{f}e{k}.gate", ff, W, 1.5)
                mat(f"{f}e{k}.up", ff, W, 1.5)
                mat(f"{f}e{k}.down", W, ff)
            mat(f + "router", ro["experts"], W, 0.3 if steady else 1.5)
            if steady:  # scores stay within 0.5 +- 0.25; where groups' sums tie, groups stand apart
                E, count = ro["experts"], (ro.get("groups") or {"count": 1})["count"]
                c = torch.randperm(E, generator=g) * 1.0 - 0.7 * E
                sums = c.view(count, -1).topk(min(2, E // count)).values.sum(-1)
                if len(set(sums.tolist())) < count:
                    c = c + torch.arange(count).repeat_interleave(E // count) * E
                w[f + "correction"] = c
            else:
                rand(f + "correction", ro["experts"], gain=0.3, mean=-0.8)
        for k in subs:
            rand(f"{p}norm{k}", W, gain=0.3, mean=1.0)
            rand(f"{p}norm{k}b", W, gain=0.3, mean=1.0)
            mat(f"{p}rg{k}", W, W, 1.5)
            rand(f"{p}rg{k}.b", W, gain=0.8)
    mat("head", cfg["vocab"], W, 3.0)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}
