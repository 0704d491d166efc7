"""Plain CPU restatement of the hybrid decoders (Dovidra: latent attention + gated delta rule layers;
Lipedra: differential attention in parallel layers; Foduzen: gated linear recurrences, and windowed
attention beside a state space mixer, behind norms of the sublayers' outputs; Tativik: latent attention with
low-rank queries and sinks, a generalized delta rule and routed experts, each gated between two norms), one
function per mechanism, whole sequences at a time, in the dtype of its weights (float64 in the tests).
Test infrastructure only: nothing under skyrl_amd/ imports it and it shares no code with it.

`w` maps tensor names to CPU tensors; `cfg` is the parsed config.json.
"""

from __future__ import annotations

import math

import torch


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotary_frequencies(rot):
    """(frequencies [dims/2], amplitude of cos and sin); YaRN interpolation when rot has 'scaling'."""
    D, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / D) for i in range(D // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def dim_of(turns):
        return D * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), D - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, positions, rot):
    """Interleaved rotary of the first rot.dims of x [T, ..., D]."""
    f, amp = rotary_frequencies(rot)
    y = x.clone()
    for i, fi in enumerate(f):
        a = positions.to(torch.float64) * fi
        c, s = (torch.cos(a) * amp).to(x.dtype), (torch.sin(a) * amp).to(x.dtype)
        shape = (-1,) + (1,) * (x.dim() - 2)
        c, s = c.view(shape), s.view(shape)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * c - v * s
        y[..., 2 * i + 1] = v * c + u * s
    return y


def window_attention(q, k, v, scale, size):
    """q, k [T, H, D], v [T, H, V]; position i sees j with 0 <= i - j < size (None: every j <= i)."""
    T = q.shape[0]
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    i = torch.arange(T)
    d = i[:, None] - i[None]
    see = d >= 0
    if size is not None:
        see &= d < size
    s = s.masked_fill(~see, float("-inf"))
    return torch.einsum("hij,jhv->ihv", torch.softmax(s, -1), v)


def latent_attention(h, w, p, m, eps):
    T = h.shape[0]
    H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    q = (h @ w[p + "q"].T).view(T, H, D + R)
    down = h @ w[p + "dkv"].T
    c = rms_norm(down[:, :C], w[p + "dkv.norm"], eps)
    qr = rotate_pairs(q[..., D:], pos, m["rot"])
    kr = rotate_pairs(down[:, C:], pos, m["rot"])
    k = (c @ w[p + "uk"].T).view(T, H, D)
    v = (c @ w[p + "uv"].T).view(T, H, V)
    q = torch.cat([q[..., :D], qr], -1)
    k = torch.cat([k, kr[:, None].expand(T, H, R)], -1)
    mask = m.get("mask")
    o = window_attention(q, k, v, m["scale"], mask["size"] if mask else None)
    return o.reshape(T, H * V) @ w[p + "o"].T


def silu(x):
    return x * torch.sigmoid(x)


def short_conv(x, w):
    """Causal per-channel convolution of x [T, C] with w [C, taps], the last tap on the current token."""
    y = torch.zeros_like(x)
    taps = w.shape[1]
    for t in range(x.shape[0]):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += x[s] * w[:, j]
    return y


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_gates(h, w, p):
    """(beta, decay g), each [T, heads]."""
    beta = torch.sigmoid(h @ w[p + "b"].T)
    z = h @ w[p + "a"].T + w[p + "dt_bias"]
    softplus = torch.where(z > 0, z, torch.zeros_like(z)) + torch.log1p(torch.exp(-z.abs()))
    return beta, torch.exp(-torch.exp(w[p + "A_log"]) * softplus)


def delta_recurrence(q, k, v, beta, g, state=None):
    """q, k [T, H, D], v [T, H, V], beta, g [T, H] -> outputs [T, H, V] and the final state [H, D, V]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            s = S[h] * g[t, h]
            u = beta[t, h] * (v[t, h] - s.T @ k[t, h])
            s = s + torch.outer(k[t, h], u)
            out[t, h] = s.T @ q[t, h]
            S[h] = s
    return out, S


def delta_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, K, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(short_conv(h @ w[p + "q"].T, w[p + "q.conv"])).view(T, K, D)
    k = silu(short_conv(h @ w[p + "k"].T, w[p + "k.conv"])).view(T, K, D)
    v = silu(short_conv(h @ w[p + "v"].T, w[p + "v.conv"])).view(T, H, V)
    group = torch.tensor([hh // (H // K) for hh in range(H)])
    q, k = (unit(q) * D ** -0.5)[:, group], unit(k)[:, group]
    beta, g = delta_gates(h, w, p)
    o, _ = delta_recurrence(q, k, v, beta, g)
    o = rms_norm(o, w[p + "norm"], eps) * silu(h @ w[p + "g"].T).view(T, H, V)
    return o.reshape(T, H * V) @ w[p + "o"].T


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def dense_ff(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def rms_norm_about_one(x, w, eps):
    """RMS norm whose stored weight is the distance from 1."""
    return rms_norm(x, 1 + w, eps)


def rotate_maps(x, rot):
    """Interleaved rotary of the first rot.dims of every map of x [T, heads, maps, dim], positions from 0."""
    d = rot["dims"]
    return torch.cat([rotate_pairs(x[..., :d], torch.arange(x.shape[0]), rot), x[..., d:]], -1)


def conv_projection(h, w, name):
    """Biased projection, then its short convolution over time."""
    return short_conv(h @ w[name].T + w[name + ".b"], w[name + ".conv"])


def attention_queries(h, w, p, m):
    T = h.shape[0]
    return rotate_maps(conv_projection(h, w, p + "q").view(T, m["heads"], 2, m["dim"]), m["rot"])


def attention_keys_values(h, w, p, m):
    T, G = h.shape[0], m["kv_heads"]
    k = rotate_maps(conv_projection(h, w, p + "k").view(T, G, 2, m["dim"]), m["rot"])
    return k, conv_projection(h, w, p + "v").view(T, G, m["vdim"])


def differential_lambda(w, p, diff):
    return (torch.exp((w[p + "lq1"] * w[p + "lk1"]).sum()) - torch.exp((w[p + "lq2"] * w[p + "lk2"]).sum()) + diff)


def differential_combine(a1, a2, lam, diff, eps):
    """Two maps' outputs [T, H, V] -> (1 - diff) times the root-mean-square-normed difference."""
    o = a1 - lam * a2
    return o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps) * (1 - diff)


def differential_attention(h, w, p, m, eps, kv):
    """kv: (keys [T, G, 2, dim], values [T, G, vdim]), this layer's own or another's."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = attention_queries(h, w, p, m)
    group = torch.tensor([hh // (H // G) for hh in range(H)])
    k, v = kv[0][:, group], kv[1][:, group]
    a1, a2 = (window_attention(q[:, :, i], k[:, :, i], v, m["scale"], None) for i in range(2))
    o = differential_combine(a1, a2, differential_lambda(w, p, m["diff"]), m["diff"], eps)
    o = o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, -1) @ w[p + "o"].T


def clamped_ff(h, w, p, limit):
    g = (h @ w[p + "gate"].T + w[p + "gate.b"]).clamp(max=limit)
    u = (h @ w[p + "up"].T + w[p + "up.b"]).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w[p + "down"].T + w[p + "down.b"]


def softplus(z):
    return torch.where(z > 0, z, torch.zeros_like(z)) + torch.log1p(torch.exp(-z.abs()))


def rms(x, eps):
    """x over its root mean square (last dimension)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sinusoid(positions, width, base=10000.0):
    """Position vectors [T, width]: sines on the even entries, cosines of the same angle after them."""
    out = torch.zeros(len(positions), width, dtype=torch.float64)
    for e in range(width):
        a = positions.double() * base ** (-(e - e % 2) / width)
        out[:, e] = torch.cos(a) if e % 2 else torch.sin(a)
    return out


def block_gates(u, w, name):
    """Sigmoid of a block-diagonal affine map: block b of u times the matrix w[name][b] [out, in]."""
    blocks, size = w[name].shape[0], w[name].shape[1]
    out = torch.zeros_like(u)
    for b in range(blocks):
        cols = slice(b * size, (b + 1) * size)
        out[:, cols] = torch.sigmoid(u[:, cols] @ w[name][b].T + w[name + ".b"][b])
    return out


def gated_linear_recurrence(u, r, i, lam, state=None):
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t per channel, log a = -8 r softplus(lam); all states [T, C]."""
    log_a = -8.0 * r * softplus(lam)
    a, into = torch.exp(log_a), torch.sqrt(-torch.expm1(2 * log_a)) * i * u
    S = torch.zeros(u.shape[1], dtype=u.dtype) if state is None else state.clone()
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        S = a[t] * S + into[t]
        out[t] = S
    return out


def rglru_mixer(h, w, p):
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = short_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"]) + w[p + "conv.b"]
    S = gated_linear_recurrence(u, block_gates(u, w, p + "ra"), block_gates(u, w, p + "ri"), w[p + "lam"])
    return (S * y) @ w[p + "o"].T


def gated_window_attention(h, w, p, m, eps):
    """Normed queries and keys, no rotation, a sliding window, an elementwise output gate."""
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    proj = lambda n: h @ w[p + n].T + w[p + n + ".b"]  # noqa: E731
    q = rms_norm(proj("q").view(T, H, D), w[p + "q.norm"], eps)
    k = rms_norm(proj("k").view(T, G, D), w[p + "k.norm"], eps)
    group = torch.tensor([hh // (H // G) for hh in range(H)])
    size = m["mask"]["size"] if m.get("mask") else None
    o = window_attention(q, k[:, group], proj("v").view(T, G, V)[:, group], m["scale"], size).reshape(T, H * V)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T + w[p + "o.b"]


def state_space_recurrence(x, B, C, dt, A_log, D, state=None):
    """x [T, H, P], B and C [T, H, N], dt [T, H] -> y [T, H, P] and the final state [H, N, P]."""
    T, H, P = x.shape
    S = torch.zeros(H, B.shape[-1], P, dtype=x.dtype) if state is None else state.clone()
    y = torch.zeros_like(x)
    for t in range(T):
        for h in range(H):
            decay = torch.exp(-torch.exp(A_log[h]) * dt[t, h])
            S[h] = decay * S[h] + dt[t, h] * torch.outer(B[t, h], x[t, h])
            y[t, h] = S[h].T @ C[t, h] + D[h] * x[t, h]
    return y, S


def grouped_gated_norm(y, z, weight, groups, eps):
    """rms over each of `groups` equal parts of y silu(z), times the weight."""
    T, n = y.shape
    return rms((y * silu(z)).view(T, groups, n // groups), eps).view(T, n) * weight


def state_space_mixer(h, w, p, m, eps):
    T, H, P, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    u = h @ w[p + "in"].T
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * G * N], u[:, 2 * inner + 2 * G * N:]
    xbc = silu(short_conv(xbc, w[p + "conv"]) + w[p + "conv.b"])
    group = torch.tensor([hh // (H // G) for hh in range(H)])
    x = xbc[:, :inner].view(T, H, P)
    B = xbc[:, inner:inner + G * N].view(T, G, N)[:, group]
    C = xbc[:, inner + G * N:].view(T, G, N)[:, group]
    y, _ = state_space_recurrence(x, B, C, softplus(dt + w[p + "dt_bias"]), w[p + "A_log"], w[p + "D"])
    y = grouped_gated_norm(y.reshape(T, inner), z, w[p + "norm"], m["norm_groups"], eps)
    return y @ w[p + "o"].T


def side_by_side(left, right, w, p, eps):
    """Half the sum of two mixers' outputs, each normed over the model width."""
    return (rms_norm(left, w[p + "left.out"], eps) + rms_norm(right, w[p + "right.out"], eps)) / 2


def xielu(z, p, q):
    neg = torch.where(z > 0, torch.zeros_like(z), z)
    return torch.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (torch.expm1(neg) - neg)) + z / 2


def xielu_ff(h, w, p):
    return xielu(h @ w[p + "up"].T, *w[p + "act"]) @ w[p + "down"].T


def output_norm_layer(x, w, i, entry, eps):
    """Foduzen: each sublayer reads the residual and its output is normed (one number as the weight)."""
    p, m = f"l{i}.", entry["mixer"]
    if entry["type"] == "rglru":
        y = rglru_mixer(x, w, p + "mix.")
    else:
        y = side_by_side(gated_window_attention(x, w, p + "mix.left.", m["left"], eps),
                         state_space_mixer(x, w, p + "mix.right.", m["right"], eps), w, p + "mix.", eps)
    x = x + rms_norm(y, w[p + "norm1"], eps)
    if entry.get("mlp"):
        x = x + rms_norm(xielu_ff(x, w, p + "mlp."), w[p + "norm2"], eps)
    return x


def grouped_rms_norm(x, w, groups, eps):
    """Every one of `groups` equal consecutive parts over its own root mean square, times the weight."""
    return rms(x.reshape(x.shape[:-1] + (groups, x.shape[-1] // groups)), eps).reshape(x.shape) * w


def rotate_halves(x, positions, rot):
    """Rotary of the first rot.dims of x [T, ..., D], dimension i paired with i + dims / 2."""
    f, amp = rotary_frequencies(rot)
    half = rot["dims"] // 2
    y = x.clone()
    for i, fi in enumerate(f):
        a = positions.to(torch.float64) * fi
        shape = (-1,) + (1,) * (x.dim() - 2)
        c, s = ((t * amp).to(x.dtype).view(shape) for t in (torch.cos(a), torch.sin(a)))
        u, v = x[..., i], x[..., half + i]
        y[..., i] = u * c - v * s
        y[..., half + i] = v * c + u * s
    return y


def sink_attention(q, k, v, scale, size, sink):
    """window_attention whose denominators also hold exp(sink[head])."""
    T = q.shape[0]
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    d = torch.arange(T)[:, None] - torch.arange(T)[None]
    see = (d >= 0) & (d < (T if size is None else size))
    s = s.masked_fill(~see, float("-inf"))
    top = torch.maximum(s.amax(-1), sink[:, None])[..., None]
    e = torch.exp(s - top)
    return torch.einsum("hij,jhv->ihv", e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None, None] - top)), v)


def latent_keys(h, w, p, m, eps):
    """(normed latents [T, rank], rotated key part [T, rot_dim]): what a layer of its own caches."""
    down, C = h @ w[p + "dkv"].T, m["kv_rank"]
    return rms_norm(down[:, :C], w[p + "dkv.norm"], eps), rotate_halves(down[:, C:], torch.arange(h.shape[0]), m["rot"])


def sink_latent_attention(h, w, p, m, eps, kv):
    """kv: (latents, rotated key part), this layer's own or another's."""
    T = h.shape[0]
    H, D, R, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c_q = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (c_q @ w[p + "uq"].T).view(T, H, D + R)
    q = torch.cat([q[..., :D], rotate_halves(q[..., D:], torch.arange(T), m["rot"])], -1)
    c, kr = kv
    k = torch.cat([(c @ w[p + "uk"].T).view(T, H, D), kr[:, None].expand(T, H, R)], -1)
    v = (c @ w[p + "uv"].T).view(T, H, V)
    size = m["mask"]["size"] if m.get("mask") else None
    o = sink_attention(q, k, v, m["scale"], size, w[p + "sink"])
    o = o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * V) @ w[p + "o"].T


def general_delta_recurrence(r, k, v, decay, a, state=None):
    """All inputs [T, H, D]: S_t = diag(decay) S - (a u) (u^T S) + k v^T with u = unit(k) and S the old state;
    outputs S_t^T r [T, H, D] and the final state [H, D, D]."""
    T, H, D = r.shape
    S = torch.zeros(H, D, D, dtype=r.dtype) if state is None else state.clone()
    u, out = unit(k), torch.zeros_like(v)
    for t in range(T):
        read = torch.einsum("hd,hdv->hv", u[t], S)
        S = decay[t][..., None] * S - (a[t] * u[t])[..., None] * read[:, None] + k[t][..., None] * v[t][:, None]
        out[t] = torch.einsum("hd,hdv->hv", r[t], S)
    return out, S


def general_delta_gates(h, w, p):
    """(decay, removal rate), each [T, heads dim]."""
    z = torch.tanh(h @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"].reshape(-1)
    return torch.exp(-math.exp(-0.5) * torch.sigmoid(z)), torch.sigmoid(h @ w[p + "a"].T + w[p + "a.b"].reshape(-1))


def general_delta_mixer(h, w, p, m, eps):
    T, H, D = h.shape[0], m["heads"], m["dim"]
    r, k, v = ((h @ w[p + n].T).view(T, H, D) for n in "rkv")
    decay, a = (t.view(T, H, D) for t in general_delta_gates(h, w, p))
    o, _ = general_delta_recurrence(r, k, v, decay, a)
    o = rms(o, eps).reshape(T, H * D) * w[p + "norm"].reshape(-1) * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def route(scores, correction, top, groups=1, keep=1):
    """Experts of every token [T, top] and their weights: the largest corrected scores among the `keep` groups whose
    two largest corrected scores sum highest; the weights are the scores themselves."""
    T, E = scores.shape
    choice = scores + correction
    per = E // groups
    best = choice.view(T, groups, per).topk(min(2, per), -1).values.sum(-1)
    kept = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, best.topk(keep, -1).indices, True)
    choice = choice.masked_fill(~kept.repeat_interleave(per, 1), float("-inf"))
    idx = choice.topk(top, -1).indices
    return idx, scores.gather(1, idx)


def experts_ff(h, w, p, m):
    """Weighted sum of the chosen experts' gated silu feed-forwards."""
    ro = m["router"]
    gr = ro.get("groups") or {"count": 1, "keep": 1}
    idx, weight = route(torch.sigmoid(h @ w[p + "router"].T), w[p + "correction"], ro["top"], gr["count"], gr["keep"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), weight[t]):
            q = f"{p}e{e}."
            out[t] += s * ((silu(w[q + "gate"] @ h[t]) * (w[q + "up"] @ h[t])) @ w[q + "down"].T)
    return out


def sandwich_layer(x, w, i, entry, cfg, kvs):
    """Tativik: each sublayer between two norms, its result gated before the second. kvs: latents by layer, extended
    here."""
    p, m, eps = f"l{i}.", entry["mixer"], cfg["norm"]["eps"]
    norm = lambda y, name: grouped_rms_norm(y, w[p + name], cfg["norm"].get("groups", 1), eps)  # noqa: E731
    gate = lambda h, name: torch.sigmoid(h @ w[p + name].T + w[p + name + ".b"])  # noqa: E731
    h = norm(x, "norm1")
    if entry["type"] == "general_delta":
        y = general_delta_mixer(h, w, p + "mix.", m, eps)
    else:
        j = m.get("kv_from")
        if j is None:
            kvs[i] = latent_keys(h, w, p + "mix.", m, eps)
        y = sink_latent_attention(h, w, p + "mix.", m, eps, kvs[i if j is None else j])
    x = x + cfg["residual_mult"] * norm(y * gate(h, "rg1"), "norm1b")
    if entry.get("mlp"):
        h = norm(x, "norm2")
        x = x + cfg["residual_mult"] * norm(experts_ff(h, w, p + "mlp.", entry["mlp"]) * gate(h, "rg2"), "norm2b")
    return x


def layer(x, w, i, entry, eps):
    """Dovidra: two halves, each behind a norm of its own."""
    p = f"l{i}."
    h = layer_norm(x, w[p + "norm1"], eps)
    mixer = {"latent_attention": latent_attention, "delta": delta_mixer}[entry["type"]]
    x = x + mixer(h, w, p + "mix.", entry["mixer"], eps)
    if entry.get("mlp"):
        x = x + dense_ff(layer_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
    return x


def parallel_layer(x, w, i, entry, eps, kvs):
    """Lipedra: mixer and feed-forward read one norm. kvs: keys and values by layer, extended here."""
    p, m = f"l{i}.", entry["mixer"]
    h = rms_norm_about_one(x, w[p + "norm1"], eps)
    if m.get("kv_from") is None:
        kvs[i] = attention_keys_values(h, w, p + "mix.", m)
    y = differential_attention(h, w, p + "mix.", m, eps, kvs[i if m.get("kv_from") is None else m["kv_from"]])
    if entry.get("mlp"):
        y = y + clamped_ff(h, w, p + "mlp.", entry["mlp"]["limit"])
    return x + y


def layer_runs(cfg):
    """[(layer, pass or None)]: None outside the loop; pass t's step vector is added before its first layer."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    runs = [(i, None) for i in range(a)]
    for t in range(lp["times"]):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def forward(tokens, w, cfg):
    """Logits [T, vocab] and the residual after every layer run [runs, T, width]."""
    eps, design = cfg["norm"]["eps"], cfg["architecture"]
    x = w["embed"][torch.as_tensor(tokens)]
    if design in ("Lipedra", "Foduzen"):
        x = x * cfg["embedding"]["scale"]
    if design == "Tativik":
        x = grouped_rms_norm(x, w["embed.norm"], cfg["norm"].get("groups", 1), eps)
    if design == "Foduzen":
        x = x + sinusoid(torch.arange(len(tokens)), cfg["width"]).to(x.dtype)
    trail, kvs = [], {}
    for i, t in layer_runs(cfg):
        if t is not None:
            x = x + w["loop.step"][t]
        e = cfg["layers"][i]
        if design == "Lipedra":
            x = parallel_layer(x, w, i, e, eps, kvs)
        elif design == "Tativik":
            x = sandwich_layer(x, w, i, e, cfg, kvs)
        else:
            x = (output_norm_layer if design == "Foduzen" else layer)(x, w, i, e, eps)
        trail.append(x)
    if design == "Tativik":
        x = grouped_rms_norm(x, w["final.norm"], cfg["norm"].get("groups", 1), eps)
    else:
        x = {"Dovidra": layer_norm, "Lipedra": rms_norm_about_one, "Foduzen": rms_norm}[design](x, w["final.norm"], eps)
    logits = x @ w["head"].T
    cap = cfg.get("logit_softcap")
    if cap:
        logits = cap * torch.tanh(logits / cap)
    return logits, torch.stack(trail)
