"""Plain, slow reference of the Fobolix decoder (torch, CPU, float64 by default), one function per mechanism.

A whole sequence goes in, the logits of every position come out; there is no cache, no batching and no chunking here.  Shares no code
with chatts_amd: the product path is checked against these equations.

A model is (cfg, sd): cfg = the dictionary of config.json, sd = name -> tensor.
"""
import math

import torch


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis"""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotary_frequencies(dims, base, scaling=None):
    """-> (angular frequency of every pair, magnitude of cos / sin): plain rotary, or YaRN when `scaling` is given"""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = base ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0

    def pair_with_turns(turns):      # index of the pair that makes `turns` turns within the original context
        return dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(pair_with_turns(scaling["fast"])), 0)
    hi = min(math.ceil(pair_with_turns(scaling["slow"])), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)
    return f / scaling["factor"] * ramp + f * (1 - ramp), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [T, ..., dims]: dimension i pairs with i + dims / 2"""
    dims = rot["dims"]
    f, mag = rotary_frequencies(dims, rot["base"], rot.get("scaling"))
    a = positions.to(torch.float64)[:, None] * f[None, :]
    cos, sin = (a.cos() * mag).to(x.dtype), (a.sin() * mag).to(x.dtype)
    while cos.dim() < x.dim():
        cos, sin = cos[:, None], sin[:, None]
    u, v, rest = x[..., :dims // 2], x[..., dims // 2:dims], x[..., dims:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], -1)


def latent_attention(h, sd, p, m, eps):
    """h [T, width] -> [T, width]; expanded keys and values, ordinary causal softmax"""
    T, H, dim, rd, vd, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    q = (h @ sd[p + "q"].T).view(T, H, dim + rd)
    q_un, q_rot = q[..., :dim], rotate(q[..., dim:], pos, m["rot"])
    ckr = h @ sd[p + "dkv"].T
    c = rms_norm(ckr[:, :R], sd[p + "dkv.norm"], eps)
    k_rot = rotate(ckr[:, R:], pos, m["rot"])
    k_un = (c @ sd[p + "uk"].T).view(T, H, dim)
    v = (c @ sd[p + "uv"].T).view(T, H, vd)
    out = torch.zeros(T, H, vd, dtype=h.dtype)
    for t in range(T):
        s = (torch.einsum("hd,jhd->hj", q_un[t], k_un[:t + 1]) + torch.einsum("hd,jd->hj", q_rot[t], k_rot[:t + 1])) * m["scale"]
        out[t] = torch.einsum("hj,jhd->hd", torch.softmax(s, -1), v[:t + 1])
    return out.reshape(T, H * vd) @ sd[p + "o"].T


def short_conv(x, w):
    """x [T, C], w [C, taps]: causal per-channel convolution (last column = the current token), then silu"""
    taps = w.shape[1]
    y = torch.zeros_like(x)
    for j in range(taps):
        lag = taps - 1 - j
        y[lag:] += x[:x.shape[0] - lag] * w[:, j] if lag < x.shape[0] else 0
    return y * torch.sigmoid(y)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_step(S, q, k, v, g, beta):
    """one token of the gated delta rule: S [H, dim, vdim], q / k / g [H, dim], v [H, vdim], beta [H] -> (S, o [H, vdim])"""
    S = g[:, :, None] * S
    u = beta[:, None] * (v - torch.einsum("hij,hi->hj", S, k))
    S = S + k[:, :, None] * u[:, None, :]
    return S, torch.einsum("hij,hi->hj", S, q)


def delta_inputs(h, sd, p, m):
    """-> q, k, g [T, H, dim], v [T, H, vdim], beta [T, H]"""
    T, H, KH, dim, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv(h @ sd[p + "q"].T, sd[p + "q.conv"]).view(T, KH, dim)
    k = short_conv(h @ sd[p + "k"].T, sd[p + "k.conv"]).view(T, KH, dim)
    v = short_conv(h @ sd[p + "v"].T, sd[p + "v.conv"]).view(T, H, vd)
    q, k = unit(q) * dim ** -0.5, unit(k)
    head = torch.arange(H) // (H // KH)
    beta = torch.sigmoid(h @ sd[p + "b"].T)
    dt = (h @ sd[p + "a1"].T) @ sd[p + "a2"].T + sd[p + "dt_bias"]
    g = torch.exp(-torch.exp(sd[p + "A_log"])[None, :, None] * torch.nn.functional.softplus(dt, threshold=1e9).view(T, H, dim))
    return q[:, head], k[:, head], g, v, beta


def channel_delta(h, sd, p, m, eps):
    T, H, dim, vd = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, g, v, beta = delta_inputs(h, sd, p, m)
    S = torch.zeros(H, dim, vd, dtype=h.dtype)
    o = torch.zeros(T, H, vd, dtype=h.dtype)
    for t in range(T):
        S, o[t] = delta_step(S, q[t], k[t], v[t], g[t], beta[t])
    gate = torch.sigmoid((h @ sd[p + "g1"].T) @ sd[p + "g2"].T).view(T, H, vd)
    o = rms_norm(o, sd[p + "norm"], eps) * gate
    return o.reshape(T, H * vd) @ sd[p + "o"].T


MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta}


def dense(h, sd, p):
    a = torch.relu(h @ sd[p + "up"].T)
    return (a * a) @ sd[p + "down"].T


def layer(x, sd, i, spec, eps):
    p = f"l{i}."
    y = MIXERS[spec["type"]](rms_norm(x, sd[p + "norm1"], eps), sd, p + "mix.", spec["mixer"], eps)
    x = x + rms_norm(y, sd[p + "norm1b"], eps)
    if spec.get("mlp"):
        y = dense(rms_norm(x, sd[p + "norm2"], eps), sd, p + "mlp.")
        x = x + rms_norm(y, sd[p + "norm2b"], eps)
    return x


def runs(cfg):
    """the layer runs in order: (layer index, pass number if this run opens a pass of the loop, else None)"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    out = [(i, None) for i in range(a)]
    for t in range(times):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def forward(cfg, sd, tokens, dtype=torch.float64, want_layers=False):
    """-> logits [T, vocab] (and the residual stream after every layer run)"""
    sd = {k: v.to(dtype) for k, v in sd.items()}
    eps = cfg["norm"]["eps"]
    x = sd["embed"][torch.as_tensor(tokens)]
    streams = []
    for i, t in runs(cfg):
        if t is not None:
            x = x + sd["loop.step"][t]
        x = layer(x, sd, i, cfg["layers"][i], eps)
        streams.append(x)
    logits = rms_norm(x, sd["final.norm"], eps) @ sd["head"].T
    return (logits, streams) if want_layers else logits


def generate(cfg, sd, tokens, n, dtype=torch.float64):
    """greedy continuation, everything recomputed for every token"""
    seq = list(tokens)
    for _ in range(n):
        seq.append(int(forward(cfg, sd, seq, dtype)[-1].argmax()))
    return seq[len(tokens):]


def random_model(cfg, seed=0):
    """bf16-representable random weights of a configuration that has, beside config.json's keys, the low-rank sizes of every
    channel_delta mixer as mixer["_rank_a"] / mixer["_rank_g"] -> name -> bfloat16 tensor"""
    gen = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(o, i, gain=1.0):
        return torch.randn(o, i, generator=gen) * gain / math.sqrt(i)

    def ones(n):
        return 1.0 + 0.2 * torch.randn(n, generator=gen)

    sd = {"embed": torch.randn(V, W, generator=gen), "final.norm": ones(W), "head": lin(V, W)}
    if cfg.get("loop"):
        sd["loop.step"] = 0.5 * torch.randn(cfg["loop"]["times"], W, generator=gen)
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if spec.get("mlp") else ()):
            sd[p + n] = ones(W)
        if spec["type"] == "latent_attention":
            H, dim, rd, vd, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            sd[p + "mix.q"] = lin(H * (dim + rd), W, 1.5)
            sd[p + "mix.dkv"] = lin(R + rd, W)
            sd[p + "mix.dkv.norm"] = ones(R)
            sd[p + "mix.uk"], sd[p + "mix.uv"] = lin(H * dim, R), lin(H * vd, R)
            sd[p + "mix.o"] = lin(W, H * vd)
        else:
            H, KH, dim, vd, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            ra, rg = m.get("_rank_a", 24), m.get("_rank_g", 24)
            for n, rows in (("q", KH * dim), ("k", KH * dim), ("v", H * vd)):
                sd[p + "mix." + n] = lin(rows, W)
                sd[p + "mix." + n + ".conv"] = torch.randn(rows, taps, generator=gen) * 0.6
            sd[p + "mix.b"] = lin(H, W)
            sd[p + "mix.A_log"] = torch.rand(H, generator=gen) * 2 - 1.5
            sd[p + "mix.dt_bias"] = torch.randn(H * dim, generator=gen) * 0.5 - 3.0
            sd[p + "mix.a1"], sd[p + "mix.a2"] = lin(ra, W), lin(H * dim, ra)
            sd[p + "mix.g1"], sd[p + "mix.g2"] = lin(rg, W), lin(H * vd, rg)
            sd[p + "mix.norm"] = ones(vd)
            sd[p + "mix.o"] = lin(W, H * vd)
        if spec.get("mlp"):
            sd[p + "mlp.up"], sd[p + "mlp.down"] = lin(spec["mlp"]["ff"], W), lin(W, spec["mlp"]["ff"])
    return {k: v.to(torch.bfloat16) for k, v in sd.items()}
