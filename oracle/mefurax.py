"""Plain, slow reference of the Mefurax decoder (torch, CPU, float64 by default), one function per mechanism.

A whole sequence goes in, the logits of every position come out; there is no cache, no batching and no chunking here.  Shares no code
with chatts_amd: the product path is checked against these equations.

A model is (cfg, sd): cfg = the dictionary of config.json, sd = name -> tensor.
"""
import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis"""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def shifted_norm(x, w, eps):
    """RMS norm whose stored weight is the distance from one"""
    return rms(x, eps) * (1 + w)


def causal_conv(u, w):
    """u [T, C], w [C, taps]: every channel's sum over its last `taps` values, the newest with the last weight; zeros before the start"""
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for back in range(min(taps, u.shape[0])):
        y[back:] += w[:, taps - 1 - back] * u[:u.shape[0] - back]
    return y


def rotate_pairs(x, base, dims):
    """x [T, H, D]: dimensions 2i and 2i + 1 (below `dims`) turned by position * base^(-2i / dims)"""
    T, y = x.shape[0], x.clone()
    pos = torch.arange(T, dtype=x.dtype)
    for i in range(dims // 2):
        a = (pos * base ** (-2.0 * i / dims))[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        y[:, :, 2 * i] = u * a.cos() - v * a.sin()
        y[:, :, 2 * i + 1] = v * a.cos() + u * a.sin()
    return y


def slopes(heads):
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap)


def in_window(i, j, size):
    """the last `size` positions, itself included (size None: every earlier one)"""
    return j <= i and (not size or i - j < size)


def in_chunk(i, j, size):
    """earlier positions of the same chunk; position 0 opens the first one"""
    return j <= i and (not size or i // size == j // size)


def attend(s, see, v):
    """s [H, T, T] scores, see [T, T], v [T, H, E] (every query head's own values) -> [T, H, E]"""
    a = torch.softmax(s.masked_fill(~see, -math.inf), -1)
    return torch.einsum("hij,jhe->ihe", a, v)


def mix_values(v, first, lam):
    return (1 - lam) * v + lam * first


def values(v, sd, p, m, shared):
    """value mixing: shared = {} at the start of a forward; the first layer that mixes leaves its values there"""
    if not m.get("v_mix"):
        return v
    if "v" not in shared:
        shared["v"] = v
        return v
    return mix_values(v, shared["v"], sd[p + "vmix"])


def see_matrix(T, rule, size):
    return torch.tensor([[rule(i, j, size) for j in range(T)] for i in range(T)])


def attention(h, sd, p, m, eps, shared):
    """short convolutions, norms over the whole projections, a distance bias per head, a sliding window"""
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_conv(h @ sd[p + n].T + sd[p + n + ".b"], sd[p + n + ".conv"]) for n in "qkv")
    q = (rms(q, eps) * sd[p + "q.norm"]).view(T, H, D)
    k = (rms(k, eps) * sd[p + "k.norm"]).view(T, G, D)
    v = values(v, sd, p, m, shared).view(T, G, E)
    head = torch.arange(H) // (H // G)
    dist = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    s = torch.einsum("ihd,jhd->hij", q, k[:, head]) * m["scale"] - torch.tensor(slopes(H), dtype=h.dtype)[:, None, None] * dist.to(h.dtype)
    o = attend(s, see_matrix(T, in_window, (m.get("mask") or {}).get("size")), v[:, head])
    return o.reshape(T, H * E) @ sd[p + "o"].T


def attention_2(h, sd, p, m, eps, shared):
    """rotated pairs, unit queries and keys after the rotation, capped scores, chunks, a gate per head"""
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = ((h @ sd[p + n].T).view(T, heads, D) for n, heads in (("q", H), ("k", G)))
    q, k = (rms(rotate_pairs(t, m["rot"]["base"], m["rot"]["dims"]), eps) for t in (q, k))
    v = values(h @ sd[p + "v"].T, sd, p, m, shared).view(T, G, E)
    head = torch.arange(H) // (H // G)
    s = soft_cap(torch.einsum("ihd,jhd->hij", q, k[:, head]) * m["scale"], m["softcap"])
    o = attend(s, see_matrix(T, in_chunk, (m.get("mask") or {}).get("size")), v[:, head])
    return (o * torch.sigmoid(h @ sd[p + "g"].T)[:, :, None]).reshape(T, H * E) @ sd[p + "o"].T


MIXERS = {"attention": attention, "attention_2": attention_2}


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def relu2(z):
    return torch.clamp(z, min=0) ** 2


def dense(h, sd, p):
    return (gelu_tanh(h @ sd[p + "gate"].T) * (h @ sd[p + "up"].T)) @ sd[p + "down"].T


def route(z, top):
    """router logits z [T, N] -> (chosen experts [T, top], their weights: softmax over the chosen logits)"""
    best = z.topk(top, -1)
    return best.indices, torch.softmax(best.values, -1)


def choice_margin(z, top):
    """how much a router's logits prefer the last chosen expert to the next one"""
    v = z.sort(-1, descending=True).values
    return v[:, top - 1] - v[:, top] if top < z.shape[1] else torch.full((z.shape[0],), math.inf, dtype=z.dtype)


def experts(h, sd, p, spec, margins=None):
    top = spec["router"]["top"]
    z = h @ sd[p + "router"].T
    idx, w = route(z, top)
    if margins is not None:
        margins.append(choice_margin(z, top))
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(idx[t].tolist(), w[t]):
            y[t] += a * (sd[f"{p}e{e}.down"] @ relu2(sd[f"{p}e{e}.up"] @ h[t]))
    if spec.get("shared"):
        y = y + relu2(h @ sd[p + "shared.up"].T) @ sd[p + "shared.down"].T
    return y


def layer(x, sd, i, spec, alpha, eps, shared, margins=None):
    """the norms stand after the sums"""
    p = f"l{i}."
    x = shifted_norm(alpha * x + MIXERS[spec["type"]](x, sd, p + "mix.", spec["mixer"], eps, shared), sd[p + "norm1"], eps)
    mlp = spec.get("mlp")
    if not mlp:
        return x
    y = experts(x, sd, p + "mlp.", mlp, margins) if mlp.get("kind", "dense") == "moe" else dense(x, sd, p + "mlp.")
    return shifted_norm(alpha * x + y, sd[p + "norm2"], eps)


def forward(cfg, sd, tokens, dtype=torch.float64, want_layers=False, margins=None):
    """-> logits [T, vocab] (and the residual stream after every layer); margins: a list that gets choice_margin of every router"""
    sd = {k: v.to(dtype) for k, v in sd.items()}
    x, eps, shared, streams = sd["embed"][torch.tensor([int(t) for t in tokens])], cfg["norm"]["eps"], {}, []
    for i, spec in enumerate(cfg["layers"]):
        x = layer(x, sd, i, spec, cfg["postln_alpha"], eps, shared, margins)
        streams.append(x)
    logits = shifted_norm(x, sd["final.norm"], eps) @ sd["head"].T
    return (logits, streams) if want_layers else logits


def generate(cfg, sd, tokens, n, dtype=torch.float64):
    """greedy continuation, everything recomputed for every token"""
    seq = list(tokens)
    for _ in range(n):
        seq.append(int(forward(cfg, sd, seq, dtype)[-1].argmax()))
    return seq[len(tokens):]


def random_model(cfg, seed=0):
    """bf16-representable random weights -> name -> bfloat16 tensor.  Queries and keys share directions, so that single scores stand out; router logits
    lie apart."""
    gen = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(o, i, gain=1.0):
        return torch.randn(o, i, generator=gen) * gain / math.sqrt(i)

    def vec(n, mean, spread):
        return mean + spread * torch.randn(n, generator=gen)

    sd = {"embed": torch.randn(V, W, generator=gen), "final.norm": vec(W, 0, 0.2), "head": lin(V, W)}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        q, H, G, D, E = p + "mix.", m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        sd[p + "norm1"] = vec(W, 0, 0.2)
        k = lin(G * D, W)
        sd[q + "k"] = k
        sd[q + "q"] = 0.6 * k.view(G, 1, D, W).expand(G, H // G, D, W).reshape(H * D, W) + lin(H * D, W, 0.8)
        sd[q + "v"], sd[q + "o"] = lin(G * E, W, 1.5), lin(W, H * E, 2.0)
        if m.get("v_mix"):
            sd[q + "vmix"] = 0.2 + 0.6 * torch.rand((), generator=gen)
        if spec["type"] == "attention":
            for n, r in (("q", H * D), ("k", G * D), ("v", G * E)):
                sd[f"{q}{n}.b"] = vec(r, 0, 0.5)
                w = 0.4 * torch.randn(r, m["conv"], generator=gen)
                w[:, -1] += 1.0
                sd[f"{q}{n}.conv"] = w
            sd[q + "q.norm"], sd[q + "k.norm"] = vec(H * D, 1.3, 0.3), vec(G * D, 1.3, 0.3)
        else:
            sd[q + "g"] = lin(H, W, 2.0)
        mlp, q = spec.get("mlp"), p + "mlp."
        if not mlp:
            continue
        sd[p + "norm2"] = vec(W, 0, 0.2)
        if mlp.get("kind", "dense") == "dense":
            sd[q + "gate"], sd[q + "up"], sd[q + "down"] = lin(mlp["ff"], W, 1.5), lin(mlp["ff"], W), lin(W, mlp["ff"])
            continue
        sd[q + "router"] = lin(mlp["router"]["experts"], W, 2.0)
        for e in range(mlp["router"]["experts"]):
            sd[f"{q}e{e}.up"], sd[f"{q}e{e}.down"] = lin(mlp["expert"]["ff"], W), lin(W, mlp["expert"]["ff"])
        if mlp.get("shared"):
            sd[q + "shared.up"], sd[q + "shared.down"] = lin(mlp["shared"]["ff"], W), lin(W, mlp["shared"]["ff"])
    return {k: v.to(torch.bfloat16) for k, v in sd.items()}
