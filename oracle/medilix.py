"""Plain, slow reference of the Medilix decoder (torch, CPU, float64 by default), one function per mechanism.

A whole sequence goes in, the logits of every position come out; there is no cache, no batching and no chunking here.  Shares no code
with chatts_amd: the product path is checked against these equations.

A model is (cfg, sd): cfg = the dictionary of config.json, sd = name -> tensor.
"""
import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis"""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    """every one of `groups` consecutive parts of the vector by its own root mean square, then the weight over all of it"""
    T, W = x.shape
    return rms(x.view(T, groups, W // groups), eps).view(T, W) * w


def embedding(cfg, sd, tokens):
    """scaled token rows plus a row per (previous token, token); the last row of that table for a sequence's first token"""
    tok = [int(t) for t in tokens]
    x = sd["embed"][torch.tensor(tok)] * cfg["embedding"].get("scale", 1.0)
    b = cfg["embedding"].get("bigram")
    if b:
        rows = [b["buckets"]] + [(p * b["mul_prev"] + t * b["mul_cur"]) % b["buckets"] for p, t in zip(tok, tok[1:])]
        x = x + sd["bigram"][torch.tensor(rows)]
    return x


def shifted(h):
    """the previous token's vector, zeros for the first token"""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def wkv_decay(z, sd, p):
    """z [T, width] -> factors in (0, 1) per (head, key channel), flat"""
    return torch.exp(-torch.exp(torch.tanh(z @ sd[p + "w1"].T) @ sd[p + "w2"].T + sd[p + "w0"]))


def wkv_step(S, r, k, v, w, u):
    """S [H, dim, dim]; r, k, v, w, u [H, dim] -> (S', o [H, dim])"""
    o = torch.einsum("hij,hi->hj", S, r) + (r * u * k).sum(-1, keepdim=True) * v
    return w[:, :, None] * S + k[:, :, None] * v[:, None, :], o


def wkv(h, sd, p, m, eps):
    T, H, D = h.shape[0], m["heads"], m["dim"]
    d = shifted(h) - h
    mix = {s: h + d * sd[p + "mu." + s] for s in "rkvgw"}
    r, k, v = ((mix[s] @ sd[p + s].T).view(T, H, D) for s in "rkv")
    z = mix["g"] @ sd[p + "g"].T
    gate = z * torch.sigmoid(z)
    w = wkv_decay(mix["w"], sd, p).view(T, H, D)
    S, o = torch.zeros(H, D, D, dtype=h.dtype), torch.zeros(T, H, D, dtype=h.dtype)
    for t in range(T):
        S, o[t] = wkv_step(S, r[t], k[t], v[t], w[t], sd[p + "u"])
    return (rms(o, eps).reshape(T, H * D) * sd[p + "norm"] * gate) @ sd[p + "o"].T


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def mlstm_step(S, n, m, q, k, v, i, f):
    """S [H, dim, vdim], n [H, dim], m [H] (running maximum); i, f [H]: logarithms of the input and forget gates -> (S, n, m, o [H, vdim])"""
    m1 = torch.maximum(f + m, i)
    a, b = torch.exp(f + m - m1), torch.exp(i - m1)
    S = a[:, None, None] * S + b[:, None, None] * k[:, :, None] * v[:, None, :]
    n = a[:, None] * n + b[:, None] * k
    den = torch.maximum((n * q).sum(-1).abs(), torch.exp(-m1)) + 1e-6
    return S, n, m1, torch.einsum("hij,hi->hj", S, q) / den[:, None]


def mlstm(h, sd, p, m, eps):
    T, H, D, E = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ sd[p + "q"].T).view(T, H, D) * D ** -0.5
    k, v = (h @ sd[p + "k"].T).view(T, H, D), (h @ sd[p + "v"].T).view(T, H, E)
    i = soft_cap(h @ sd[p + "i"].T + sd[p + "i.b"], m["gate_cap"])
    f = torch.nn.functional.logsigmoid(soft_cap(h @ sd[p + "f"].T + sd[p + "f.b"], m["gate_cap"]))
    S, n, mx = (torch.zeros(*s, dtype=h.dtype) for s in ((H, D, E), (H, D), (H,)))
    o = torch.zeros(T, H, E, dtype=h.dtype)
    for t in range(T):
        S, n, mx, o[t] = mlstm_step(S, n, mx, q[t], k[t], v[t], i[t], f[t])
    return (rms(o, eps).reshape(T, H * E) * sd[p + "norm"] * torch.sigmoid(h @ sd[p + "g"].T)) @ sd[p + "o"].T


def visible(i, j, mask):
    """does position i see position j: causal, the last `size` positions (itself included) and the first `keep_first` ones"""
    if j > i:
        return False
    return not mask or i - j < mask["size"] or j < mask.get("keep_first", 0)


def sink_softmax(s):
    """exp(s) / (1 + sum exp(s)) over the last axis"""
    top = torch.clamp(s.max(-1, keepdim=True).values, min=0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attention(h, sd, p, m, eps):
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ sd[p + "q"].T).view(T, H, D), eps) * sd[p + "q.norm"]
    k = rms((h @ sd[p + "k"].T).view(T, G, D), eps) * sd[p + "k.norm"]
    v = (h @ sd[p + "v"].T).view(T, G, E)
    head = torch.arange(H) // (H // G)
    see = torch.tensor([[visible(i, j, m.get("mask")) for j in range(T)] for i in range(T)])
    s = torch.einsum("ihd,jhd->hij", q, k[:, head]) * m["scale"]
    a = sink_softmax(s.masked_fill(~see, -math.inf))
    o = torch.einsum("hij,jhe->ihe", a, v[:, head]).reshape(T, H * E)
    return (o * torch.sigmoid(h @ sd[p + "g"].T)) @ sd[p + "o"].T


MIXERS = {"wkv": wkv, "mlstm": mlstm, "attention": attention}


def dense(h, sd, p, spec):
    g = torch.clamp(h @ sd[p + "gate"].T, max=spec["limit"])
    u = torch.clamp(h @ sd[p + "up"].T, -spec["limit"], spec["limit"])
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ sd[p + "down"].T


def route(z, correction, r):
    """router logits z [T, N] -> (chosen outputs [T, top], their weights [T, top])"""
    s = torch.softmax(z, -1)
    choice = s + correction
    groups = r.get("groups") or {"count": 1, "keep": 1}
    T, N = z.shape
    best = choice.view(T, groups["count"], -1).max(-1).values
    keep = torch.zeros(T, groups["count"], dtype=torch.bool).scatter_(1, best.topk(groups["keep"], -1).indices, True)
    choice = choice.masked_fill(~keep.repeat_interleave(N // groups["count"], 1), -math.inf)
    idx = choice.topk(r["top"], -1).indices
    w = s.gather(1, idx)
    return idx, w / (w.sum(-1, keepdim=True) + 1e-20)


def choice_margin(z, correction, r):
    """how much a router's logits z [T, N] prefer what is chosen to the next best, groups and outputs: a much smaller rounding changes nothing"""
    choice, groups, T = torch.softmax(z, -1) + correction, r.get("groups") or {"count": 1, "keep": 1}, z.shape[0]

    def gap(v, n):
        v = v.sort(-1, descending=True).values
        return v[:, n - 1] - v[:, n] if n < v.shape[1] else torch.full((T,), math.inf, dtype=z.dtype)
    best = choice.view(T, groups["count"], -1).max(-1).values
    out = best < best.sort(-1, descending=True).values[:, groups["keep"] - 1:groups["keep"]]
    return torch.minimum(gap(best, groups["keep"]), gap(choice.masked_fill(out.repeat_interleave(z.shape[1] // groups["count"], 1), -1e9), r["top"]))


def experts(h, sd, p, spec, margins=None):
    r = spec["router"]
    z = h @ sd[p + "router"].T
    idx, w = route(z, sd[p + "correction"], r)
    if margins is not None:
        margins.append(choice_margin(z, sd[p + "correction"], r))
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(idx[t].tolist(), w[t]):
            if e >= r["experts"]:
                y[t] += a * h[t]
                continue
            q = f"{p}e{e}."
            g = sd[q + "gate"] @ h[t]
            y[t] += a * (sd[q + "down"] @ (g * torch.sigmoid(g) * (sd[q + "up"] @ h[t])))
    return y


def layer(x, sd, i, spec, norm, margins=None):
    p = f"l{i}."
    y = MIXERS[spec["type"]](group_norm(x, sd[p + "norm1"], norm["groups"], norm["eps"]), sd, p + "mix.", spec["mixer"], norm["eps"])
    if spec.get("mlp"):
        h = group_norm(x, sd[p + "norm2"], norm["groups"], norm["eps"])
        y = y + (experts(h, sd, p + "mlp.", spec["mlp"], margins) if spec["mlp"]["kind"] == "moe" else dense(h, sd, p + "mlp.", spec["mlp"]))
    return x + y


def runs(cfg):
    """the layer runs in order: (layer index, pass number if this run opens a pass of the loop, else None)"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def forward(cfg, sd, tokens, dtype=torch.float64, want_layers=False, margins=None):
    """-> logits [T, vocab] (and the residual stream after every layer run); margins: a list that gets choice_margin of every router run"""
    sd = {k: v.to(dtype) for k, v in sd.items()}
    x = x0 = embedding(cfg, sd, tokens)
    streams = []
    for i, t in runs(cfg):
        if t is not None:
            x = torch.cat([x, x0], -1) @ sd["loop.in"].T
        x = layer(x, sd, i, cfg["layers"][i], cfg["norm"], margins)
        streams.append(x)
    logits = group_norm(x, sd["final.norm"], cfg["norm"]["groups"], cfg["norm"]["eps"]) @ sd["head"].T
    return (logits, streams) if want_layers else logits


def generate(cfg, sd, tokens, n, dtype=torch.float64):
    """greedy continuation, everything recomputed for every token"""
    seq = list(tokens)
    for _ in range(n):
        seq.append(int(forward(cfg, sd, seq, dtype)[-1].argmax()))
    return seq[len(tokens):]


def random_model(cfg, seed=0):
    """bf16-representable random weights of a configuration that has, beside config.json's keys, the low-rank size of every wkv mixer as
    mixer["_rank"] -> name -> bfloat16 tensor.  Decays reach from almost none to strong; some gates saturate; queries and keys of the
    attention layers share directions, so that single scores stand out."""
    gen = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(o, i, gain=1.0):
        return torch.randn(o, i, generator=gen) * gain / math.sqrt(i)

    def ones(n):
        return 1.0 + 0.2 * torch.randn(n, generator=gen)

    scale = cfg["embedding"].get("scale", 1.0)
    sd = {"embed": torch.randn(V, W, generator=gen) / scale, "final.norm": ones(W), "head": lin(V, W)}
    if cfg["embedding"].get("bigram"):
        sd["bigram"] = 0.5 * torch.randn(cfg["embedding"]["bigram"]["buckets"] + 1, W, generator=gen)
    if cfg.get("loop"):
        sd["loop.in"] = torch.cat([torch.eye(W) + lin(W, W, 0.3), lin(W, W, 0.5)], 1)
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        q = p + "mix."
        sd[p + "norm1"] = ones(W)
        if spec["type"] == "wkv":
            n, R = m["heads"] * m["dim"], m.get("_rank", 8)
            for s in "rkvgw":
                sd[q + "mu." + s] = torch.rand(W, generator=gen)
            for s in "rkvg":
                sd[q + s] = lin(n, W)
            sd[q + "w1"], sd[q + "w2"] = lin(R, W), lin(n, R)
            sd[q + "w0"] = torch.rand(n, generator=gen) * 8 - 7
            sd[q + "u"] = torch.randn(m["heads"], m["dim"], generator=gen)
            sd[q + "norm"], sd[q + "o"] = ones(n), lin(W, n)
        elif spec["type"] == "mlstm":
            H, D, E = m["heads"], m["dim"], m["vdim"]
            sd[q + "q"], sd[q + "k"], sd[q + "v"] = lin(H * D, W, 1.5), lin(H * D, W, 1.5), lin(H * E, W)
            sd[q + "i"], sd[q + "f"] = lin(H, W), lin(H, W)
            sd[q + "i.b"], sd[q + "f.b"] = torch.randn(H, generator=gen), torch.rand(H, generator=gen) * 7
            sd[q + "g"], sd[q + "norm"], sd[q + "o"] = lin(H * E, W), ones(H * E), lin(W, H * E)
        else:
            H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            k = lin(G * D, W)
            sd[q + "k"] = k
            sd[q + "q"] = 0.6 * k.view(G, 1, D, W).expand(G, H // G, D, W).reshape(H * D, W) + lin(H * D, W, 0.8)
            sd[q + "v"], sd[q + "g"] = lin(G * E, W), lin(H * E, W)
            sd[q + "q.norm"], sd[q + "k.norm"] = 1.3 * ones(D), 1.3 * ones(D)
            sd[q + "o"] = lin(W, H * E)
        mlp = spec.get("mlp")
        if not mlp:
            continue
        sd[p + "norm2"] = ones(W)
        if mlp["kind"] == "moe":
            r, ff = mlp["router"], mlp["expert"]["ff"]
            N = r["experts"] + r.get("identity", 0)
            for e in range(r["experts"]):
                sd[f"{p}mlp.e{e}.gate"], sd[f"{p}mlp.e{e}.up"], sd[f"{p}mlp.e{e}.down"] = lin(ff, W), lin(ff, W), lin(W, ff)
            sd[p + "mlp.router"], sd[p + "mlp.correction"] = lin(N, W, 2.0), torch.randn(N, generator=gen) * 0.2 - 0.5
        else:
            sd[p + "mlp.gate"], sd[p + "mlp.up"], sd[p + "mlp.down"] = lin(mlp["ff"], W, 1.5), lin(mlp["ff"], W, 1.5), lin(W, mlp["ff"])
    return {k: v.to(torch.bfloat16) for k, v in sd.items()}
