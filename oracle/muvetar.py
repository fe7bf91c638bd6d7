"""Plain, slow reference of the Muvetar decoder (torch, CPU, float64 by default), one function per mechanism.

A whole sequence goes in, the logits of every position come out; there is no cache, no batching and no chunking here.  Shares no code
with chatts_amd: the product path is checked against these equations.

A model is (cfg, sd): cfg = the dictionary of config.json, sd = name -> tensor.
"""
import math

import torch

GATE_SLOPE = 1.702


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def sinusoid(positions, width, dtype=torch.float64):
    """[T, width]: sine and cosine in turn of position * 10000^(-2 i / width)"""
    p = torch.zeros(len(positions), width, dtype=torch.float64)
    for i in range((width + 1) // 2):
        a = torch.tensor([float(t) for t in positions], dtype=torch.float64) * 10000.0 ** (-2.0 * i / width)
        p[:, 2 * i] = a.sin()
        if 2 * i + 1 < width:
            p[:, 2 * i + 1] = a.cos()
    return p.to(dtype)


def embedding(cfg, sd, tokens):
    e = sd["embed"][torch.tensor([int(t) for t in tokens])]
    return e + sinusoid(range(len(tokens)), cfg["width"], e.dtype)


# ---- minGRU ----
def candidate(u):
    return torch.where(u >= 0, u + 0.5, torch.sigmoid(u))


def gru_step(S, z, c):
    return (1 - z) * S + z * c


def mingru(h, sd, p, m, eps):
    z, c = torch.sigmoid(h @ sd[p + "z"].T + sd[p + "z.b"]), candidate(h @ sd[p + "x"].T + sd[p + "x.b"])
    S, states = torch.zeros_like(z[0]), []
    for t in range(h.shape[0]):
        S = gru_step(S, z[t], c[t])
        states.append(S)
    return (torch.stack(states) * silu(h @ sd[p + "g"].T)) @ sd[p + "o"].T


# ---- attention with a logarithmic distance bias ----
def distance_bias(r1, r2, d):
    """r1, r2 [H], d [..]: distances -> [H, ..], to be taken off the scores"""
    at = (-1,) + (1,) * d.dim()
    return r1.view(at) * torch.log(1 + r2.view(at) * d)


def causal_softmax(s):
    T = s.shape[-1]
    return torch.softmax(s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf), -1)


def attention(h, sd, p, m):
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = ((h @ sd[p + n].T).view(T, heads, size) for n, heads, size in (("q", H, D), ("k", G, D), ("v", G, E)))
    head = torch.arange(H) // (H // G)
    i = torch.arange(T)
    d = (i[:, None] - i[None, :]).clamp(min=0).to(h.dtype)      # (what lies ahead is masked anyway)
    s = torch.einsum("ihd,jhd->hij", q, k[:, head]) * m["scale"] - distance_bias(sd[p + "r1"], sd[p + "r2"], d)
    return torch.einsum("hij,jhe->ihe", causal_softmax(s), v[:, head]).reshape(T, H * E) @ sd[p + "o"].T


# ---- selective scan ----
def causal_conv(u, w, b):
    """u [T, C], w [C, taps]: every channel's sum over its last `taps` values, the newest with the last weight; zeros before the start"""
    taps = w.shape[1]
    y = torch.zeros_like(u) + b
    for back in range(min(taps, u.shape[0])):
        y[back:] += w[:, taps - 1 - back] * u[:u.shape[0] - back]
    return y


def scan_step(S, dt, A, B, x):
    """S, A [C, N]; dt, x [C]; B [N]"""
    return torch.exp(dt[:, None] * A) * S + (dt * x)[:, None] * B[None, :]


def selective_scan(h, sd, p, m):
    C, N, R = m["inner"], m["state"], m["dt_rank"]
    x, z = (h @ sd[p + "in"].T).split([C, C], -1)
    x = silu(causal_conv(x, sd[p + "conv"], sd[p + "conv.b"]))
    dt, B, Cn = (x @ sd[p + "x"].T).split([R, N, N], -1)
    dt = softplus(dt @ sd[p + "dt"].T + sd[p + "dt.b"])
    A = -torch.exp(sd[p + "A_log"])
    S, y = torch.zeros_like(A), torch.zeros_like(x)
    for t in range(h.shape[0]):
        S = scan_step(S, dt[t], A, B[t], x[t])
        y[t] = S @ Cn[t] + sd[p + "D"] * x[t]
    return (y * silu(z)) @ sd[p + "o"].T


def parallel(h, sd, p, m, eps):
    return m["left_scale"] * attention(h, sd, p + "left.", m["left"]) + m["right_scale"] * selective_scan(h, sd, p + "right.", m["right"])


MIXERS = {"mingru": mingru, "parallel": parallel}


# ---- experts ----
def clamped_glu(h, sd, p, limit):
    g = torch.clamp(h @ sd[p + "gate"].T, max=limit)
    u = torch.clamp(h @ sd[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(GATE_SLOPE * g) * (u + 1)) @ sd[p + "down"].T


def route(z, top, scale):
    """router logits z [T, N] -> (chosen experts [T, top], their weights: softmax over ALL experts, times scale)"""
    best = torch.softmax(z, -1).topk(top, -1)
    return best.indices, best.values * scale


def choice_margin(z, top):
    """how much a router's logits prefer the last chosen expert to the next one"""
    v = z.sort(-1, descending=True).values
    return v[:, top - 1] - v[:, top] if top < z.shape[1] else torch.full((z.shape[0],), math.inf, dtype=z.dtype)


def experts(h, sd, p, spec, margins=None):
    r = spec["router"]
    z = h @ sd[p + "router"].T
    idx, w = route(z, r["top"], r["scale"])
    if margins is not None:
        margins.append(choice_margin(z, r["top"]))
    y = torch.zeros_like(h)
    for e in range(r["experts"]):
        t, j = (idx == e).nonzero(as_tuple=True)
        if len(t):
            y[t] += w[t, j, None] * clamped_glu(h[t], sd, f"{p}e{e}.", spec["expert"]["limit"])
    if spec.get("shared"):
        y = y + clamped_glu(h, sd, p + "shared.", spec["shared"]["limit"])
    return y


# ---- layers ----
def depth_average(w, streams):
    """w [n], streams: the embedding output and every layer's result so far"""
    return sum(a * x for a, x in zip(w, streams))


def layer(x, sd, i, spec, mult, eps, margins=None):
    p = f"l{i}."
    x = x + mult * MIXERS[spec["type"]](rms_norm(x, sd[p + "norm1"], eps), sd, p + "mix.", spec["mixer"], eps)
    if spec.get("mlp"):
        x = x + mult * experts(rms_norm(x, sd[p + "norm2"], eps), sd, p + "mlp.", spec["mlp"], margins)
    return x


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def forward(cfg, sd, tokens, dtype=torch.float64, want_layers=False, margins=None):
    """-> logits [T, vocab] (and the residual stream after every layer); margins: a list that gets choice_margin of every router"""
    sd = {k: v.to(dtype) for k, v in sd.items()}
    x, eps = embedding(cfg, sd, tokens), cfg["norm"]["eps"]
    streams, after = [x], []
    for i, spec in enumerate(cfg["layers"]):
        streams.append(layer(x, sd, i, spec, cfg["residual_mult"], eps, margins))
        x = depth_average(sd[f"l{i}.dwa"], streams)
        after.append(x)
    logits = soft_cap(rms_norm(x, sd["final.norm"], eps) @ sd["head"].T, cfg["logit_softcap"])
    return (logits, after) if want_layers else logits


def generate(cfg, sd, tokens, n, dtype=torch.float64):
    """greedy continuation, everything recomputed for every token"""
    seq = list(tokens)
    for _ in range(n):
        seq.append(int(forward(cfg, sd, seq, dtype)[-1].argmax()))
    return seq[len(tokens):]


def random_model(cfg, seed=0):
    """bf16-representable random weights -> name -> bfloat16 tensor.  Queries and keys share directions, so that single scores stand out against the distance
    bias; states that forget at once and states that keep thousands of tokens; router logits lie apart; every earlier stream has its share."""
    gen = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def lin(o, i, gain=1.0):
        return torch.randn(o, i, generator=gen) * gain / math.sqrt(i)

    def vec(n, mean, spread):
        return mean + spread * torch.randn(n, generator=gen)

    sd = {"embed": torch.randn(V, W, generator=gen), "final.norm": vec(W, 1, 0.2), "head": lin(V, W, 2.0)}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        q = p + "mix."
        sd[p + "norm1"] = vec(W, 1, 0.2)
        sd[p + "dwa"] = torch.cat([vec(i + 1, 0, 0.3), vec(1, 0.9, 0.1)])
        if spec["type"] == "mingru":
            C = m["width"]
            sd.update({q + "z": lin(C, W, 1.5), q + "z.b": vec(C, -2.0, 2.5), q + "x": lin(C, W, 1.5), q + "x.b": vec(C, 0, 0.3), q + "g": lin(C, W),
                       q + "o": lin(W, C, 1.5)})
        else:
            l, r = m["left"], m["right"]
            H, G, D, E, a = l["heads"], l["kv_heads"], l["dim"], l["vdim"], q + "left."
            k = lin(G * D, W)
            sd[a + "k"] = k
            sd[a + "q"] = 1.5 / (l["scale"] * math.sqrt(D)) * k.view(G, 1, D, W).expand(G, H // G, D, W).reshape(H * D, W) + lin(H * D, W, 0.5)
            sd.update({a + "v": lin(G * E, W, 1.5), a + "r1": 1.5 * torch.rand(H, generator=gen), a + "r2": 0.02 + 0.5 * torch.rand(H, generator=gen),
                       a + "o": lin(W, H * E, 2.0)})
            C, N, R, b = r["inner"], r["state"], r["dt_rank"], q + "right."
            w = 0.4 * torch.randn(C, r["conv"], generator=gen)
            w[:, -1] += 1.0
            sd.update({b + "in": lin(2 * C, W), b + "conv": w, b + "conv.b": vec(C, 0, 0.2), b + "x": lin(R + 2 * N, C, 2.0), b + "dt": lin(C, R, 1.0),
                       b + "dt.b": vec(C, -3.0, 1.0), b + "A_log": vec(C * N, -1.5, 2.0).view(C, N), b + "D": vec(C, 0.8, 0.2), b + "o": lin(W, C, 2.0)})
        mlp, q = spec.get("mlp"), p + "mlp."
        if not mlp:
            continue
        sd[p + "norm2"] = vec(W, 1, 0.2)
        sd[q + "router"] = lin(mlp["router"]["experts"], W, 2.0)
        for name, ff in [(f"e{e}", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])] + ([("shared", mlp["shared"]["ff"])] if mlp.get("shared") else []):
            sd.update({f"{q}{name}.gate": lin(ff, W, 1.5), f"{q}{name}.up": lin(ff, W, 1.5), f"{q}{name}.down": lin(W, ff)})
    return {k: v.to(torch.bfloat16) for k, v in sd.items()}
