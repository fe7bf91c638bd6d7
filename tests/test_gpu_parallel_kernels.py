"""The kernels of parallel layers, each alone, against the plain equations: pair embedding, two norms, token shift, gated linear recurrences, windowed
attention, experts, the clamped gated unit."""
import math

import pytest
import torch

from chatts_amd import _lib
from oracle import medilix as F
from tests.test_gpu_mixed_kernels import DEV, call, gen, operand, rel

pytestmark = pytest.mark.gpu
up = lambda n, m: (n + m - 1) // m * m


def rows_of(segs, dev=DEV):
    """segs: (first row, rows, first position, slot) -> ChattsRow table, ChattsSpan table"""
    meta = [[slot, pos + i, r0, t - 1 - i] for r0, t, pos, slot in segs for i in range(t)]
    spans = [[r0, t, pos, slot, -1] for r0, t, pos, slot in segs]
    return torch.tensor(meta, dtype=torch.int32, device=dev), torch.tensor(spans, dtype=torch.int32, device=dev)


def planes_of(t):
    hi = t.to(torch.bfloat16)
    return torch.stack([hi, (t - hi.float()).to(torch.bfloat16)])


# ---- embedding ---------------------------------------------------------------------------------------------------------------------
def test_embed_pair_over_portions_and_slots():
    g, V, W, buckets, scale = gen(0), 50, 72, 13, 2.5
    emb, big = torch.randn(V, W, generator=g).to(torch.bfloat16), torch.randn(buckets + 1, W, generator=g).to(torch.bfloat16)
    cfg = {"embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": 7, "mul_cur": 3}}}
    sd = {"embed": emb.double(), "bigram": big.double()}
    toks = torch.randint(0, V, (2, 12), generator=g)
    want = [F.embedding(cfg, sd, t.tolist()) for t in toks]
    ed, bd = emb.to(DEV), big.to(DEV)
    prev = torch.full((3,), 49, dtype=torch.int64, device=DEV)      # (rubbish: a sequence that starts must not see it)

    def step(segs, ids, single):
        rows, _ = rows_of(segs)
        T = rows.shape[0]
        x, x0, td = torch.full((T, W), 9.0, device=DEV), torch.full((T, W), 9.0, device=DEV), torch.tensor(ids, device=DEV)
        call("chatts_embed_pair", _lib.EmbedPairArgs(tokens=td.data_ptr(), rows=rows.data_ptr(), t=T, single=single, width_p=W, vocab=V, embed=ed.data_ptr(), scale=scale,
                                                     bigram=bd.data_ptr(), buckets=buckets, mul_prev=7, mul_cur=3, prev=prev.data_ptr(), x=x.data_ptr(), x0=x0.data_ptr()))
        assert torch.equal(x, x0)
        return x.cpu().double()
    a, b = toks.tolist()
    out = step([(0, 4, 0, 2), (4, 1, 0, 0)], a[:4] + b[:1], 0)      # an even number of rows, a single one
    assert rel(out, torch.cat([want[0][:4], want[1][:1]])) < 1e-6
    out = step([(0, 1, 4, 2), (1, 1, 1, 0)], [a[4], b[1]], 1)
    assert rel(out, torch.stack([want[0][4], want[1][1]])) < 1e-6
    out = step([(0, 2, 5, 2), (2, 3, 2, 0)], a[5:7] + b[2:5], 0)
    assert rel(out, torch.cat([want[0][5:7], want[1][2:5]])) < 1e-6
    before = prev.clone()
    rows = torch.tensor([[0, -1, 0, 0]], dtype=torch.int32, device=DEV)      # a parked row keeps the slot as it is
    x, td = torch.zeros(1, W, device=DEV), torch.tensor([3], device=DEV)
    call("chatts_embed_pair", _lib.EmbedPairArgs(tokens=td.data_ptr(), rows=rows.data_ptr(), t=1, single=1, width_p=W, vocab=V, embed=ed.data_ptr(), scale=scale,
                                                 bigram=bd.data_ptr(), buckets=buckets, mul_prev=7, mul_cur=3, prev=prev.data_ptr(), x=x.data_ptr()))
    assert torch.equal(prev, before)


# ---- norms --------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("width,groups", [(64, 1), (90, 3), (90, 90), (192, 6), (1540, 4), (5120, 5)])
@pytest.mark.parametrize("planes", [False, True])
def test_pair_norm_with_experts_sum_and_join(width, groups, planes):
    g, T, wp, eps, top = gen(width), 5, up(width, 64), 1e-3, 3
    pad = lambda t: torch.cat([t, torch.zeros(*t.shape[:-1], wp - width)], -1)
    x, x0, h = (pad(torch.randn(T, width, generator=g) * (1 + 4 * torch.rand(width, generator=g))) for _ in range(3))
    y = pad(torch.randn(9, width, generator=g))
    w1, w2 = pad(torch.randn(width, generator=g)), pad(torch.randn(width, generator=g))
    place = torch.tensor([[0, 8, 3], [1, -1, -1], [-1, -1, -1], [2, 4, -1], [5, 6, 7]], dtype=torch.int32)
    weight, kept = torch.rand(T, top, generator=g), torch.tensor([0.0, 0.3, 1.0, 0.2, 0.0])
    dev = {n: t.to(DEV) for n, t in dict(x0=x0, h=h, y=y, w1=w1, w2=w2, place=place, weight=weight, kept=kept).items()}
    hp = planes_of(dev["h"])

    for experts in (0, 1):
        want = x.double()
        if experts:
            want = want.clone()
            for t in range(T):
                for j in range(top):
                    if place[t, j] >= 0:
                        want[t] += weight[t, j].double() * y[place[t, j]].double()
                want[t] += kept[t].double() * h[t].double()
        for join in (0, 1):
            xd, n = x.to(DEV), 2 * wp if join else wp
            outs = [torch.full((2, T, n), 7.0, dtype=torch.bfloat16, device=DEV) if planes else torch.full((T, n), 7.0, device=DEV) for _ in range(2)]
            op = lambda o: operand(None if planes else o, o if planes else None, n)
            a = _lib.PairNormArgs(x=xd.data_ptr(), t=T, width=width, ldx=wp, groups=groups, eps=eps, out1=op(outs[0]), out2=op(outs[1]))
            if join:
                a.x0 = dev["x0"].data_ptr()
            else:
                a.w1, a.w2 = dev["w1"].data_ptr(), dev["w2"].data_ptr()
            if experts:
                a.y, a.place, a.weight, a.kept, a.top = dev["y"].data_ptr(), dev["place"].data_ptr(), dev["weight"].data_ptr(), dev["kept"].data_ptr(), top
                a.h = operand(None if planes else dev["h"], hp if planes else None, wp)
            call("chatts_pair_norm", a)
            got = [o[0].float() + o[1].float() if planes else o for o in outs]
            assert rel(xd, want) < (2e-5 if planes else 1e-6)
            if join:
                assert rel(got[0], torch.cat([want, x0.double()], 1)) < (2e-5 if planes else 1e-6)
            else:
                for o, w in zip(got, (w1, w2)):
                    assert rel(o[:, :width], F.group_norm(want[:, :width], w.double()[:width], groups, eps)) < (4e-5 if planes else 1e-6)
                    assert float(o[:, width:].abs().sum()) == 0


@pytest.mark.parametrize("width", [90, 2050])
def test_token_shift_over_portions(width):
    """segments of several tokens, then single tokens (in the norm's launch); slots are used again"""
    g, wp, eps, n = gen(width), up(width, 64), 1e-4, 3
    pad = lambda t: torch.cat([t, torch.zeros(*t.shape[:-1], wp - width)], -1)
    mu, w1 = pad(torch.rand(n, width, generator=g)), pad(torch.randn(width, generator=g))
    x = pad(torch.randn(11, width, generator=g))
    h = F.group_norm(x.double()[:, :width], w1.double()[:width], 1, eps)
    want = h[None] + (F.shifted(h) - h)[None] * mu.double()[:, None, :width]
    prev = torch.randn(2, wp, generator=g).to(DEV)      # rubbish
    mud, wd = mu.to(DEV), w1.to(DEV)
    for slot in (0, 1, 0):
        hd = pad(h[:6].float()).to(DEV)
        rows, _ = rows_of([(0, 6, 0, slot)])
        mix = torch.zeros(n, 7, wp, device=DEV)
        call("chatts_token_shift", _lib.TokenShiftArgs(h=hd.data_ptr(), t=6, ldx=wp, n_mix=n, mu=mud.data_ptr(), mix=operand(mix, None, wp), mix_stride=7 * wp,
                                                       prev=prev.data_ptr(), rows=rows.data_ptr()))
        assert rel(mix[:, :6, :width], want[:, :6]) < 1e-6
        prev[slot] = hd[5]
        for t in range(6, 11):
            rows, _ = rows_of([(0, 1, t, slot)])
            xd, out2 = x[t:t + 1].to(DEV), torch.zeros(1, wp, device=DEV)
            call("chatts_pair_norm", _lib.PairNormArgs(x=xd.data_ptr(), t=1, width=width, ldx=wp, groups=1, eps=eps, w1=wd.data_ptr(), w2=wd.data_ptr(), out2=operand(out2, None, wp),
                                                       n_mix=n, mu=mud.data_ptr(), mix=operand(mix, None, wp), mix_stride=7 * wp, prev=prev.data_ptr(), rows=rows.data_ptr()))
            assert rel(mix[:, 0, :width], want[:, t]) < 1e-6 and rel(out2[0, :width], h[t]) < 1e-6


# ---- recurrences ----------------------------------------------------------------------------------------------------------------------
class Recur:
    """one recurrent mixer with given raw inputs: the kernels on slots of a state pool, and the plain recurrence"""

    def __init__(self, kind, H, D, E, rank=12, seed=0, slots=3):
        g = gen(seed)
        self.kind, self.H, self.D, self.E, self.eps, self.cap = kind, H, D, E, 1e-4, 5.0
        self.rank, self.rp = rank, up(rank, 64)
        blocks = [("q", H * D), ("k", H * D), ("v", H * E), ("g", H * E)] + ([("a", self.rp)] if kind == "wkv" else [("i", H), ("f", H)])
        self.off, at = {}, 0
        for n, r in blocks:
            self.off[n] = at
            at += up(r, 64)
        self.ld, self.vals = at, dict(blocks)
        self.w2 = (torch.randn(H * D, rank, generator=g) / math.sqrt(rank)).to(torch.bfloat16)
        self.w0, self.u = torch.rand(H * D, generator=g) * 9 - 8, torch.randn(H * D, generator=g)
        self.bi, self.bf, self.norm = torch.randn(H, generator=g), torch.rand(H, generator=g) * 7, 1 + 0.2 * torch.randn(H * E, generator=g)
        w2 = torch.zeros(H * D, self.rp, dtype=torch.bfloat16)
        w2[:, :rank] = self.w2
        t = dict(w2d=w2.view(H * D, -1, 8).transpose(0, 1), w0=self.w0, u=self.u, bi=self.bi, bf=self.bf, nw=self.norm)
        self.t = {k: v.contiguous().to(DEV) for k, v in t.items()}
        self.state = torch.randn(slots, H, D, up(E, 4), generator=g).to(DEV)      # rubbish of an earlier sequence
        self.n, self.m = torch.randn(slots, H, D, generator=g).to(DEV), torch.full((slots, H), 3.0, device=DEV)

    def inputs(self, T, seed):
        x = torch.randn(T, self.ld, generator=gen(seed))
        if self.kind == "wkv":
            x[:, self.off["a"] + self.rank:] = 0
        return x

    def plain(self, x):
        x = x.double()
        T, H, D, E = x.shape[0], self.H, self.D, self.E
        blk = lambda n, c: x[:, self.off[n]:self.off[n] + c]
        q, k, v = blk("q", H * D).view(T, H, D), blk("k", H * D).view(T, H, D), blk("v", H * E).view(T, H, E)
        o, S = torch.zeros(T, H, E, dtype=torch.float64), torch.zeros(H, D, E, dtype=torch.float64)
        gate = blk("g", H * E)
        if self.kind == "wkv":
            w = torch.exp(-torch.exp(torch.tanh(blk("a", self.rank)) @ self.w2.double().T + self.w0.double())).view(T, H, D)
            for t in range(T):
                S, o[t] = F.wkv_step(S, q[t], k[t], v[t], w[t], self.u.double().view(H, D))
            gate = gate * torch.sigmoid(gate)
        else:
            i, f = F.soft_cap(blk("i", H) + self.bi.double(), self.cap), torch.nn.functional.logsigmoid(F.soft_cap(blk("f", H) + self.bf.double(), self.cap))
            n, m = torch.zeros(H, D, dtype=torch.float64), torch.zeros(H, dtype=torch.float64)
            for t in range(T):
                S, n, m, o[t] = F.mlstm_step(S, n, m, q[t] * D ** -0.5, k[t], v[t], i[t], f[t])
            gate = torch.sigmoid(gate)
        return F.rms(o, self.eps).reshape(T, H * E) * self.norm.double() * gate

    def run(self, x, segs, single=False, planes=False):
        xd, (rows, spans), H, D, E = x.to(DEV), rows_of(segs), self.H, self.D, self.E
        T = x.shape[0]
        out = torch.zeros(2, T, H * E, dtype=torch.bfloat16, device=DEV) if planes else torch.zeros(T, H * E, device=DEV)
        P = lambda n: self.t[n].data_ptr()
        a = _lib.RecurArgs(kind=_lib.RECUR_WKV if self.kind == "wkv" else _lib.RECUR_MLSTM, proj=xd.data_ptr(), ld_proj=self.ld, off_q=self.off["q"], off_k=self.off["k"],
                           off_v=self.off["v"], off_gate=self.off["g"], heads=H, dim=D, vdim=E, w2d=P("w2d"), w0=P("w0"), u=P("u"), bias_i=P("bi"), bias_f=P("bf"),
                           cap=self.cap, eps=self.eps, norm_w=P("nw"), state=self.state.data_ptr(), n_state=self.n.data_ptr(), m_state=self.m.data_ptr(),
                           rows=rows.data_ptr(), n_rows=T, spans=spans.data_ptr(), n_spans=len(segs), out=operand(None if planes else out, out if planes else None, H * E))
        if self.kind == "wkv":
            a.off_a, a.rank = self.off["a"], self.rp
        else:
            a.off_i, a.off_f = self.off["i"], self.off["f"]
        if single:
            call("chatts_recur_decode", a)
        else:
            chunks = torch.zeros(int(_lib.load().chatts_recur_chunk_floats(H, D, T, len(segs))), device=DEV)
            gates, o, den = torch.zeros(T, H, 4, device=DEV), torch.zeros(T, H * E, device=DEV), torch.zeros(T, H, device=DEV)
            decay = (torch.tanh(xd[:, self.off["a"]:self.off["a"] + self.rank]).double() @ self.w2.double().to(DEV).T).float() if self.kind == "wkv" else None
            a.chunks, a.gates, a.o, a.den = (t.data_ptr() for t in (chunks, gates, o, den))
            if decay is not None:
                a.decay, a.ld_decay = decay.data_ptr(), H * D
            call("chatts_recur_scan", a)
            call("chatts_recur_out", a)
        return (out[0].float() + out[1].float() if planes else out).cpu()


SIZES = [("wkv", 3, 20, 20), ("wkv", 2, 64, 64), ("wkv", 1, 160, 160), ("wkv", 1, 250, 250), ("mlstm", 3, 20, 37), ("mlstm", 2, 64, 64), ("mlstm", 1, 136, 96),
         ("mlstm", 1, 200, 250), ("mlstm", 5, 1, 3)]


@pytest.mark.parametrize("kind,H,D,E", SIZES)
def test_recurrence_token_by_token_and_in_portions(kind, H, D, E):
    r = Recur(kind, H, D, E, seed=D)
    x = r.inputs(75, 1)
    want = r.plain(x)
    got = torch.cat([r.run(x[t:t + 1], [(0, 1, t, 0)], single=True) for t in range(40)])
    assert rel(got, want[:40]) < 2e-6
    assert rel(r.run(x, [(0, 75, 0, 1)]), want) < 2e-6
    assert rel(r.run(x, [(0, 75, 0, 1)], planes=True), want) < 4e-5      # the slot again, from the start
    at, out = 0, []
    for n in (2, 16, 1, 17, 2, 3, 33, 1):      # portions around a chunk's size; the state passes between the two forms
        out.append(r.run(x[at:at + n], [(0, n, at, 2)], single=n == 1))
        at += n
    assert at == 75 and rel(torch.cat(out), want) < 2e-6


@pytest.mark.parametrize("kind,H,D,E", SIZES[:2] + SIZES[4:6])
def test_recurrence_of_unequal_segments(kind, H, D, E):
    r = Recur(kind, H, D, E, seed=3)
    xs = [r.inputs(n, 10 + n) for n in (41, 23, 60)]
    want = [r.plain(x) for x in xs]
    cut = (20, 1, 33)
    first = r.run(torch.cat([x[:c] for x, c in zip(xs, cut)]), [(0, 20, 0, 1), (20, 1, 0, 2), (21, 33, 0, 0)])
    rest = r.run(torch.cat([x[c:] for x, c in zip(xs, cut)]), [(0, 21, 20, 1), (21, 22, 1, 2), (43, 27, 33, 0)])
    assert rel(first, torch.cat([w[:c] for w, c in zip(want, cut)])) < 2e-6
    assert rel(rest, torch.cat([w[c:] for w, c in zip(want, cut)])) < 2e-6


def test_wkv_remembers_and_forgets():
    """channels whose decay is 1 - 2e-5 keep a key of 300 tokens ago, channels whose decay underflows keep nothing but the bonus"""
    r = Recur("wkv", 1, 32, 32)
    r.w2.zero_(); r.t["w2d"].zero_()
    r.w0[:16], r.w0[16:] = -11.0, 8.0
    r.t["w0"].copy_(r.w0)
    x = r.inputs(320, 7) * 0.01
    x[10, r.off["k"]:r.off["k"] + 32] = 5.0
    x[10, r.off["v"]:r.off["v"] + 32] = torch.randn(32, generator=gen(2)) * 5
    x[310, r.off["q"]:r.off["q"] + 32] = 3.0
    want = r.plain(x)
    assert rel(r.run(x, [(0, 320, 0, 0)])[310], want[310]) < 5e-6
    r.run(x[:300], [(0, 300, 0, 1)])
    got = torch.cat([r.run(x[t:t + 1], [(0, 1, t, 1)], single=True) for t in range(300, 320)])
    assert rel(got[10], want[310]) < 5e-6


@pytest.mark.parametrize("f_in,i_in", [(60.0, 60.0), (-60.0, 60.0), (60.0, -60.0), (-60.0, -60.0)])
def test_mlstm_saturated_gates(f_in, i_in):
    """both gates at their caps: the running maximum and the floor exp(-m) of the normaliser"""
    r = Recur("mlstm", 2, 24, 20)
    x = r.inputs(90, 5)
    x[:, r.off["f"]:r.off["f"] + 2] = f_in
    x[:, r.off["i"]:r.off["i"] + 2] = i_in
    x[40, r.off["i"]] = -i_in
    want = r.plain(x)
    assert rel(r.run(x, [(0, 90, 0, 0)]), want) < 5e-6
    assert rel(torch.cat([r.run(x[t:t + 1], [(0, 1, t, 1)], single=True) for t in range(90)]), want) < 5e-6


def test_recur_tanh_operand_and_last_rows():
    r = Recur("wkv", 2, 20, 20)
    x = r.inputs(9, 1) * 3
    xd, (rows, spans) = x.to(DEV), rows_of([(0, 4, 3, 2), (4, 5, 0, 0)])
    a = _lib.RecurArgs(kind=_lib.RECUR_WKV, proj=xd.data_ptr(), ld_proj=r.ld, off_q=0, off_k=0, off_v=0, off_gate=0, off_a=r.off["a"], heads=2, dim=20, vdim=20, rank=64,
                       w2d=r.t["w2d"].data_ptr(), w0=r.t["w0"].data_ptr(), u=r.t["u"].data_ptr(), norm_w=r.t["nw"].data_ptr(), state=r.state.data_ptr(), rows=rows.data_ptr(),
                       n_rows=9, spans=spans.data_ptr(), n_spans=2)
    import ctypes as C
    out = torch.zeros(9, 64, device=DEV)
    op = operand(out, None, 64)
    _lib.check(_lib.load().chatts_recur_tanh(C.byref(a), C.byref(op), _lib.stream_ptr()))
    assert rel(out, torch.tanh(x[:, r.off["a"]:r.off["a"] + 64].double())) < 1e-6
    h, prev, o, res = torch.randn(9, 128, device=DEV), torch.zeros(3, 128, device=DEV), torch.randn(9, 40, device=DEV), torch.zeros(9, 40, device=DEV)
    a.o, a.out, a.h, a.prev, a.ld_h = o.data_ptr(), operand(res, None, 40), h.data_ptr(), prev.data_ptr(), 128
    call("chatts_recur_out", a)
    assert torch.equal(prev[2], h[3]) and torch.equal(prev[0], h[8]) and float(prev[1].abs().sum()) == 0


# ---- windowed attention ------------------------------------------------------------------------------------------------------------------
class Window:
    """paged keys and values of a few slots, the plain formula over whole sequences"""

    def __init__(self, H, G, D, E, window=0, keep=0, sink=1, gate=True, f32=False, scale=0.25, seed=0, slots=3, pages=5):
        g = gen(seed)
        self.H, self.G, self.D, self.E, self.window, self.keep, self.sink, self.gate, self.f32, self.scale, self.eps = H, G, D, E, window, keep, sink, gate, f32, scale, 1e-4
        self.Dp, self.Ep = up(D, 32), up(E, 16)
        self.off, at = {}, 0
        for n, r in (("q", H * D), ("k", G * D), ("v", G * E), ("g", H * E)):
            self.off[n] = at
            at += up(r, 64)
        self.ld = at
        self.qn, self.kn = 1.5 + 0.2 * torch.randn(D, generator=g), 1.5 + 0.2 * torch.randn(D, generator=g)
        dt = torch.float32 if f32 else torch.bfloat16
        self.kc = torch.randn(slots * pages, G, 64, self.Dp, generator=g).to(dt).to(DEV) * 50      # rubbish in rows never written
        self.vc = torch.randn(slots * pages, G, 64, self.Ep, generator=g).to(dt).to(DEV) * 50
        self.table = torch.randperm(slots * pages, generator=g).view(slots, pages).to(torch.int32).to(DEV)
        self.t = dict(qn=self.qn.to(DEV), kn=self.kn.to(DEV))

    def inputs(self, T, seed):
        return torch.randn(T, self.ld, generator=gen(seed))

    def plain(self, x):
        x = x.double()
        T, H, G, D, E = x.shape[0], self.H, self.G, self.D, self.E
        blk = lambda n, c: x[:, self.off[n]:self.off[n] + c]
        rnd = (lambda t: t) if self.f32 else (lambda t: t.float().to(torch.bfloat16).double())      # what the pages and the queries hold
        q, k = rnd(F.rms(blk("q", H * D).view(T, H, D), self.eps) * self.qn.double()), rnd(F.rms(blk("k", G * D).view(T, G, D), self.eps) * self.kn.double())
        v, head = rnd(blk("v", G * E).view(T, G, E)), torch.arange(H) // (H // G)
        mask = {"size": self.window, "keep_first": self.keep} if self.window else None
        see = torch.tensor([[F.visible(i, j, mask) for j in range(T)] for i in range(T)])
        s = (torch.einsum("ihd,jhd->hij", q, k[:, head]) * self.scale).masked_fill(~see, -math.inf)
        a = F.sink_softmax(s) if self.sink else torch.softmax(s, -1)
        o = torch.einsum("hij,jhe->ihe", a, v[:, head]).reshape(T, H * E)
        return o * torch.sigmoid(blk("g", H * E)) if self.gate else o

    def run(self, x, segs, form, splits=1, planes=False):
        xd, (rows, spans), T = x.to(DEV), rows_of(segs), x.shape[0]
        q = torch.zeros(T, self.H * self.Dp, dtype=torch.float32 if self.f32 else torch.bfloat16, device=DEV)
        n = self.H * self.E
        out = torch.zeros(2, T, n, dtype=torch.bfloat16, device=DEV) if planes else torch.zeros(T, n, device=DEV)
        part = torch.zeros(T * self.H * splits * (self.Ep + 4), device=DEV)
        a = _lib.WindowArgs(proj=xd.data_ptr(), ld_proj=self.ld, off_q=self.off["q"], off_k=self.off["k"], off_v=self.off["v"], off_gate=self.off["g"] if self.gate else -1,
                            heads=self.H, kv_heads=self.G, dim=self.D, vdim=self.E, dim_p=self.Dp, vdim_p=self.Ep, scale=self.scale, eps=self.eps, q_norm=self.t["qn"].data_ptr(),
                            k_norm=self.t["kn"].data_ptr(), window=self.window, keep_first=self.keep, sink=self.sink, kcache=self.kc.data_ptr(), vcache=self.vc.data_ptr(),
                            cache_f32=int(self.f32), table=self.table.data_ptr(), table_stride=self.table.shape[1], log_block=6, rows=rows.data_ptr(), n_rows=T,
                            spans=spans.data_ptr(), n_spans=len(segs), longest=max(s[1] for s in segs), n_splits=splits, partial=part.data_ptr(),
                            q=_lib.Operand(f32=q.data_ptr() if self.f32 else None, hi=None if self.f32 else q.data_ptr(), lo=None, ld=self.H * self.Dp),
                            out=operand(None if planes else out, out if planes else None, n))
        call("chatts_window_prep", a)
        call("chatts_window_" + form, a)
        return (out[0].float() + out[1].float() if planes else out).cpu()


WINDOWS = [dict(H=6, G=2, D=24, E=42, window=30, keep=5), dict(H=20, G=1, D=32, E=32), dict(H=6, G=3, D=136, E=200, window=65, keep=70, scale=0.1),
           dict(H=4, G=4, D=64, E=64, window=64, keep=64), dict(H=8, G=2, D=128, E=128, window=100, keep=0, scale=0.1, gate=False), dict(H=2, G=1, D=48, E=18, window=1, keep=2),
           dict(H=3, G=1, D=20, E=16, window=17, keep=130, sink=0), dict(H=2, G=2, D=256, E=256, sink=0, scale=0.06)]


@pytest.mark.parametrize("case", range(len(WINDOWS)))
def test_window_attention(case):
    """prompts, portions and single rows with one and several ranges of keys; 32-bit; a slot again"""
    w = Window(**WINDOWS[case], seed=case)
    x = w.inputs(210, case)
    want = w.plain(x)
    tol = 6e-3      # probabilities enter the second product in bf16
    assert rel(w.run(x, [(0, 210, 0, 1)], "prefill"), want) < tol
    assert rel(w.run(x, [(0, 210, 0, 2)], "attend", planes=True), want) < tol
    at, out = 0, []
    for n in (3, 61, 2, 70, 1, 24, 49):
        out.append(w.run(x[at:at + n], [(0, n, at, 1)], "prefill"))
        at += n
    assert at == 210 and rel(torch.cat(out), want) < tol
    got = [w.run(x[:150], [(0, 150, 0, 0)], "prefill")] + [w.run(x[t:t + 1], [(0, 1, t, 0)], "attend", splits=t % 4 + 1) for t in range(150, 210)]
    assert rel(torch.cat(got), want) < tol
    e = Window(**WINDOWS[case], f32=True, seed=case)
    assert rel(e.run(x, [(0, 210, 0, 1)], "attend"), e.plain(x)) < 2e-6


@pytest.mark.parametrize("form", ["prefill", "attend"])
def test_window_edges(form):
    """one key that would take all the weight: the queries just inside and just outside the window, and around the kept tokens, see it or not"""
    W, K = 37, 6
    for target in (0, 3, K - 1, K, K + 1, 50, 63, 64, 65, 100):
        w = Window(H=2, G=1, D=32, E=32, window=W, keep=K, scale=1.0, gate=False, seed=target)
        x = w.inputs(180, 3) * 0.3
        for b, r in (("q", 64), ("k", 32)):
            x[:, w.off[b]:w.off[b] + r] = 0.2 * x[:, w.off[b]:w.off[b] + r]
        x[:, w.off["q"]] = x[:, w.off["q"] + 32] = 4.0          # every query looks along the first dimension ...
        x[:, w.off["k"]] = -1.0
        x[target, w.off["k"]] = 4.0                             # ... where one key lies
        x[target, w.off["v"]:w.off["v"] + 32] = 9.0
        want, got = w.plain(x), w.run(x, [(0, 180, 0, 1)], form)
        sees = [F.visible(i, target, {"size": W, "keep_first": K}) for i in range(180)]
        for i in {target, target + 1, target + W - 1, target + W, target + W + 1, 179}:
            if i < 180:
                assert (float(want[i].mean()) > 5) == sees[i] and float((got[i].double() - want[i]).abs().max()) < 0.05, (target, i)
        assert rel(got, want) < 6e-3


@pytest.mark.parametrize("f32", [False, True])
def test_sink_takes_weight_when_scores_are_low(f32):
    w = Window(H=4, G=2, D=32, E=16, scale=4.0, gate=False, f32=f32)
    x = w.inputs(70, 2)
    x[:, w.off["q"]] = x[:, w.off["q"] + 32] = x[:, w.off["q"] + 64] = x[:, w.off["q"] + 96] = 30.0
    x[:, w.off["k"]] = x[:, w.off["k"] + 32] = -30.0
    x[40, w.off["k"]] = x[40, w.off["k"] + 32] = 30.0
    want = w.plain(x)
    assert float(want[39].abs().max()) < 1e-6 < 1e-2 < float(want[40].abs().max())
    got = w.run(x, [(0, 70, 0, 0)], "attend")
    assert float((got.double() - want).abs().max()) < (1e-5 if f32 else 0.05)
    if not f32:
        assert float((w.run(x, [(0, 70, 0, 1)], "prefill").double() - want).abs().max()) < 0.05
        for s in (2, 5):
            assert float((w.run(x[69:], [(0, 1, 69, 1)], "attend", splits=s).double() - want[69]).abs().max()) < 0.05


def test_window_unequal_segments():
    w = Window(H=6, G=2, D=24, E=40, window=30, keep=5)
    xs = [w.inputs(n, n) for n in (90, 33, 140)]
    want, cut = [w.plain(x) for x in xs], (64, 1, 100)
    a = w.run(torch.cat([x[:c] for x, c in zip(xs, cut)]), [(0, 64, 0, 2), (64, 1, 0, 0), (65, 100, 0, 1)], "prefill")
    b = w.run(torch.cat([x[c:] for x, c in zip(xs, cut)]), [(0, 26, 64, 2), (26, 32, 1, 0), (58, 40, 100, 1)], "prefill")
    assert rel(a, torch.cat([t[:c] for t, c in zip(want, cut)])) < 6e-3 and rel(b, torch.cat([t[c:] for t, c in zip(want, cut)])) < 6e-3


# ---- experts --------------------------------------------------------------------------------------------------------------------------
MOES = [dict(experts=6, identity=2, top=3, count=4, keep=2, W=90, ff=40), dict(experts=5, identity=0, top=1, count=1, keep=1, W=128, ff=64),
        dict(experts=40, identity=8, top=6, count=8, keep=3, W=192, ff=96), dict(experts=3, identity=3, top=4, count=2, keep=2, W=64, ff=200)]


@pytest.mark.parametrize("case", range(len(MOES)))
@pytest.mark.parametrize("T", [1, 7, 16, 33, 300])
@pytest.mark.parametrize("exact", [0, 1])
def test_experts(case, T, exact):
    c = MOES[case]
    g, E, N, W, ff, top = gen(case), c["experts"], c["experts"] + c["identity"], c["W"], c["ff"], c["top"]
    Wp, fp = up(W, 64), up(ff, 64)
    h = torch.randn(T, W, generator=g)
    lin = lambda o, i: (torch.randn(o, i, generator=g) / math.sqrt(i)).to(torch.bfloat16)
    sd = {"router": lin(N, W) * 3, "correction": torch.randn(N, generator=g) * 0.3 - 0.8}      # (negative choice scores)
    sd.update({f"e{e}.{n}": lin(*s) for e in range(E) for n, s in (("gate", (ff, W)), ("up", (ff, W)), ("down", (W, ff)))})
    sd64 = {k: v.double() for k, v in sd.items()}
    spec = {"router": {"experts": E, "identity": c["identity"], "top": top, "groups": {"count": c["count"], "keep": c["keep"]}}}
    z = h.double() @ sd64["router"].T
    idx, wt = F.route(z, sd64["correction"], spec["router"])
    want = F.experts(h.double(), sd64, "", spec)
    gu, dn = torch.zeros(E, fp // 16, 2, 16, Wp, dtype=torch.bfloat16), torch.zeros(E, Wp, fp, dtype=torch.bfloat16)
    for e in range(E):
        for j, n in enumerate(("gate", "up")):
            full = torch.zeros(fp, Wp, dtype=torch.bfloat16)
            full[:ff, :W] = sd[f"e{e}.{n}"]
            gu[e, :, j] = full.view(fp // 16, 16, Wp)
        dn[e, :W, :ff] = sd[f"e{e}.down"]
    hd = torch.zeros(T, Wp)
    hd[:, :W] = h
    hd, zd = hd.to(DEV), z.float().to(DEV)
    hp = planes_of(hd)
    parked = T == 7
    rows = torch.tensor([[i, -1 if parked and i == 2 else 5, i, 0] for i in range(T)], dtype=torch.int32, device=DEV)
    I = lambda n: torch.full((n,), -7, dtype=torch.int32, device=DEV)
    ids, place, order, offsets, tiles = I(T * top), I(T * top), I(T * top), I(E + 2), I(4 * int(_lib.load().chatts_moe_tiles(T, top, E)))
    weight, kept, y = torch.zeros(T, top, device=DEV), torch.zeros(T, device=DEV), torch.zeros(T * top, Wp, device=DEV)
    act = torch.zeros(T * top, fp, device=DEV) if exact else torch.zeros(2, T * top, fp, dtype=torch.bfloat16, device=DEV)
    gud, dnd, cd = gu.to(DEV), dn.to(DEV), sd["correction"].to(DEV)
    a = _lib.MoeArgs(experts=E, identity=c["identity"], top=top, groups=c["count"], keep=c["keep"], width_p=Wp, ff_p=fp, gate_up=gud.data_ptr(), down=dnd.data_ptr(),
                     correction=cd.data_ptr(), logits=zd.data_ptr(), ld_logits=N, h=operand(hd if exact else None, None if exact else hp, Wp), rows=rows.data_ptr(), n_rows=T,
                     exact=exact, ids=ids.data_ptr(), place=place.data_ptr(), order=order.data_ptr(), offsets=offsets.data_ptr(), tiles=tiles.data_ptr(),
                     weight=weight.data_ptr(), kept=kept.data_ptr(), act=operand(act if exact else None, None if exact else act, fp), y=y.data_ptr())
    call("chatts_moe_route", a)
    chosen, at = ids.view(T, top).cpu(), place.view(T, top).cpu()
    live = [t for t in range(T) if not (parked and t == 2)]
    for t in live:
        assert sorted(i for i in chosen[t].tolist() if i >= 0) == sorted(i for i in idx[t].tolist() if i < E)
    if parked:
        assert (chosen[2] == -1).all() and (at[2] == -1).all() and float(kept[2]) == 0
    used = at[at >= 0].tolist()
    assert sorted(used) == list(range(len(used)))                    # the places are packed, experts in order
    assert torch.equal(chosen.view(-1)[order.cpu()[:len(used)].long()], chosen[chosen >= 0].sort().values)
    x = torch.zeros(T, Wp, device=DEV)
    tiled = [torch.empty_like(t) for t in (gud, dnd)]
    for src, dst, n, k in ((gud, tiled[0], 2 * fp, Wp), (dnd, tiled[1], Wp, fp)):
        for e in range(E):
            _lib.check(_lib.load().chatts_tile_bf16(src[e].data_ptr(), n, k, k, dst[e].data_ptr(), _lib.stream_ptr()))
    if not exact:                                                    # the weights' tiled copies: the same products
        a.gate_up_t, a.down_t = (t.data_ptr() for t in tiled)
        call("chatts_moe_experts", a)
        from_tiles = y.clone()
        y.zero_()
        a.gate_up_t = a.down_t = None
    call("chatts_moe_experts", a)
    assert exact or torch.equal(y, from_tiles)
    call("chatts_pair_norm", _lib.PairNormArgs(x=x.data_ptr(), t=T, width=W, ldx=Wp, groups=1, eps=1e-5, y=y.data_ptr(), place=place.data_ptr(), weight=weight.data_ptr(),
                                               kept=kept.data_ptr(), h=a.h, top=top))
    assert rel(x.cpu()[live][:, :W], want[live]) < (2e-6 if exact else 5e-5)
    assert float(x[:, W:].abs().sum()) == 0


# ---- the clamped gated unit -------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("m", [1, 3, 16, 40, 130, 600])
@pytest.mark.parametrize("exact", [0, 1])
@pytest.mark.parametrize("n,k", [(96, 320), (320, 1536)])
def test_linear_clamp_glu(m, exact, n, k):
    g, limit, alpha = gen(m), 0.8, 1.3
    a, w = torch.randn(m, k, generator=g), (torch.randn(2 * n, k, generator=g) / math.sqrt(k)).to(torch.bfloat16)
    z = a.double() @ w.double().T
    gate, lin = z.view(m, n // 16, 2, 16)[:, :, 0].reshape(m, n), z.view(m, n // 16, 2, 16)[:, :, 1].reshape(m, n)
    gate, lin = gate.clamp_max(limit), lin.clamp(-limit, limit)
    want = gate * torch.sigmoid(alpha * gate) * (lin + 1)
    ad, wd, c = a.to(DEV), w.to(DEV), torch.zeros(m, n, device=DEV)
    ws = torch.zeros(max(16, int(_lib.load().chatts_linear_workspace(m, 2 * n, k))), dtype=torch.uint8, device=DEV)
    kw = dict(w=wd.data_ptr(), m=m, n=2 * n, k=k, ldw=k, ldc=n, epilogue=_lib.EPI_CLAMPGLU, glu_limit=limit, glu_alpha=alpha, workspace=ws.data_ptr(), workspace_bytes=ws.numel())
    call("chatts_linear", _lib.LinearArgs(a=ad.data_ptr(), lda=k, c=c.data_ptr(), exact_f32=exact, **kw))
    assert rel(c, want) < (2e-6 if exact or m == 1 else 2e-5)
    if m > 1 and not exact:
        hp, out = planes_of(ad), torch.zeros(2, m, n, dtype=torch.bfloat16, device=DEV)
        call("chatts_linear", _lib.LinearArgs(a_hi=hp[0].data_ptr(), a_lo=hp[1].data_ptr(), ld_planes=k, c_hi=out[0].data_ptr(), c_lo=out[1].data_ptr(), ld_cplanes=n, **kw))
        assert rel(out[0].float() + out[1].float(), want) < 4e-5


# ---- several projections of one shape ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("m", [1, 2, 16, 40, 130])
@pytest.mark.parametrize("exact", [0, 1])
@pytest.mark.parametrize("n,k", [(64, 128), (192, 2048)])
def test_linear_batch(m, exact, n, k):
    g, B = gen(m), 3
    a, w = torch.randn(B, m + 1, k, generator=g), (torch.randn(B, n, k, generator=g) / math.sqrt(k)).to(torch.bfloat16)
    want = torch.stack([a[i, :m].double() @ w[i].double().T for i in range(B)], 1)
    ad, wd = a.to(DEV), w.to(DEV)
    ws = torch.zeros(max(16, int(_lib.load().chatts_linear_workspace_batch(m, n, k, B))), dtype=torch.uint8, device=DEV)
    kw = dict(w=wd.data_ptr(), m=m, n=n, k=k, ldw=k, ldc=B * n + 64, epilogue=_lib.EPI_NONE, exact_f32=exact, workspace=ws.data_ptr(), workspace_bytes=ws.numel(), batch=B,
              a_stride=(m + 1) * k, w_stride=n * k, c_stride=n)
    forms = [dict(a=ad.data_ptr(), lda=k)]
    if m > 1 and not exact:
        hp = planes_of(ad)
        forms.append(dict(a_hi=hp[0].data_ptr(), a_lo=hp[1].data_ptr(), ld_planes=k))
    for f in forms:
        c = torch.zeros(m, B * n + 64, device=DEV)
        call("chatts_linear", _lib.LinearArgs(c=c.data_ptr(), **f, **kw))
        assert rel(c[:, :B * n].reshape(m, B, n), want) < (1e-6 if exact or m == 1 else 2e-5)
        assert float(c[:, B * n:].abs().sum()) == 0
