"""The kernels of pre-norm layers, each alone, against the plain equations: sinusoidal positions, factors and averages over depth with the next norm, the minimal
gated recurrence, the selective scan, attention with a logarithmic distance bias, clamped experts weighted by their scores, the cap of the logits."""
import ctypes as C
import math

import pytest
import torch

from chatts_amd import _lib
from chatts_amd.rotary import sinusoid_tables
from oracle import muvetar as F
from tests.test_gpu_mixed_kernels import DEV, call, gen, operand, rel
from tests.test_gpu_parallel_kernels import planes_of, rows_of, up
from tests.test_gpu_postnorm_kernels import TOL, Attn

pytestmark = pytest.mark.gpu


# ---- the stream -----------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("W", [64, 90, 1540])
def test_embedding_with_positions(W):
    """positions of a page's edges and far ones; a parked row; the copy that averages over depth start from"""
    g, V, wp = gen(W), 50, up(W, 64)
    pos = [0, 1, 2, 63, 64, 65, 127, 128, 1000, 4095, -1]
    emb = torch.zeros(V, wp, dtype=torch.bfloat16)
    emb[:, :W] = torch.randn(V, W, generator=g)
    toks = torch.randint(0, V, (len(pos),), generator=g)
    want = emb[toks].double()[:, :W] + F.sinusoid([max(p, 0) for p in pos], W)
    fine, coarse = sinusoid_tables(W, wp, 4096, 10000.0, DEV)
    rows = torch.tensor([[0, p, i, 0] for i, p in enumerate(pos)], dtype=torch.int32, device=DEV)
    x, x0, ed, td = torch.full((len(pos), wp), 7.0, device=DEV), torch.full((len(pos), wp), 7.0, device=DEV), emb.to(DEV), toks.to(DEV)
    call("chatts_embed_pair", _lib.EmbedPairArgs(tokens=td.data_ptr(), rows=rows.data_ptr(), t=len(pos), single=0, width_p=wp, vocab=V, embed=ed.data_ptr(), scale=1.0,
                                                 x=x.data_ptr(), x0=x0.data_ptr(), width=W, pos_fine=fine.data_ptr(), pos_coarse=coarse.data_ptr()))
    live = [i for i, p in enumerate(pos) if p >= 0]
    assert float((x.cpu().double()[live, :W] - want[live]).abs().max()) < 1e-6 and float(x[:, W:].abs().sum()) == 0 and torch.equal(x, x0)


@pytest.mark.parametrize("width,T", [(64, 5), (90, 5), (1540, 70), (3000, 3), (5120, 3), (5120, 66), (9000, 2)])
@pytest.mark.parametrize("planes", [False, True])
def test_depth_norm(width, T, planes):
    g, wp, eps, top, mult = gen(width + T), up(width, 64), 1e-3, 3, 0.6
    pad = lambda t: torch.cat([t, torch.zeros(*t.shape[:-1], wp - width)], -1)
    x, y, w = pad(torch.randn(T, width, generator=g) * (1 + 4 * torch.rand(width, generator=g))), pad(torch.randn(T, width, generator=g) * 3), pad(torch.randn(width, generator=g))
    ey, streams = pad(torch.randn(9, width, generator=g)), pad(torch.randn(8, T + 1, width, generator=g))
    place, weight, depth = torch.randint(-1, 9, (T, top), generator=g, dtype=torch.int32), torch.rand(T, top, generator=g), torch.randn(9, generator=g)
    dev = {n: t.to(DEV) for n, t in dict(y=y, ey=ey, w=w, place=place, weight=weight, depth=depth).items()}
    for use_y, experts, n, keep, norm in ((0, 0, -1, 0, 1), (1, 0, -1, 0, 1), (1, 1, 1, 1, 1), (0, 1, 7, 1, 1), (1, 1, 8, 0, 0), (1, 0, 5, 0, 1), (0, 0, 0, 1, 1)):
        add = torch.zeros(T, wp, dtype=torch.float64)
        if use_y:
            add += y.double()
        if experts:
            for t in range(T):
                for j in range(top):
                    if place[t, j] >= 0:
                        add[t] += weight[t, j].double() * ey[place[t, j]].double()
        s = x.double() + mult * add
        v = s if n < 0 else F.depth_average(depth[:n + 1].double(), [streams[j, :T].double() for j in range(n)] + [s])
        want = F.rms_norm(v[:, :width], w.double()[:width], eps)
        xd, sd = x.to(DEV), streams.to(DEV)
        out = torch.full((2, T, wp), 7.0, dtype=torch.bfloat16, device=DEV) if planes else torch.full((T, wp), 7.0, device=DEV)
        a = _lib.DepthNormArgs(x=xd.data_ptr(), t=T, width=width, ldx=wp, mult=mult, eps=eps, y=dev["y"].data_ptr() if use_y else None, w=dev["w"].data_ptr() if norm else None,
                               out=operand(None if planes else out, out if planes else None, wp))
        if experts:
            a.ey, a.place, a.weight, a.top = dev["ey"].data_ptr(), dev["place"].data_ptr(), dev["weight"].data_ptr(), top
        if n >= 0:
            a.depth, a.streams, a.stream_stride, a.n_streams, a.keep = dev["depth"].data_ptr(), sd.data_ptr(), (T + 1) * wp, n, keep
        call("chatts_depth_norm", a)
        assert rel(xd[:, :width], v[:, :width]) < 1e-6 and float(xd[:, width:].abs().sum()) == 0
        kept = streams.clone()
        if keep:
            kept[n, :T] = s.float()
        assert rel(sd, kept) < 1e-6 and (keep or torch.equal(sd.cpu(), streams))
        got = out[0].float() + out[1].float() if planes else out
        if norm:
            assert rel(got[:, :width], want) < (2e-5 if planes else 1e-6) and float(got[:, width:].abs().sum()) == 0
        else:
            assert float((got - (14.0 if planes else 7.0)).abs().max()) == 0


@pytest.mark.parametrize("n", [1, 3, 4, 1023, 5000])
def test_soft_cap(n):
    x = torch.cat([torch.tensor([0.0, 1e-4, -1e-4, 300.0, -300.0, 1e30]), torch.randn(5000, generator=gen(n)) * 20])[:n]
    xd = torch.cat([x, torch.full((4,), 3.0)]).to(DEV)
    _lib.check(_lib.load().chatts_soft_cap(xd.data_ptr(), n, 15.0, _lib.stream_ptr()))
    assert float((xd[:n].cpu().double() - F.soft_cap(x.double(), 15.0)).abs().max()) < 5e-6 and float((xd[n:] - 3.0).abs().sum()) == 0


# ---- minimal gated recurrence -------------------------------------------------------------------------------------------------------------
class Gru:
    """raw projections in, read-outs out, on slots full of rubbish; and the plain recurrence"""

    def __init__(self, W, seed=0, slots=3, scale=1.0):
        self.W, self.scale, g = W, scale, gen(seed)
        self.off = {n: i * up(W, 64) for i, n in enumerate("zxg")}
        self.ld = 3 * up(W, 64)
        self.state = torch.randn(slots, up(W, 4), generator=g).to(DEV) * 50

    def inputs(self, T, seed, gate=0.0):
        x = torch.zeros(T, self.ld)
        for n, o in self.off.items():
            x[:, o:o + self.W] = torch.randn(T, self.W, generator=gen(seed + ord(n))) * 2 + (gate if n == "z" else 0)
        return x

    def plain(self, x):
        z, c, gate = (x[:, self.off[n]:self.off[n] + self.W].double() for n in "zxg")
        z, c, S, out = torch.sigmoid(z), F.candidate(c), torch.zeros(self.W, dtype=torch.float64), []
        for t in range(x.shape[0]):
            S = F.gru_step(S, z[t], c[t])
            out.append(S)
        return torch.stack(out) * F.silu(gate) * self.scale

    def run(self, x, segs, single=False, planes=False):
        xd, (rows, spans), T, ld = x.to(DEV), rows_of(segs), x.shape[0], up(self.W, 64)
        out = torch.zeros(2, T, ld, dtype=torch.bfloat16, device=DEV) if planes else torch.zeros(T, ld, device=DEV)
        a = _lib.GruArgs(proj=xd.data_ptr(), ld_proj=self.ld, off_z=self.off["z"], off_x=self.off["x"], off_g=self.off["g"], width=self.W, out_scale=self.scale,
                         state=self.state.data_ptr(), rows=rows.data_ptr(), n_rows=T, spans=spans.data_ptr(), n_spans=len(segs),
                         out=operand(None if planes else out, out if planes else None, ld))
        call("chatts_gru_decode" if single else "chatts_gru_scan", a)
        return (out[0].float() + out[1].float() if planes else out)[:, :self.W].cpu()


@pytest.mark.parametrize("W", [3, 16, 75, 130, 1028])
@pytest.mark.parametrize("gate", [0.0, -7.0, 7.0])
def test_minimal_recurrence(W, gate):
    """whole prompts over several tiles, portions down to one token, token by token, slots used again; gates that keep thousands of tokens, or none"""
    T = 2300 if W in (16, 75) else 300
    w = Gru(W, W, scale=0.7)
    x = w.inputs(T, 1, gate)
    want = w.plain(x)
    assert rel(w.run(x, [(0, T, 0, 1)]), want) < 2e-6 and rel(w.run(x, [(0, T, 0, 0)], planes=True), want) < 2e-5
    at, out = 0, []
    for n in (1, 2, 61, 3, 128, 100, T - 295):
        out.append(w.run(x[at:at + n], [(0, n, at, 1)]))
        at += n
    assert at == T and rel(torch.cat(out), want) < 2e-6
    got = [w.run(x[:200], [(0, 200, 0, 2)])] + [w.run(x[t:t + 1], [(0, 1, t, 2)], single=True) for t in range(200, 240)]
    assert rel(torch.cat(got), want[:240]) < 2e-6
    assert rel(torch.cat([w.run(x[t:t + 1], [(0, 1, t, 0)], single=True) for t in range(5)]), want[:5]) < 2e-6


def test_minimal_recurrence_of_unequal_segments():
    """sequences side by side, then their next portions; a parked row and a slot without a segment keep their states"""
    w = Gru(75, 3)
    xs = [w.inputs(n, n) for n in (90, 33, 700)]
    want, cut = [w.plain(x) for x in xs], (64, 1, 500)
    a = w.run(torch.cat([x[:c] for x, c in zip(xs, cut)]), [(0, 64, 0, 2), (64, 1, 0, 0), (65, 500, 0, 1)])
    b = w.run(torch.cat([x[c:] for x, c in zip(xs, cut)]), [(0, 26, 64, 2), (26, 32, 1, 0), (58, 200, 500, 1)])
    assert rel(a, torch.cat([t[:c] for t, c in zip(want, cut)])) < 2e-6 and rel(b, torch.cat([t[c:] for t, c in zip(want, cut)])) < 2e-6
    before = w.state.clone()
    w.run(w.inputs(2, 9), [(0, 1, -1, 0), (1, 1, 0, 2)], single=True)
    assert torch.equal(w.state[:2], before[:2]) and not torch.equal(w.state[2], before[2])


# ---- selective scan -----------------------------------------------------------------------------------------------------------------------
class Select:
    """raw x and z projections in, read-outs out, on states and rings full of rubbish; and the plain scan"""

    def __init__(self, C_, N, R, taps, seed=0, slots=3, scale=1.0, a_mean=-1.0, a_spread=2.0, dt_mean=-2.0):
        g = gen(seed)
        self.__dict__.update({k: v for k, v in locals().items() if k not in ("self", "g")}, C=C_)
        self.rank, self.n4, self.c4, self.k = up(R, 64), up(N, 4), up(C_, 4), up(C_, 64)
        self.off = {"x": 64, "z": 64 + up(C_, 64)}
        self.ld = 64 + 2 * up(C_, 64)
        bf = lambda t: t.to(torch.bfloat16).float()
        self.w = {"conv": 0.5 * torch.randn(C_, taps, generator=g), "conv.b": 0.3 * torch.randn(C_, generator=g), "x": bf(torch.randn(R + 2 * N, C_, generator=g) * 2 / math.sqrt(C_)),
                  "dt": bf(torch.randn(C_, R, generator=g) / math.sqrt(R)), "dt.b": dt_mean + torch.randn(C_, generator=g), "A_log": a_mean + a_spread * torch.randn(C_, N, generator=g),
                  "D": torch.randn(C_, generator=g)}
        # the second projection: the blocks dt, B, C at columns of their own
        self.at = {"dt": 0, "b": self.rank, "c": self.rank + up(N, 16)}
        self.ldl = up(self.at["c"] + up(N, 16), 64)
        low = torch.zeros(self.ldl, self.k)
        for n, a, b in (("dt", 0, R), ("b", R, R + N), ("c", R + N, R + 2 * N)):
            low[self.at[n]:self.at[n] + b - a, :C_] = self.w["x"][a:b]
        dt, conv, a = torch.zeros(self.k, self.rank), torch.zeros(taps, self.c4), torch.zeros(C_, self.n4)
        dt[:C_, :R], conv[:, :C_], a[:, :N] = self.w["dt"], self.w["conv"].t(), -torch.exp(self.w["A_log"].double()).float() * math.log2(math.e)
        pad = lambda t: torch.cat([t, torch.zeros(self.c4 - C_)])
        self.t = {n: t.to(DEV) for n, t in dict(conv=conv, conv_b=pad(self.w["conv.b"]), dt=dt.to(torch.bfloat16), dt_b=pad(self.w["dt.b"]), a=a, d=pad(self.w["D"])).items()}
        self.low, self.wdt = low.to(DEV), dt.to(DEV)
        self.s, self.ring = torch.randn(slots, C_, self.n4, generator=g).to(DEV) * 50, torch.randn(slots, taps, self.c4, generator=g).to(DEV) * 50

    def inputs(self, T, seed):
        x = torch.zeros(T, self.ld)
        for n, o in self.off.items():
            x[:, o:o + self.C] = torch.randn(T, self.C, generator=gen(seed + ord(n)))
        return x

    def plain(self, x):
        w = {k: v.double() for k, v in self.w.items()}
        u, z = (x[:, self.off[n]:self.off[n] + self.C].double() for n in "xz")
        u = F.silu(F.causal_conv(u, w["conv"], w["conv.b"]))
        dt, B, Cn = (u @ w["x"].T).split([self.R, self.N, self.N], -1)
        dt, A = F.softplus(dt @ w["dt"].T + w["dt.b"]), -torch.exp(w["A_log"])
        S, out = torch.zeros_like(A), []
        for t in range(x.shape[0]):
            S = F.scan_step(S, dt[t], A, B[t], u[t])
            out.append(S @ Cn[t] + w["D"] * u[t])
        return torch.stack(out) * F.silu(z) * self.scale

    def run(self, x, segs, single=False, planes=False):
        xd, (rows, spans), T = x.to(DEV), rows_of(segs), x.shape[0]
        u, up_ = torch.zeros(T, self.k, device=DEV), torch.zeros(2, T, self.k, dtype=torch.bfloat16, device=DEV)
        out = torch.zeros(2, T, self.k, dtype=torch.bfloat16, device=DEV) if planes else torch.zeros(T, self.k, device=DEV)
        P = {n: t.data_ptr() for n, t in self.t.items()}
        a = _lib.SelectArgs(proj=xd.data_ptr(), ld_proj=self.ld, off_x=self.off["x"], off_z=self.off["z"], inner=self.C, state=self.N, taps=self.taps, conv_ch=self.c4,
                            conv_w=P["conv"], conv_b=P["conv_b"], ld_low=self.ldl, off_dt=self.at["dt"], off_b=self.at["b"], off_c=self.at["c"], rank=self.rank, w_dt=P["dt"],
                            dt_bias=P["dt_b"], a=P["a"], d=P["d"], out_scale=self.scale, s=self.s.data_ptr(), ring=self.ring.data_ptr(), rows=rows.data_ptr(), n_rows=T,
                            spans=spans.data_ptr(), n_spans=0 if single else len(segs), u=operand(u, up_, self.k), out=operand(None if planes else out, out if planes else None, self.k))
        call("chatts_select_conv", a)
        assert rel(up_[0].float() + up_[1].float(), u.cpu()) < 2e-5
        low = u @ self.low.t()                       # (a projection of the framework's in the product)
        delta = low[:, :self.rank].contiguous() @ self.wdt.t()
        a.low, a.delta, a.ld_delta = low.data_ptr(), delta.data_ptr(), self.k
        if planes and not single and self.rank <= 384:                    # the step sizes by the kernel for many rows
            steps, hp = torch.zeros(T, self.k, device=DEV), torch.zeros(2, up(T, 16), self.rank, dtype=torch.bfloat16, device=DEV)
            frags = self.wdt.to(torch.bfloat16).view(self.k // 16, 16, self.rank // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous()
            a.delta, a.delta_steps, a.w_dt_f, a.dt_hi, a.dt_lo = steps.data_ptr(), 1, frags.data_ptr(), hp[0].data_ptr(), hp[1].data_ptr()
            call("chatts_select_steps", a)
            want = F.softplus(delta.double().cpu()[:, :self.C] + self.w["dt.b"].double())
            assert float((steps.cpu().double()[:, :self.C] / want - 1).abs().max()) < 1e-4
        call("chatts_select_decode" if single else "chatts_select_scan", a)
        return (out[0].float() + out[1].float() if planes else out)[:, :self.C].cpu()


SELECTS = [dict(C_=50, N=5, R=7, taps=5), dict(C_=91, N=19, R=70, taps=1), dict(C_=128, N=1, R=8, taps=2), dict(C_=64, N=16, R=16, taps=4), dict(C_=200, N=32, R=130, taps=3),
           dict(C_=70, N=40, R=30, taps=4), dict(C_=33, N=128, R=3, taps=9), dict(C_=20, N=200, R=12, taps=4), dict(C_=1100, N=8, R=64, taps=4, scale=0.3),
           dict(C_=300, N=12, R=256, taps=4), dict(C_=130, N=16, R=320, taps=4), dict(C_=70, N=4, R=500, taps=4)]
STOL = 1e-5


@pytest.mark.parametrize("case", SELECTS, ids=lambda c: "-".join(f"{k}{v}" for k, v in c.items()))
def test_selective_scan(case):
    """prompts, portions down to one and two tokens, token by token; slots used again; more taps than a portion has tokens"""
    T = 210
    w = Select(**case)
    x = w.inputs(T, 1)
    want = w.plain(x)
    assert rel(w.run(x, [(0, T, 0, 1)]), want) < STOL and rel(w.run(x, [(0, T, 0, 0)], planes=True), want) < 3e-5
    at, out = 0, []
    for n in (1, 2, 61, 3, 70, 2, 2, 69):
        out.append(w.run(x[at:at + n], [(0, n, at, 1)]))
        at += n
    assert at == T and rel(torch.cat(out), want) < STOL
    got = [w.run(x[:150], [(0, 150, 0, 2)])] + [w.run(x[t:t + 1], [(0, 1, t, 2)], single=True) for t in range(150, 180)]
    assert rel(torch.cat(got), want[:180]) < STOL
    got = [w.run(x[t:t + 1], [(0, 1, t, 0)], single=True) for t in range(12)] + [w.run(x[12:40], [(0, 28, 12, 0)])]
    assert rel(torch.cat(got), want[:40]) < STOL


@pytest.mark.parametrize("case", SELECTS[:4], ids=lambda c: f"N{c['N']}")
def test_selective_scan_of_unequal_segments(case):
    w = Select(**case)
    xs = [w.inputs(n, n) for n in (90, 33, 140)]
    want, cut = [w.plain(x) for x in xs], (64, 1, 100)
    a = w.run(torch.cat([x[:c] for x, c in zip(xs, cut)]), [(0, 64, 0, 2), (64, 1, 0, 0), (65, 100, 0, 1)])
    b = w.run(torch.cat([x[c:] for x, c in zip(xs, cut)]), [(0, 26, 64, 2), (26, 32, 1, 0), (58, 40, 100, 1)])
    assert rel(a, torch.cat([t[:c] for t, c in zip(want, cut)])) < STOL and rel(b, torch.cat([t[c:] for t, c in zip(want, cut)])) < STOL
    before = w.s.clone(), w.ring.clone()
    w.run(w.inputs(2, 9), [(0, 1, -1, 0), (1, 1, 0, 2)], single=True)
    assert torch.equal(w.s[:2], before[0][:2]) and torch.equal(w.ring[:2], before[1][:2]) and not torch.equal(w.s[2], before[0][2])


@pytest.mark.parametrize("case", [dict(C_=8200, N=7, R=8, taps=2), dict(C_=8200, N=13, R=8, taps=3), dict(C_=8300, N=25, R=8, taps=4), dict(C_=4100, N=16, R=16, taps=4)],
                         ids=lambda c: f"C{c['C_']}-N{c['N']}")
def test_selective_scan_of_many_channels(case):
    """the forms for more workgroups than there are CUs, with three sequences"""
    w = Select(**case)
    xs = [w.inputs(n, n) for n in (70, 33, 47)]
    want, cut = [w.plain(x) for x in xs], (40, 1, 16)
    a = w.run(torch.cat([x[:c] for x, c in zip(xs, cut)]), [(0, 40, 0, 2), (40, 1, 0, 0), (41, 16, 0, 1)])
    b = w.run(torch.cat([x[c:] for x, c in zip(xs, cut)]), [(0, 30, 40, 2), (30, 32, 1, 0), (62, 31, 16, 1)])
    assert rel(a, torch.cat([t[:c] for t, c in zip(want, cut)])) < STOL and rel(b, torch.cat([t[c:] for t, c in zip(want, cut)])) < STOL
    assert rel(w.run(xs[0], [(0, 70, 0, 1)]), want[0]) < STOL


@pytest.mark.parametrize("case", SELECTS[:6], ids=lambda c: f"N{c['N']}")
def test_selective_decoding_of_many_sequences(case):
    """sequences at different positions in one step (groups of rows share weights), a parked one among them, some from their first token"""
    w = Select(**case, slots=7)
    xs = [w.inputs(30, 20 + i) for i in range(7)]
    want, start = [w.plain(x) for x in xs], [0, 3, 17, 1, 0, 9, 5]
    for i, n in enumerate(start):
        if n:
            w.run(xs[i][:n], [(0, n, 0, i)])
    for step in range(8):
        parked = step % 7 if step < 4 else -1
        rows = [(i, 1, -1 if i == parked else start[i], i) for i in range(7)]
        got = w.run(torch.cat([xs[i][start[i]:start[i] + 1] for i in range(7)]), rows, single=True)
        for i in range(7):
            if i != parked:
                assert rel(got[i], want[i][start[i]]) < STOL, (step, i)
                start[i] += 1


@pytest.mark.parametrize("kw", [dict(a_mean=-9.0, a_spread=1.0), dict(a_mean=6.0, a_spread=1.0), dict(dt_mean=-12.0), dict(dt_mean=30.0)], ids=lambda k: str(k))
def test_selective_scan_with_extreme_decays(kw):
    """states that keep everything, states that forget at once, step sizes from 1e-5 to 30"""
    w = Select(C_=70, N=16, R=8, taps=4, **kw)
    x = w.inputs(1500, 1)
    want = w.plain(x)
    assert torch.isfinite(want).all() and rel(w.run(x, [(0, 1500, 0, 1)]), want) < 3e-5
    assert rel(w.run(x[:1], [(0, 1, 0, 0)], single=True), want[:1]) < 3e-5


# ---- attention with a logarithmic distance bias -----------------------------------------------------------------------------------------------
LOGS = [dict(H=6, G=2, D=21, E=18), dict(H=20, G=1, D=32, E=32, out_scale=0.7), dict(H=6, G=3, D=136, E=200, scale=0.1), dict(H=2, G=2, D=64, E=64, window=30, out_scale=1.9),
        dict(H=4, G=4, D=256, E=256, scale=0.06, gate="values", out_scale=0.5), dict(H=8, G=4, D=128, E=128, scale=0.1, gate="heads", out_scale=2.0),
        dict(H=4, G=2, D=50, E=18, softcap=6.0, chunk=40, sink=1, keep=3, slopes=True), dict(H=3, G=3, D=42, E=9, taps=4, whole=True, out_scale=1.2)]


@pytest.mark.parametrize("case", LOGS, ids=lambda c: "-".join(f"{k}{v}" for k, v in c.items()))
def test_attention_with_a_logarithmic_bias(case):
    T = 210
    for f32, tol in ((False, TOL), (True, 3e-6)):
        w = Attn(**case, log=True, f32=f32, seed=T)
        x = w.inputs(T, 3)
        want = w.plain(x)
        forms = ("attend",) if f32 else ("prefill", "attend")
        for form in forms:
            assert rel(w.run(x, [(0, T, 0, 1)], form), want) < tol, form
        at, out = 0, []
        for n in (3, 61, 2, 70, 1, 24, 49):
            out.append(w.run(x[at:at + n], [(0, n, at, 1)], forms[0]))
            at += n
        assert rel(torch.cat(out), want) < tol
        got = [w.run(x[:150], [(0, 150, 0, 0)], forms[0])]
        got += [w.run(x[t:t + 1], [(0, 1, t, 0)], "attend", splits=1 if f32 else t % 4 + 1, single=True) for t in range(150, T)]
        assert rel(torch.cat(got), want) < tol


@pytest.mark.parametrize("form", ["prefill", "attend", "f32"])
def test_far_key_with_a_logarithmic_bias(form):
    """one key near the start: a bias of 8 ln(1 + d) takes its score of 40 back before the end, one of 2 ln(1 + d) never does; the first token, a page's edge"""
    T = 500
    for target in (0, 20, 63, 64):
        w = Attn(H=4, G=2, D=32, E=16, scale=1.0, log=True, pages=8, f32=form == "f32")
        w.r1, w.r2 = torch.tensor([8.0, 2.0, 8.0, 2.0]), torch.tensor([1.0, 1.0, 0.5, 0.01])
        w.t["r1"], w.t["r2"] = w.r1.to(DEV), w.r2.to(DEV)
        x = w.inputs(T, 3) * 0.1
        for h in range(4):
            x[:, w.off["q"] + 32 * h] = 5.0
        for h in range(2):
            x[:, w.off["k"] + 32 * h] = 0.0
            x[target, w.off["k"] + 32 * h] = 8.0
            x[target, w.off["v"] + 16 * h:w.off["v"] + 16 * h + 16] = 5.0
        want, got = w.plain(x), w.run(x, [(0, T, 0, 1)], "attend" if form == "f32" else form)
        assert float(want[target + 20, :16].mean()) > 4 > 1 > float(want[450, :16].mean().abs()) and float(want[450, 16:32].mean()) > 4 and float(want[450, 48:].mean()) > 4
        assert rel(got, want) < (1e-5 if form == "f32" else TOL), target


# ---- experts -----------------------------------------------------------------------------------------------------------------------------
MOES = [dict(experts=6, top=3, W=90, ff=40, limit=0.7, scale=2.5), dict(experts=5, top=1, W=128, ff=64, limit=7.0, scale=1.0),
        dict(experts=40, top=6, W=192, ff=96, limit=1.5, scale=0.3), dict(experts=4, top=4, W=64, ff=200, limit=0.2, scale=1.7)]


@pytest.mark.parametrize("case", range(len(MOES)))
@pytest.mark.parametrize("T", [1, 7, 16, 33, 700])
@pytest.mark.parametrize("exact", [0, 1])
def test_clamped_experts_weighted_by_scores(case, T, exact):
    c = MOES[case]
    g, E, W, ff, top = gen(case), c["experts"], c["W"], c["ff"], c["top"]
    Wp, fp = up(W, 64), up(ff, 64)
    h = torch.randn(T, W, generator=g)
    lin = lambda o, i: (torch.randn(o, i, generator=g) / math.sqrt(i)).to(torch.bfloat16)
    sd = {"router": lin(E, W) * 3}
    sd.update({f"e{e}.{n}": lin(*s) for e in range(E) for n, s in (("gate", (ff, W)), ("up", (ff, W)), ("down", (W, ff)))})
    sd64 = {k: v.double() for k, v in sd.items()}
    spec = {"router": {"experts": E, "top": top, "scale": c["scale"]}, "expert": {"ff": ff, "limit": c["limit"]}}
    z = h.double() @ sd64["router"].T
    idx, wt = F.route(z, top, c["scale"])
    want = F.experts(h.double(), sd64, "", spec)
    gu, dn = torch.zeros(E, fp // 16, 2, 16, Wp, dtype=torch.bfloat16), torch.zeros(E, Wp, fp, dtype=torch.bfloat16)
    for e in range(E):
        for j, n in enumerate(("gate", "up")):
            t = torch.zeros(fp, Wp, dtype=torch.bfloat16)
            t[:ff, :W] = sd[f"e{e}.{n}"]
            gu[e, :, j] = t.view(fp // 16, 16, Wp)
        dn[e, :W, :ff] = sd[f"e{e}.down"]
    hd = torch.zeros(T, Wp)
    hd[:, :W] = h
    hd, zd, gud, dnd = hd.to(DEV), z.float().to(DEV), gu.view(E, 2 * fp, Wp).to(DEV), dn.to(DEV)
    hp = planes_of(hd)
    parked = T == 7
    rows = torch.tensor([[i, -1 if parked and i == 2 else 5, i, 0] for i in range(T)], dtype=torch.int32, device=DEV)
    I = lambda n: torch.full((n,), -7, dtype=torch.int32, device=DEV)
    ids, place, order, offsets, tiles = I(T * top), I(T * top), I(T * top), I(E + 2), I(4 * int(_lib.load().chatts_moe_tiles(T, top, E)))
    weight, kept, y = torch.zeros(T, top, device=DEV), torch.zeros(T, device=DEV), torch.zeros(T * top, Wp, device=DEV)
    act = torch.zeros(T * top, fp, device=DEV) if exact else torch.zeros(2, T * top, fp, dtype=torch.bfloat16, device=DEV)
    a = _lib.MoeArgs(experts=E, identity=0, top=top, groups=1, keep=1, choose=_lib.CHOOSE_SCORES, act_kind=_lib.EXPERT_CLAMPGLU, width_p=Wp, ff_p=fp, gate_up=gud.data_ptr(),
                     down=dnd.data_ptr(), logits=zd.data_ptr(), ld_logits=E, h=operand(hd if exact else None, None if exact else hp, Wp), rows=rows.data_ptr(), n_rows=T,
                     exact=exact, ids=ids.data_ptr(), place=place.data_ptr(), order=order.data_ptr(), offsets=offsets.data_ptr(), tiles=tiles.data_ptr(),
                     weight=weight.data_ptr(), kept=kept.data_ptr(), act=operand(act if exact else None, None if exact else act, fp), y=y.data_ptr(),
                     weight_scale=c["scale"], glu_limit=c["limit"], glu_alpha=F.GATE_SLOPE)
    call("chatts_moe_route", a)
    live = [t for t in range(T) if not (parked and t == 2)]
    chosen = ids.view(T, top).cpu()
    for t in live:
        assert sorted(chosen[t].tolist()) == sorted(idx[t].tolist())
    assert float((weight.cpu()[live].sort(-1, descending=True).values - wt[live]).abs().max()) < 1e-5
    call("chatts_moe_experts", a)
    if not exact:                                                    # the weights' tiled copies: the same products
        plain, tiled = y.clone(), [torch.empty_like(t) for t in (gud, dnd)]
        for src, dst, n, k in ((gud, tiled[0], 2 * fp, Wp), (dnd, tiled[1], Wp, fp)):
            for e in range(E):
                _lib.check(_lib.load().chatts_tile_bf16(src[e].data_ptr(), n, k, k, dst[e].data_ptr(), _lib.stream_ptr()))
        y.zero_()
        a.gate_up_t, a.down_t = (t.data_ptr() for t in tiled)
        call("chatts_moe_experts", a)
        assert torch.equal(y, plain)
    yc, at = y.cpu().double(), place.view(T, top).cpu()
    got = torch.stack([sum(weight[t, j].cpu().double() * yc[at[t, j]] for j in range(top)) for t in live])
    assert rel(got[:, :W], want[live]) < (3e-6 if exact else 5e-5)


def test_refusals():
    """what the kernels cannot do is an error on the host, not a launch"""
    x = torch.zeros(64, device=DEV)
    assert _lib.load().chatts_soft_cap(x.data_ptr(), 64, 0.0, _lib.stream_ptr()) < 0
    with pytest.raises(_lib.ChattsError):
        Select(C_=8, N=300, R=4, taps=2).run(torch.zeros(2, 192), [(0, 2, 0, 0)])
    for fn, args in (("chatts_gru_scan", _lib.GruArgs()), ("chatts_select_scan", _lib.SelectArgs()), ("chatts_depth_norm", _lib.DepthNormArgs())):
        assert getattr(_lib.load(), fn)(C.byref(args), _lib.stream_ptr()) < 0
    w = Attn(H=2, G=1, D=32, E=16, log=True)
    w.t["r2"] = torch.zeros(0, device=DEV)
    with pytest.raises(_lib.ChattsError):
        w.run(w.inputs(4, 0), [(0, 4, 0, 0)], "attend")
