"""The kernels of post-norm layers, each alone, against the plain equations: the norm of a sum, attention's optional steps (short convolutions, norms over all
heads, rotated pairs, unit queries and keys, mixed values, capped scores, distance bias, chunks, gates per head), experts chosen by logits, the gelu unit."""
import math

import pytest
import torch

from chatts_amd import _lib
from chatts_amd.rotary import rotary_tables
from oracle import mefurax as F
from oracle import muvetar as M
from tests.test_gpu_mixed_kernels import DEV, call, gen, operand, rel
from tests.test_gpu_parallel_kernels import planes_of, rows_of, up

pytestmark = pytest.mark.gpu


# ---- norm of a sum --------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("width,T", [(64, 5), (90, 5), (1540, 5), (1540, 70), (5120, 3), (5120, 66), (9000, 2)])
@pytest.mark.parametrize("planes", [False, True])
def test_post_norm(width, T, planes):
    g, wp, eps, top, alpha = gen(width + T), up(width, 64), 1e-3, 3, 1.7
    pad = lambda t: torch.cat([t, torch.zeros(*t.shape[:-1], wp - width)], -1)
    x, y = pad(torch.randn(T, width, generator=g) * (1 + 4 * torch.rand(width, generator=g))), pad(torch.randn(T, width, generator=g) * 3)
    ey, w = pad(torch.randn(9, width, generator=g)), pad(torch.randn(width, generator=g))
    place, weight = torch.randint(-1, 9, (T, top), generator=g, dtype=torch.int32), torch.rand(T, top, generator=g)
    dev = {n: t.to(DEV) for n, t in dict(y=y, ey=ey, w=w, place=place, weight=weight).items()}
    for use_y, experts in ((1, 0), (1, 1), (0, 1), (0, 0)):
        s = alpha * x.double() + (y.double() if use_y else 0)
        if experts:
            for t in range(T):
                for j in range(top):
                    if place[t, j] >= 0:
                        s[t] += weight[t, j].double() * ey[place[t, j]].double()
        want = F.rms(s[:, :width], eps) * w.double()[:width]
        xd, out = x.to(DEV), torch.full((2, T, wp), 7.0, dtype=torch.bfloat16, device=DEV) if planes else torch.full((T, wp), 7.0, device=DEV)
        a = _lib.PostNormArgs(x=xd.data_ptr(), t=T, width=width, ldx=wp, alpha=alpha, eps=eps, y=dev["y"].data_ptr() if use_y else None, w=dev["w"].data_ptr(),
                              out=operand(None if planes else out, out if planes else None, wp))
        if experts:
            a.ey, a.place, a.weight, a.top = dev["ey"].data_ptr(), dev["place"].data_ptr(), dev["weight"].data_ptr(), top
        call("chatts_post_norm", a)
        got = out[0].float() + out[1].float() if planes else out
        assert rel(xd[:, :width], want) < 1e-6 and float(xd[:, width:].abs().sum()) == 0
        assert rel(got[:, :width], want) < (2e-5 if planes else 1e-6) and float(got[:, width:].abs().sum()) == 0


# ---- attention ---------------------------------------------------------------------------------------------------------------------------
class Attn:
    """paged keys and values and convolution rings of a few slots; the plain formula over whole sequences"""

    def __init__(self, H, G, D, E, window=0, chunk=0, keep=0, sink=0, gate=None, f32=False, scale=0.25, softcap=0.0, slopes=False, taps=0, whole=False, heads_norm=False, rot=0,
                 base=1000.0, unit=False, mix=None, log=False, out_scale=0.0, seed=0, slots=3, pages=5):
        g = gen(seed)
        self.__dict__.update({k: v for k, v in locals().items() if k not in ("self", "g")}, eps=1e-4, Dp=up(D, 32), Ep=up(E, 16))
        self.off, at = {}, 0
        for n, r in (("q", H * D), ("k", G * D), ("v", G * E), ("g", H * E if gate == "values" else H)):
            self.off[n] = at
            at += up(r, 64)
        self.ld, self.conv_ch = at, self.off["g"]
        self.w = {n: torch.randn(r, max(taps, 1), generator=g) for n, r in (("q", H * D), ("k", G * D), ("v", G * E))}
        wide = (H * D, G * D) if whole else (D, D)
        self.qn, self.kn = (1.3 + 0.3 * torch.randn(n, generator=g) for n in wide)
        dt = torch.float32 if f32 else torch.bfloat16
        self.kc = torch.randn(slots * pages, G, 64, self.Dp, generator=g).to(dt).to(DEV) * 50      # rubbish in rows never written
        self.vc = torch.randn(slots * pages, G, 64, self.Ep, generator=g).to(dt).to(DEV) * 50
        self.ring = torch.randn(slots, max(taps, 1), self.conv_ch, generator=g).to(DEV) * 50
        self.table = torch.randperm(slots * pages, generator=g).view(slots, pages).to(torch.int32).to(DEV)
        conv = torch.zeros(max(taps, 1), self.conv_ch)
        for n, t in self.w.items():
            conv[:, self.off[n]:self.off[n] + t.shape[0]] = t.t()
        self.r1, self.r2 = 2.5 * torch.rand(H, generator=g), 0.02 + 0.6 * torch.rand(H, generator=g)
        padded = lambda t: torch.cat([t, torch.zeros(-t.numel() % 4)]).to(DEV)
        cos, sin = rotary_tables(max(rot, 2), base, pages * 64)
        self.t = dict(qn=padded(self.qn), kn=padded(self.kn), conv=conv.to(DEV), cos=cos.to(DEV), sin=sin.to(DEV), slopes=torch.tensor(F.slopes(H), device=DEV), r1=self.r1.to(DEV), r2=self.r2.to(DEV))

    def inputs(self, T, seed):
        x = torch.zeros(T, self.ld)
        for n, r in (("q", self.H * self.D), ("k", self.G * self.D), ("v", self.G * self.E), ("g", self.ld - self.off["g"])):      # (padding is zero, as projections leave it)
            x[:, self.off[n]:self.off[n] + r] = torch.randn(T, r, generator=gen(seed + ord(n)))
        return x

    def firsts(self, T, seed):
        return torch.randn(T, self.G * self.E, generator=gen(seed + 1000))

    def plain(self, x, first=None):
        x = x.double()
        T, H, G, D, E = x.shape[0], self.H, self.G, self.D, self.E
        q, k, v = (x[:, self.off[n]:self.off[n] + r] for n, r in (("q", H * D), ("k", G * D), ("v", G * E)))
        if self.taps:
            q, k, v = (F.causal_conv(t, self.w[n].double()) for n, t in (("q", q), ("k", k), ("v", v)))
        self.values = v
        if self.whole:
            q, k = F.rms(q, self.eps) * self.qn.double(), F.rms(k, self.eps) * self.kn.double()
        q, k = q.reshape(T, H, D), k.reshape(T, G, D)
        if self.heads_norm:
            q, k = F.rms(q, self.eps) * self.qn.double(), F.rms(k, self.eps) * self.kn.double()
        if self.rot:
            q, k = (F.rotate_pairs(t, self.base, self.rot) for t in (q, k))
        if self.unit:
            q, k = (F.rms(t, self.eps) for t in (q, k))
        if first is not None:
            v = F.mix_values(v, first.double(), self.mix)
        rnd = (lambda t: t) if self.f32 else (lambda t: t.float().to(torch.bfloat16).double())      # what the pages and the queries hold
        q, k, v, head = rnd(q), rnd(k), rnd(v).reshape(T, G, E), torch.arange(H) // (H // G)
        s = torch.einsum("ihd,jhd->hij", q, k[:, head]) * self.scale
        if self.softcap:
            s = F.soft_cap(s, self.softcap)
        dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).double()
        if self.slopes:
            s = s - torch.tensor(F.slopes(H), dtype=torch.float64)[:, None, None] * dist
        if self.log:
            s = s - M.distance_bias(self.r1.double(), self.r2.double(), dist.clamp(min=0))
        if self.sink:
            s = torch.cat([torch.zeros(H, T, 1, dtype=torch.float64), s], -1)
        see = self.sees(T)
        a = torch.softmax(s.masked_fill(~torch.cat([torch.ones(T, self.sink, dtype=torch.bool), see], 1), -math.inf), -1)[:, :, self.sink:]
        o = torch.einsum("hij,jhe->ihe", a, v[:, head]) * (self.out_scale or 1.0)
        gate = x[:, self.off["g"]:].double()
        if self.gate == "heads":
            o = o * torch.sigmoid(gate[:, :H])[:, :, None]
        o = o.reshape(T, H * E)
        return o * torch.sigmoid(gate[:, :H * E]) if self.gate == "values" else o

    def sees(self, T):
        rule = (lambda i, j: F.in_window(i, j, self.window)) if self.window or not self.chunk else (lambda i, j: F.in_chunk(i, j, self.chunk))
        return torch.tensor([[rule(i, j) or (j <= i and j < self.keep) for j in range(T)] for i in range(T)])

    def run(self, x, segs, form, splits=1, first=None, write=None, single=False):
        xd, (rows, spans), T = x.to(DEV), rows_of(segs), x.shape[0]
        q = torch.full((T, self.H * self.Dp), 1e3, dtype=torch.float32 if self.f32 else torch.bfloat16, device=DEV)      # (another layer's numbers)
        n = self.H * self.E
        out, part = torch.zeros(T, n, device=DEV), torch.zeros(T * self.H * splits * (self.Ep + 4), device=DEV)
        ldv = up(self.G * self.E, 4)
        fv = torch.zeros(T, ldv, device=DEV)
        if first is not None:
            fv[:, :self.G * self.E] = first.to(DEV)
        norms = self.whole or self.heads_norm
        P = {k: t.data_ptr() for k, t in self.t.items()}
        a = _lib.WindowArgs(proj=xd.data_ptr(), ld_proj=self.ld, off_q=self.off["q"], off_k=self.off["k"], off_v=self.off["v"], off_gate=self.off["g"] if self.gate else -1,
                            heads=self.H, kv_heads=self.G, dim=self.D, vdim=self.E, dim_p=self.Dp, vdim_p=self.Ep, scale=self.scale, eps=self.eps,
                            q_norm=P["qn"] if norms else None, k_norm=P["kn"] if norms else None, window=self.window, keep_first=self.keep, sink=self.sink, chunk=self.chunk,
                            softcap=self.softcap, slopes=P["slopes"] if self.slopes else None, gate_heads=int(self.gate == "heads"), norm_whole=int(self.whole), rot=self.rot,
                            unit=int(self.unit), cos_tab=P["cos"] if self.rot else None, sin_tab=P["sin"] if self.rot else None, taps=self.taps, conv_ch=self.conv_ch,
                            conv_w=P["conv"] if self.taps else None, ring=self.ring.data_ptr() if self.taps else None, vmix=self.mix or 0.0,
                            vfirst=fv.data_ptr() if first is not None or write else None, ld_vfirst=ldv, vfirst_write=int(bool(write)), kcache=self.kc.data_ptr(),
                            vcache=self.vc.data_ptr(), cache_f32=int(self.f32), table=self.table.data_ptr(), table_stride=self.table.shape[1], log_block=6, rows=rows.data_ptr(),
                            n_rows=T, spans=spans.data_ptr(), n_spans=0 if single else len(segs), longest=max(s[1] for s in segs), n_splits=splits, partial=part.data_ptr(),
                            q=_lib.Operand(f32=q.data_ptr() if self.f32 else None, hi=None if self.f32 else q.data_ptr(), lo=None, ld=self.H * self.Dp),
                            out=operand(out, None, n), log_r1=P["r1"] if self.log else None, log_r2=P["r2"] if self.log else None, out_scale=self.out_scale)
        call("chatts_window_prep", a)
        call("chatts_window_" + form, a)
        if write:
            self.written = fv[:, :self.G * self.E].cpu()
        return out.cpu()


CONV = [dict(H=6, G=2, D=24, E=42, taps=3, whole=True, slopes=True, window=30, mix=0.3), dict(H=20, G=1, D=32, E=32, taps=1, whole=True, slopes=True),
        dict(H=6, G=3, D=136, E=200, taps=4, whole=True, slopes=True, window=65, scale=0.1, mix=0.8), dict(H=3, G=3, D=21, E=9, taps=6, whole=True, slopes=True, window=64, mix=0.5),
        dict(H=4, G=4, D=96, E=32, taps=2, window=100, scale=0.1), dict(H=2, G=1, D=64, E=64, whole=True, slopes=True, window=1, gate="values"),
        dict(H=4, G=2, D=50, E=18, taps=4, slopes=True, softcap=6.0, chunk=40, sink=1, keep=3, gate="heads")]
ROT = [dict(H=4, G=4, D=64, E=32, rot=32, unit=True, softcap=4.0, chunk=40, gate="heads", scale=2.0, mix=0.4), dict(H=6, G=2, D=21, E=9, rot=10, unit=True, softcap=9.0, chunk=64, gate="heads"),
       dict(H=20, G=1, D=32, E=48, rot=32, unit=True, softcap=2.0, gate="heads", mix=0.6), dict(H=6, G=3, D=136, E=200, rot=62, unit=True, softcap=30.0, chunk=100, gate="heads", scale=0.1),
       dict(H=3, G=1, D=42, E=22, rot=42, softcap=5.0, chunk=1), dict(H=2, G=2, D=256, E=256, rot=128, unit=True, softcap=20.0, chunk=70, scale=0.06, gate="values"),
       dict(H=4, G=2, D=48, E=50, rot=6, heads_norm=True, unit=True, chunk=50, keep=5, sink=1), dict(H=4, G=2, D=40, E=20, heads_norm=True, slopes=True, softcap=3.0, window=33, mix=0.5)]
TOL = 8e-3      # queries, keys, values and probabilities in bf16; weights that one rounding of a query moves


@pytest.mark.parametrize("case", CONV + ROT, ids=lambda c: "-".join(f"{k}{v}" for k, v in c.items()))
def test_attention_with_its_optional_steps(case):
    """prompts, portions down to one and two tokens, single rows with one and several ranges of keys; slots used again; 32-bit"""
    T = 210
    for f32, tol in ((False, TOL), (True, 3e-6)):
        w = Attn(**case, f32=f32, seed=T)
        x = w.inputs(T, 3)
        first = w.firsts(T, 3) if w.mix else None
        cut = lambda a, b: None if first is None else first[a:b]
        want = w.plain(x, first)
        forms = ("attend",) if f32 else ("prefill", "attend")
        for form in forms:
            assert rel(w.run(x, [(0, T, 0, 1)], form, first=first), want) < tol, form
        at, out = 0, []
        for i, n in enumerate((3, 61, 2, 70, 1, 24, 49)):
            out.append(w.run(x[at:at + n], [(0, n, at, 1)], forms[0], first=cut(at, at + n)))
            at += n
        assert at == T and rel(torch.cat(out), want) < tol
        got = [w.run(x[:150], [(0, 150, 0, 0)], forms[0], first=cut(0, 150))]
        got += [w.run(x[t:t + 1], [(0, 1, t, 0)], "attend", splits=1 if f32 else t % 4 + 1, first=cut(t, t + 1), single=True) for t in range(150, T)]
        assert rel(torch.cat(got), want) < tol
        got = torch.cat([w.run(x[t:t + 1], [(0, 1, t, 2)], "attend", first=cut(t, t + 1), single=True) for t in range(9)])      # from the first token on
        assert rel(got, want[:9]) < tol


@pytest.mark.parametrize("case", [CONV[0], CONV[3], ROT[0], ROT[1]])
def test_unequal_segments(case):
    """three sequences in a step, prompts beside a single token, then their next portions"""
    w = Attn(**case)
    xs = [w.inputs(n, n) for n in (90, 33, 140)]
    fs = [w.firsts(len(x), len(x)) if w.mix else None for x in xs]
    want, cut = [w.plain(x, f) for x, f in zip(xs, fs)], (64, 1, 100)
    both = lambda s: torch.cat([f[s(c)] for f, c in zip(fs, cut)]) if w.mix else None
    a = w.run(torch.cat([x[:c] for x, c in zip(xs, cut)]), [(0, 64, 0, 2), (64, 1, 0, 0), (65, 100, 0, 1)], "prefill", first=both(lambda c: slice(0, c)))
    b = w.run(torch.cat([x[c:] for x, c in zip(xs, cut)]), [(0, 26, 64, 2), (26, 32, 1, 0), (58, 40, 100, 1)], "prefill", first=both(lambda c: slice(c, None)))
    assert rel(a, torch.cat([t[:c] for t, c in zip(want, cut)])) < TOL and rel(b, torch.cat([t[c:] for t, c in zip(want, cut)])) < TOL


@pytest.mark.parametrize("case", [CONV[0], CONV[3], ROT[0], ROT[1]])
def test_first_values_are_left_behind(case):
    """the first layer of those that mix caches its own values and leaves them (after their convolution) for the others"""
    w = Attn(**case)
    x = w.inputs(80, 1)
    want = w.plain(x)
    assert rel(w.run(x, [(0, 80, 0, 1)], "prefill", write=True), want) < TOL
    assert rel(w.written, w.values) < 1e-6
    assert rel(w.run(x[:1], [(0, 1, 0, 1)], "attend", write=True, single=True), want[:1]) < TOL and rel(w.written, w.values[:1]) < 1e-6


EDGES = [dict(window=37, slopes=True), dict(chunk=37, softcap=60.0), dict(chunk=64, softcap=60.0), dict(window=64), dict(chunk=50, slopes=True, softcap=60.0)]


@pytest.mark.parametrize("mask", EDGES, ids=lambda m: "-".join(m))
@pytest.mark.parametrize("form", ["prefill", "attend", "decode", "f32"])
def test_edges(form, mask):
    """one key that would take all the weight: the queries just inside and just outside the window or chunk see it or not"""
    T, S = 180, mask.get("window") or mask["chunk"]
    targets = (0, 3, S - 1, S, S + 1, 63, 64, 65, 2 * S - 1, 2 * S)
    for target in targets:
        w = Attn(H=2, G=1, D=32, E=32, scale=1.0, seed=target, f32=form == "f32", **mask)
        x = w.inputs(T, 3) * 0.3
        x[:, :w.off["v"]] *= 0.2
        x[:, w.off["q"]] = x[:, w.off["q"] + 32] = 7.0          # every query looks along the first dimension ...
        x[:, w.off["k"]] = -1.0
        x[target, w.off["k"]] = 7.0                             # ... where one key lies
        x[target, w.off["v"]:w.off["v"] + 32] = 9.0
        want, sees = w.plain(x), w.sees(T)[:, target].tolist()
        tests = [i for i in sorted({target, target + 1, target + S - 1, target + S, target - target % S + S - 1, target - target % S + S, T - 1}) if i < T]
        for i in tests:
            assert (float(want[i].mean()) > 5) == sees[i], (target, i)
        if form == "decode":
            w.run(x[:target + 1], [(0, target + 1, 0, 1)], "prefill")
            got = torch.cat([w.run(x[t:t + 1], [(0, 1, t, 1)], "attend", splits=t % 3 + 1, single=True) for t in range(target + 1, T)])
            assert rel(got, want[target + 1:]) < TOL, target
            continue
        got = w.run(x, [(0, T, 0, 1)], "attend" if form == "f32" else form)
        for i in tests:
            assert float((got[i].double() - want[i]).abs().max()) < 0.06, (target, i)
        assert rel(got, want) < (1e-5 if form == "f32" else TOL), target


@pytest.mark.parametrize("form", ["prefill", "attend"])
def test_far_key_with_a_distance_bias(form):
    """a key hundreds of tokens back whose score outweighs the bias, and one whose score does not; heads differ in their slopes"""
    w = Attn(H=4, G=4, D=32, E=16, scale=1.0, slopes=True, pages=8)
    T = 500
    x = w.inputs(T, 3) * 0.1
    for h in range(4):
        x[:, w.off["q"] + 32 * h] = 5.0
        x[:, w.off["k"] + 32 * h] = 0.0
        x[20, w.off["k"] + 32 * h] = 8.0                       # score 40: slopes 1/4, 1/16, 1/64, 1/256 leave it behind after 160, 640, .. tokens
        x[20, w.off["v"] + 16 * h:w.off["v"] + 16 * h + 16] = 5.0
    want, got = w.plain(x), w.run(x, [(0, T, 0, 1)], form)
    assert float(want[60, :16].mean()) > 4 > 1 > float(want[300, :16].mean().abs()) and float(want[450, 48:].mean()) > 4
    assert rel(got, want) < TOL


def test_scores_far_above_the_cap():
    """saturated scores become equal weights; moderate ones keep their order"""
    for form, f32 in (("prefill", False), ("attend", False), ("attend", True)):
        w = Attn(H=2, G=1, D=32, E=16, scale=50.0, softcap=2.0, f32=f32)
        x = w.inputs(100, 4)
        want = w.plain(x)
        assert rel(w.run(x, [(0, 100, 0, 1)], form), want) < (1e-5 if f32 else TOL)


# ---- experts -----------------------------------------------------------------------------------------------------------------------------
MOES = [dict(experts=6, top=3, W=90, ff=40), dict(experts=5, top=1, W=128, ff=64), dict(experts=40, top=6, W=192, ff=96), dict(experts=4, top=4, W=64, ff=200)]


@pytest.mark.parametrize("case", range(len(MOES)))
@pytest.mark.parametrize("T", [1, 7, 16, 33, 700])
@pytest.mark.parametrize("exact", [0, 1])
def test_experts_by_logits(case, T, exact):
    """squared-relu experts; weights are a softmax over the chosen logits, also where a softmax over all of them would round to zero"""
    c = MOES[case]
    g, E, W, ff, top = gen(case), c["experts"], c["W"], c["ff"], c["top"]
    Wp, fp = up(W, 64), up(ff, 64)
    h = torch.randn(T, W, generator=g)
    lin = lambda o, i: (torch.randn(o, i, generator=g) / math.sqrt(i)).to(torch.bfloat16)
    sd = {"router": lin(E, W) * (30 if T == 33 else 3)}
    sd.update({f"e{e}.{n}": lin(*s) for e in range(E) for n, s in (("up", (ff, W)), ("down", (W, ff)))})
    sd64 = {k: v.double() for k, v in sd.items()}
    z = h.double() @ sd64["router"].T
    if T == 33:
        z[:, 0] += 400.0
    idx, wt = F.route(z, top)
    want = torch.zeros(T, W, dtype=torch.float64)
    for t in range(T):
        for e, a in zip(idx[t].tolist(), wt[t]):
            want[t] += a * (sd64[f"e{e}.down"] @ F.relu2(sd64[f"e{e}.up"] @ h[t].double()))
    upw, dn = torch.zeros(E, fp, Wp, dtype=torch.bfloat16), torch.zeros(E, Wp, fp, dtype=torch.bfloat16)
    for e in range(E):
        upw[e, :ff, :W], dn[e, :W, :ff] = sd[f"e{e}.up"], sd[f"e{e}.down"]
    hd = torch.zeros(T, Wp)
    hd[:, :W] = h
    hd, zd, upd, dnd = hd.to(DEV), z.float().to(DEV), upw.to(DEV), dn.to(DEV)
    hp = planes_of(hd)
    parked = T == 7
    rows = torch.tensor([[i, -1 if parked and i == 2 else 5, i, 0] for i in range(T)], dtype=torch.int32, device=DEV)
    I = lambda n: torch.full((n,), -7, dtype=torch.int32, device=DEV)
    ids, place, order, offsets, tiles = I(T * top), I(T * top), I(T * top), I(E + 2), I(4 * int(_lib.load().chatts_moe_tiles(T, top, E)))
    weight, kept, y = torch.zeros(T, top, device=DEV), torch.zeros(T, device=DEV), torch.zeros(T * top, Wp, device=DEV)
    act = torch.zeros(T * top, fp, device=DEV) if exact else torch.zeros(2, T * top, fp, dtype=torch.bfloat16, device=DEV)
    a = _lib.MoeArgs(experts=E, identity=0, top=top, groups=1, keep=1, choose=_lib.CHOOSE_LOGITS, act_kind=_lib.EXPERT_RELU2, width_p=Wp, ff_p=fp, gate_up=upd.data_ptr(),
                     down=dnd.data_ptr(), logits=zd.data_ptr(), ld_logits=E, h=operand(hd if exact else None, None if exact else hp, Wp), rows=rows.data_ptr(), n_rows=T,
                     exact=exact, ids=ids.data_ptr(), place=place.data_ptr(), order=order.data_ptr(), offsets=offsets.data_ptr(), tiles=tiles.data_ptr(),
                     weight=weight.data_ptr(), kept=kept.data_ptr(), act=operand(act if exact else None, None if exact else act, fp), y=y.data_ptr())
    call("chatts_moe_route", a)
    live = [t for t in range(T) if not (parked and t == 2)]
    chosen = ids.view(T, top).cpu()
    for t in live:
        assert sorted(chosen[t].tolist()) == sorted(idx[t].tolist())
    assert float((weight.cpu()[live].sort(-1, descending=True).values - wt[live]).abs().max()) < 1e-5
    call("chatts_moe_experts", a)
    if not exact:                                                    # the weights' tiled copies: the same products
        plain, tiled = y.clone(), [torch.empty_like(t) for t in (upd, dnd)]
        for src, dst, n, k in ((upd, tiled[0], fp, Wp), (dnd, tiled[1], Wp, fp)):
            for e in range(E):
                _lib.check(_lib.load().chatts_tile_bf16(src[e].data_ptr(), n, k, k, dst[e].data_ptr(), _lib.stream_ptr()))
        y.zero_()
        a.gate_up_t, a.down_t = (t.data_ptr() for t in tiled)
        call("chatts_moe_experts", a)
        assert torch.equal(y, plain)
    yc, at = y.cpu().double(), place.view(T, top).cpu()
    got = torch.stack([sum(weight[t, j].cpu().double() * yc[at[t, j]] for j in range(top)) for t in live])
    assert rel(got[:, :W], want[live]) < (3e-6 if exact else 5e-5)


# ---- the gelu unit -----------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("m", [1, 3, 16, 40, 130, 600])
@pytest.mark.parametrize("exact", [0, 1])
@pytest.mark.parametrize("n,k", [(96, 320), (320, 1536)])
def test_linear_geglu(m, exact, n, k):
    g = gen(m)
    a, w = 3 * torch.randn(m, k, generator=g), (torch.randn(2 * n, k, generator=g) / math.sqrt(k)).to(torch.bfloat16)
    z = (a.double() @ w.double().T).view(m, n // 16, 2, 16)
    want = F.gelu_tanh(z[:, :, 0].reshape(m, n)) * z[:, :, 1].reshape(m, n)
    ad, wd, c = a.to(DEV), w.to(DEV), torch.zeros(m, n, device=DEV)
    ws = torch.zeros(max(16, int(_lib.load().chatts_linear_workspace(m, 2 * n, k))), dtype=torch.uint8, device=DEV)
    kw = dict(w=wd.data_ptr(), m=m, n=2 * n, k=k, ldw=k, ldc=n, epilogue=_lib.EPI_GEGLU, workspace=ws.data_ptr(), workspace_bytes=ws.numel())
    call("chatts_linear", _lib.LinearArgs(a=ad.data_ptr(), lda=k, c=c.data_ptr(), exact_f32=exact, **kw))
    assert rel(c, want) < (2e-6 if exact or m == 1 else 2e-5)
    if m > 1 and not exact:
        hp, out = planes_of(ad), torch.zeros(2, m, n, dtype=torch.bfloat16, device=DEV)
        call("chatts_linear", _lib.LinearArgs(a_hi=hp[0].data_ptr(), a_lo=hp[1].data_ptr(), ld_planes=k, c_hi=out[0].data_ptr(), c_lo=out[1].data_ptr(), ld_cplanes=n, **kw))
        assert rel(out[0].float() + out[1].float(), want) < 4e-5


def test_refusals():
    """what the kernels cannot do is an error on the host, not a launch"""
    w = Attn(H=2, G=1, D=32, E=16)
    x = w.inputs(4, 0)
    for change in (dict(window=4, chunk=4), dict(rot=3), dict(rot=34), dict(taps=2, rot=4), dict(softcap=-1.0), dict(taps=2, heads_norm=True)):
        bad = Attn(**{**dict(H=2, G=1, D=32, E=16), **change})
        with pytest.raises(_lib.ChattsError):
            bad.run(x, [(0, 4, 0, 0)], "attend")
