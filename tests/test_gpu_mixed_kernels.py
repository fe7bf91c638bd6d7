"""The kernels of mixed-layer decoders, each alone, against plain float64 formulas."""
import ctypes as C
import math

import numpy as np
import pytest
import torch

from chatts_amd import _lib
from oracle import fobolix as F

pytestmark = pytest.mark.gpu
DEV = "cuda"


def gen(seed):
    return torch.Generator().manual_seed(seed)


def rel(got, want):
    got, want = got.double().cpu(), want.double()
    return float((got - want).norm() / want.norm().clamp_min(1e-30))


def operand(f32=None, planes=None, ld=0):
    return _lib.Operand(f32=_lib.ptr(f32), hi=None if planes is None else planes[0].data_ptr(), lo=None if planes is None else planes[1].data_ptr(), ld=ld)


def call(fn, args):
    _lib.check(getattr(_lib.load(), fn)(C.byref(args), _lib.stream_ptr()))
    torch.cuda.synchronize()


# ---- norms -------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("width", [64, 90, 1500, 5000])
@pytest.mark.parametrize("planes", [False, True])
def test_residual_norm(width, planes):
    g, T, wp, eps = gen(width), 5, (width + 63) // 64 * 64, 1e-3
    x, y = torch.zeros(T, wp), torch.zeros(T, wp)
    x[:, :width], y[:, :width] = torch.randn(T, width, generator=g), torch.randn(T, width, generator=g) * 3
    w = [torch.cat([torch.randn(width, generator=g), torch.zeros(wp - width)]) for _ in range(3)]
    for use_y, use_post, use_add in ((1, 1, 1), (1, 0, 0), (0, 0, 1), (0, 0, 0), (1, 1, 0)):
        xd, yd, wd = x.to(DEV), y.to(DEV), [t.to(DEV) for t in w]
        out = torch.full((T, wp), 7.0, device=DEV)
        pl = torch.full((2, T, wp), 7.0, dtype=torch.bfloat16, device=DEV)
        a = _lib.ResidualNormArgs(x=xd.data_ptr(), y=yd.data_ptr() if use_y else None, post_w=wd[0].data_ptr() if use_post else None,
                                  add=wd[1].data_ptr() if use_add else None, pre_w=wd[2].data_ptr(), out=operand(None if planes else out, pl if planes else None, wp),
                                  t=T, width=width, ldx=wp, ldy=wp, eps=eps)
        call("chatts_residual_norm", a)
        want = x.double()[:, :width]
        if use_y:
            yy = y.double()[:, :width]
            want = want + (F.rms_norm(yy, w[0].double()[:width], eps) if use_post else yy)
        if use_add:
            want = want + w[1].double()[:width]
        assert rel(xd[:, :width], want) < 1e-6 and float(xd[:, width:].abs().sum()) == 0
        got = pl[0].float() + pl[1].float() if planes else out
        assert rel(got[:, :width], F.rms_norm(want, w[2].double()[:width], eps)) < (2e-5 if planes else 1e-6)
        assert float(got[:, width:].abs().sum()) == 0


# ---- projections -----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("m", [1, 3, 16, 40, 130])
@pytest.mark.parametrize("exact", [0, 1])
def test_linear_relu2_and_exact(m, exact):
    g, n, k = gen(m), 208, 320
    a, w = torch.randn(m, k, generator=g), (torch.randn(n, k, generator=g) / math.sqrt(k)).to(torch.bfloat16)
    ad, wd = a.to(DEV), w.to(DEV)
    for epi in (_lib.EPI_NONE, _lib.EPI_RELU2):
        want = a.double() @ w.double().T
        if epi == _lib.EPI_RELU2:
            want = want.clamp_min(0) ** 2
        c = torch.zeros(m, n, device=DEV)
        la = _lib.LinearArgs(a=ad.data_ptr(), w=wd.data_ptr(), c=c.data_ptr(), m=m, n=n, k=k, lda=k, ldw=k, ldc=n, epilogue=epi, exact_f32=exact)
        ws = torch.zeros(max(16, int(_lib.load().chatts_linear_workspace(m, n, k))), dtype=torch.uint8, device=DEV)
        la.workspace, la.workspace_bytes = ws.data_ptr(), ws.numel()
        call("chatts_linear", la)
        assert rel(c, want) < (1e-6 if exact or m == 1 else 2e-5)
        if m > 1 and not exact:                       # plane operands in, planes out
            hi = ad.to(torch.bfloat16)
            lo = (ad - hi.float()).to(torch.bfloat16)
            out = torch.zeros((2, m, n), dtype=torch.bfloat16, device=DEV)
            la = _lib.LinearArgs(w=wd.data_ptr(), m=m, n=n, k=k, ldw=k, ldc=n, epilogue=epi, a_hi=hi.data_ptr(), a_lo=lo.data_ptr(), ld_planes=k,
                                 c_hi=out[0].data_ptr(), c_lo=out[1].data_ptr(), ld_cplanes=n, workspace=ws.data_ptr(), workspace_bytes=ws.numel())
            call("chatts_linear", la)
            assert rel(out[0].float() + out[1].float(), want) < 4e-5


@pytest.mark.parametrize("m,heads,n,k", [(1, 3, 32, 64), (7, 2, 96, 32), (33, 5, 48, 160), (70, 1, 144, 96)])
def test_head_linear(m, heads, n, k):
    g = gen(m)
    a, w = torch.randn(m, heads, k, generator=g), (torch.randn(heads, n, k, generator=g) / math.sqrt(k)).to(torch.bfloat16)
    want = torch.stack([a[:, h].double() @ w[h].double().T for h in range(heads)], 1)
    ad, wd = a.to(DEV), w.to(DEV)
    for exact in (0, 1):
        ld = heads * (n + 16)
        out = torch.zeros(m, ld, device=DEV)
        call("chatts_head_linear", _lib.HeadLinearArgs(a=ad.data_ptr(), w=wd.data_ptr(), out=operand(out, None, ld), m=m, heads=heads, n=n, k=k, lda=heads * k,
                                                       a_head=k, out_head=n + 16, exact=exact))
        assert rel(out.view(m, heads, n + 16)[..., :n], want) < (1e-6 if exact else 2e-5)
        assert float(out.view(m, heads, n + 16)[..., n:].abs().sum()) == 0
    pl = torch.zeros((2, m, heads * n), dtype=torch.bfloat16, device=DEV)
    call("chatts_head_linear", _lib.HeadLinearArgs(a=ad.data_ptr(), w=wd.data_ptr(), out=operand(None, pl, heads * n), m=m, heads=heads, n=n, k=k, lda=heads * k,
                                                   a_head=k, out_head=n, exact=0))
    assert rel((pl[0].float() + pl[1].float()).view(m, heads, n), want) < 4e-5


# ---- gated delta rule --------------------------------------------------------------------------------------------------------------
class Delta:
    """one delta mixer with random parameters: the kernels on a slot of a state pool, and the plain recurrence"""

    def __init__(self, H, KH, dim, vd, taps, ra, rg, seed=0, slots=3):
        g = gen(seed)
        self.H, self.KH, self.dim, self.vd, self.taps, self.slots = H, KH, dim, vd, taps, slots
        up = lambda n, m: (n + m - 1) // m * m
        self.ra, self.rg = ra, rg
        self.off, at = {}, 0
        for n, rows in (("q", KH * dim), ("k", KH * dim), ("v", H * vd), ("a", ra), ("g", rg), ("b", H)):
            self.off[n] = at
            at += up(rows, 64)
        self.ld, self.conv_ch = at, self.off["a"]
        self.rap, self.rgp = up(ra, 64), up(rg, 64)
        bf = lambda t: t.to(torch.bfloat16)
        self.conv = {"q": torch.randn(KH * dim, taps, generator=g) * 0.6, "k": torch.randn(KH * dim, taps, generator=g) * 0.6, "v": torch.randn(H * vd, taps, generator=g) * 0.6}
        self.a2, self.g2 = bf(torch.randn(H * dim, ra, generator=g) / math.sqrt(ra)), bf(torch.randn(H * vd, rg, generator=g) / math.sqrt(rg))
        self.dt_bias, self.a_log = torch.randn(H * dim, generator=g) * 0.5 - 3, torch.rand(H, generator=g) - 1
        self.norm, self.eps = 1 + 0.2 * torch.randn(vd, generator=g), 1e-4
        cw = torch.zeros(taps, self.conv_ch)
        for n, t in self.conv.items():
            cw[:, self.off[n]:self.off[n] + t.shape[0]] = t.T
        pad = lambda t, c: torch.cat([t, torch.zeros(t.shape[0], c - t.shape[1], dtype=t.dtype)], 1)
        self.t = dict(cw=cw, a2=pad(self.a2, self.rap), g2=pad(self.g2, self.rgp), dt=self.dt_bias, na=-torch.exp(self.a_log).repeat_interleave(dim), nw=self.norm)
        for n in ("a2", "g2"):
            self.t[n + "d"] = self.t[n].view(self.t[n].shape[0], -1, 8).transpose(0, 1)
        self.t = {k: v.contiguous().to(DEV) for k, v in self.t.items()}
        # used slots hold rubbish: a sequence that starts must not see it
        self.state = torch.randn(slots, H, dim, up(vd, 4), generator=g).to(DEV)
        self.ring = torch.randn(slots, taps, self.conv_ch, generator=g).to(DEV)

    def inputs(self, T, seed):
        x = torch.zeros(T, self.ld)
        g = gen(seed)
        for n, rows in (("q", self.KH * self.dim), ("k", self.KH * self.dim), ("v", self.H * self.vd), ("a", self.ra), ("g", self.rg), ("b", self.H)):
            x[:, self.off[n]:self.off[n] + rows] = torch.randn(T, rows, generator=g)
        return x

    def reference(self, x):
        """[T, H * vd] of a sequence from its start"""
        x = x.double()
        T, H, KH, dim, vd = x.shape[0], self.H, self.KH, self.dim, self.vd
        cut = lambda n, rows: x[:, self.off[n]:self.off[n] + rows]
        q = F.short_conv(cut("q", KH * dim).clone(), self.conv["q"].double()).view(T, KH, dim)
        k = F.short_conv(cut("k", KH * dim).clone(), self.conv["k"].double()).view(T, KH, dim)
        v = F.short_conv(cut("v", H * vd).clone(), self.conv["v"].double()).view(T, H, vd)
        q, k = F.unit(q) * dim ** -0.5, F.unit(k)
        head = torch.arange(H) // (H // KH)
        dt = cut("a", self.ra) @ self.a2.double().T + self.dt_bias.double()
        g = torch.exp(-torch.exp(self.a_log.double())[None, :, None] * torch.log1p(dt.exp()).view(T, H, dim))
        beta = torch.sigmoid(cut("b", H))
        S, o = torch.zeros(H, dim, vd, dtype=torch.float64), torch.zeros(T, H, vd, dtype=torch.float64)
        for t in range(T):
            S, o[t] = F.delta_step(S, q[t][head], k[t][head], v[t], g[t], beta[t])
        gate = torch.sigmoid(cut("g", self.rg) @ self.g2.double().T).view(T, H, vd)
        return (F.rms_norm(o, self.norm.double(), self.eps) * gate).reshape(T, H * vd), S

    def args(self, x, rows, out, spans=None):
        t, T = self.t, x.shape[0]
        a = _lib.DeltaArgs(proj=x.data_ptr(), ld_proj=self.ld, off_q=self.off["q"], off_k=self.off["k"], off_v=self.off["v"], off_a=self.off["a"], off_g=self.off["g"],
                           off_b=self.off["b"], conv_ch=self.conv_ch, heads=self.H, kv_heads=self.KH, dim=self.dim, vdim=self.vd, taps=self.taps, rank_a=self.rap,
                           rank_g=self.rgp, conv_w=t["cw"].data_ptr(), a2=t["a2"].data_ptr(), g2=t["g2"].data_ptr(), a2d=t["a2d"].data_ptr(), g2d=t["g2d"].data_ptr(), ld_a2=self.rap, ld_g2=self.rgp,
                           dt_bias=t["dt"].data_ptr(), neg_a=t["na"].data_ptr(), norm_w=t["nw"].data_ptr(), eps=self.eps, state=self.state.data_ptr(),
                           ring=self.ring.data_ptr(), rows=rows.data_ptr(), n_rows=T, out=operand(out, None, self.H * self.vd))
        if spans is not None:
            a.spans, a.n_spans = spans.data_ptr(), spans.shape[0]
        return a

    def step(self, segs, forms):
        """segs: list of (slot, pos0, x [t, ld]) -> list of [t, H * vd]; forms 'decode' (every t == 1), 'scan' or 'scan32'"""
        x = torch.cat([s[2] for s in segs]).to(DEV)
        rows, spans, at = [], [], 0
        for slot, pos0, xs in segs:
            n = xs.shape[0]
            rows += [(slot, pos0 + i, at, n - 1 - i) for i in range(n)]
            spans.append((at, n, pos0, slot, -1))
            at += n
        rows, spans = torch.tensor(rows, dtype=torch.int32, device=DEV), torch.tensor(spans, dtype=torch.int32, device=DEV)
        out = torch.zeros(at, self.H * self.vd, device=DEV)
        a = self.args(x, rows, out, spans)
        if forms == "decode":
            call("chatts_delta_decode", a)
        else:
            H, KH, dim, vd = self.H, self.KH, self.dim, self.vd
            z = lambda n: torch.full((at, n), float("nan"), device=DEV)
            q, k, v, g, beta, o = z(KH * dim), z(KH * dim), z(H * vd), z(H * dim), z(H), z(H * vd)
            chunks = torch.full((int(_lib.load().chatts_delta_chunk_floats(H, dim, at, len(segs))),), float("nan"), device=DEV)
            gate = z(H * vd)
            a.q, a.k, a.v, a.g, a.beta, a.chunks, a.o, a.gate = (t.data_ptr() for t in (q, k, v, g, beta, chunks, o, gate))
            a.exact = int(forms == "scan32")
            for fn in ("chatts_delta_prep", "chatts_delta_scan", "chatts_delta_out"):
                call(fn, a)
        res, at = [], 0
        for _, _, xs in segs:
            res.append(out[at:at + xs.shape[0]].cpu())
            at += xs.shape[0]
        return res


SHAPES = [(6, 2, 20, 36, 4, 12, 21), (4, 4, 33, 17, 2, 9, 8), (2, 1, 128, 128, 4, 128, 128), (3, 3, 64, 200, 3, 24, 24), (2, 2, 200, 256, 1, 16, 70), (2, 2, 256, 256, 5, 8, 8)]


@pytest.mark.parametrize("shape", SHAPES)
def test_delta_token_by_token_and_whole(shape):
    m = Delta(*shape)
    T = 37
    x = m.inputs(T, 5)
    want, S = m.reference(x)
    got = torch.cat([m.step([(1, t, x[t:t + 1])], "decode")[0] for t in range(T)])
    assert rel(got, want) < 2e-5
    assert rel(m.state[1, :, :, :m.vd], S) < 2e-5
    for form, tol in (("scan", 1e-4), ("scan32", 2e-5)):
        got = m.step([(2, 0, x)], form)[0]
        assert rel(got, want) < tol
        assert rel(m.state[2, :, :, :m.vd], S) < tol


@pytest.mark.parametrize("shape", SHAPES[:3])
def test_delta_portions_batches_and_reused_slots(shape):
    m = Delta(*shape)
    T = 90
    x, y, z = m.inputs(T, 7), m.inputs(41, 8), m.inputs(5, 9)
    want = {"x": m.reference(x)[0], "y": m.reference(y)[0], "z": m.reference(z)[0]}
    got, at, turn = {"x": [], "y": [], "z": []}, 0, 0
    cuts = [2, 3, 1, 16, 17, 2, 33, 1, 1, 14]
    assert sum(cuts) == T
    ya = 0
    for c in cuts:                                       # x in portions; y rides along in slot 2 with other sizes, then z takes y's slot
        segs, names = [(0, at, x[at:at + c])], ["x"]
        n = min(7, 41 - ya)
        if n > 0:
            segs.append((2, ya, y[ya:ya + n])); names.append("y"); ya += n
        elif not got["z"]:
            segs.append((2, 0, z)); names.append("z")
        form = "decode" if all(s[2].shape[0] == 1 for s in segs) else "scan"
        for n_, r in zip(names, m.step(segs, form)):
            got[n_].append(r)
        at += c
    for n in got:
        assert rel(torch.cat(got[n]), want[n]) < 1e-4, n


@pytest.mark.parametrize("a_log,dt,what", [(4.0, 3.0, "forgets at once"), (1.5, 1.0, "fades within a chunk"), (-6.0, -9.0, "keeps everything")])
def test_delta_extreme_decays_and_repeated_keys(a_log, dt, what):
    """decay products that vanish within a few tokens or stay at 1, and one key written over and over at full strength"""
    m = Delta(2, 1, 48, 32, 2, 8, 8)
    m.a_log, m.dt_bias = torch.tensor([a_log, a_log - 1]), m.dt_bias * 0.5 + 1.5 + dt
    m.t["na"], m.t["dt"] = (-torch.exp(m.a_log).repeat_interleave(m.dim)).to(DEV), m.dt_bias.to(DEV)
    T = 70
    x = m.inputs(T, 3)
    k0, nk = m.off["k"], m.KH * m.dim
    x[20:60, k0:k0 + nk] = x[20, k0:k0 + nk]
    x[:, m.off["b"]:m.off["b"] + m.H] = 9.0
    want, S = m.reference(x)
    for cuts in ([T], [17, 2, 31, 20]):
        got, at = [], 0
        for c in cuts:
            got += m.step([(1, at, x[at:at + c])], "scan32")
            at += c
        assert rel(torch.cat(got), want) < 5e-5, (what, cuts)
        assert rel(m.state[1, :, :, :m.vd], S) < 5e-5, (what, cuts)


def test_delta_parked_rows_touch_nothing():
    m = Delta(2, 2, 16, 16, 3, 8, 8)
    before = m.state.clone(), m.ring.clone()
    x = m.inputs(2, 1).to(DEV)
    rows = torch.tensor([[0, -1, 0, 0], [1, -1, 1, 0]], dtype=torch.int32, device=DEV)
    out = torch.full((2, 32), 3.0, device=DEV)
    call("chatts_delta_decode", m.args(x, rows, out))
    assert torch.equal(m.state, before[0]) and torch.equal(m.ring, before[1]) and float((out - 3).abs().sum()) == 0


# ---- latent attention --------------------------------------------------------------------------------------------------------------
class Latent:
    """pages of latents + the absorbed attention, against softmax over the cached rows"""

    def __init__(self, heads, rank, rot, f32, slots=2, ctx=512, block=64, seed=0):
        self.heads, self.rank, self.rot, self.f32, self.block = heads, rank, rot, f32, block
        self.rp, self.rotp = (rank + 31) // 32 * 32, (rot + 31) // 32 * 32
        self.cw = self.rp + self.rotp
        g = np.random.default_rng(seed)
        nblk = slots * ctx // block
        self.table = torch.from_numpy(g.permutation(nblk).astype(np.int32).reshape(slots, -1)).to(DEV)      # scattered pages
        self.cache = torch.full((nblk, block, self.cw), float("nan"), dtype=torch.float32 if f32 else torch.bfloat16, device=DEV)

    def put(self, slot, rows):
        """rows [n, rank + rot] -> cache rows 0 .. n, padded; what lies behind them stays NaN"""
        full = torch.zeros(rows.shape[0], self.cw)
        full[:, :self.rank], full[:, self.rp:self.rp + self.rot] = rows[:, :self.rank], rows[:, self.rank:]
        t = self.table.cpu()
        for j in range(rows.shape[0]):
            self.cache[t[slot, j // self.block], j % self.block] = full[j].to(self.cache.dtype).to(DEV)
        return full.to(self.cache.dtype).double()

    def attend(self, q, where, scale, splits=1):
        """q [T, heads, rank + rot], where: (slot, position) per row -> [T, heads, rank]"""
        T = q.shape[0]
        full = torch.zeros(T, self.heads, self.cw)
        full[..., :self.rank], full[..., self.rp:self.rp + self.rot] = q[..., :self.rank], q[..., self.rank:]
        qd = full.reshape(T, -1).to(DEV)
        hi = qd.to(torch.bfloat16)
        pl = torch.stack([hi, (qd - hi.float()).to(torch.bfloat16)])
        rows = torch.tensor([(s, p, i, 0) for i, (s, p) in enumerate(where)], dtype=torch.int32, device=DEV)
        out = torch.zeros(T, self.heads, self.rp, device=DEV)
        part = torch.zeros(T * self.heads * splits * (self.rp + 4), device=DEV)
        a = _lib.LatentArgs(heads=self.heads, dim=8, rot=self.rot, rank=self.rank, vdim=8, rank_p=self.rp, rot_p=self.rotp, scale=scale, eps=1e-6,
                            cache=self.cache.data_ptr(), cache_f32=int(self.f32), table=self.table.data_ptr(), table_stride=self.table.shape[1],
                            log_block=int(math.log2(self.block)), rows=rows.data_ptr(), n_rows=T,
                            q=operand(qd, None, self.heads * self.cw) if self.f32 else operand(None, pl, self.heads * self.cw),
                            o=out.data_ptr(), n_splits=splits, partial=part.data_ptr())
        call("chatts_latent_attend", a)
        return out[..., :self.rank].cpu()


def soft(q, rows, pos, scale, rank):
    """q [heads, n], rows [m, n] (float64)"""
    p = torch.softmax(q.double() @ rows[:pos + 1].T * scale, -1)
    return p @ rows[:pos + 1, :rank]


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("heads,rank,rot,block", [(3, 50, 10, 64), (20, 160, 32, 128), (16, 512, 64, 64), (4, 600, 8, 64)])
@pytest.mark.parametrize("splits", [1, 3])
def test_latent_attend(f32, heads, rank, rot, block, splits):
    m = Latent(heads, rank, rot, f32, block=block)
    g = gen(rank)
    rows = [torch.randn(400, rank + rot, generator=g), torch.randn(130, rank + rot, generator=g)]
    stored = [m.put(s, r) for s, r in enumerate(rows)]
    where = [(0, 0), (0, 63), (0, 64), (0, 399), (1, 1), (1, 127), (1, 128), (1, 129)]
    q = torch.randn(len(where), heads, rank + rot, generator=g) * 2
    got = m.attend(q, where, 1 / math.sqrt(rank), splits)
    for i, (s, p) in enumerate(where):
        full = torch.zeros(heads, m.cw, dtype=torch.float64)
        full[:, :rank], full[:, m.rp:m.rp + rot] = q[i, :, :rank], q[i, :, rank:]
        want = soft(full, stored[s], p, 1 / math.sqrt(rank), rank)
        assert rel(got[i], want) < (1e-5 if f32 else 1e-2), (s, p)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("splits", [1, 4])
def test_latent_attend_finds_one_key_among_many(f32, splits):
    """one key stands out by a large score: its latent is the result wherever it lies, unless it is in the future"""
    heads, rank, rot = 4, 64, 16
    m = Latent(heads, rank, rot, f32)
    g = gen(3)
    rows = torch.randn(400, rank + rot, generator=g) * 0.1
    for key in (0, 1, 62, 63, 64, 65, 127, 128, 255, 256, 383, 384, 398, 399):
        r = rows.clone()
        r[key] = torch.randn(rank + rot, generator=gen(key + 100))
        stored = m.put(0, r)
        q = (r[key] * 40 / float(r[key].norm() ** 2)).repeat(1, heads, 1).float()
        got = m.attend(q, [(0, 399)], 1.0, splits)[0]
        assert rel(got, stored[key, :rank].repeat(heads, 1)) < 1e-2, key
        if key > 0:
            got = m.attend(q, [(0, key - 1)], 1.0, splits)[0]
            assert rel(got, stored[key, :rank].repeat(heads, 1)) > 0.5, key


@pytest.mark.parametrize("f32", [True, False])
def test_latent_prep(f32):
    heads, dim, rot, rank, T = 3, 24, 10, 50, 4
    m = Latent(heads, rank, rot, f32)
    dim_p, g = 32, gen(0)
    off_qr, off_c, off_kr, ld = heads * dim_p, heads * dim_p + 64, heads * dim_p + 128, heads * dim_p + 192
    x = torch.randn(T, ld, generator=g)
    cn = 1 + 0.2 * torch.randn(rank, generator=g)
    rspec = {"dims": rot, "base": 5000.0, "scaling": {"factor": 5.0, "original": 48, "fast": 16.0, "slow": 1.5}}
    from chatts_amd.rotary import rotary_tables
    cos, sin = rotary_tables(rot, 5000.0, 512, rspec["scaling"], DEV)
    where = [(0, 0), (0, 63), (1, 64), (1, 300)]
    rows = torch.tensor([(s, p, i, 0) for i, (s, p) in enumerate(where)], dtype=torch.int32, device=DEV)
    xd, cnd = x.to(DEV), cn.to(DEV)
    q = torch.zeros(T, heads * m.cw, device=DEV)
    pl = torch.zeros((2, T, heads * m.cw), dtype=torch.bfloat16, device=DEV)
    call("chatts_latent_prep", _lib.LatentArgs(proj=xd.data_ptr(), ld_proj=ld, off_q=0, off_qr=off_qr, off_c=off_c, off_kr=off_kr, heads=heads, dim=dim, rot=rot,
                                               rank=rank, vdim=8, rank_p=m.rp, rot_p=m.rotp, scale=1.0, eps=1e-3, c_norm=cnd.data_ptr(), cos_tab=cos.data_ptr(),
                                               sin_tab=sin.data_ptr(), cache=m.cache.data_ptr(), cache_f32=int(f32), table=m.table.data_ptr(),
                                               table_stride=m.table.shape[1], log_block=6, rows=rows.data_ptr(), n_rows=T,
                                               q=operand(q, None, heads * m.cw) if f32 else operand(None, pl, heads * m.cw), n_splits=1))
    if not f32:
        q = pl[0].float() + pl[1].float()
    pos = torch.tensor([p for _, p in where])
    want_q = F.rotate(x.double()[:, off_qr:off_qr + heads * rot].view(T, heads, rot), pos, rspec)
    assert rel(q.view(T, heads, m.cw)[..., m.rp:m.rp + rot], want_q) < (1e-6 if f32 else 2e-5)
    c = F.rms_norm(x.double()[:, off_c:off_c + rank], cn.double(), 1e-3)
    kr = F.rotate(x.double()[:, off_kr:off_kr + rot], pos, rspec)
    tab = m.table.cpu()
    for i, (s, p) in enumerate(where):
        row = m.cache[tab[s, p // 64], p % 64].double().cpu()
        tol = 1e-6 if f32 else 4e-3
        assert rel(row[:rank], c[i]) < tol and rel(row[m.rp:m.rp + rot], kr[i]) < tol
        assert float(row[rank:m.rp].abs().sum()) == 0 and float(row[m.rp + rot:].abs().sum()) == 0
    assert int(torch.isfinite(m.cache.float()).all(-1).sum()) == T                # nothing else was written


@pytest.mark.parametrize("heads,dim,rot,vdim,rank", [(3, 24, 10, 40, 50), (2, 128, 64, 128, 512), (4, 64, 32, 64, 128), (2, 200, 32, 150, 96)])
def test_latent_expanded(heads, dim, rot, vdim, rank):
    """spans of many tokens, one of them behind earlier ones, beside a span that is left out; against softmax over expanded float64 keys"""
    up = lambda n, m: (n + m - 1) // m * m
    m = Latent(heads, rank, rot, False, slots=3)
    m.rp = up(rank, 64)
    m.cw = m.rp + m.rotp
    m.cache = torch.full((m.cache.shape[0], m.block, m.cw), float("nan"), dtype=torch.bfloat16, device=DEV)
    dp, vp, lib = up(dim, 32), up(vdim, 16), _lib.load()
    assert lib.chatts_latent_can_expand(dp, m.rotp, vp, m.rp)
    g = gen(dim)
    bf = lambda *s: (torch.randn(*s, generator=g) / math.sqrt(s[-1])).to(torch.bfloat16)
    uk, uv = bf(heads, dim, rank), bf(heads, vdim, rank)
    ukp, uvp = torch.zeros(heads, dp, m.rp, dtype=torch.bfloat16), torch.zeros(heads, vp, m.rp, dtype=torch.bfloat16)
    ukp[:, :dim, :rank], uvp[:, :vdim, :rank] = uk, uv
    spans = [(0, 150, 0, 0), (150, 3, 70, 1), (153, 70, 130, 2)]
    bases, at = [], 0
    for r0, t, p0, s in spans:
        ok = t >= 8
        bases.append(at if ok else -1)
        at += up(p0 + t, 64) if ok else 0
    T = 223
    stored = {s: m.put(s, torch.randn(p0 + t, rank + rot, generator=g)) for r0, t, p0, s in spans}
    q = torch.randn(T, heads, dim + rot, generator=g) * 1.5
    qx = torch.zeros(T, heads, dp + m.rotp)
    qx[..., :dim], qx[..., dp:dp + rot] = q[..., :dim], q[..., dim:]
    qx = qx.to(torch.bfloat16)
    host = (_lib.Span * 3)(*[_lib.Span(*s, b) for s, b in zip(spans, bases)])
    dev = torch.tensor([list(s) + [b] for s, b in zip(spans, bases)], dtype=torch.int32, device=DEV)
    z = lambda *s: torch.zeros(*s, dtype=torch.bfloat16, device=DEV)
    cb, kr, zero, kh, kl, vh, vl = z(at, m.rp), z(at, m.rotp), z(max(at, heads * vp), m.rp), z(at, heads * dp + 128), z(at, heads * dp + 128), z(heads * vp, at + 128), z(heads * vp, at + 128)
    ukd, uvd, qd = ukp.to(DEV), uvp.to(DEV), qx.reshape(T, -1).contiguous().to(DEV)
    out = torch.full((T, heads * (vp + 4)), 5.0, device=DEV)
    ws = torch.zeros(64 << 20, dtype=torch.uint8, device=DEV)
    scale = 1 / math.sqrt(dim + rot)
    rows = torch.zeros(T, 4, dtype=torch.int32, device=DEV)
    a = _lib.LatentArgs(heads=heads, dim=dim, rot=rot, rank=rank, vdim=vdim, rank_p=m.rp, rot_p=m.rotp, dim_p=dp, scale=scale, eps=1e-6, cache=m.cache.data_ptr(),
                        cache_f32=0, table=m.table.data_ptr(), table_stride=m.table.shape[1], log_block=6, rows=rows.data_ptr(), n_rows=T, q=operand(None, None, heads * m.cw),
                        n_splits=1, qx=qd.data_ptr())
    x = _lib.LatentExpandArgs(latent=C.pointer(a), spans=host, spans_dev=dev.data_ptr(), n_spans=3, vdim_p=vp, out_head=vp + 4, max_rows=at, uk=ukd.data_ptr(),
                              uv=uvd.data_ptr(), cbuf=cb.data_ptr(), krbuf=kr.data_ptr(), zero=zero.data_ptr(), k_hi=kh.data_ptr(), k_lo=kl.data_ptr(),
                              v_hi=vh.data_ptr(), v_lo=vl.data_ptr(), out=operand(out, None, heads * (vp + 4)), workspace=ws.data_ptr(), workspace_bytes=ws.numel())
    call("chatts_latent_expanded", x)
    got = out.view(T, heads, vp + 4).cpu()
    for (r0, t, p0, s), b in zip(spans, bases):
        if b < 0:
            assert float((got[r0:r0 + t] - 5).abs().sum()) == 0
            continue
        c, krot = stored[s][:, :rank], stored[s][:, m.rp:m.rp + rot]
        k = torch.einsum("jr,hdr->jhd", c, uk.double())
        v = torch.einsum("jr,hdr->jhd", c, uv.double())
        for i in range(0, t, 7):
            n = p0 + i + 1
            qq = qx[r0 + i].double()
            sc = (torch.einsum("hd,jhd->hj", qq[:, :dim], k[:n]) + torch.einsum("hd,jd->hj", qq[:, dp:dp + rot], krot[:n])) * scale
            want = torch.einsum("hj,jhd->hd", torch.softmax(sc, -1), v[:n])
            assert rel(got[r0 + i, :, :vdim], want) < 1e-2, (s, i)


def test_bad_shapes_are_refused_on_the_host():
    lib = _lib.load()
    t = torch.zeros(4096, device=DEV)
    a = _lib.DeltaArgs(proj=t.data_ptr(), rows=t.data_ptr(), state=t.data_ptr(), ring=t.data_ptr(), conv_w=t.data_ptr(), dt_bias=t.data_ptr(), neg_a=t.data_ptr(),
                       norm_w=t.data_ptr(), heads=3, kv_heads=2, dim=8, vdim=8, taps=2)
    assert lib.chatts_delta_decode(C.byref(a), _lib.stream_ptr()) == _lib.E_SHAPE
    a = _lib.LatentArgs(cache=t.data_ptr(), table=t.data_ptr(), rows=t.data_ptr(), heads=1, dim=8, rot=8, rank=2000, rank_p=2016, rot_p=32, log_block=6,
                        q=operand(t, None, 4096))
    assert lib.chatts_latent_attend(C.byref(a), _lib.stream_ptr()) == _lib.E_SHAPE
    h = _lib.HeadLinearArgs(a=t.data_ptr(), w=t.data_ptr(), out=operand(t, None, 64), m=1, heads=1, n=20, k=32, lda=32, a_head=32, out_head=20)
    assert lib.chatts_head_linear(C.byref(h), _lib.stream_ptr()) == _lib.E_SHAPE
