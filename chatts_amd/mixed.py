"""MixedDecoder - a served model whose layers each name their mixer, run by csrc/mixdec.hip.

A sequential layer is norm1 -> mixer -> norm1b -> residual, then optionally norm2 -> squared-relu feed-forward -> norm2b -> residual; a parallel one adds
mixer(norm1(x)) + feed-forward(norm2(x)) to x, both norms of the same x in groups (csrc/pair.hip); a post-norm one is x <- norm1(alpha x + mixer(x)), then
x <- norm2(alpha x + feed-forward(x)) (csrc/postnorm.hip); a pre-norm one adds factors of mixer(norm1(x)) and feed-forward(norm2(x)) in turn and may average the
streams of all layers so far (csrc/depth.hip).  Mixers:
  LatentMixer   attention over a paged cache of one latent + one rotated key part per token (csrc/latent.hip)
  DeltaMixer    gated delta rule: a float32 state and a ring of convolution inputs per slot (csrc/delta.hip)
  WindowMixer   grouped-head attention over paged keys and values (csrc/window.hip); by its fields: short convolutions with a ring of inputs per slot, norms
                per head / over all heads / after a rotation, values mixed with an earlier layer's, window or chunks, kept first tokens, sink, capped
                scores, a distance bias (linear or logarithmic), a gate per value or per head
  WkvMixer, MlstmMixer   gated linear recurrences: a float32 state per slot (csrc/recur.hip)
  MinGruMixer   a gated recurrence per channel whose gates read the current token alone: a float32 state per slot (csrc/gru.hip)
  SelectMixer   selective scan: a float32 state and a ring of convolution inputs per slot (csrc/select.hip)
  SideBySide    two of WindowMixer, MinGruMixer, SelectMixer reading the same rows, their outputs added with a factor each
Feed-forwards of parallel, post-norm and pre-norm layers: ClampGlu, GeluGlu, Experts (csrc/moe.hip).
A design (chatts_amd/fobolix.py, medilix.py, mefurax.py, muvetar.py) says in which order layers run (config.runs(): a layer may run several times, every run has
its own pages or state) and maps its tensor names onto LayerWeights.

Everything is padded once, at load: widths and feed-forwards to multiples of 64, the stacked input projections block by block, heads to
what the kernels tile by.  Padding is zero weights, so activations never need clearing.

Slots, pages, sampling, scheduling and generation are SlotModel's.  A recurrent state is a function of the whole prefix and is not kept per
position, so prefixes are not reused between requests.
"""
import ctypes as C
import glob
import math
import os
from dataclasses import dataclass
from types import SimpleNamespace
from typing import Any, Optional

import torch

from . import _lib
from .kv_blocks import BlockPool
from .rotary import rotary_tables, sinusoid_tables
from .slot_model import SlotModel
from .tp import LocalComm


@dataclass
class LatentMixer:
    heads: int
    dim: int
    rot: int
    vdim: int
    rank: int
    scale: float
    rot_base: float
    rot_scaling: Optional[dict]
    q: Any          # [heads * (dim + rot), width], head by head
    dkv: Any        # [rank + rot, width]
    c_norm: Any
    uk: Any         # [heads * dim, rank]
    uv: Any         # [heads * vdim, rank]
    o: Any          # [width, heads * vdim]


@dataclass
class DeltaMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    q: Any
    k: Any
    v: Any
    q_conv: Any     # [channels, taps]
    k_conv: Any
    v_conv: Any
    b: Any
    a_log: Any
    a1: Any
    a2: Any
    dt_bias: Any
    g1: Any
    g2: Any
    norm: Any
    o: Any


@dataclass
class WindowMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int     # 0: every earlier position
    keep_first: int
    sink: bool
    q: Any
    k: Any
    v: Any
    g: Any          # output gate [heads * vdim, width] or None
    q_norm: Any     # [dim] (norm_whole: [heads * dim], [kv_heads * dim]) or None
    k_norm: Any
    o: Any
    bias: Any = None            # of q, k, v: (3 vectors) or None
    conv: Any = None            # of q, k, v: ([channels, taps] each) or None
    norm_whole: bool = False    # the norms run over all heads at once
    rot: int = 0                # rotated dimensions, paired (2 i, 2 i + 1)
    rot_base: float = 0.0
    unit: bool = False          # queries and keys divided by their root mean square, after the rotation
    chunk: int = 0              # 0: none
    softcap: float = 0.0        # 0: none
    slopes: Any = None          # [heads] or None
    gate_heads: bool = False    # g is [heads, width]: one gate per head
    log_bias: Any = None        # (r1, r2), [heads] each: r1 ln(1 + r2 distance) is taken off the scores; or None
    vmix: Optional[float] = None    # values become (1 - vmix) v + vmix v_first, v_first those of the first layer that has a vmix


@dataclass
class WkvMixer:
    heads: int
    dim: int
    mu: Any         # of r, k, v, g, w
    r: Any
    k: Any
    v: Any
    g: Any
    w1: Any
    w2: Any
    w0: Any
    u: Any
    norm: Any
    o: Any


@dataclass
class MlstmMixer:
    heads: int
    dim: int
    vdim: int
    cap: float
    q: Any
    k: Any
    v: Any
    g: Any
    i: Any
    f: Any
    bias_i: Any
    bias_f: Any
    norm: Any
    o: Any


@dataclass
class MinGruMixer:
    z: Any          # [channels, width]: gate, candidate, output gate
    x: Any
    g: Any
    bias_z: Any
    bias_x: Any
    o: Any


@dataclass
class SelectMixer:
    state: int      # states per channel
    rank: int       # of the step sizes
    w_in: Any       # [x: channels | z: channels, width]
    conv: Any       # [channels, taps]
    conv_bias: Any
    x: Any          # [dt: rank | B: state | C: state, channels]
    dt: Any         # [channels, rank]
    dt_bias: Any
    a_log: Any      # [channels, state]
    d: Any
    o: Any


@dataclass
class SideBySide:
    left: Any
    right: Any      # of another kind than left
    left_scale: float
    right_scale: float


@dataclass
class ClampGlu:
    gate: Any
    up: Any
    down: Any
    limit: float
    alpha: float


@dataclass
class GeluGlu:
    gate: Any
    up: Any
    down: Any


@dataclass
class Experts:
    router: Any         # [experts + identity, width]
    correction: Any     # or None
    experts: Any        # (gate, up, down) each; (up, down): squared relu
    identity: int
    top: int
    groups: int
    keep: int
    by_logits: bool = False     # chosen by logits, weights: softmax over the chosen ones
    shared: Any = None          # an expert that every token uses: (up, down), squared relu, in post-norm layers; (gate, up, down), clamped, in pre-norm ones
    weight_scale: Optional[float] = None    # weights: the chosen softmax values as they are, times this
    clamp: Optional[tuple] = None           # (limit, alpha): experts are clamped gated units
    shared_clamp: Optional[tuple] = None


@dataclass
class LayerWeights:
    mixer: Any
    norm1: Any
    norm1b: Any = None
    norm2: Any = None
    norm2b: Any = None
    up: Any = None      # squared-relu feed-forward of a sequential layer
    down: Any = None
    ff: Any = None      # ClampGlu, GeluGlu or Experts of a parallel, post-norm or pre-norm layer
    parallel: bool = False
    post: bool = False  # norms after the sums; norm1 / norm2 as they multiply
    pre: bool = False   # norms before the sublayers only
    depth: Any = None   # pre: weights of the embedding output and of every layer's result so far, whose sum goes on


def _up(n, m):
    return (int(n) + m - 1) // m * m


def _pad(t, rows, cols):
    out = torch.zeros((rows, cols), dtype=t.dtype, device=t.device)
    out[:t.shape[0], :t.shape[1]] = t
    return out


class MixedDecoder(SlotModel):
    step_is_idempotent = False       # a decode step advances recurrent states

    def __init__(self, config, device="cuda", comm=None, max_ctx=2048, max_prefill_tokens=2048, use_graph=True, max_batch=1, kv_block_size=None,
                 kv_pool_blocks=None, dtype="bfloat16", prefill_tiled_weights=None, weight_format="bf16", **unused):
        """dtype "bfloat16": bf16 hi / lo operand planes and a bf16 latent cache; "float32": every product and sum in 32-bit (checks)."""
        if not torch.cuda.is_available():
            raise RuntimeError("chatts_amd needs a ROCm GPU: there is no CPU fallback for the model")
        if dtype not in ("bfloat16", "float32"):
            raise ValueError("dtype must be 'bfloat16' or 'float32'")
        if weight_format != "bf16":
            raise ValueError(f"{type(config).__name__} is served with bf16 weights, not {weight_format!r}")
        self.comm = comm or LocalComm()
        if self.comm.world != 1:
            raise ValueError("decoders of mixed layers run on one GPU (tensor_parallel_size 1)")
        self.lib = _lib.load()
        self.config, self.device = config, torch.device(device)
        self.dtype, self.exact = dtype, dtype == "float32"
        self.max_batch = max(1, int(max_batch))
        self.kv_block_size = int(kv_block_size or 64)
        if self.kv_block_size < 64 or self.kv_block_size & (self.kv_block_size - 1):
            raise ValueError(f"kv_block_size={kv_block_size} must be a power of two >= 64")
        self.max_ctx = _up(max_ctx, self.kv_block_size)
        self.t_max = int(max(min(max_prefill_tokens, self.max_ctx * self.max_batch), self.max_batch))
        self._kv_pool_blocks = None if kv_pool_blocks is None else int(kv_pool_blocks)
        self.use_graph, self._graph, self._graph_batched, self._tp = use_graph, None, None, None
        if prefill_tiled_weights is None:
            prefill_tiled_weights = self.t_max >= 96 and os.environ.get("CHATTS_TILED_WEIGHTS", "1") != "0"
        self.tiled = bool(prefill_tiled_weights) and not self.exact
        self.plan = SimpleNamespace(world=1, rank=0, vocab=config.vocab_size, v0=0)
        self.enable_prefix_caching = False
        self._slot_idents = [[] for _ in range(self.max_batch)]
        self._slot_seen = [0] * self.max_batch
        self._kv_replaced = {}
        self.prefix_stats = {"requests": 0, "hits": 0, "tokens_reused": 0, "tokens_prefilled": 0}
        self._decoder, self._keep, self.loaded = None, [], set()

    # ---- weights -------------------------------------------------------------------------------------------------------------
    def layer_weights(self, sd, i):
        raise NotImplementedError

    def model_weights(self, sd):
        raise NotImplementedError

    @classmethod
    def from_pretrained(cls, path, config=None, torch_dtype=None, device_map=None, trust_remote_code=None, **kw):
        from safetensors import safe_open
        from .registry import load_config
        if torch_dtype is not None and "dtype" not in kw:
            kw["dtype"] = str(torch_dtype).replace("torch.", "")
        m = cls(config or load_config(path), **kw)

        def pairs():
            for f in sorted(glob.glob(os.path.join(path, "*.safetensors"))):
                with safe_open(f, framework="pt", device="cpu") as h:
                    for k in h.keys():
                        yield k, h.get_tensor(k)
        m.load_weights(pairs())
        return m

    @classmethod
    def from_synthetic(cls, config, seed=0, rank_a=None, rank_g=None, **kw):
        """random weights of the configuration's shapes, made on the device (speed measurements)"""
        m = cls(config, **kw)
        gen = torch.Generator(device=m.device).manual_seed(seed)
        big = max((l["mixer"].get("dim", 64) for l in config.layers), default=64)
        sd = {}
        for name, shape in config.tensor_shapes(rank_a or big, rank_g or big).items():
            t = torch.randn(shape, generator=gen, device=m.device)
            if len(shape) == 2 and not name.endswith((".conv", ".u")) and name not in ("embed", "bigram"):
                t *= shape[1] ** -0.5
            if name.endswith(("norm", "norm1", "norm2", "norm1b", "norm2b")):
                t = 1.0 + 0.1 * t
            if name.endswith("dt_bias"):
                t = 0.5 * t - 3.0
            if name.endswith(("mix.w0", "mix.f.b")):
                t = t + (-4.0 if name.endswith("w0") else 4.0)
            if ".mu." in name:
                t = 0.5 + 0.1 * t
            if name.endswith(".correction"):
                t = 0.01 * t        # (larger ones would send every token to the same few experts)
            if name.endswith(".dt.b"):
                t = 0.5 * t - 3.0
            if name.endswith((".r1", ".r2")):
                t = 0.5 * t.abs()
            if name.endswith(".dwa"):
                t = t / shape[0]
            sd[name] = t.to(torch.bfloat16)
        m.load_weights(sd.items())
        return m

    def load_weights(self, weights):
        """consume (name, tensor) pairs; returns the set of names taken"""
        sd = {n: t.to(self.device) for n, t in weights}
        want = self.config.tensor_shapes()
        missing = sorted(set(want) - set(sd))
        if missing:
            raise ValueError(f"checkpoint lacks {missing[:5]}{' ...' if len(missing) > 5 else ''}")
        for n, shape in want.items():
            if any(s is not None and s != g for s, g in zip(shape, sd[n].shape)) or len(shape) != sd[n].dim():
                raise ValueError(f"{n}: shape {tuple(sd[n].shape)}, the configuration says {shape}")
        self._build(sd)
        self.loaded = set(want)
        return self.loaded

    def _dev(self, t):
        t = t.contiguous()
        self._keep.append(t)
        return t.data_ptr()

    def _f32(self, t, n=None):
        t = t.to(torch.float32).reshape(-1)
        if n is not None and n > t.numel():
            t = torch.cat([t, torch.zeros(n - t.numel(), dtype=torch.float32, device=self.device)])
        return self._dev(t)

    def _mat(self, t, rows=None, cols=None, tile=False):
        """bf16 matrix, zero padded -> (pointer, pointer of its tiled copy or None)"""
        t = t.to(torch.bfloat16)
        t = _pad(t, rows or t.shape[0], cols or t.shape[1]).contiguous()
        p, pt = self._dev(t), None
        if tile and self.tiled:
            out = torch.empty(int(self.lib.chatts_tile_bf16_elems(t.shape[0], t.shape[1])), dtype=torch.bfloat16, device=self.device)
            _lib.check(self.lib.chatts_tile_bf16(p, t.shape[0], t.shape[1], t.shape[1], out.data_ptr(), _lib.stream_ptr()))
            pt = self._dev(out)
        return p, pt

    def _pieces(self, t, cols):
        """[rows, rank] -> [rank / 8, rows, 8]: what neighbouring threads read of neighbouring rows lies side by side"""
        t = _pad(t.to(torch.bfloat16), t.shape[0], cols)
        return self._dev(t.view(t.shape[0], cols // 8, 8).transpose(0, 1).contiguous())

    def _stack(self, blocks, cols=None):
        """stacked projection: (name, [rows, width], padded rows) -> (matrix, {name: first row}); cols: padded width of its input"""
        off, at = {}, 0
        for name, t, rows in blocks:
            off[name] = at
            at += rows
        out = torch.zeros((_up(at, 64), cols or self._wp), dtype=torch.bfloat16, device=self.device)
        for name, t, rows in blocks:
            out[off[name]:off[name] + t.shape[0], :t.shape[1]] = t.to(torch.bfloat16)
        return out, off

    def _state(self, shape):
        t = torch.zeros(shape, dtype=torch.float32, device=self.device)
        self.state_bytes += 4 * t.numel()
        return self._dev(t)

    def _latent_layer(self, L, m):
        H, W = m.heads, self.config.hidden_size
        dim_p, rank_p, rot_p, vdim_p = _up(m.dim, 32), _up(m.rank, 64), _up(m.rot, 32), _up(m.vdim, 16)
        q = m.q.view(H, m.dim + m.rot, W)
        un = torch.zeros((H, dim_p, W), dtype=q.dtype, device=self.device)
        un[:, :m.dim] = q[:, :m.dim]
        w, off = self._stack([("q", un.view(H * dim_p, W), H * dim_p), ("qr", q[:, m.dim:].reshape(H * m.rot, W), _up(H * m.rot, 64)),
                              ("c", m.dkv[:m.rank], _up(m.rank, 64)), ("kr", m.dkv[m.rank:], _up(m.rot, 64))])
        L.kind, L.in_n = _lib.MIX_LATENT, w.shape[0]
        L.w_in, L.in_t = self._mat(w, tile=True)
        o = torch.zeros((W, H, vdim_p), dtype=m.o.dtype, device=self.device)
        o[:, :, :m.vdim] = m.o.view(W, H, m.vdim)
        L.out_k, L.out_head, L.dim_p, L.vdim_p = _up(H * vdim_p, 64), vdim_p, dim_p, vdim_p
        L.out, L.out_t = self._mat(o.view(W, H * vdim_p), self._wp, L.out_k, tile=True)
        uk = torch.zeros((H, rank_p, dim_p), dtype=torch.bfloat16, device=self.device)
        uk[:, :m.rank, :m.dim] = m.uk.view(H, m.dim, m.rank).transpose(1, 2).to(torch.bfloat16)
        uv = torch.zeros((H, vdim_p, rank_p), dtype=torch.bfloat16, device=self.device)
        uv[:, :m.vdim, :m.rank] = m.uv.view(H, m.vdim, m.rank).to(torch.bfloat16)
        L.uk, L.uv = self._dev(uk), self._dev(uv)
        if self.expand_rows and self.lib.chatts_latent_can_expand(dim_p, rot_p, vdim_p, rank_p):      # prompts: keys and values written out
            L.ukx, L.uvx = self._dev(uk.transpose(1, 2).reshape(H * dim_p, rank_p)), L.uv
            self._exp = [max(a, b) for a, b in zip(self._exp, (rank_p, rot_p, H * dim_p, H * vdim_p, H * (dim_p + rot_p)))]
        cos, sin = rotary_tables(m.rot, m.rot_base, self.max_ctx, m.rot_scaling, self.device)
        L.latent = _lib.LatentArgs(off_q=off["q"], off_qr=off["qr"], off_c=off["c"], off_kr=off["kr"], heads=H, dim=m.dim, rot=m.rot, rank=m.rank,
                                   vdim=m.vdim, rank_p=rank_p, rot_p=rot_p, scale=m.scale, c_norm=self._f32(m.c_norm), cos_tab=self._dev(cos),
                                   sin_tab=self._dev(sin))
        self._lat_q, self._lat_o = max(self._lat_q, H * (rank_p + rot_p)), max(self._lat_o, H * rank_p)

    def _delta_layer(self, L, m):
        qk, v, ra, rg = m.kv_heads * m.dim, m.heads * m.vdim, m.a1.shape[0], m.g1.shape[0]
        ra_p, rg_p = _up(ra, 64), _up(rg, 64)
        w, off = self._stack([("q", m.q, _up(qk, 64)), ("k", m.k, _up(qk, 64)), ("v", m.v, _up(v, 64)), ("a", m.a1, ra_p), ("g", m.g1, rg_p),
                              ("b", m.b, _up(m.heads, 64))])
        L.kind, L.in_n = _lib.MIX_DELTA, w.shape[0]
        L.w_in, L.in_t = self._mat(w, tile=True)
        L.out_k, L.out_head = _up(v, 64), m.vdim
        L.out, L.out_t = self._mat(m.o, self._wp, L.out_k, tile=True)
        conv = torch.zeros((m.taps, off["a"]), dtype=torch.float32, device=self.device)
        for n, t in (("q", m.q_conv), ("k", m.k_conv), ("v", m.v_conv)):
            conv[:, off[n]:off[n] + t.shape[0]] = t.to(torch.float32).t()
        L.delta = _lib.DeltaArgs(off_q=off["q"], off_k=off["k"], off_v=off["v"], off_a=off["a"], off_g=off["g"], off_b=off["b"], conv_ch=off["a"],
                                 heads=m.heads, kv_heads=m.kv_heads, dim=m.dim, vdim=m.vdim, taps=m.taps, rank_a=ra_p, rank_g=rg_p,
                                 conv_w=self._dev(conv), a2=self._mat(m.a2, None, ra_p)[0], g2=self._mat(m.g2, None, rg_p)[0],
                                 a2d=self._pieces(m.a2, ra_p), g2d=self._pieces(m.g2, rg_p), ld_a2=ra_p, ld_g2=rg_p,
                                 dt_bias=self._f32(m.dt_bias), neg_a=self._f32(-torch.exp(m.a_log.to(torch.float32)).repeat_interleave(m.dim)), norm_w=self._f32(m.norm))

    def _blocks(self, L, blocks, split=False, bias=None):
        """stacked input projection of a layer -> {name: first row}; split: every block has an operand of its own; bias: {name: vector}"""
        w, off = self._stack([(n, t, _up(t.shape[0], 64)) for n, t in blocks])
        L.in_n = w.shape[0]
        if bias:
            b = torch.zeros(L.in_n, dtype=torch.float32, device=self.device)
            for n, t in bias.items():
                b[off[n]:off[n] + t.shape[0]] = t.to(torch.float32)
            L.in_bias = self._dev(b)
        L.w_in, L.in_t = self._mat(w, tile=not split)
        if split:
            L.n_mix = len(blocks)
            for j, (n, _) in enumerate(blocks):
                L.mix_row[j] = off[n]
            L.mix_row[len(blocks)] = L.in_n
            for j in range(len(blocks)):
                L.mix_t[j] = self._mat(w[L.mix_row[j]:L.mix_row[j + 1]], tile=True)[1] if self.tiled else None
        return off

    # a mixer that may stand beside another: its blocks of the stacked input projection and their biases, and what its kernels need (off: first rows of its blocks)
    def _window_blocks(self, m):
        return [("q", m.q), ("k", m.k), ("v", m.v)] + ([("g", m.g)] if m.g is not None else []), dict(zip("qkv", m.bias)) if m.bias else {}

    def _window_args(self, L, m, off, scale):
        dim_p, vdim_p = _up(m.dim, 32), _up(m.vdim, 16)
        L.window = _lib.WindowArgs(off_q=off["q"], off_k=off["k"], off_v=off["v"], off_gate=off.get("g", -1), heads=m.heads, kv_heads=m.kv_heads, dim=m.dim,
                                   vdim=m.vdim, dim_p=dim_p, vdim_p=vdim_p, scale=m.scale, window=m.window, keep_first=m.keep_first if m.window or m.chunk else 0, sink=int(m.sink),
                                   chunk=m.chunk, softcap=m.softcap, gate_heads=int(m.gate_heads), norm_whole=int(m.norm_whole), rot=m.rot, unit=int(m.unit), out_scale=scale)
        a = L.window
        if m.log_bias is not None:
            a.log_r1, a.log_r2 = (self._f32(t) for t in m.log_bias)
        if m.q_norm is not None:
            a.q_norm, a.k_norm = (self._f32(t, _up(t.shape[0], 4)) for t in (m.q_norm, m.k_norm))
        if m.slopes is not None:
            a.slopes = self._f32(torch.tensor(m.slopes, device=self.device))
        if m.rot:
            cos, sin = rotary_tables(m.rot, m.rot_base, self.max_ctx, None, self.device)
            a.cos_tab, a.sin_tab = self._dev(cos), self._dev(sin)
        if m.conv:
            a.taps, a.conv_ch = m.conv[0].shape[1], off["v"] + _up(m.v.shape[0], 64)
            conv = torch.zeros((a.taps, a.conv_ch), dtype=torch.float32, device=self.device)
            for n_, t in zip("qkv", m.conv):
                conv[:, off[n_]:off[n_] + t.shape[0]] = t.to(torch.float32).t()
            a.conv_w = self._dev(conv)
        if m.vmix is not None:
            a.vmix, a.ld_vfirst = m.vmix, _up(m.kv_heads * m.vdim, 4)
        self._lat_q, self._lat_o = max(self._lat_q, m.heads * dim_p), max(self._lat_o, m.heads * (vdim_p + 4))

    def _gru_blocks(self, m):
        return [("z", m.z), ("x", m.x), ("g", m.g)], {"z": m.bias_z, "x": m.bias_x}

    def _gru_args(self, L, m, off, scale):
        L.gru = _lib.GruArgs(off_z=off["z"], off_x=off["x"], off_g=off["g"], width=m.z.shape[0], out_scale=scale)

    def _select_blocks(self, m):
        n = m.conv.shape[0]
        return [("x", m.w_in[:n]), ("z", m.w_in[n:])], {}

    def _select_args(self, L, m, off, scale):
        (n, taps), N, rank = m.conv.shape, m.state, _up(m.rank, 64)
        n4, N4, L.sel_k = _up(n, 4), _up(N, 4), _up(n, 64)
        low, at = self._stack([("dt", m.x[:m.rank], rank), ("b", m.x[m.rank:m.rank + N], _up(N, 16)), ("c", m.x[m.rank + N:], _up(N, 16))], L.sel_k)
        L.sel_low, L.sel_low_t = self._mat(low, tile=True)
        L.sel_dt_n = L.sel_k
        L.sel_dt = self._mat(m.dt, L.sel_dt_n, rank)[0]
        frags = None
        if not self.exact and self.lib.chatts_select_can_steps(rank):
            frags = self._dev(_pad(m.dt.to(torch.bfloat16), L.sel_k, rank).view(L.sel_k // 16, 16, rank // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous())
        conv, a = torch.zeros((taps, n4), dtype=torch.float32, device=self.device), torch.zeros((n, N4), dtype=torch.float32, device=self.device)
        conv[:, :n] = m.conv.to(torch.float32).t()
        a[:, :N] = (-torch.exp(m.a_log.to(torch.float64)) * math.log2(math.e)).float()
        L.select = _lib.SelectArgs(off_x=off["x"], off_z=off["z"], inner=n, state=N, taps=taps, conv_ch=n4, conv_w=self._dev(conv), conv_b=self._f32(m.conv_bias, n4),
                                   ld_low=low.shape[0], off_dt=at["dt"], off_b=at["b"], off_c=at["c"], rank=rank, w_dt=L.sel_dt, w_dt_f=frags, dt_bias=self._f32(m.dt_bias, n4),
                                   a=self._dev(a), d=self._f32(m.d, n4), out_scale=scale)

    def _mixers(self, L, parts):
        """one mixer, or two side by side: (mixer, factor of its output) each"""
        about = {WindowMixer: (_lib.MIX_WINDOW, self._window_blocks, self._window_args), MinGruMixer: (_lib.MIX_GRU, self._gru_blocks, self._gru_args),
                 SelectMixer: (_lib.MIX_SELECT, self._select_blocks, self._select_args)}
        blocks, bias = [], {}
        for j, (m, _) in enumerate(parts):
            rows, b = about[type(m)][1](m)
            blocks += [((j, n), t) for n, t in rows]
            bias.update({(j, n): t for n, t in b.items()})
        off = self._blocks(L, blocks, bias=bias)
        cols = [_up(m.o.shape[1], 64) for m, _ in parts]
        L.kind, L.out_k = about[type(parts[0][0])][0], sum(cols)
        out = torch.zeros((self._wp, L.out_k), dtype=torch.bfloat16, device=self.device)
        for j, (m, scale) in enumerate(parts):
            at = sum(cols[:j])
            if scale:      # (the kernels take a factor of zero for none)
                out[:m.o.shape[0], at:at + m.o.shape[1]] = m.o.to(torch.bfloat16)
            about[type(m)][2](L, m, {n: r for (i, n), r in off.items() if i == j}, scale)
        L.out, L.out_t = self._mat(out, tile=True)
        if len(parts) > 1:
            L.beside, L.beside_col = about[type(parts[1][0])][0], cols[0]

    def _single_layer(self, L, m):
        self._mixers(L, [(m, 1.0)])

    def _side_by_side(self, L, m):
        self._mixers(L, [(m.left, m.left_scale), (m.right, m.right_scale)])

    def _wkv_layer(self, L, m):
        n, rank = m.heads * m.dim, _up(m.w1.shape[0], 64)
        L.kind = _lib.MIX_RECUR
        off = self._blocks(L, [("r", m.r), ("k", m.k), ("v", m.v), ("g", m.g), ("w", m.w1)], split=True)
        mu = torch.zeros((len(m.mu), self._wp), dtype=torch.float32, device=self.device)
        for j, t in enumerate(m.mu):
            mu[j, :t.shape[0]] = t.to(torch.float32)
        L.mu, L.out_k, L.w2_n = self._dev(mu), _up(n, 64), _up(n, 64)
        L.out, L.out_t = self._mat(m.o, self._wp, L.out_k, tile=True)
        L.w2 = self._mat(m.w2, L.w2_n, rank)[0]
        L.recur = _lib.RecurArgs(kind=_lib.RECUR_WKV, off_q=off["r"], off_k=off["k"], off_v=off["v"], off_gate=off["g"], off_a=off["w"], heads=m.heads, dim=m.dim,
                                 vdim=m.dim, rank=rank, w2d=self._pieces(m.w2, rank), w0=self._f32(m.w0), u=self._f32(m.u), norm_w=self._f32(m.norm))

    def _mlstm_layer(self, L, m):
        L.kind = _lib.MIX_RECUR
        off = self._blocks(L, [("q", m.q), ("k", m.k), ("v", m.v), ("g", m.g), ("i", m.i), ("f", m.f)])
        L.out_k = _up(m.heads * m.vdim, 64)
        L.out, L.out_t = self._mat(m.o, self._wp, L.out_k, tile=True)
        L.recur = _lib.RecurArgs(kind=_lib.RECUR_MLSTM, off_q=off["q"], off_k=off["k"], off_v=off["v"], off_gate=off["g"], off_i=off["i"], off_f=off["f"],
                                 heads=m.heads, dim=m.dim, vdim=m.vdim, bias_i=self._f32(m.bias_i), bias_f=self._f32(m.bias_f), cap=m.cap, norm_w=self._f32(m.norm))

    def _gate_up(self, gate, up, ff):
        """[2 ff, width_p]: gate and up rows in turn, 16 of each"""
        w = torch.zeros((ff // 16, 2, 16, self._wp), dtype=torch.bfloat16, device=self.device)
        for j, t in enumerate((gate, up)):
            w[:, j] = _pad(t.to(torch.bfloat16), ff, self._wp).view(ff // 16, 16, self._wp)
        return w.view(2 * ff, self._wp)

    def _tiles(self, t):
        """chatts_tile_bf16 copies of [n, rows, cols], one after the other"""
        out = torch.empty_like(t)
        for e in range(t.shape[0]):
            _lib.check(self.lib.chatts_tile_bf16(t[e].data_ptr(), t.shape[1], t.shape[2], t.shape[2], out[e].data_ptr(), _lib.stream_ptr()))
        return self._dev(out)

    def _glu(self, L, m):
        L.ff_kind, L.ff, L.glu_limit, L.glu_alpha = _lib.FF_CLAMPGLU, _up(m.gate.shape[0], 64), m.limit, m.alpha
        L.up, L.up_t = self._mat(self._gate_up(m.gate, m.up, L.ff), tile=True)
        L.down, L.down_t = self._mat(m.down, self._wp, L.ff, tile=True)

    def _gelu_glu(self, L, m):
        L.ff_kind, L.ff = _lib.FF_GEGLU, _up(m.gate.shape[0], 64)
        L.up, L.up_t = self._mat(self._gate_up(m.gate, m.up, L.ff), tile=True)
        L.down, L.down_t = self._mat(m.down, self._wp, L.ff, tile=True)

    def _experts(self, L, m):
        n, ff, gated = len(m.experts), _up(m.experts[0][0].shape[0], 64), len(m.experts[0]) == 3
        gu = torch.empty((n, 2 * ff if gated else ff, self._wp), dtype=torch.bfloat16, device=self.device)
        dn = torch.empty((n, self._wp, ff), dtype=torch.bfloat16, device=self.device)
        for e, x in enumerate(m.experts):
            gu[e], dn[e] = self._gate_up(x[0], x[1], ff) if gated else _pad(x[0].to(torch.bfloat16), ff, self._wp), _pad(x[-1].to(torch.bfloat16), self._wp, ff)
        gut, dnt = (self._tiles(t) if self.tiled else None for t in (gu, dn))
        L.ff_kind, L.router_n = _lib.FF_MOE, _up(n + m.identity, 64)
        L.router, L.router_t = self._mat(m.router, L.router_n, self._wp, tile=True)
        L.moe = _lib.MoeArgs(experts=n, identity=m.identity, top=m.top, groups=m.groups, keep=m.keep,
                             choose=_lib.CHOOSE_LOGITS if m.by_logits else (_lib.CHOOSE_SOFTMAX if m.weight_scale is None else _lib.CHOOSE_SCORES),
                             act_kind=_lib.EXPERT_CLAMPGLU if m.clamp else (_lib.EXPERT_SWIGLU if gated else _lib.EXPERT_RELU2), weight_scale=m.weight_scale or 0.0,
                             glu_limit=m.clamp[0] if m.clamp else 0.0, glu_alpha=m.clamp[1] if m.clamp else 0.0,
                             width_p=self._wp, ff_p=ff, gate_up=self._dev(gu), down=self._dev(dn), gate_up_t=gut, down_t=dnt,
                             correction=None if m.correction is None else self._f32(m.correction))
        if m.shared is not None:
            L.ff = _up(m.shared[0].shape[0], 64)
            if m.shared_clamp:
                L.glu_limit, L.glu_alpha = m.shared_clamp
            L.up, L.up_t = self._mat(self._gate_up(m.shared[0], m.shared[1], L.ff) if m.shared_clamp else m.shared[0], None if m.shared_clamp else L.ff, self._wp, tile=True)
            L.down, L.down_t = self._mat(m.shared[-1], self._wp, L.ff, tile=True)

    def _build(self, sd):
        cfg, lib, dev = self.config, self.lib, self.device
        W, self._wp = cfg.hidden_size, _up(cfg.hidden_size, 64)
        Wp, V, Vp, MB, T = self._wp, cfg.vocab_size, _up(cfg.vocab_size, 64), self.max_batch, self.t_max
        self.vocab_p = Vp
        self._lat_q = self._lat_o = 1
        self.expand_rows = 0 if self.exact else _up(min(self.max_ctx, max(8192, 2 * T)), 64) + 64 * MB
        self._exp = [0] * 5                              # latent, rotated part, keys, values, queries of the expanded form: widest layer
        mixers, arr = [], (_lib.MixLayer * len(cfg.layers))()
        build = {LatentMixer: self._latent_layer, DeltaMixer: self._delta_layer, WindowMixer: self._single_layer, WkvMixer: self._wkv_layer,
                 MlstmMixer: self._mlstm_layer, MinGruMixer: self._single_layer, SelectMixer: self._single_layer, SideBySide: self._side_by_side}
        for i in range(len(cfg.layers)):
            lw, L = self.layer_weights(sd, i), arr[i]
            L.norm1, L.parallel, L.post, L.pre = self._f32(lw.norm1, Wp), int(lw.parallel), int(lw.post), int(lw.pre)
            if lw.depth is not None:
                L.depth = self._f32(lw.depth)
            if lw.norm1b is not None:
                L.norm1b = self._f32(lw.norm1b, Wp)
            build[type(lw.mixer)](L, lw.mixer)
            if lw.ff is not None:
                L.norm2 = self._f32(lw.norm2, Wp)
                {ClampGlu: self._glu, GeluGlu: self._gelu_glu, Experts: self._experts}[type(lw.ff)](L, lw.ff)
            if lw.up is not None:
                L.ff_kind = _lib.FF_RELU2
                L.norm2, L.norm2b, L.ff = self._f32(lw.norm2, Wp), self._f32(lw.norm2b, Wp), _up(lw.up.shape[0], 64)
                L.up, L.up_t = self._mat(lw.up, L.ff, Wp, tile=True)
                L.down, L.down_t = self._mat(lw.down, Wp, L.ff, tile=True)
            mixers.append(lw.mixer)
        mw = self.model_weights(sd)
        f32 = dict(dtype=torch.float32, device=dev)
        # every run's pages / states
        bps = self.max_ctx // self.kv_block_size
        nblk = MB * bps if self._kv_pool_blocks is None else self._kv_pool_blocks
        if nblk < 1 or nblk > MB * bps:
            raise ValueError(f"kv_pool_blocks={nblk} must lie in 1..{MB * bps} (max_batch x max_ctx / kv_block_size)")
        self._kv = BlockPool(nblk, self.kv_block_size, MB, bps)
        self._kv_dynamic = nblk < MB * bps
        cache_dtype = torch.float32 if self.exact else torch.bfloat16
        order = cfg.runs()
        runs = (_lib.MixRun * len(order))()
        self.cache_bytes = self.state_bytes = 0
        join = None
        if mw.get("join") is not None:                   # [x | x0], each half padded
            w = torch.zeros((Wp, 2, Wp), dtype=torch.bfloat16, device=dev)
            w[:W, :, :W] = mw["join"].view(W, 2, W).to(torch.bfloat16)
            join = self._mat(w.view(Wp, 2 * Wp), tile=True)
        for r, (i, opens) in enumerate(order):
            runs[r].layer = i
            if opens is not None and mw.get("steps") is not None:
                runs[r].add = self._f32(mw["steps"][opens], Wp)
            if opens is not None and mw.get("join") is not None:
                runs[r].join, runs[r].join_t = join
            if isinstance(mixers[i], LatentMixer):
                a = arr[i].latent
                t = torch.zeros((nblk, self.kv_block_size, a.rank_p + a.rot_p), dtype=cache_dtype, device=dev)
                runs[r].cache = self._dev(t)
                self.cache_bytes += t.numel() * t.element_size()
            elif arr[i].kind in (_lib.MIX_WINDOW, _lib.MIX_GRU, _lib.MIX_SELECT):
                kinds = (arr[i].kind, arr[i].beside)
                if _lib.MIX_WINDOW in kinds:
                    a = arr[i].window
                    k, v = (torch.zeros((nblk, a.kv_heads, self.kv_block_size, d), dtype=cache_dtype, device=dev) for d in (a.dim_p, a.vdim_p))
                    runs[r].cache, runs[r].vcache = self._dev(k), self._dev(v)
                    self.cache_bytes += (k.numel() + v.numel()) * k.element_size()
                    if a.taps:
                        runs[r].ring = self._state((MB, a.taps, a.conv_ch))
                if _lib.MIX_GRU in kinds:
                    runs[r].gru_state = self._state((MB, _up(arr[i].gru.width, 4)))
                if _lib.MIX_SELECT in kinds:
                    a = arr[i].select
                    runs[r].sel_state, runs[r].sel_ring = self._state((MB, a.inner, _up(a.state, 4))), self._state((MB, a.taps, a.conv_ch))
            elif arr[i].kind == _lib.MIX_RECUR:
                a = arr[i].recur
                mem = [torch.zeros((MB, a.heads, a.dim, _up(a.vdim, 4)), **f32), torch.zeros((MB, Wp), **f32) if arr[i].n_mix else None]
                mem += [torch.zeros((MB, a.heads, a.dim), **f32), torch.zeros((MB, a.heads), **f32)] if a.kind == _lib.RECUR_MLSTM else [None, None]
                runs[r].state, runs[r].ring, runs[r].n_state, runs[r].m_state = [None if t is None else self._dev(t) for t in mem]
                self.state_bytes += sum(4 * t.numel() for t in mem if t is not None)
            else:
                a = arr[i].delta
                s = torch.zeros((MB, a.heads, a.dim, _up(a.vdim, 4)), **f32)
                ring = torch.zeros((MB, a.taps, a.conv_ch), **f32)
                runs[r].state, runs[r].ring = self._dev(s), self._dev(ring)
                self.state_bytes += 4 * (s.numel() + ring.numel())
        head, head_t = self._mat(mw["head"], Vp, Wp, tile=True)
        embed = self._mat(mw["embed"], V, Wp)[0]
        kmax = max([2 * Wp if join else Wp] + [max(L.out_k, L.ff, L.recur.rank) for L in arr])
        deltas, recurs, moes = ([L for L in arr if c(L)] for c in (lambda L: L.kind == _lib.MIX_DELTA, lambda L: L.kind == _lib.MIX_RECUR,
                                                                lambda L: L.ff_kind == _lib.FF_MOE))
        most = lambda f: max([f(L) for L in deltas], default=1)
        over = lambda layers, f: max([f(L) for L in layers], default=1)
        shifts, pairs, n_mix = bool(over(recurs, lambda L: L.n_mix) > 1), T * over(moes, lambda L: L.moe.top), over(arr, lambda L: L.n_mix)
        selects = [L for L in arr if _lib.MIX_SELECT in (L.kind, L.beside)]
        depth = any(L.depth for L in arr)
        mixing = [i for i, _ in order if isinstance(mixers[i], WindowMixer) and mixers[i].vmix is not None]      # value mixing: the first leaves its values
        if mixing:
            if len({mixers[i].kv_heads * mixers[i].vdim for i in mixing}) > 1:
                raise ValueError("layers that mix their values with the first one's must have as many")
            arr[mixing[0]].window.vfirst_write = 1
        ldv = arr[mixing[0]].window.ld_vfirst if mixing else 4
        bigram = mw.get("bigram")
        mc = _lib.MixConfig(width=W, width_p=Wp, n_layers=len(arr), n_runs=len(order), exact=int(self.exact), t_max=T, max_slots=MB, max_ctx=self.max_ctx,
                            expand_rows=self.expand_rows if self._exp[0] else 0,
                            vocab=V, vocab_p=Vp, eps=cfg.rms_norm_eps, block_size=self.kv_block_size, table_stride=bps,
                            norm_groups=getattr(cfg, "norm_groups", 1), embed_scale=mw.get("embed_scale", 1.0),
                            alpha=mw.get("alpha", 1.0), mult=mw.get("mult", 1.0), logit_cap=mw.get("logit_cap", 0.0))
        if bigram:
            mc.bigram_buckets, mc.bigram_prev, mc.bigram_cur = bigram[1:]
        ws = int(lib.chatts_mixdec_workspace(C.byref(mc), arr))
        rows = T + 1                                     # (kernels may read one row past the last)
        bf = dict(dtype=torch.bfloat16, device=dev)
        xr = self.expand_rows if self._exp[0] else 0
        self.buf = B = {
            "x": torch.zeros((rows, Wp), **f32), "y": torch.zeros((rows, Wp), **f32), "proj": torch.zeros((rows, max(L.in_n for L in arr)), **f32),
            "a_f32": torch.zeros((rows, Wp), **f32), "b_f32": torch.zeros((rows, kmax), **f32),
            "a_planes": torch.zeros((2, rows, Wp), **bf), "b_planes": torch.zeros((2, rows, kmax), **bf),
            "q_f32": torch.zeros((rows, self._lat_q) if self.exact else (1, 1), **f32),
            "q_planes": torch.zeros((2, 1, 1) if self.exact else (2, rows, self._lat_q), **bf),
            "o_lat": torch.zeros((rows, self._lat_o), **f32), "partial": torch.zeros(max(64, MB) * 8 * self._lat_o + 65536, **f32),
            "x_q": torch.zeros(rows * self._exp[4] + 16, **bf), "x_c": torch.zeros(xr * self._exp[0] + 16, **bf), "x_kr": torch.zeros(xr * self._exp[1] + 16, **bf),
            "x_k": torch.zeros((2, xr * (self._exp[2] + _lib.EXPAND_PAD) + 16), **bf),
            "x_v": torch.zeros((2, self._exp[3] * (xr + _lib.EXPAND_PAD) + 16), **bf),
            "x_zero": torch.zeros(max(xr, self._exp[3]) * self._exp[0] + 16, **bf),
            "dq": torch.zeros((rows, most(lambda L: L.delta.kv_heads * L.delta.dim)), **f32),
            "dk": torch.zeros((rows, most(lambda L: L.delta.kv_heads * L.delta.dim)), **f32),
            "dv": torch.zeros((rows, most(lambda L: L.delta.heads * L.delta.vdim)), **f32),
            "dg": torch.zeros((rows, max(most(lambda L: L.delta.heads * L.delta.dim), over(recurs, lambda L: L.w2_n))), **f32),
            "dgate": torch.zeros((rows, most(lambda L: L.delta.heads * L.delta.vdim)), **f32), "dbeta": torch.zeros((rows, most(lambda L: L.delta.heads)), **f32),
            "dchunks": torch.zeros(max(most(lambda L: int(lib.chatts_delta_chunk_floats(L.delta.heads, L.delta.dim, T, MB))),
                                       over(recurs, lambda L: int(lib.chatts_recur_chunk_floats(L.recur.heads, L.recur.dim, T, MB)))), **f32),
            "dout": torch.zeros((rows, max(most(lambda L: L.delta.heads * L.delta.vdim), over(recurs, lambda L: L.recur.heads * L.recur.vdim))), **f32),
            "prev_token": torch.zeros(MB, dtype=torch.int64, device=dev), "x0": torch.zeros((rows, Wp) if join else (1, 1), **f32),
            "h": torch.zeros((rows, Wp) if shifts else (1, 1), **f32), "m_f32": torch.zeros((n_mix, rows, Wp) if shifts else (1, 1), **f32),
            "m_planes": torch.zeros((2, n_mix, rows, Wp) if shifts and not self.exact else (2, 1, 1), **bf),
            "n_f32": torch.zeros((rows, Wp), **f32), "n_planes": torch.zeros((2, rows, Wp) if not self.exact else (2, 1, 1), **bf),
            "gates": torch.zeros((rows, 4 * over(recurs, lambda L: L.recur.heads)), **f32), "den": torch.zeros((rows, over(recurs, lambda L: L.recur.heads)), **f32),
            "moe_ids": torch.zeros(pairs, dtype=torch.int32, device=dev), "moe_place": torch.zeros(pairs, dtype=torch.int32, device=dev),
            "moe_order": torch.zeros(pairs, dtype=torch.int32, device=dev),
            "moe_offsets": torch.zeros(over(moes, lambda L: L.moe.experts) + 2, dtype=torch.int32, device=dev),
            "moe_tiles": torch.zeros(4 * over(moes, lambda L: int(lib.chatts_moe_tiles(T, L.moe.top, L.moe.experts))), dtype=torch.int32, device=dev),
            "moe_weight": torch.zeros(pairs, **f32), "moe_kept": torch.zeros(rows, **f32), "moe_logits": torch.zeros((rows, over(moes, lambda L: L.router_n)), **f32),
            "moe_y": torch.zeros((pairs, Wp) if moes else (1, 1), **f32),
            "act_f32": torch.zeros((pairs, over(moes, lambda L: L.moe.ff_p)) if self.exact else (1, 1), **f32),
            "act_planes": torch.zeros((2, pairs, over(moes, lambda L: L.moe.ff_p)) if not self.exact else (2, 1, 1), **bf),
            "vfirst": torch.zeros((rows, ldv) if mixing else (1, 4), **f32),
            "streams": torch.zeros((len(order), rows, Wp) if depth else (1, 1, 4), **f32),
            "sel_u": torch.zeros((rows, over(selects, lambda L: L.sel_k)), **f32), "sel_low": torch.zeros((rows, over(selects, lambda L: L.select.ld_low)), **f32),
            "sel_delta": torch.zeros((rows, over(selects, lambda L: L.sel_dt_n)), **f32),
            "sel_u_planes": torch.zeros((2, 1, 1) if self.exact else (2, rows, over(selects, lambda L: L.sel_k)), **bf),
            "sel_dt_planes": torch.zeros((2, 1, 1) if self.exact else (2, _up(rows, 16), over(selects, lambda L: L.select.rank)), **bf),
            "rows": torch.zeros((rows, 4), dtype=torch.int32, device=dev), "spans": torch.zeros((MB, 5), dtype=torch.int32, device=dev),
            "kv_table": torch.zeros((MB, bps), dtype=torch.int32, device=dev), "ids": torch.zeros(rows, dtype=torch.int64, device=dev),
            "logits_all": torch.zeros((MB, Vp), **f32), "ws": torch.zeros(ws, dtype=torch.uint8, device=dev),
            "pos_all": torch.full((MB,), -1, dtype=torch.int32, device=dev), "step_all": torch.zeros(MB, dtype=torch.int32, device=dev),
            "token_all": torch.zeros(MB, dtype=torch.int64, device=dev), "token_logit_all": torch.zeros(MB, **f32),
            "out_tokens_all": torch.zeros((MB, self.max_ctx + 8), dtype=torch.int64, device=dev),
        }
        B["pos"], B["step"], B["token"], B["out_tokens"] = B["pos_all"][:1], B["step_all"][:1], B["token_all"][:1], B["out_tokens_all"][0]
        P = _lib.ptr
        fine, coarse = (self._dev(t) for t in sinusoid_tables(W, Wp, self.max_ctx, mw["sinusoid"], dev)) if mw.get("sinusoid") else (None, None)
        mb = _lib.MixBuffers(embed=embed, head=head, head_t=head_t, final_norm=self._f32(mw["final_norm"], Wp), x=P(B["x"]), y=P(B["y"]), proj=P(B["proj"]),
                             a_f32=P(B["a_f32"]), b_f32=P(B["b_f32"]), a_hi=P(B["a_planes"][0]), a_lo=P(B["a_planes"][1]), b_hi=P(B["b_planes"][0]),
                             b_lo=P(B["b_planes"][1]), q_f32=P(B["q_f32"]), o_lat=P(B["o_lat"]), partial=P(B["partial"]), q_hi=P(B["q_planes"][0]),
                             q_lo=P(B["q_planes"][1]), partial_elems=B["partial"].numel(), qx=P(B["x_q"]), cbuf=P(B["x_c"]), krbuf=P(B["x_kr"]),
                             kx_hi=P(B["x_k"][0]), kx_lo=P(B["x_k"][1]), vx_hi=P(B["x_v"][0]), vx_lo=P(B["x_v"][1]), zero=P(B["x_zero"]), rows=P(B["rows"]), spans=P(B["spans"]), table=P(B["kv_table"]),
                             logits=P(B["logits_all"]), workspace=P(B["ws"]), workspace_bytes=ws,
                             bigram=self._mat(bigram[0], None, Wp)[0] if bigram else None, x0=P(B["x0"]) if join else None, mix_stride=rows * Wp, vfirst=P(B["vfirst"]), ld_vfirst=ldv,
                             pos_fine=fine, pos_coarse=coarse, streams=P(B["streams"]) if depth else None, stream_stride=rows * Wp,
                             **{f"{n}_{h}": P(B[f"{n}_planes"][j]) for n in ("m", "n", "act", "sel_u", "sel_dt") for j, h in enumerate(("hi", "lo"))},
                             **{n: P(B[n]) for n in ("dq", "dk", "dv", "dg", "dgate", "dbeta", "dchunks", "dout", "prev_token", "h", "m_f32", "n_f32", "gates", "den",
                                                     "moe_ids", "moe_place", "moe_order", "moe_offsets", "moe_tiles", "moe_weight", "moe_kept", "moe_logits", "moe_y",
                                                     "act_f32", "sel_u", "sel_low", "sel_delta")})
        h = lib.chatts_mixdec_create(C.byref(mc), arr, runs, C.byref(mb))
        if not h:
            raise _lib.ChattsError(-1, lib.chatts_last_error().decode())
        self._decoder, self._layer_arr, self._mix_config = C.c_void_p(h), arr, mc
        if not self._kv_dynamic:
            for s in range(MB):
                self._kv.reserve(s, self.max_ctx)
                self._kv.retire(s)
                self._push_kv_row(s)

    def __del__(self):
        try:
            if self._decoder:
                self.lib.chatts_mixdec_destroy(self._decoder)
        except Exception:
            pass

    # ---- the step ------------------------------------------------------------------------------------------------------------
    def _forward(self, ids, segs):
        """ids: all tokens of the batch; segs: (first row, tokens, first position, slot), slots distinct"""
        B, T = self.buf, len(ids)
        if T > self.t_max:
            raise ValueError(f"{T} tokens exceed max_prefill_tokens={self.t_max}")
        self.check_ids(ids)
        B["ids"][:T].copy_(torch.tensor(ids, dtype=torch.int64))
        meta = torch.empty((T, 4), dtype=torch.int32)
        for row, t, pos0, slot in segs:
            r = torch.arange(t, dtype=torch.int32)
            meta[row:row + t, 0], meta[row:row + t, 1], meta[row:row + t, 2], meta[row:row + t, 3] = slot, pos0 + r, row, t - 1 - r
        B["rows"][:T].copy_(meta)
        single = all(s[1] == 1 for s in segs)
        spans = (_lib.Span * len(segs))(*[_lib.Span(r, t, p, s, -1) for r, t, p, s in segs])
        if not single:
            _lib.check(self.lib.chatts_mixdec_plan(self._decoder, spans, len(segs)))
            B["spans"][:len(segs)].copy_(torch.frombuffer(spans, dtype=torch.int32).view(-1, 5))
        _lib.check(self.lib.chatts_mixdec_forward(self._decoder, _lib.ptr(B["ids"]), T, spans, len(segs), int(single), _lib.stream_ptr()))

    def _logits(self, index):
        """logits of rows `index` of the last forward -> [n, vocab_p] float32"""
        out = torch.empty((len(index), self.vocab_p), dtype=torch.float32, device=self.device)
        idx = torch.tensor(index, dtype=torch.int32, device=self.device)
        for a in range(0, len(index), 256):
            n = min(256, len(index) - a, self.t_max)
            _lib.check(self.lib.chatts_mixdec_logits(self._decoder, idx[a:].data_ptr(), n, out[a:].data_ptr(), _lib.stream_ptr()))
        return out

    def _run_segments(self, ids, segs, index):
        self._forward(ids, segs)
        return self._logits(index)[:, :self.config.vocab_size] if index else None

    def _select(self, logits, slot, n, sampling, pos):
        """tokens of rows slot .. slot + n from `logits` [n, vocab_p]: appended to out_tokens, step (and position, when pos) advanced"""
        B, lib, st, V = self.buf, self.lib, _lib.stream_ptr(), self.config.vocab_size
        out, stride = B["out_tokens_all"][slot:].data_ptr(), B["out_tokens_all"].shape[1]
        at = lambda k: B[k][slot:].data_ptr()
        posp, limit = (at("pos_all"), self.max_ctx - 1) if pos else (None, 0)
        if sampling is None:
            _lib.check(lib.chatts_argmax_batched_ws(logits.data_ptr(), n, self.vocab_p, V, 0, at("token_all"), at("token_logit_all"), out, stride, at("step_all"),
                                                    posp, limit, B["ws"].data_ptr(), B["ws"].numel(), st))
        else:
            _lib.check(lib.chatts_sample_batched(logits.data_ptr(), n, self.vocab_p, V, 0, C.byref(sampling), at("token_all"), at("token_logit_all"), out, stride,
                                                 at("step_all"), posp, limit, st))

    def _batched_step_eager(self):
        B = self.buf
        _lib.check(self.lib.chatts_mixdec_decode(self._decoder, self.max_batch, _lib.ptr(B["token_all"]), _lib.ptr(B["pos_all"]), _lib.ptr(B["logits_all"]),
                                                 _lib.stream_ptr()))
        self._select(B["logits_all"], 0, self.max_batch, getattr(self, "_sampling", None), True)

    def decode_step(self):
        self.batched_step()

    def _install_sampling(self, args):
        pass                                             # (_select reads self._sampling when the step is enqueued or captured)

    # ---- admission -----------------------------------------------------------------------------------------------------------
    def request_tokens(self, ids, series=None, lengths=None):
        return len(ids)

    def check_ids(self, ids):
        if not len(ids):
            raise ValueError("an empty prompt")
        if min(ids) < 0 or max(ids) >= self.config.vocab_size:
            raise ValueError(f"token ids must lie in 0..{self.config.vocab_size - 1}")

    def _request_idents(self, ids, series, lengths):
        return None

    def admit_begin(self, slot, ids, series=None, lengths=None, max_new_tokens=1):
        if series is not None and len(series):
            raise ValueError(f"{self.config.name} takes token ids only, no time series")
        ids = [int(t) for t in ids]
        self.check_ids(ids)
        T = len(ids)
        if T + max_new_tokens > self.max_ctx:
            raise ValueError(f"prompt ({T}) + max_new_tokens ({max_new_tokens}) exceeds max_ctx={self.max_ctx}")
        self.reserve_kv(slot, T + max_new_tokens)
        self.prefix_stats["requests"] += 1
        self.prefix_stats["tokens_prefilled"] += T
        return {"slot": slot, "ids": ids, "T": T, "done": 0}

    def admit_step(self, st, max_rows=None):
        slot, T, a = st["slot"], st["T"], st["done"]
        end = T if max_rows is None else min(T, a + max(int(max_rows), 1))
        while a < end:
            n = min(self.t_max, end - a)
            self._forward(st["ids"][a:a + n], [(0, n, a, slot)])
            a += n
        st["done"] = a
        if a < T:
            return False
        self._first_token(slot, n - 1, T)
        return True

    def _first_token(self, slot, row, T):
        B = self.buf
        lg = self._logits([row])
        B["pos_all"][slot] = T
        B["step_all"][slot] = 0
        sa = getattr(self, "_sampling", None)
        if getattr(self, "_sampling_key", None) == "rows":
            sa = self._rows_args(slot)
        elif sa is not None:                             # (a later step draws with (seed, slot, step): fold the slot into this one's seed)
            sa = _lib.SamplingArgs(temperature=sa.temperature, top_k=sa.top_k, top_p=sa.top_p, seed=(sa.seed ^ (0x51ED27 * (slot + 1))) & 0xFFFFFFFF,
                                   n_kept=None, kept_mass=None)
        self._select(lg, slot, 1, sa, False)

    def _admit_packed(self, items):
        """several prompts in one ragged pass (plan_pack has checked that they fit t_max)"""
        states = []
        try:
            for it in items:
                states.append(self.admit_begin(*it))
        except Exception:
            for st in states:                            # nothing ran yet: others may take these reservations
                self._kv.retire(st["slot"])
            raise
        ids, segs = [], []
        for st in states:
            segs.append((len(ids), st["T"], 0, st["slot"]))
            ids += st["ids"]
        self._forward(ids, segs)
        self.prefix_stats["packed_prefills"] = self.prefix_stats.get("packed_prefills", 0) + 1
        for row, t, _, slot in segs:
            self._first_token(slot, row + t - 1, t)
        return [st["T"] for st in states]

    def _prefill_request(self, ids, series, lengths, max_new_tokens):
        return self._admit(0, ids, series, lengths, max_new_tokens)

    # ---- call surface --------------------------------------------------------------------------------------------------------
    @torch.no_grad()
    def generate(self, input_ids=None, attention_mask=None, max_new_tokens=64, max_length=None, eos_token_id=None, do_sample=False, temperature=None,
                 top_k=None, top_p=None, seed=0, **kw):
        """like the other models' generate(): LongTensor [B, T_in + new], rows right-padded with pad_token_id"""
        if do_sample:
            self.set_sampling(1.0 if temperature is None else temperature, 50 if top_k is None else top_k, 1.0 if top_p is None else top_p, seed)
        else:
            self.set_sampling(0.0)
        ids = input_ids if isinstance(input_ids, torch.Tensor) else torch.tensor(input_ids)
        ids = (ids[None] if ids.dim() == 1 else ids).cpu()
        mask = attention_mask.cpu() if attention_mask is not None else torch.ones_like(ids)
        reqs = [(ids[b][mask[b].bool()].tolist(), None, None) for b in range(ids.shape[0])]
        budget = max_new_tokens if max_length is None else max(1, max_length - max(len(r[0]) for r in reqs))
        outs = self.generate_batch(reqs, budget, self.config.eos_token_id if eos_token_id is None else eos_token_id)
        rows = [ids[b].tolist() + outs[b] for b in range(ids.shape[0])]
        n = max(len(r) for r in rows)
        return torch.tensor([r + [self.config.pad_token_id] * (n - len(r)) for r in rows], dtype=torch.long)
