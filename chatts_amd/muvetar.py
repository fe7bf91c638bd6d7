"""Muvetar: a small decoder-only design with norms before its sublayers, a factor on what they add, sinusoidal positions, and weighted averages over the streams of
all earlier layers after each.  Mixers: a minimal gated recurrence, or attention with a logarithmic distance bias beside a selective scan.  Feed-forwards: clamped
gated experts, weighted by their softmax scores as they are, beside a shared one.  The logits are capped.

This file is the design's configuration and its tensor names; everything that runs is MixedDecoder (chatts_amd/mixed.py).
"""
import copy
import json
import os

from .mixed import Experts, LayerWeights, MinGruMixer, MixedDecoder, SelectMixer, SideBySide, WindowMixer

GLU_ALPHA = 1.702
POSITION_BASE = 10000.0
MIXER_KEYS = {"mingru": ("width",), "parallel": ("left", "right", "left_scale", "right_scale")}
LEFT_KEYS, RIGHT_KEYS = ("heads", "kv_heads", "dim", "vdim", "scale"), ("inner", "state", "dt_rank", "conv")


def _exactly(d, keys, where, optional=()):
    missing, extra = [k for k in keys if k not in d], sorted(set(d) - set(keys) - set(optional))
    if missing:
        raise ValueError(f"config.json: {where} lacks {missing}")
    if extra:
        raise ValueError(f"config.json: {where} has the unknown entries {extra}")


def _positive(d, keys, where):
    for k in keys:
        if int(d[k]) < 1:
            raise ValueError(f"config.json: {where} has {k} = {d[k]}")


class MuvetarConfig:
    architecture = "Muvetar"

    def __init__(self, vocab, width, layers, norm, residual_mult, logit_softcap, architecture="Muvetar", name="muvetar", **extra):
        if architecture != "Muvetar":
            raise ValueError(f"architecture {architecture!r} is not Muvetar")
        self.vocab_size, self.hidden_size = int(vocab), int(width)
        self.layers, self.norm = copy.deepcopy(layers), copy.deepcopy(norm)
        self.residual_mult, self.logit_softcap = float(residual_mult), float(logit_softcap)
        _exactly(self.norm, ("eps",), "norm")
        self.rms_norm_eps = float(norm["eps"])
        self.name, self.extra = name, extra
        eos = extra.get("eos_token_id", [])                  # (the design itself has no special tokens)
        self.eos_token_id = list(eos) if isinstance(eos, (list, tuple)) else [int(eos)]
        self.pad_token_id = int(extra.get("pad_token_id", 0))
        self.num_hidden_layers = len(self.layers)
        if not self.layers:
            raise ValueError("config.json: no layers")
        if self.logit_softcap <= 0:
            raise ValueError(f"config.json: logits are capped at {logit_softcap}")
        for i, l in enumerate(self.layers):
            self._check_layer(i, l)

    @staticmethod
    def _check_layer(i, l):
        _exactly(l, ("type", "mixer"), f"layer {i}", ("mlp",))
        if l["type"] not in MIXER_KEYS:
            raise ValueError(f"config.json: layer {i} has the unknown mixer {l['type']!r}")
        m, where = l["mixer"], f"mixer of layer {i}"
        _exactly(m, MIXER_KEYS[l["type"]], where)
        if l["type"] == "mingru":
            _positive(m, ("width",), where)
        else:
            _exactly(m["left"], LEFT_KEYS, f"left {where}")
            _exactly(m["right"], RIGHT_KEYS, f"right {where}")
            _positive(m["left"], ("heads", "kv_heads", "dim", "vdim"), f"left {where}")
            _positive(m["right"], RIGHT_KEYS, f"right {where}")
            if m["left"]["heads"] % m["left"]["kv_heads"]:
                raise ValueError(f"config.json: layer {i} shares {m['left']['kv_heads']} key / value heads among {m['left']['heads']}")
        mlp = l.get("mlp")
        if not mlp:
            return
        where = f"mlp of layer {i}"
        _exactly(mlp, ("kind", "expert", "router"), where, ("shared",))
        if mlp["kind"] != "moe":
            raise ValueError(f"config.json: layer {i} has the unknown feed-forward {mlp['kind']!r}")
        _exactly(mlp["router"], ("experts", "top", "scale"), f"router of layer {i}")
        if not 1 <= mlp["router"]["top"] <= mlp["router"]["experts"]:
            raise ValueError(f"config.json: layer {i} chooses {mlp['router']['top']} of {mlp['router']['experts']} experts")
        for n in ("expert", "shared"):
            if mlp.get(n):
                _exactly(mlp[n], ("ff", "limit"), f"{n} of layer {i}")
                _positive(mlp[n], ("ff",), f"{n} of layer {i}")

    def to_dict(self):
        return dict(copy.deepcopy(self.extra), architecture="Muvetar", vocab=self.vocab_size, width=self.hidden_size, layers=copy.deepcopy(self.layers),
                    norm=copy.deepcopy(self.norm), residual_mult=self.residual_mult, logit_softcap=self.logit_softcap)

    @classmethod
    def from_dict(cls, d):
        return cls(**copy.deepcopy(d))

    @classmethod
    def from_pretrained(cls, path):
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f))

    def save_pretrained(self, path):
        os.makedirs(path, exist_ok=True)
        with open(os.path.join(path, "config.json"), "w") as f:
            json.dump(self.to_dict(), f, indent=1)

    def runs(self):
        """layer runs in order: every layer once"""
        return [(i, None) for i in range(len(self.layers))]

    def tensor_shapes(self, *_):
        """name -> shape of every tensor of a checkpoint"""
        W, V = self.hidden_size, self.vocab_size
        s = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
        for i, l in enumerate(self.layers):
            p, m = f"l{i}.", l["mixer"]
            q = p + "mix."
            s.update({p + "norm1": (W,), p + "dwa": (i + 2,)})
            if l["type"] == "mingru":
                C = m["width"]
                s.update({q + "z": (C, W), q + "z.b": (C,), q + "x": (C, W), q + "x.b": (C,), q + "g": (C, W), q + "o": (W, C)})
            else:
                a, b = m["left"], m["right"]
                H, G, C, N, R = a["heads"], a["kv_heads"], b["inner"], b["state"], b["dt_rank"]
                s.update({q + "left.q": (H * a["dim"], W), q + "left.k": (G * a["dim"], W), q + "left.v": (G * a["vdim"], W), q + "left.r1": (H,), q + "left.r2": (H,),
                          q + "left.o": (W, H * a["vdim"])})
                s.update({q + "right.in": (2 * C, W), q + "right.conv": (C, b["conv"]), q + "right.conv.b": (C,), q + "right.x": (R + 2 * N, C), q + "right.dt": (C, R),
                          q + "right.dt.b": (C,), q + "right.A_log": (C, N), q + "right.D": (C,), q + "right.o": (W, C)})
            mlp, q = l.get("mlp"), p + "mlp."
            if not mlp:
                continue
            s.update({p + "norm2": (W,), q + "router": (mlp["router"]["experts"], W)})
            units = [(f"e{e}", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])] + ([("shared", mlp["shared"]["ff"])] if mlp.get("shared") else [])
            for n, ff in units:
                s.update({f"{q}{n}.gate": (ff, W), f"{q}{n}.up": (ff, W), f"{q}{n}.down": (W, ff)})
        return s


class MuvetarForCausalLM(MixedDecoder):
    def layer_weights(self, sd, i):
        """tensors of layer i -> what MixedDecoder builds from"""
        p, l = f"l{i}.", self.config.layers[i]
        m, mlp, t = l["mixer"], l.get("mlp"), lambda n: sd[p + n]
        if l["type"] == "mingru":
            mixer = MinGruMixer(z=t("mix.z"), x=t("mix.x"), g=t("mix.g"), bias_z=t("mix.z.b"), bias_x=t("mix.x.b"), o=t("mix.o"))
        else:
            a, b, left, right = m["left"], m["right"], lambda n: t("mix.left." + n), lambda n: t("mix.right." + n)
            mixer = SideBySide(
                left=WindowMixer(heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], scale=float(a["scale"]), window=0, keep_first=0, sink=False,
                                 q=left("q"), k=left("k"), v=left("v"), g=None, q_norm=None, k_norm=None, o=left("o"), log_bias=(left("r1"), left("r2"))),
                right=SelectMixer(state=b["state"], rank=b["dt_rank"], w_in=right("in"), conv=right("conv"), conv_bias=right("conv.b"), x=right("x"), dt=right("dt"),
                                  dt_bias=right("dt.b"), a_log=right("A_log"), d=right("D"), o=right("o")),
                left_scale=float(m["left_scale"]), right_scale=float(m["right_scale"]))
        ff = None
        if mlp:
            r, unit = mlp["router"], lambda n: [t(f"mlp.{n}.{x}") for x in ("gate", "up", "down")]
            shared = mlp.get("shared")
            ff = Experts(router=t("mlp.router"), correction=None, experts=[unit(f"e{e}") for e in range(r["experts"])], identity=0, top=r["top"], groups=1, keep=1,
                         weight_scale=float(r["scale"]), clamp=(float(mlp["expert"]["limit"]), GLU_ALPHA), shared=unit("shared") if shared else None,
                         shared_clamp=(float(shared["limit"]), GLU_ALPHA) if shared else None)
        return LayerWeights(mixer=mixer, norm1=t("norm1"), norm2=t("norm2") if mlp else None, ff=ff, pre=True, depth=t("dwa"))

    def model_weights(self, sd):
        return dict(embed=sd["embed"], head=sd["head"], final_norm=sd["final.norm"], mult=self.config.residual_mult, logit_cap=self.config.logit_softcap,
                    sinusoid=POSITION_BASE)
