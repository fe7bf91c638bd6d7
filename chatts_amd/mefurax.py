"""Mefurax: a small decoder-only design whose norms stand after the sums (x <- norm(alpha x + sublayer(x)), weights stored around zero).  Two kinds of
attention: one with short convolutions on queries, keys and values, norms over the whole projections, a distance bias and a sliding window; one with
rotated pairs, unit queries and keys, capped scores, chunks and a gate per head.  Layers may mix their values with the first such layer's.  Feed-forwards: a
gated one (tanh gelu), or experts (squared relu, chosen by logits) with a shared one.

This file is the design's configuration and its tensor names; everything that runs is MixedDecoder (chatts_amd/mixed.py).
"""
import copy
import json
import os

from .mixed import Experts, GeluGlu, LayerWeights, MixedDecoder, WindowMixer

MIXER_KEYS = {"attention": ("heads", "kv_heads", "dim", "vdim", "scale", "conv"), "attention_2": ("heads", "kv_heads", "dim", "vdim", "scale", "rot", "softcap")}
OPTIONAL_KEYS = ("mask", "v_mix")


def _need(d, keys, where):
    missing = [k for k in keys if k not in d]
    if missing:
        raise ValueError(f"config.json: {where} lacks {missing}")


def _only(d, keys, where):
    extra = sorted(set(d) - set(keys))
    if extra:
        raise ValueError(f"config.json: {where} has the unknown entries {extra}")


class MefuraxConfig:
    architecture = "Mefurax"

    def __init__(self, vocab, width, layers, norm, postln_alpha, architecture="Mefurax", name="mefurax", **extra):
        if architecture != "Mefurax":
            raise ValueError(f"architecture {architecture!r} is not Mefurax")
        self.vocab_size, self.hidden_size = int(vocab), int(width)
        self.layers, self.norm, self.postln_alpha = copy.deepcopy(layers), copy.deepcopy(norm), float(postln_alpha)
        _need(self.norm, ("eps",), "norm")
        self.rms_norm_eps = float(norm["eps"])
        self.name, self.extra = name, extra
        eos = extra.get("eos_token_id", [])                  # (the design itself has no special tokens)
        self.eos_token_id = list(eos) if isinstance(eos, (list, tuple)) else [int(eos)]
        self.pad_token_id = int(extra.get("pad_token_id", 0))
        self.num_hidden_layers = len(self.layers)
        if not self.layers:
            raise ValueError("config.json: no layers")
        for i, l in enumerate(self.layers):
            self._check_layer(i, l)
        sizes = {l["mixer"]["kv_heads"] * l["mixer"]["vdim"] for l in self.layers if l["mixer"].get("v_mix")}
        if len(sizes) > 1:
            raise ValueError(f"config.json: layers that mix their values have {sorted(sizes)} of them")

    @staticmethod
    def _check_layer(i, l):
        _need(l, ("type", "mixer"), f"layer {i}")
        if l["type"] not in MIXER_KEYS:
            raise ValueError(f"config.json: layer {i} has the unknown mixer {l['type']!r}")
        m = l["mixer"]
        _need(m, MIXER_KEYS[l["type"]], f"mixer of layer {i}")
        _only(m, MIXER_KEYS[l["type"]] + OPTIONAL_KEYS, f"mixer of layer {i}")
        if m["heads"] % m["kv_heads"]:
            raise ValueError(f"config.json: layer {i} shares {m['kv_heads']} key / value heads among {m['heads']}")
        if m.get("mask"):
            _need(m["mask"], ("size",), f"mask of layer {i}")
            _only(m["mask"], ("size",), f"mask of layer {i}")
            if m["mask"]["size"] < 1:
                raise ValueError(f"config.json: layer {i} sees {m['mask']['size']} positions")
        if l["type"] == "attention":
            if m["conv"] < 1:
                raise ValueError(f"config.json: layer {i} has convolutions over {m['conv']} tokens")
        else:
            _need(m["rot"], ("base", "dims"), f"rot of layer {i}")
            _only(m["rot"], ("base", "dims"), f"rot of layer {i}")
            if m["rot"]["dims"] % 2 or m["rot"]["dims"] > m["dim"]:
                raise ValueError(f"config.json: layer {i} rotates {m['rot']['dims']} of {m['dim']} dimensions")
            if m["softcap"] <= 0:
                raise ValueError(f"config.json: layer {i} caps its scores at {m['softcap']}")
        mlp = l.get("mlp")
        if not mlp:
            return
        kind = mlp.get("kind", "dense")
        if kind == "dense":
            _need(mlp, ("ff",), f"mlp of layer {i}")
        elif kind == "moe":
            _need(mlp, ("expert", "router"), f"mlp of layer {i}")
            _need(mlp["expert"], ("ff",), f"expert of layer {i}")
            _need(mlp["router"], ("experts", "top"), f"router of layer {i}")
            _only(mlp["router"], ("experts", "top"), f"router of layer {i}")
            if not 1 <= mlp["router"]["top"] <= mlp["router"]["experts"]:
                raise ValueError(f"config.json: layer {i} chooses {mlp['router']['top']} of {mlp['router']['experts']} experts")
            if mlp.get("shared"):
                _need(mlp["shared"], ("ff",), f"shared expert of layer {i}")
        else:
            raise ValueError(f"config.json: layer {i} has the unknown feed-forward {kind!r}")

    def to_dict(self):
        return dict(copy.deepcopy(self.extra), architecture="Mefurax", vocab=self.vocab_size, width=self.hidden_size, layers=copy.deepcopy(self.layers),
                    norm=copy.deepcopy(self.norm), postln_alpha=self.postln_alpha)

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
            q, H, G = p + "mix.", m["heads"], m["kv_heads"]
            rows = {"q": H * m["dim"], "k": G * m["dim"], "v": G * m["vdim"]}
            s[p + "norm1"] = (W,)
            s.update({q + n: (r, W) for n, r in rows.items()})
            s[q + "o"] = (W, H * m["vdim"])
            if m.get("v_mix"):
                s[q + "vmix"] = ()
            if l["type"] == "attention":
                s.update({f"{q}{n}.b": (r,) for n, r in rows.items()})
                s.update({f"{q}{n}.conv": (r, m["conv"]) for n, r in rows.items()})
                s.update({q + "q.norm": (rows["q"],), q + "k.norm": (rows["k"],)})
            else:
                s[q + "g"] = (H, W)
            mlp, q = l.get("mlp"), p + "mlp."
            if not mlp:
                continue
            s[p + "norm2"] = (W,)
            if mlp.get("kind", "dense") == "dense":
                s.update({q + "gate": (mlp["ff"], W), q + "up": (mlp["ff"], W), q + "down": (W, mlp["ff"])})
                continue
            s[q + "router"] = (mlp["router"]["experts"], W)
            for e in range(mlp["router"]["experts"]):
                s.update({f"{q}e{e}.up": (mlp["expert"]["ff"], W), f"{q}e{e}.down": (W, mlp["expert"]["ff"])})
            if mlp.get("shared"):
                s.update({q + "shared.up": (mlp["shared"]["ff"], W), q + "shared.down": (W, mlp["shared"]["ff"])})
        return s


class MefuraxForCausalLM(MixedDecoder):
    def layer_weights(self, sd, i):
        """tensors of layer i -> what MixedDecoder builds from"""
        p, l = f"l{i}.", self.config.layers[i]
        m, mlp, t = l["mixer"], l.get("mlp"), lambda n: sd[p + n]
        size = int((m.get("mask") or {}).get("size", 0))
        kw = dict(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]), keep_first=0, sink=False, q=t("mix.q"), k=t("mix.k"),
                  v=t("mix.v"), o=t("mix.o"), vmix=float(t("mix.vmix")) if m.get("v_mix") else None)
        if l["type"] == "attention":
            mixer = WindowMixer(window=size, g=None, q_norm=t("mix.q.norm"), k_norm=t("mix.k.norm"), norm_whole=True, bias=[t(f"mix.{n}.b") for n in "qkv"],
                                conv=[t(f"mix.{n}.conv") for n in "qkv"], slopes=[2.0 ** (-8.0 * (h + 1) / m["heads"]) for h in range(m["heads"])], **kw)
        else:
            mixer = WindowMixer(window=0, chunk=size, g=t("mix.g"), gate_heads=True, q_norm=None, k_norm=None, rot=m["rot"]["dims"], rot_base=float(m["rot"]["base"]),
                                unit=True, softcap=float(m["softcap"]), **kw)
        ff = None
        if mlp and mlp.get("kind", "dense") == "dense":
            ff = GeluGlu(gate=t("mlp.gate"), up=t("mlp.up"), down=t("mlp.down"))
        elif mlp:
            r = mlp["router"]
            ff = Experts(router=t("mlp.router"), correction=None, experts=[[t(f"mlp.e{e}.{n}") for n in ("up", "down")] for e in range(r["experts"])], identity=0,
                         top=r["top"], groups=1, keep=1, by_logits=True, shared=[t("mlp.shared.up"), t("mlp.shared.down")] if mlp.get("shared") else None)
        return LayerWeights(mixer=mixer, norm1=1.0 + t("norm1").float(), norm2=1.0 + t("norm2").float() if mlp else None, ff=ff, post=True)

    def model_weights(self, sd):
        return dict(embed=sd["embed"], head=sd["head"], final_norm=1.0 + sd["final.norm"].float(), alpha=self.config.postln_alpha)
