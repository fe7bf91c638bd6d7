"""Fobolix: a small decoder-only design of mixed layers - latent attention (YaRN rotary part) and the gated delta rule with channel decays,
squared-relu feed-forwards, norms before and after every sublayer, and a range of layers that runs several times per token.

This file is the design's configuration and its tensor names; everything that runs is MixedDecoder (chatts_amd/mixed.py).
"""
import copy
import json
import os

from .mixed import DeltaMixer, LatentMixer, LayerWeights, MixedDecoder


def _need(d, keys, where):
    missing = [k for k in keys if k not in d]
    if missing:
        raise ValueError(f"config.json: {where} lacks {missing}")


class FobolixConfig:
    architecture = "Fobolix"

    def __init__(self, vocab, width, layers, norm, loop=None, architecture="Fobolix", name="fobolix", **extra):
        if architecture != "Fobolix":
            raise ValueError(f"architecture {architecture!r} is not Fobolix")
        self.vocab_size, self.hidden_size = int(vocab), int(width)
        self.layers, self.norm, self.loop = copy.deepcopy(layers), copy.deepcopy(norm), copy.deepcopy(loop)
        self.rms_norm_eps = float(norm["eps"])
        self.name, self.extra = name, extra
        eos = extra.get("eos_token_id", [])                  # (the design itself has no special tokens)
        self.eos_token_id = list(eos) if isinstance(eos, (list, tuple)) else [int(eos)]
        self.pad_token_id = int(extra.get("pad_token_id", 0))
        self.num_hidden_layers = len(self.layers)
        for i, l in enumerate(self.layers):
            _need(l, ("type", "mixer"), f"layer {i}")
            if l["type"] == "latent_attention":
                _need(l["mixer"], ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot"), f"mixer of layer {i}")
                rot = l["mixer"]["rot"]
                _need(rot, ("base", "dims"), f"rot of layer {i}")
                if rot["dims"] != l["mixer"]["rot_dim"]:
                    raise ValueError(f"config.json: layer {i} rotates {rot['dims']} of {l['mixer']['rot_dim']} dimensions")
                if rot.get("scaling"):
                    _need(rot["scaling"], ("factor", "original", "fast", "slow"), f"rot.scaling of layer {i}")
            elif l["type"] == "channel_delta":
                _need(l["mixer"], ("heads", "kv_heads", "dim", "vdim", "conv"), f"mixer of layer {i}")
            else:
                raise ValueError(f"config.json: layer {i} has the unknown mixer {l['type']!r}")
            if l.get("mlp") and l["mlp"].get("kind", "dense") != "dense":
                raise ValueError(f"config.json: layer {i} has the unknown feed-forward {l['mlp']['kind']!r}")
        if self.loop:
            _need(self.loop, ("start", "stop", "times"), "loop")
            if not (0 <= self.loop["start"] < self.loop["stop"] <= len(self.layers) and self.loop["times"] >= 1):
                raise ValueError(f"config.json: loop {self.loop} does not fit {len(self.layers)} layers")

    def to_dict(self):
        return dict(copy.deepcopy(self.extra), architecture="Fobolix", vocab=self.vocab_size, width=self.hidden_size, layers=copy.deepcopy(self.layers),
                    norm=copy.deepcopy(self.norm), loop=copy.deepcopy(self.loop))

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
        """layer runs in order: (layer, number of the pass that this run opens, or None)"""
        n = len(self.layers)
        if not self.loop:
            return [(i, None) for i in range(n)]
        a, b = self.loop["start"], self.loop["stop"]
        passes = [(i, t if i == a else None) for t in range(self.loop["times"]) for i in range(a, b)]
        return [(i, None) for i in range(a)] + passes + [(i, None) for i in range(b, n)]

    def tensor_shapes(self, rank_a=None, rank_g=None):
        """name -> shape of every tensor of a checkpoint (rank_a / rank_g: low-rank sizes of the delta mixers, which only the tensors
        themselves tell; None leaves them out of the shapes)"""
        W, V = self.hidden_size, self.vocab_size
        s = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
        if self.loop:
            s["loop.step"] = (self.loop["times"], W)
        for i, l in enumerate(self.layers):
            p, m = f"l{i}.", l["mixer"]
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l.get("mlp") else ()):
                s[p + n] = (W,)
            if l["type"] == "latent_attention":
                H, R = m["heads"], m["kv_rank"]
                s.update({p + "mix.q": (H * (m["dim"] + m["rot_dim"]), W), p + "mix.dkv": (R + m["rot_dim"], W), p + "mix.dkv.norm": (R,),
                          p + "mix.uk": (H * m["dim"], R), p + "mix.uv": (H * m["vdim"], R), p + "mix.o": (W, H * m["vdim"])})
            else:
                H, qk, v = m["heads"], m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
                for n, rows in (("q", qk), ("k", qk), ("v", v)):
                    s[p + "mix." + n] = (rows, W)
                    s[p + "mix." + n + ".conv"] = (rows, m["conv"])
                s.update({p + "mix.b": (H, W), p + "mix.A_log": (H,), p + "mix.norm": (m["vdim"],), p + "mix.dt_bias": (H * m["dim"],),
                          p + "mix.a1": (rank_a, W), p + "mix.a2": (H * m["dim"], rank_a), p + "mix.g1": (rank_g, W),
                          p + "mix.g2": (v, rank_g), p + "mix.o": (W, v)})
            if l.get("mlp"):
                s[p + "mlp.up"], s[p + "mlp.down"] = (l["mlp"]["ff"], W), (W, l["mlp"]["ff"])
        return s


class FobolixForCausalLM(MixedDecoder):
    def layer_weights(self, sd, i):
        """tensors of layer i -> what MixedDecoder builds from"""
        p, l = f"l{i}.", self.config.layers[i]
        m, t = l["mixer"], lambda n: sd[p + n]
        if l["type"] == "latent_attention":
            mixer = LatentMixer(heads=m["heads"], dim=m["dim"], rot=m["rot_dim"], vdim=m["vdim"], rank=m["kv_rank"], scale=float(m["scale"]),
                                rot_base=float(m["rot"]["base"]), rot_scaling=m["rot"].get("scaling"), q=t("mix.q"), dkv=t("mix.dkv"),
                                c_norm=t("mix.dkv.norm"), uk=t("mix.uk"), uv=t("mix.uv"), o=t("mix.o"))
        else:
            mixer = DeltaMixer(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], taps=m["conv"], q=t("mix.q"), k=t("mix.k"),
                               v=t("mix.v"), q_conv=t("mix.q.conv"), k_conv=t("mix.k.conv"), v_conv=t("mix.v.conv"), b=t("mix.b"), a_log=t("mix.A_log"),
                               a1=t("mix.a1"), a2=t("mix.a2"), dt_bias=t("mix.dt_bias"), g1=t("mix.g1"), g2=t("mix.g2"), norm=t("mix.norm"), o=t("mix.o"))
        ff = bool(l.get("mlp"))
        return LayerWeights(mixer=mixer, norm1=t("norm1"), norm1b=t("norm1b"), norm2=t("norm2") if ff else None, norm2b=t("norm2b") if ff else None,
                            up=t("mlp.up") if ff else None, down=t("mlp.down") if ff else None)

    def model_weights(self, sd):
        return dict(embed=sd["embed"], head=sd["head"], final_norm=sd["final.norm"], steps=sd.get("loop.step"))
