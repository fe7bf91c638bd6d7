"""Medilix: a small decoder-only design whose layers read two norms of the same x in parallel - a mixer (wkv time mixing, mLSTM matrix memory, or windowed
attention with kept first tokens and a sink) beside a clamped gated feed-forward or a mixture of experts - with a row per token pair in the
embedding and a range of layers that runs several times, joined to the embedding at each pass.

This file is the design's configuration and its tensor names; everything that runs is MixedDecoder (chatts_amd/mixed.py).
"""
import copy
import json
import os

from .mixed import ClampGlu, Experts, LayerWeights, MixedDecoder, MlstmMixer, WindowMixer, WkvMixer

GLU_ALPHA = 1.702
SHIFTS = ("r", "k", "v", "g", "w")
MIXER_KEYS = {"wkv": ("heads", "dim"), "mlstm": ("heads", "dim", "vdim", "gate_cap"), "attention": ("heads", "kv_heads", "dim", "vdim", "scale")}


def _need(d, keys, where):
    missing = [k for k in keys if k not in d]
    if missing:
        raise ValueError(f"config.json: {where} lacks {missing}")


def _only(d, keys, where):
    extra = sorted(set(d) - set(keys))
    if extra:
        raise ValueError(f"config.json: {where} has the unknown entries {extra}")


class MedilixConfig:
    architecture = "Medilix"

    def __init__(self, vocab, width, layers, norm, embedding=None, loop=None, architecture="Medilix", name="medilix", **extra):
        if architecture != "Medilix":
            raise ValueError(f"architecture {architecture!r} is not Medilix")
        self.vocab_size, self.hidden_size = int(vocab), int(width)
        self.layers, self.norm, self.loop, self.embedding = copy.deepcopy(layers), copy.deepcopy(norm), copy.deepcopy(loop), copy.deepcopy(embedding or {})
        _need(self.norm, ("eps",), "norm")
        self.rms_norm_eps, self.norm_groups = float(norm["eps"]), int(norm.get("groups", 1))
        self.name, self.extra = name, extra
        eos = extra.get("eos_token_id", [])                  # (the design itself has no special tokens)
        self.eos_token_id = list(eos) if isinstance(eos, (list, tuple)) else [int(eos)]
        self.pad_token_id = int(extra.get("pad_token_id", 0))
        self.num_hidden_layers = len(self.layers)
        if self.norm_groups < 1 or self.hidden_size % self.norm_groups:
            raise ValueError(f"config.json: a width of {width} does not split into {self.norm_groups} groups")
        _only(self.embedding, ("scale", "bigram"), "embedding")
        if self.embedding.get("bigram"):
            _need(self.embedding["bigram"], ("buckets", "mul_prev", "mul_cur"), "embedding.bigram")
        for i, l in enumerate(self.layers):
            self._check_layer(i, l)
        if self.loop:
            _need(self.loop, ("start", "stop", "times"), "loop")
            if not (0 <= self.loop["start"] < self.loop["stop"] <= len(self.layers) and self.loop["times"] >= 1):
                raise ValueError(f"config.json: loop {self.loop} does not fit {len(self.layers)} layers")

    @staticmethod
    def _check_layer(i, l):
        _need(l, ("type", "mixer"), f"layer {i}")
        if l["type"] not in MIXER_KEYS:
            raise ValueError(f"config.json: layer {i} has the unknown mixer {l['type']!r}")
        m = l["mixer"]
        _need(m, MIXER_KEYS[l["type"]], f"mixer of layer {i}")
        _only(m, MIXER_KEYS[l["type"]] + (("mask",) if l["type"] == "attention" else ()), f"mixer of layer {i}")
        if l["type"] == "attention":
            if m["heads"] % m["kv_heads"]:
                raise ValueError(f"config.json: layer {i} shares {m['kv_heads']} key / value heads among {m['heads']}")
            if m.get("mask"):
                _need(m["mask"], ("size",), f"mask of layer {i}")
                _only(m["mask"], ("size", "keep_first"), f"mask of layer {i}")
        mlp = l.get("mlp")
        if not mlp:
            return
        kind = mlp.get("kind", "dense")
        if kind == "dense":
            _need(mlp, ("ff", "limit"), f"mlp of layer {i}")
        elif kind == "moe":
            _need(mlp, ("expert", "router"), f"mlp of layer {i}")
            r = mlp["router"]
            _need(mlp["expert"], ("ff",), f"expert of layer {i}")
            _need(r, ("experts", "top"), f"router of layer {i}")
            _only(r, ("experts", "top", "identity", "groups"), f"router of layer {i}")
            n, g = r["experts"] + r.get("identity", 0), r.get("groups") or {"count": 1, "keep": 1}
            _need(g, ("count", "keep"), f"router.groups of layer {i}")
            if n % g["count"] or not 1 <= g["keep"] <= g["count"] or r["top"] > n // g["count"] * g["keep"]:
                raise ValueError(f"config.json: layer {i} chooses {r['top']} of {n} outputs in {g['keep']} of {g['count']} groups")
        else:
            raise ValueError(f"config.json: layer {i} has the unknown feed-forward {kind!r}")

    def to_dict(self):
        return dict(copy.deepcopy(self.extra), architecture="Medilix", vocab=self.vocab_size, width=self.hidden_size, layers=copy.deepcopy(self.layers),
                    norm=copy.deepcopy(self.norm), embedding=copy.deepcopy(self.embedding), loop=copy.deepcopy(self.loop))

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

    def tensor_shapes(self, rank=None, *_):
        """name -> shape of every tensor of a checkpoint (rank: low-rank size of the wkv decays, which only the tensors themselves tell; None
        leaves it out of the shapes)"""
        W, V = self.hidden_size, self.vocab_size
        s = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
        if self.embedding.get("bigram"):
            s["bigram"] = (self.embedding["bigram"]["buckets"] + 1, W)
        if self.loop:
            s["loop.in"] = (W, 2 * W)
        for i, l in enumerate(self.layers):
            p, m = f"l{i}.", l["mixer"]
            q, H, D = p + "mix.", m["heads"], m["dim"]
            s[p + "norm1"] = (W,)
            if l["type"] == "wkv":
                s.update({q + "mu." + n: (W,) for n in SHIFTS})
                s.update({q + n: (H * D, W) for n in "rkvg"})
                s.update({q + "w1": (rank, W), q + "w2": (H * D, rank), q + "w0": (H * D,), q + "u": (H, D), q + "norm": (H * D,), q + "o": (W, H * D)})
            elif l["type"] == "mlstm":
                v = H * m["vdim"]
                s.update({q + "q": (H * D, W), q + "k": (H * D, W), q + "v": (v, W), q + "g": (v, W), q + "i": (H, W), q + "f": (H, W), q + "i.b": (H,),
                          q + "f.b": (H,), q + "norm": (v,), q + "o": (W, v)})
            else:
                G, v = m["kv_heads"], H * m["vdim"]
                s.update({q + "q": (H * D, W), q + "k": (G * D, W), q + "v": (G * m["vdim"], W), q + "g": (v, W), q + "q.norm": (D,), q + "k.norm": (D,),
                          q + "o": (W, v)})
            mlp, q = l.get("mlp"), p + "mlp."
            if not mlp:
                continue
            s[p + "norm2"] = (W,)
            if mlp.get("kind", "dense") == "dense":
                s.update({q + "gate": (mlp["ff"], W), q + "up": (mlp["ff"], W), q + "down": (W, mlp["ff"])})
            else:
                r, ff = mlp["router"], mlp["expert"]["ff"]
                n = r["experts"] + r.get("identity", 0)
                s.update({q + "router": (n, W), q + "correction": (n,)})
                for e in range(r["experts"]):
                    s.update({f"{q}e{e}.gate": (ff, W), f"{q}e{e}.up": (ff, W), f"{q}e{e}.down": (W, ff)})
        return s


class MedilixForCausalLM(MixedDecoder):
    def layer_weights(self, sd, i):
        """tensors of layer i -> what MixedDecoder builds from"""
        p, l = f"l{i}.", self.config.layers[i]
        m, mlp, t = l["mixer"], l.get("mlp"), lambda n: sd[p + n]
        if l["type"] == "wkv":
            mixer = WkvMixer(heads=m["heads"], dim=m["dim"], mu=[t("mix.mu." + n) for n in SHIFTS], r=t("mix.r"), k=t("mix.k"), v=t("mix.v"), g=t("mix.g"),
                             w1=t("mix.w1"), w2=t("mix.w2"), w0=t("mix.w0"), u=t("mix.u"), norm=t("mix.norm"), o=t("mix.o"))
        elif l["type"] == "mlstm":
            mixer = MlstmMixer(heads=m["heads"], dim=m["dim"], vdim=m["vdim"], cap=float(m["gate_cap"]), q=t("mix.q"), k=t("mix.k"), v=t("mix.v"), g=t("mix.g"),
                               i=t("mix.i"), f=t("mix.f"), bias_i=t("mix.i.b"), bias_f=t("mix.f.b"), norm=t("mix.norm"), o=t("mix.o"))
        else:
            mask = m.get("mask") or {}
            mixer = WindowMixer(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]), window=int(mask.get("size", 0)),
                                keep_first=int(mask.get("keep_first", 0)), sink=True, q=t("mix.q"), k=t("mix.k"), v=t("mix.v"), g=t("mix.g"),
                                q_norm=t("mix.q.norm"), k_norm=t("mix.k.norm"), o=t("mix.o"))
        ff = None
        if mlp and mlp.get("kind", "dense") == "dense":
            ff = ClampGlu(gate=t("mlp.gate"), up=t("mlp.up"), down=t("mlp.down"), limit=float(mlp["limit"]), alpha=GLU_ALPHA)
        elif mlp:
            r = mlp["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            ff = Experts(router=t("mlp.router"), correction=t("mlp.correction"), experts=[[t(f"mlp.e{e}.{n}") for n in ("gate", "up", "down")] for e in range(r["experts"])],
                         identity=r.get("identity", 0), top=r["top"], groups=g["count"], keep=g["keep"])
        return LayerWeights(mixer=mixer, norm1=t("norm1"), norm2=t("norm2") if mlp else None, ff=ff, parallel=True)

    def model_weights(self, sd):
        b = self.config.embedding.get("bigram")
        return dict(embed=sd["embed"], head=sd["head"], final_norm=sd["final.norm"], embed_scale=float(self.config.embedding.get("scale", 1.0)), join=sd.get("loop.in"),
                    bigram=(sd["bigram"], b["buckets"], b["mul_prev"], b["mul_cur"]) if b else None)
