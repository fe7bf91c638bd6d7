"""Small Medilix configurations of the tests: sizes that divide nothing evenly, sizes that fill tiles, and the optional branches."""
import copy


def _wkv(heads, dim, rank):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim, "_rank": rank}}


def _mlstm(heads, dim, vdim, cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def _attention(heads, kv_heads, dim, vdim, scale, size=0, keep_first=0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size:
        m["mask"] = {"size": size, "keep_first": keep_first}
    return {"type": "attention", "mixer": m}


def _dense(layer, ff, limit):
    return dict(layer, mlp={"kind": "dense", "ff": ff, "limit": limit} if ff else None)


def _moe(layer, ff, experts, top, identity=0, count=0, keep=0):
    r = {"experts": experts, "top": top}
    if identity:
        r["identity"] = identity
    if count:
        r["groups"] = {"count": count, "keep": keep}
    return dict(layer, mlp={"kind": "moe", "expert": {"ff": ff}, "router": r})


CONFIGS = {
    # uneven sizes, groups that split no quad of columns evenly, a loop over the middle, a layer without a feed-forward
    "odd": {"vocab": 130, "width": 90, "norm": {"eps": 3e-5, "groups": 3}, "embedding": {"scale": 3.0, "bigram": {"buckets": 37, "mul_prev": 5, "mul_cur": 11}},
            "loop": {"start": 1, "stop": 3, "times": 2},
            "layers": [_dense(_mlstm(3, 20, 37, 6.0), 70, 1.5), _moe(_wkv(3, 22, 12), 40, 6, 3, 2, 4, 2), _dense(_attention(6, 2, 24, 42, 0.3, 30, 5), 0, 0),
                       _moe(_attention(4, 4, 40, 18, 0.2, 7), 33, 5, 2, 1)]},
    # no loop, no pairs, one group, no window, experts without groups or identity outputs, one choice
    "plain": {"vocab": 96, "width": 128, "norm": {"eps": 1e-6, "groups": 1}, "embedding": {}, "loop": None,
              "layers": [_moe(_attention(20, 1, 32, 32, 0.2), 64, 4, 1), _dense(_wkv(2, 64, 64), 192, 7.0), _dense(_mlstm(2, 64, 64, 15.0), 128, 0.5)]},
    # the whole stack looped, larger heads, a window of several pages, more first tokens kept than a page holds
    "wide": {"vocab": 200, "width": 192, "norm": {"eps": 1e-5, "groups": 6}, "embedding": {"scale": 0.5, "bigram": {"buckets": 64, "mul_prev": 1, "mul_cur": 1}},
             "loop": {"start": 0, "stop": 3, "times": 2},
             "layers": [_moe(_mlstm(2, 136, 96, 3.0), 96, 12, 4, 4, 2, 1), _dense(_wkv(1, 160, 20), 256, 2.0), _dense(_attention(6, 3, 136, 200, 0.1, 65, 70), 64, 3.0)]},
}


def model(name, seed=0):
    """(configuration with the low-rank hints, config.json dictionary, weights)"""
    from oracle import medilix as F
    cfg = copy.deepcopy(CONFIGS[name])
    sd = F.random_model(cfg, seed)
    public = copy.deepcopy(cfg)
    public["architecture"] = "Medilix"
    for l in public["layers"]:
        l["mixer"] = {k: v for k, v in l["mixer"].items() if not k.startswith("_")}
    return cfg, public, sd
