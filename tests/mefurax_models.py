"""Small Mefurax configurations of the tests: sizes that divide nothing evenly, sizes that fill tiles, and the optional branches."""
import copy


def _conv(heads, kv_heads, dim, vdim, scale, conv, size=0, v_mix=False):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "conv": conv, "v_mix": v_mix}
    if size:
        m["mask"] = {"size": size}
    return {"type": "attention", "mixer": m}


def _rot(heads, kv_heads, dim, vdim, scale, softcap, base, dims, size=0, v_mix=False):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap, "rot": {"base": base, "dims": dims}, "v_mix": v_mix}
    if size:
        m["mask"] = {"size": size}
    return {"type": "attention_2", "mixer": m}


def _dense(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff} if ff else None)


def _moe(layer, ff, experts, top, shared=0):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared}
    return dict(layer, mlp=mlp)


CONFIGS = {
    # uneven sizes; heads that no quad of channels fits; five taps; masks shorter than a page, none; a layer without a feed-forward; one expert chosen
    "odd": {"vocab": 130, "width": 90, "norm": {"eps": 3e-5}, "postln_alpha": 1.7,
            "layers": [_moe(_conv(6, 2, 21, 18, 0.3, 3, 30, True), 40, 6, 3, 70), _dense(_rot(4, 4, 24, 9, 0.4, 3.0, 1000.0, 10, 17, True), 70),
                       _dense(_rot(3, 1, 42, 22, 0.2, 9.0, 50.0, 42), 0), _moe(_conv(4, 4, 12, 9, 0.25, 5, 0, True), 33, 5, 1)]},
    # every expert chosen, one tap, one key head for many queries, a chunk that is a page, no mixed values
    "plain": {"vocab": 96, "width": 128, "norm": {"eps": 1e-6}, "postln_alpha": 1.0,
              "layers": [_moe(_rot(20, 1, 32, 32, 0.25, 20.0, 10000.0, 16, 64), 64, 4, 4, 64), _dense(_conv(4, 1, 32, 32, 0.2, 1, 64), 192)]},
    # larger heads, windows and chunks of several pages, values mixed from a layer with chunks, the first layer of all without
    "wide": {"vocab": 200, "width": 192, "norm": {"eps": 1e-5}, "postln_alpha": 4.0,
             "layers": [_dense(_conv(2, 2, 64, 64, 0.15, 4, 100), 64), _moe(_rot(6, 3, 136, 200, 0.3, 30.0, 500000.0, 60, 150, True), 96, 12, 4, 32),
                        _moe(_conv(6, 3, 136, 200, 0.1, 2, 65, True), 128, 8, 2, 256), _dense(_rot(5, 5, 48, 120, 0.3, 5.0, 100.0, 48, 1, True), 256)]},
}


def model(name, seed=0, all_experts=False):
    """(configuration, config.json dictionary, weights); all_experts: every expert is chosen, so that no rounding changes a choice"""
    from oracle import mefurax as F
    cfg = copy.deepcopy(CONFIGS[name])
    for l in cfg["layers"]:
        if all_experts and (l.get("mlp") or {}).get("kind") == "moe":
            l["mlp"]["router"]["top"] = l["mlp"]["router"]["experts"]
    return cfg, dict(copy.deepcopy(cfg), architecture="Mefurax"), F.random_model(cfg, seed)
