"""Small Muvetar configurations of the tests: sizes that divide nothing evenly, sizes that fill tiles, and the optional branches."""
import copy


def _gru(width):
    return {"type": "mingru", "mixer": {"width": width}}


def _par(heads, kv_heads, dim, vdim, scale, inner, state, dt_rank, conv, scales):
    return {"type": "parallel", "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale},
                                          "right": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv},
                                          "left_scale": scales[0], "right_scale": scales[1]}}


def _moe(layer, ff, limit, experts, top, scale, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        mlp["shared"] = {"ff": shared[0], "limit": shared[1]}
    return dict(layer, mlp=mlp)


CONFIGS = {
    # uneven sizes; heads and states that no quad fits; five taps, one tap; a layer without a feed-forward; one expert chosen; limits of their own
    "odd": {"vocab": 130, "width": 90, "norm": {"eps": 3e-5}, "residual_mult": 0.7, "logit_softcap": 9.0,
            "layers": [_moe(_par(6, 2, 21, 18, 0.3, 50, 5, 7, 5, (0.6, 1.3)), 40, 1.1, 6, 3, 2.5, (70, 0.6)), _moe(_gru(75), 33, 2.0, 5, 1, 0.8),
                       dict(_gru(130), mlp=None), _moe(_par(3, 3, 42, 9, 0.2, 91, 19, 70, 1, (1.0, 0.4)), 20, 0.9, 7, 2, 1.0, (17, 3.0))]},
    # every expert chosen, one key head for many queries, one state per channel, factors of one, the recurrence first
    "plain": {"vocab": 96, "width": 128, "norm": {"eps": 1e-6}, "residual_mult": 1.0, "logit_softcap": 40.0,
              "layers": [_moe(_gru(128), 64, 7.0, 4, 4, 1.0, (64, 7.0)), _moe(_par(20, 1, 32, 32, 0.25, 128, 1, 8, 2, (1.0, 1.0)), 64, 7.0, 4, 4, 1.0)]},
    # larger heads and states, more layers than streams are requested at once, wider than a workgroup of the norms
    "wide": {"vocab": 200, "width": 1100, "norm": {"eps": 1e-5}, "residual_mult": 0.3, "logit_softcap": 25.0,
             "layers": [_moe(_par(6, 3, 136, 200, 0.1, 160, 40, 30, 4, (0.9, 0.5)), 96, 1.5, 12, 4, 1.7, (32, 1.0)), dict(_gru(2048), mlp=None),
                        _moe(_gru(68), 128, 3.0, 8, 2, 1.3, (256, 2.0)), dict(_par(2, 2, 64, 64, 0.15, 64, 128, 16, 3, (0.5, 0.8)), mlp=None), dict(_gru(40), mlp=None),
                        dict(_par(5, 5, 48, 120, 0.2, 200, 200, 65, 4, (0.4, 1.0)), mlp=None)]},
}


def model(name, seed=0, all_experts=False):
    """(configuration, config.json dictionary, weights); all_experts: every expert is chosen, so that no rounding changes a choice"""
    from oracle import muvetar as F
    cfg = copy.deepcopy(CONFIGS[name])
    for l in cfg["layers"]:
        if all_experts and l.get("mlp"):
            l["mlp"]["router"]["top"] = l["mlp"]["router"]["experts"]
    return cfg, dict(copy.deepcopy(cfg), architecture="Muvetar"), F.random_model(cfg, seed)
