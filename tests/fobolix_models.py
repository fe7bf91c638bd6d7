"""Small Fobolix configurations of the tests: sizes that divide nothing evenly, sizes that fill tiles, and the optional branches."""
import copy


def _latent(heads, dim, rot, vdim, rank, scale, base=10000.0, scaling=None):
    r = {"base": base, "dims": rot}
    if scaling:
        r["scaling"] = scaling
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale, "rot": r}}


def _delta(heads, kv_heads, dim, vdim, conv, rank_a, rank_g):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "_rank_a": rank_a, "_rank_g": rank_g}}


def _ff(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff} if ff else None)


YARN = {"factor": 5.0, "original": 48, "fast": 16.0, "slow": 1.5}

CONFIGS = {
    # grouped delta heads, uneven sizes, a loop over the middle, a layer without a feed-forward
    "odd": {"vocab": 130, "width": 90, "norm": {"eps": 3e-5}, "loop": {"start": 1, "stop": 3, "times": 3},
            "layers": [_ff(_delta(6, 2, 20, 36, 4, 12, 21), 70), _ff(_latent(3, 24, 10, 40, 50, 0.19, 5000.0, YARN), 0), _ff(_delta(4, 4, 33, 17, 2, 9, 8), 111),
                       _ff(_latent(5, 18, 8, 22, 36, 0.2), 64)]},
    # no loop, one tap, two head tiles, plain rotary
    "plain": {"vocab": 96, "width": 128, "norm": {"eps": 1e-6}, "loop": None,
              "layers": [_ff(_latent(20, 32, 32, 32, 160, 0.125), 192), _ff(_delta(8, 4, 16, 16, 1, 16, 16), 192)]},
    # the whole stack looped, attention first, larger heads
    "wide": {"vocab": 200, "width": 192, "norm": {"eps": 1e-5}, "loop": {"start": 0, "stop": 2, "times": 2},
             "layers": [_ff(_latent(4, 48, 16, 72, 96, 0.125, 1e6, YARN), 256), _ff(_delta(3, 1, 72, 96, 3, 32, 40), 256)]},
}


def model(name, seed=0, sharp=True):
    """(configuration with the low-rank hints, config.json dictionary, weights).  sharp: larger query weights, so that attention picks a few
    keys out of many instead of averaging them"""
    from oracle import fobolix as F
    cfg = copy.deepcopy(CONFIGS[name])
    sd = F.random_model(cfg, seed)
    if sharp:
        for k in sd:
            if k.endswith("mix.q") and k.replace("mix.q", "mix.dkv") in sd:
                sd[k] = sd[k] * 2
    public = copy.deepcopy(cfg)
    public["architecture"] = "Fobolix"
    for l in public["layers"]:
        l["mixer"] = {k: v for k, v in l["mixer"].items() if not k.startswith("_")}
    return cfg, public, sd
