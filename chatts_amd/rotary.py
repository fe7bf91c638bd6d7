"""Rotary position tables with optional YaRN scaling, and sinusoidal position vectors (constants as parameters)."""
import math

import torch


def yarn_frequencies(dims, base, factor, original, fast, slow):
    """float64 angular frequencies of the dims / 2 pairs.  Pairs that turn more than `fast` times within the `original` context keep their
    frequency, those below `slow` turns are slowed down by `factor`, the ones between are blended linearly over the pair index."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.exp(i * (-2.0 / dims * math.log(base)))
    index_at = lambda turns: dims * math.log(original / (turns * 2.0 * math.pi)) / (2.0 * math.log(base))
    first = max(math.floor(index_at(fast)), 0)
    last = min(math.ceil(index_at(slow)), dims - 1)
    blend = torch.clamp((i - first) / max(last - first, 0.001), 0.0, 1.0)
    return f * (1.0 - blend) + f / factor * blend


def rotary_tables(dims, base, n, scaling=None, device=None):
    """float32 cos / sin [n, dims / 2] of positions 0 .. n - 1, rotate-half layout (dimension i pairs with i + dims / 2).  scaling: None, or
    YaRN's {factor, original, fast, slow}; both tables then carry its magnitude 0.1 ln(factor) + 1."""
    if scaling:
        f = yarn_frequencies(dims, base, scaling["factor"], scaling["original"], scaling["fast"], scaling["slow"])
        mag = 0.1 * math.log(scaling["factor"]) + 1.0
    else:
        f, mag = torch.exp(torch.arange(dims // 2, dtype=torch.float64) * (-2.0 / dims * math.log(base))), 1.0
    a = torch.arange(n, dtype=torch.float64)[:, None] * f[None, :]
    return (a.cos() * mag).float().contiguous().to(device), (a.sin() * mag).float().contiguous().to(device)


def sinusoid_tables(width, width_p, n, base, device=None):
    """float32 tables [64, width_p] of positions 0 .. 63 and [n / 64, width_p] of positions 0, 64, 128, ...: columns 2 i and 2 i + 1 hold sine and cosine of
    position * base^(-2 i / width).  A position's vector is the sum of the angles of one row of each."""
    f = torch.exp(torch.arange((width + 1) // 2, dtype=torch.float64) * (-2.0 / width * math.log(base)))

    def table(pos):
        a = torch.tensor(pos, dtype=torch.float64)[:, None] * f[None, :]
        t = torch.zeros((len(pos), width_p), dtype=torch.float32)
        pairs = torch.stack([a.sin(), a.cos()], -1).view(len(pos), -1).float()
        t[:, :pairs.shape[1]] = pairs
        return t.to(device)
    return table(list(range(64))), table(list(range(0, max(n, 1), 64)))
