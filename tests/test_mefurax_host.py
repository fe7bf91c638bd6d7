"""Mefurax without a GPU: configuration reader, registry, tensor shapes, the reference's own consistency."""
import json
import math

import numpy as np
import pytest
import torch

from chatts_amd import registry
from chatts_amd.mefurax import MefuraxConfig
from oracle import mefurax as F
from tests.mefurax_models import CONFIGS, model


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_config_round_trip_and_registry(name, tmp_path):
    _, public, _ = model(name)
    c = MefuraxConfig.from_dict(public)
    assert c.runs() == [(i, None) for i in range(len(public["layers"]))]
    c.save_pretrained(str(tmp_path))
    again = registry.load_config(str(tmp_path))
    assert isinstance(again, MefuraxConfig) and again.to_dict() == c.to_dict()
    assert registry.model_class(again).__name__ == "MefuraxForCausalLM"


def test_config_reads_every_value_and_refuses_what_it_does_not_know():
    _, public, _ = model("odd")
    c = MefuraxConfig.from_dict(public)
    assert (c.vocab_size, c.hidden_size, c.rms_norm_eps, c.postln_alpha, c.eos_token_id) == (130, 90, 3e-5, 1.7, [])

    def broken(change):
        bad = json.loads(json.dumps(public))
        change(bad)
        with pytest.raises(ValueError):
            MefuraxConfig.from_dict(bad)
    broken(lambda d: d["layers"][0].update(type="conv"))
    broken(lambda d: d["layers"][0]["mlp"].update(kind="sparse"))
    broken(lambda d: d["layers"][0]["mixer"].pop("conv"))
    broken(lambda d: d["layers"][0]["mixer"].update(conv=0))
    broken(lambda d: d["layers"][0]["mixer"].update(softcap=4.0))
    broken(lambda d: d["layers"][0]["mixer"].update(kv_heads=4))
    broken(lambda d: d["layers"][0]["mixer"]["mask"].update(keep_first=2))
    broken(lambda d: d["layers"][0]["mixer"]["mask"].update(size=0))
    broken(lambda d: d["layers"][0]["mixer"].update(vdim=17))
    broken(lambda d: d["layers"][1]["mixer"]["rot"].update(dims=26))
    broken(lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7))
    broken(lambda d: d["layers"][1]["mixer"]["rot"].update(scaling={}))
    broken(lambda d: d["layers"][1]["mixer"].pop("softcap"))
    broken(lambda d: d["layers"][0]["mlp"]["router"].update(top=7))
    broken(lambda d: d["layers"][0]["mlp"]["router"].update(groups=2))
    broken(lambda d: d["norm"].pop("eps"))
    broken(lambda d: d.update(architecture="Medilix"))
    broken(lambda d: d.update(layers=[]))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_tensor_shapes_cover_the_model(name):
    _, public, sd = model(name)
    shapes = MefuraxConfig.from_dict(public).tensor_shapes()
    assert set(shapes) == set(sd)
    for n, s in shapes.items():
        assert tuple(s) == tuple(sd[n].shape), n


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_reference_is_causal(name):
    cfg, _, sd = model(name)
    toks = np.random.default_rng(0).integers(0, cfg["vocab"], 20).tolist()
    full, streams = F.forward(cfg, sd, toks, want_layers=True)
    assert len(streams) == len(cfg["layers"])
    assert torch.allclose(F.forward(cfg, sd, toks[:11]), full[:11])


def test_reference_mechanisms():
    """properties that single out the equations' readings"""
    g = torch.Generator().manual_seed(1)
    u, w = torch.randn(6, 4, generator=g, dtype=torch.float64), torch.randn(4, 3, generator=g, dtype=torch.float64)
    y = F.causal_conv(u, w)
    assert torch.allclose(y[0], w[:, 2] * u[0]) and torch.allclose(y[4], w[:, 0] * u[2] + w[:, 1] * u[3] + w[:, 2] * u[4])
    x = torch.randn(7, 2, 10, generator=g, dtype=torch.float64)
    r = F.rotate_pairs(x, 100.0, 6)
    assert torch.equal(r[0], x[0]) and torch.equal(r[:, :, 6:], x[:, :, 6:])
    pairs = lambda t: t[:, :, :6].reshape(7, 2, 3, 2).norm(dim=-1)
    assert torch.allclose(pairs(r), pairs(x))
    same = x[:1].expand(7, 2, 10)                     # of equal vectors the product depends on the distance alone
    t = F.rotate_pairs(same, 100.0, 6)
    assert torch.allclose((t[5] * t[2]).sum(-1), (t[3] * t[0]).sum(-1)) and not torch.allclose((t[5] * t[2]).sum(-1), (t[5] * t[5]).sum(-1))
    assert F.slopes(4) == [0.25, 0.0625, 2.0 ** -6, 2.0 ** -8]
    assert [j for j in range(12) if F.in_window(9, j, 4)] == [6, 7, 8, 9] and [j for j in range(12) if F.in_chunk(9, j, 4)] == [8, 9]
    assert [j for j in range(12) if F.in_chunk(3, j, None)] == [0, 1, 2, 3]
    idx, wt = F.route(torch.tensor([[1.0, 3.0, 2.0, -5.0]]), 2)
    assert idx.tolist() == [[1, 2]] and math.isclose(float(wt[0, 0]), 1 / (1 + math.exp(-1)), rel_tol=1e-6)
    shared, p = {}, "l0.mix."
    a = F.values(u, {p + "vmix": torch.tensor(0.25)}, p, {"v_mix": True}, shared)
    b = F.values(2 * u, {p + "vmix": torch.tensor(0.25)}, p, {"v_mix": True}, shared)
    c = F.values(3 * u, {}, p, {}, shared)
    assert torch.equal(a, u) and torch.allclose(b, 1.75 * u) and torch.equal(c, 3 * u)
    z = torch.linspace(-6, 6, 25, dtype=torch.float64)
    assert torch.allclose(F.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert torch.allclose(F.shifted_norm(z, torch.zeros(25, dtype=torch.float64), 0.0).pow(2).mean(), torch.tensor(1.0, dtype=torch.float64))
