"""Muvetar without a GPU: configuration reader, registry, tensor shapes, position tables, the reference's own consistency."""
import json
import math

import numpy as np
import pytest
import torch

from chatts_amd import registry
from chatts_amd.muvetar import MuvetarConfig
from chatts_amd.rotary import sinusoid_tables
from oracle import muvetar as F
from tests.muvetar_models import CONFIGS, model


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_config_round_trip_and_registry(name, tmp_path):
    _, public, _ = model(name)
    c = MuvetarConfig.from_dict(public)
    assert c.runs() == [(i, None) for i in range(len(public["layers"]))]
    c.save_pretrained(str(tmp_path))
    again = registry.load_config(str(tmp_path))
    assert isinstance(again, MuvetarConfig) and again.to_dict() == c.to_dict()
    assert registry.model_class(again).__name__ == "MuvetarForCausalLM"


def test_config_reads_every_value_and_refuses_what_it_does_not_know():
    _, public, _ = model("odd")
    c = MuvetarConfig.from_dict(public)
    assert (c.vocab_size, c.hidden_size, c.rms_norm_eps, c.residual_mult, c.logit_softcap, c.eos_token_id) == (130, 90, 3e-5, 0.7, 9.0, [])

    def broken(change):
        bad = json.loads(json.dumps(public))
        change(bad)
        with pytest.raises(ValueError):
            MuvetarConfig.from_dict(bad)
    broken(lambda d: d["layers"][0].update(type="attention"))
    broken(lambda d: d["layers"][0].update(norm="post"))
    broken(lambda d: d["layers"][0]["mixer"].pop("left_scale"))
    broken(lambda d: d["layers"][0]["mixer"]["left"].update(mask={"size": 8}))
    broken(lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=4))
    broken(lambda d: d["layers"][0]["mixer"]["left"].pop("scale"))
    broken(lambda d: d["layers"][0]["mixer"]["right"].update(conv=0))
    broken(lambda d: d["layers"][0]["mixer"]["right"].update(heads=2))
    broken(lambda d: d["layers"][0]["mixer"]["right"].pop("state"))
    broken(lambda d: d["layers"][1]["mixer"].update(width=0))
    broken(lambda d: d["layers"][1]["mixer"].update(heads=1))
    broken(lambda d: d["layers"][0]["mlp"].update(kind="dense"))
    broken(lambda d: d["layers"][0]["mlp"]["router"].update(top=7))
    broken(lambda d: d["layers"][0]["mlp"]["router"].pop("scale"))
    broken(lambda d: d["layers"][0]["mlp"]["expert"].pop("limit"))
    broken(lambda d: d["layers"][0]["mlp"]["shared"].update(alpha=1.0))
    broken(lambda d: d["norm"].update(groups=2))
    broken(lambda d: d.pop("norm") and d.update(norm={}))
    broken(lambda d: d.update(logit_softcap=0.0))
    broken(lambda d: d.update(architecture="Mefurax"))
    broken(lambda d: d.update(layers=[]))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_tensor_shapes_cover_the_model(name):
    _, public, sd = model(name)
    shapes = MuvetarConfig.from_dict(public).tensor_shapes()
    assert set(shapes) == set(sd)
    for n, s in shapes.items():
        assert tuple(s) == tuple(sd[n].shape), n


@pytest.mark.parametrize("width,width_p", [(64, 64), (90, 128), (7, 64)])
def test_position_tables_add_up(width, width_p):
    """sine and cosine of the sum of a fine and a coarse angle, far beyond where a float32 product would still hold them"""
    fine, coarse = sinusoid_tables(width, width_p, 200000, 10000.0)
    want = F.sinusoid([0, 1, 63, 64, 65, 4095, 199999], width)
    for row, p in zip(want, [0, 1, 63, 64, 65, 4095, 199999]):
        a, b = fine[p % 64].view(-1, 2), coarse[p // 64].view(-1, 2)
        got = torch.stack([a[:, 0] * b[:, 1] + a[:, 1] * b[:, 0], a[:, 1] * b[:, 1] - a[:, 0] * b[:, 0]], -1).view(-1)[:width]
        assert float((got.double() - row).abs().max()) < 3e-7


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
    d64 = dict(generator=g, dtype=torch.float64)
    p = F.sinusoid([0, 3], 6)
    assert p[0].tolist() == [0, 1, 0, 1, 0, 1] and math.isclose(float(p[1, 2]), math.sin(3 * 10000 ** (-2 / 6))) and math.isclose(float(p[1, 5]), math.cos(3 * 10000 ** (-4 / 6)))
    assert F.candidate(torch.tensor([0.0, 2.0, -1.0])).tolist() == pytest.approx([0.5, 2.5, 1 / (1 + math.e)])
    assert F.gru_step(torch.tensor(2.0), torch.tensor(0.25), torch.tensor(4.0)).item() == 2.5
    b = F.distance_bias(torch.tensor([2.0, 0.5]), torch.tensor([1.0, 3.0]), torch.tensor([0.0, 1.0]))
    assert torch.allclose(b, torch.tensor([[0.0, 2 * math.log(2)], [0.0, 0.5 * math.log(4)]]))
    u, w = torch.randn(6, 4, **d64), torch.randn(4, 3, **d64)
    y = F.causal_conv(u, w, torch.ones(4, dtype=torch.float64))
    assert torch.allclose(y[0], 1 + w[:, 2] * u[0]) and torch.allclose(y[4], 1 + w[:, 0] * u[2] + w[:, 1] * u[3] + w[:, 2] * u[4])
    S = F.scan_step(torch.full((1, 2), 2.0), torch.tensor([0.5]), torch.tensor([[-1.0, -2.0]]), torch.tensor([1.0, 3.0]), torch.tensor([4.0]))
    assert torch.allclose(S, torch.tensor([[2 * math.exp(-0.5) + 2, 2 * math.exp(-1) + 6]]))
    z = torch.linspace(-30, 30, 25, dtype=torch.float64)
    assert torch.allclose(F.softplus(z), torch.nn.functional.softplus(z), rtol=1e-6) and torch.allclose(F.silu(z), torch.nn.functional.silu(z))
    idx, wt = F.route(torch.tensor([[1.0, 3.0, 2.0, -5.0]]), 2, 3.0)
    s = torch.softmax(torch.tensor([1.0, 3.0, 2.0, -5.0]), 0)
    assert idx.tolist() == [[1, 2]] and torch.allclose(wt, 3 * s[[1, 2]][None])
    one = torch.eye(2, dtype=torch.float64)
    glu = lambda h, limit: F.clamped_glu(torch.tensor([h], dtype=torch.float64), {"gate": one[:1], "up": one[1:], "down": one[:, :1]}, "", limit)[0, 0].item()
    gate = lambda x: x / (1 + math.exp(-1.702 * x))
    assert glu([5.0, 5.0], 2.0) == pytest.approx(gate(2.0) * 3) and glu([-5.0, -5.0], 2.0) == pytest.approx(gate(-5.0) * -1) and glu([1.0, 0.5], 2.0) == pytest.approx(gate(1.0) * 1.5)
    assert torch.allclose(F.depth_average(torch.tensor([2.0, -1.0]), [u, u]), u)
    assert float(F.soft_cap(torch.tensor(1000.0), 5.0)) == 5.0 and math.isclose(float(F.soft_cap(torch.tensor(1.0), 5.0)), 5 * math.tanh(0.2), rel_tol=1e-6)


def test_reference_streams_are_results_before_their_averages():
    cfg, _, sd = model("plain")
    toks = [5, 9, 1]
    _, after = F.forward(cfg, sd, toks, want_layers=True)
    s64 = {k: v.double() for k, v in sd.items()}
    x0 = F.embedding(cfg, s64, toks)
    x1 = F.layer(x0, s64, 0, cfg["layers"][0], 1.0, 1e-6)
    a = s64["l0.dwa"][0] * x0 + s64["l0.dwa"][1] * x1
    x2 = F.layer(a, s64, 1, cfg["layers"][1], 1.0, 1e-6)
    w = s64["l1.dwa"]
    assert torch.allclose(after[0], a) and torch.allclose(after[1], w[0] * x0 + w[1] * x1 + w[2] * x2)
