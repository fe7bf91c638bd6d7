"""Fobolix without a GPU: configuration reader, registry, rotary tables, the reference's own consistency, slot bookkeeping of a replay."""
import ctypes as C
import json
import os
import subprocess

import numpy as np
import pytest
import torch

from chatts_amd import registry, rotary
from chatts_amd.fobolix import FobolixConfig
from oracle import fobolix as F
from tests.fobolix_models import CONFIGS, YARN, model

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_config_round_trip_and_runs(name, tmp_path):
    _, public, _ = model(name)
    c = FobolixConfig.from_dict(public)
    assert c.runs() == F.runs(public)
    c.save_pretrained(str(tmp_path))
    again = registry.load_config(str(tmp_path))
    assert isinstance(again, FobolixConfig) and again.to_dict() == c.to_dict()
    assert registry.model_class(again).__name__ == "FobolixForCausalLM"


def test_config_reads_every_value_and_refuses_what_it_does_not_know():
    _, public, _ = model("odd")
    c = FobolixConfig.from_dict(public)
    assert (c.vocab_size, c.hidden_size, c.rms_norm_eps) == (130, 90, 3e-5) and c.loop["times"] == 3 and c.eos_token_id == []
    for change in ({"type": "window"}, {"mlp": {"kind": "experts"}}):
        bad = json.loads(json.dumps(public))
        bad["layers"][0].update(change)
        with pytest.raises(ValueError):
            FobolixConfig.from_dict(bad)
    bad = json.loads(json.dumps(public))
    del bad["layers"][1]["mixer"]["kv_rank"]
    with pytest.raises(ValueError, match="kv_rank"):
        FobolixConfig.from_dict(bad)
    bad = dict(public, loop={"start": 2, "stop": 9, "times": 1})
    with pytest.raises(ValueError, match="loop"):
        FobolixConfig.from_dict(bad)


def test_registry_by_config_json(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nothing"}))
    with pytest.raises(ValueError, match="Nothing"):
        registry.load_config(str(tmp_path))
    (tmp_path / "config.json").write_text(json.dumps({"model_type": "qwen2", "hidden_size": 256, "num_attention_heads": 2}))
    assert type(registry.load_config(str(tmp_path))).__name__ == "ChatTSConfig"


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_tensor_shapes_cover_the_model(name):
    _, public, sd = model(name)
    shapes = FobolixConfig.from_dict(public).tensor_shapes()
    assert set(shapes) == set(sd)
    for n, s in shapes.items():
        assert all(a is None or a == b for a, b in zip(s, sd[n].shape)), n


@pytest.mark.parametrize("scaling", [None, YARN, {"factor": 1.0, "original": 32, "fast": 4.0, "slow": 4.0}, {"factor": 40.0, "original": 4096, "fast": 32, "slow": 1}])
@pytest.mark.parametrize("dims", [2, 10, 64])
def test_rotary_tables(dims, scaling):
    cos, sin = rotary.rotary_tables(dims, 10000.0, 300, scaling)
    f, mag = F.rotary_frequencies(dims, 10000.0, scaling)
    a = torch.arange(300, dtype=torch.float64)[:, None] * f
    assert torch.allclose(cos.double(), a.cos() * mag, atol=1e-6) and torch.allclose(sin.double(), a.sin() * mag, atol=1e-6)


def test_reference_is_causal_and_looped():
    cfg, _, sd = model("odd")
    rng = np.random.default_rng(0)
    toks = rng.integers(0, 130, 20).tolist()
    full, streams = F.forward(cfg, sd, toks, want_layers=True)
    assert len(streams) == len(F.runs(cfg)) == 1 + 2 * 3 + 1
    assert torch.allclose(F.forward(cfg, sd, toks[:11]), full[:11])
    once = dict(cfg, loop=dict(cfg["loop"], times=1))
    assert not torch.allclose(F.forward(once, sd, toks), full, atol=1e-2)


def test_reference_delta_rule_writes_before_it_reads():
    """a single token from an empty state: o = (q . k) beta v"""
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(2, n, generator=g, dtype=torch.float64) for n in (5, 5, 3))
    S, o = F.delta_step(torch.zeros(2, 5, 3, dtype=torch.float64), q, k, v, torch.full((2, 5), 0.5, dtype=torch.float64), torch.tensor([0.25, 1.0], dtype=torch.float64))
    want = (q * k).sum(-1, keepdim=True) * torch.tensor([[0.25], [1.0]], dtype=torch.float64) * v
    assert torch.allclose(o, want)


def test_struct_layouts_match_the_header(tmp_path):
    from chatts_amd import _lib
    names = {"ChattsRow": 16, "ChattsSpan": C.sizeof(_lib.Span), "ChattsLatentExpandArgs": C.sizeof(_lib.LatentExpandArgs), "ChattsOperand": C.sizeof(_lib.Operand), "ChattsResidualNormArgs": C.sizeof(_lib.ResidualNormArgs),
             "ChattsHeadLinearArgs": C.sizeof(_lib.HeadLinearArgs), "ChattsDeltaArgs": C.sizeof(_lib.DeltaArgs), "ChattsLatentArgs": C.sizeof(_lib.LatentArgs),
             "ChattsEmbedPairArgs": C.sizeof(_lib.EmbedPairArgs), "ChattsPairNormArgs": C.sizeof(_lib.PairNormArgs),
             "ChattsTokenShiftArgs": C.sizeof(_lib.TokenShiftArgs), "ChattsRecurArgs": C.sizeof(_lib.RecurArgs),
             "ChattsPostNormArgs": C.sizeof(_lib.PostNormArgs), "ChattsDepthNormArgs": C.sizeof(_lib.DepthNormArgs), "ChattsGruArgs": C.sizeof(_lib.GruArgs),
             "ChattsSelectArgs": C.sizeof(_lib.SelectArgs),
             "ChattsWindowArgs": C.sizeof(_lib.WindowArgs), "ChattsMoeArgs": C.sizeof(_lib.MoeArgs),
             "ChattsMixLayer": C.sizeof(_lib.MixLayer), "ChattsMixRun": C.sizeof(_lib.MixRun), "ChattsMixConfig": C.sizeof(_lib.MixConfig),
             "ChattsMixBuffers": C.sizeof(_lib.MixBuffers), "ChattsLinearArgs": C.sizeof(_lib.LinearArgs)}
    src = tmp_path / "s.c"
    src.write_text(f'#include "{ROOT}/include/chatts_amd.h"\n#include <stdio.h>\nint main(void) {{\n' +
                   "".join(f'  printf("%zu\\n", sizeof({n}));\n' for n in names) + "  return 0;\n}\n")
    subprocess.run(["gcc", str(src), "-o", str(tmp_path / "s")], check=True)
    got = [int(x) for x in subprocess.run([str(tmp_path / "s")], check=True, capture_output=True, text=True).stdout.split()]
    assert dict(zip(names, got)) == names


class _FakeModel:
    def __init__(self):
        self.calls, self.released = [], []

    def step_tokens(self, batch):
        self.calls.append(batch)
        return torch.zeros((sum(len(w) for _, _, w in batch), 3))

    def release_slot(self, slot):
        self.released.append(slot)


def test_replay_hands_slots_out_and_back():
    from chatts_amd.trace_run import Replay
    m = _FakeModel()
    r = Replay(m, 2)
    assert r.step([{"id": "a", "tokens": [1, 2], "want": [1]}, {"id": "b", "tokens": [3], "want": []}], []).shape[0] == 1
    sa, sb = r.slot_of["a"], r.slot_of["b"]
    with pytest.raises(RuntimeError):
        r.step([{"id": "c", "tokens": [1], "want": []}], [])
    r.step([{"id": "b", "tokens": [4, 5], "want": [0, 1]}], ["b"])
    assert m.released == [sb]
    r.step([{"id": "c", "tokens": [1], "want": []}, {"id": "a", "tokens": [9], "want": [0]}], ["a", "c"])
    assert r.slot_of == {} and m.calls[-1][0][0] == sb and m.calls[-1][1][0] == sa
    with pytest.raises(ValueError):
        r.step([{"id": "d", "tokens": [1], "want": [1]}], [])


def test_token_id_prompts_without_a_tokenizer():
    from chatts_amd.processing import TextProcessor
    from chatts_amd.tokenizer import TokenIdTokenizer
    t = TokenIdTokenizer()
    assert t.encode("5 17 3") == [5, 17, 3] and t.decode([5, 17]) == "5 17"
    with pytest.raises(ValueError):
        t.encode("hello")
    with pytest.raises(ValueError):
        TextProcessor(t).splice("1 2", [[1.0]])
