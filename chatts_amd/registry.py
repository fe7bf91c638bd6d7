"""Which configuration and model class serve a checkpoint directory, decided by its config.json.

A design names itself under "architecture"; a config.json without that key is a ChatTS / Qwen decoder (HF keys).
"""
import importlib
import json
import os

# architecture -> (module, configuration class, model class); None = no "architecture" key
ARCHITECTURES = {
    None: ("chatts_amd", "ChatTSConfig", "ChatTSForCausalLM"),
    "Fobolix": ("chatts_amd.fobolix", "FobolixConfig", "FobolixForCausalLM"),
    "Medilix": ("chatts_amd.medilix", "MedilixConfig", "MedilixForCausalLM"),
    "Muvetar": ("chatts_amd.muvetar", "MuvetarConfig", "MuvetarForCausalLM"),
    "Mefurax": ("chatts_amd.mefurax", "MefuraxConfig", "MefuraxForCausalLM"),
}


def _entry(architecture):
    if architecture not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {architecture!r}; known: {sorted(k for k in ARCHITECTURES if k)} and ChatTS / Qwen checkpoints")
    return ARCHITECTURES[architecture]


def load_config(path):
    """config.json of a checkpoint directory -> configuration object of its design"""
    with open(os.path.join(path, "config.json")) as f:
        d = json.load(f)
    module, cls, _ = _entry(d.get("architecture"))
    return getattr(importlib.import_module(module), cls).from_dict(d)


def model_class(config):
    """the model class that runs a configuration object"""
    module, _, cls = _entry(getattr(config, "architecture", None))
    return getattr(importlib.import_module(module), cls)
