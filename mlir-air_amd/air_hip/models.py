"""Model registry: a checkpoint directory's config.json names the architecture, the architecture names the class.

Every class is a generation.CausalLM with `load(path, config, dtype, device)`; `library` is the shared library its
kernels are in (mlir-air_amd/build.py builds them one by one).
"""

import dataclasses
import importlib
import json
import os

import torch


@dataclasses.dataclass(frozen=True)
class Entry:
    module: str
    cls: str
    library: str


REGISTRY = {
    "LlamaForCausalLM": Entry("decode", "LlamaModel", "w4a16"),
    "Kuvonex": Entry("kuvonex", "KuvonexModel", "dense_lm"),
    "Sitirax": Entry("sitirax", "SitiraxModel", "dense_lm"),
}


def read_config(path):
    file = os.path.join(path, "config.json")
    if not os.path.isfile(file):
        raise FileNotFoundError(f"{file} does not exist")
    with open(file) as f:
        return json.load(f)


def entry_for(config):
    """Registry entry of a parsed config.json (`architecture`, or HuggingFace's list `architectures`)."""
    names = [config["architecture"]] if "architecture" in config else list(config.get("architectures") or [])
    for name in names:
        if name in REGISTRY:
            return REGISTRY[name]
    raise ValueError(f"no model for architecture {names or '(none named)'}; known: {', '.join(sorted(REGISTRY))}")


def load_model(path, dtype=torch.bfloat16, device="cuda"):
    """The model of a local checkpoint directory, on the device."""
    config = read_config(path)
    entry = entry_for(config)
    cls = getattr(importlib.import_module(f".{entry.module}", __package__), entry.cls)
    return cls.load(path, config, dtype=dtype, device=device)
