"""Model registry: configuration type -> model class, and model folders (config.json + model.safetensors) or names -> both."""
from __future__ import annotations

import json
from pathlib import Path
from typing import Any, Callable, Dict

from . import bulodra, dugalix, genusun, models, mosurax

# config.json "architecture" -> reader of the file
ARCHITECTURES: Dict[str, Callable[[dict, str], Any]] = {"Genusun": genusun.GenusunConfig.from_dict, "Mosurax": mosurax.MosuraxConfig.from_dict,
                                                        "Bulodra": bulodra.BulodraConfig.from_dict, "Dugalix": dugalix.DugalixConfig.from_dict}
_MODELS = {models.ModelConfig: models.CausalLM, genusun.GenusunConfig: genusun.GenusunForCausalLM,
           mosurax.MosuraxConfig: mosurax.MosuraxForCausalLM, bulodra.BulodraConfig: bulodra.BulodraForCausalLM,
           dugalix.DugalixConfig: dugalix.DugalixForCausalLM}
# HIP units (sglang_amd/csrc) a model's path needs; a model that is not listed uses the whole library
_UNITS = {genusun.GenusunConfig: "hybrid", mosurax.MosuraxConfig: "grouped", bulodra.BulodraConfig: "layered",
          dugalix.DugalixConfig: "shifted"}
_NAMED = (models.CONFIGS, genusun.CONFIGS, mosurax.CONFIGS, bulodra.CONFIGS, dugalix.CONFIGS)


def model_class(config):
    for kind, cls in _MODELS.items():
        if isinstance(config, kind):
            return cls
    raise ValueError(f"no model is registered for a {type(config).__name__}")


def unit_group(config) -> str:
    return next((g for kind, g in _UNITS.items() if isinstance(config, kind)), "all")


def load_config(path):
    """The configuration of a model folder, by its "architecture"."""
    path = Path(path)
    d = json.loads((path / "config.json").read_text())
    arch = d.get("architecture") or next(iter(d.get("architectures") or []), None)
    if arch not in ARCHITECTURES:
        raise ValueError(f"{path}: architecture {arch!r} is not registered (have {sorted(ARCHITECTURES)})")
    return ARCHITECTURES[arch](d, path.name)


def named_config(name: str):
    for table in _NAMED:
        if name in table:
            return table[name]
    raise KeyError(f"unknown model {name!r} (have {config_names()})")


def config_names():
    return sorted(n for table in _NAMED for n in table)


def runner_for(model: str, dtype=None, device=None, **kw):
    """A ModelRunner for a model folder (its weights) or a named configuration (seeded random weights)."""
    import torch

    from .. import native
    from .engine import ModelRunner
    from .weights import TensorWeights

    dtype = dtype or torch.bfloat16
    folder = Path(model)
    is_dir = (folder / "config.json").exists()
    config = load_config(folder) if is_dir else named_config(model)
    native.ensure(unit_group(config))
    device = device if device is not None else torch.device("cuda", torch.cuda.current_device())
    if is_dir:
        kw["weights"] = TensorWeights.from_dir(folder, device, dtype)
    return ModelRunner(config, device=device, dtype=dtype, **kw)
