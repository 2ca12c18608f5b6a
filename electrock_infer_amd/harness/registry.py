"""Which model a checkpoint directory holds: config.json names an architecture, the registry maps it to the model's
configuration and class.  A configuration is made from config.json and the shapes of the checkpoint's tensors (sizes
that config.json does not give are read off those)."""
import json
import os
from dataclasses import dataclass
from glob import glob
from typing import Any, Callable, Dict, Tuple

import torch

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


@dataclass
class ModelEntry:
    config_class: Any                   # has from_checkpoint(config, shapes, dtype)
    build: Callable[[Any], torch.nn.Module]    # EngineConfig -> model
    libraries: Tuple[Callable[[], str], ...]   # what has to be compiled for it


REGISTRY: Dict[str, ModelEntry] = {}


def register(architecture: str, config_class, build, *libraries) -> None:
    REGISTRY[architecture] = ModelEntry(config_class, build, libraries)


def checkpoint_shapes(model_dir: str) -> Dict[str, Tuple[int, ...]]:
    """Name -> shape of every tensor, from the headers of the safetensors files alone."""
    shapes = {}
    for file in sorted(glob(os.path.join(model_dir, "*.safetensors"))):
        with open(file, "rb") as f:
            header = json.loads(f.read(int.from_bytes(f.read(8), "little")))
        shapes.update({name: tuple(t["shape"]) for name, t in header.items() if name != "__metadata__"})
    return shapes


def load_config(model_dir: str, dtype: str = "bfloat16"):
    with open(os.path.join(model_dir, "config.json")) as f:
        config = json.load(f)
    names = [config["architecture"]] if "architecture" in config else config.get("architectures", [])
    for name in names:
        if name in REGISTRY:
            return REGISTRY[name].config_class.from_checkpoint(config, checkpoint_shapes(model_dir), DTYPES[dtype])
    raise ValueError(f"no registered architecture among {names}; known: {sorted(REGISTRY)}")


def entry_of(config) -> ModelEntry:
    for entry in REGISTRY.values():
        if isinstance(config, entry.config_class):
            return entry
    raise ValueError(f"no registered model for a {type(config).__name__}")


def build_model(engine_config) -> torch.nn.Module:
    return entry_of(engine_config.model).build(engine_config)


def ensure_libraries(config) -> None:
    """Compile what the model of this configuration needs and is not built yet."""
    for ensure in entry_of(config).libraries:
        ensure()


def _register_all() -> None:
    from .. import _build
    from .config import ModelConfig
    from .feguvik import FeguvikConfig, FeguvikForCausalLM
    from .model import MixtralForCausalLM
    from .nunivik import NunivikConfig, NunivikForCausalLM
    register("MixtralForCausalLM", ModelConfig, lambda c: MixtralForCausalLM(c.model, fused_moe_tail=c.fused_moe_tail),
             _build.ensure_moe)
    register("Feguvik", FeguvikConfig, lambda c: FeguvikForCausalLM(c.model), _build.ensure_decoder)
    register("Nunivik", NunivikConfig, lambda c: NunivikForCausalLM(c.model), _build.ensure_decoder)


_register_all()
