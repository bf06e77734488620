"""The models the engine knows: which class serves a configuration, and how its shape is read."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Any, Callable

from .kapolorn import Kapolorn, KapolornShape
from .mefupel import Mefupel, MefupelShape
from .pedivik import Pedivik, PedivikShape
from .qwen3 import Qwen3, Qwen3Shape
from .rutevik import Rutevik, RutevikShape
from .weights import read_folder


@dataclass(frozen=True)
class Architecture:
    name: str                                # as config.json names it
    model: type
    shape: type
    from_config: Callable[[dict], Any]
    libs: tuple[str, ...]                    # the kernels it needs (names in zipage_amd/build.py)
    loads_weights: bool = True


ARCHITECTURES = {a.name: a for a in (
    Architecture("Qwen3ForCausalLM", Qwen3, Qwen3Shape, Qwen3Shape.from_config, ("LIB",), loads_weights=False),
    Architecture("Pedivik", Pedivik, PedivikShape, PedivikShape.from_config, ("MODELS_LIB", "LATENT_LIB")),
    Architecture("Kapolorn", Kapolorn, KapolornShape, KapolornShape.from_config,
                 ("MODELS_LIB", "GROUPED_LIB", "RECURRENT_LIB", "MOE_LIB")),
    Architecture("Rutevik", Rutevik, RutevikShape, RutevikShape.from_config,
                 ("MODELS_LIB", "LATENT_LIB", "GROUPED_LIB", "MOE_LIB")),
    Architecture("Mefupel", Mefupel, MefupelShape, MefupelShape.from_config,
                 ("MODELS_LIB", "GROUPED_LIB", "LINEAR_LIB")),
)}


def architecture_of(config: dict) -> Architecture:
    names = [config["architecture"]] if "architecture" in config else config.get("architectures", [])
    for n in names:
        if n in ARCHITECTURES:
            return ARCHITECTURES[n]
    raise ValueError(f"no model for architecture {names}; known: {sorted(ARCHITECTURES)}")


def read_shape(folder: str):
    """The shape a model folder's config.json describes."""
    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    return architecture_of(config).from_config(config)


def arch_for_shape(shape) -> Architecture:
    for a in ARCHITECTURES.values():
        if isinstance(shape, a.shape):
            return a
    raise TypeError(f"no model for shape {type(shape).__name__}")


def build_model(shape, device, dtype, seed: int = 0, folder: str | None = None):
    """The model of `shape`, with the weights of `folder` or, without one, drawn from `seed`."""
    arch = arch_for_shape(shape)
    kw = {}
    if folder is not None:
        if not arch.loads_weights:
            raise NotImplementedError(f"{arch.name} is random-initialised only")
        kw["weights"] = read_folder(folder)
    return arch.model(shape, device, dtype=dtype, seed=seed, **kw)
