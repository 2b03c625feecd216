"""Model registry: config.json -> the class that serves it.

An entry is a loader `load(path, dtype, capacity, slots, max_portion, device)` returning an object with the engine's
interface: `architecture`, `vocab`, `capacity`, `slots`, `forward(slot, tokens, pos, want)` -> logits and
`decode(slot, token, pos, n)` -> tokens."""
from __future__ import annotations

from typing import Callable, Dict, List, Tuple

import torch

from .weights import read_config

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32, "float16": torch.float16}


def _nibotar(*args, **kw):
    from . import nibotar
    return nibotar.load(*args, **kw)


def _kagapel(*args, **kw):
    from . import kagapel
    return kagapel.load(*args, **kw)


def _neox(*args, **kw):
    from .build import ensure_neox
    ensure_neox()
    from . import model
    return model.load_neox(*args, **kw)


# architecture name -> (loader, element types it runs in)
_REGISTRY: Dict[str, Tuple[Callable, Tuple[str, ...]]] = {
    "Nibotar": (_nibotar, ("bfloat16", "float32")),
    "Kagapel": (_kagapel, ("bfloat16", "float32")),
    "GPTNeoXForCausalLM": (_neox, ("float16",)),
}


def architectures() -> List[str]:
    return sorted(_REGISTRY)


def architecture_of(config: dict) -> str:
    """The architecture's name: the `architecture` entry, or HuggingFace's `architectures` list."""
    name = config.get("architecture") or (config.get("architectures") or [None])[0]
    if name not in _REGISTRY:
        raise ValueError(f"unknown architecture {name!r}; known: {', '.join(architectures())}")
    return name


def dtypes_of(config: dict) -> Tuple[str, ...]:
    """The element types this model runs in; the first one is the default."""
    return _REGISTRY[architecture_of(config)][1]


def load_model(path: str, dtype: str = "", capacity: int = 4096, slots: int = 1, max_portion: int = 2048, device="cuda"):
    """Loads the checkpoint folder `path` with the class its config.json names."""
    config = read_config(path)
    loader, types = _REGISTRY[architecture_of(config)]
    dtype = dtype or types[0]
    if dtype not in types:
        raise ValueError(f"{architecture_of(config)} does not run in {dtype}; it runs in {', '.join(types)}")
    return loader(path, DTYPES[dtype], capacity=capacity, slots=slots, max_portion=max_portion, device=device)
