"""The architectures this package serves, by the name a checkpoint's config.json gives, and how each is read, loaded
and run.  ``load_engine`` is the way from a checkpoint folder to an engine that prefills and generates."""
from __future__ import annotations

import dataclasses
from typing import Callable, Dict, Tuple

import torch

from . import checkpoint
from ._capi import TahDuoError


@dataclasses.dataclass(frozen=True)
class Architecture:
    name: str
    load: Callable          # (config dict, tensors by name, device, dtype) -> weights
    engine: Callable        # (weights, batch, max_len, device=..., **options) -> engine
    dtypes: Tuple[torch.dtype, ...] = (torch.bfloat16,)


_ARCHITECTURES: Dict[str, Architecture] = {}


def register(arch: Architecture) -> Architecture:
    _ARCHITECTURES[arch.name] = arch
    return arch


def architectures():
    return sorted(_ARCHITECTURES)


def of_config(config: dict) -> Architecture:
    """The architecture of a parsed config.json ('architecture', or Hugging Face's list 'architectures')."""
    names = [config["architecture"]] if "architecture" in config else list(config.get("architectures") or [])
    for n in names:
        if n in _ARCHITECTURES:
            return _ARCHITECTURES[n]
    raise TahDuoError(f"no architecture for {names or 'a config without a name'} (known: {', '.join(architectures())})")


def load_weights(folder: str, device="cuda", dtype: torch.dtype = torch.bfloat16):
    """(architecture, weights) of a checkpoint folder."""
    config = checkpoint.read_config(folder)
    arch = of_config(config)
    if dtype not in arch.dtypes:
        raise TahDuoError(f"{arch.name} does not run in {dtype}")
    return arch, arch.load(config, checkpoint.read_tensors(folder), device, dtype)


def load_engine(folder: str, batch: int, max_len: int, *, device="cuda", dtype: torch.dtype = torch.bfloat16, **options):
    arch, weights = load_weights(folder, device, dtype)
    return arch.engine(weights, batch, max_len, device=device, **options)


def _zozosun() -> None:
    from . import zozosun

    register(Architecture(zozosun.NAME, zozosun.load, zozosun.engine, (torch.bfloat16, torch.float32)))


def _zedudra() -> None:
    from . import zedudra

    register(Architecture(zedudra.NAME, zedudra.load, zedudra.engine, (torch.bfloat16, torch.float32)))


def _qwen3() -> None:
    from .engine import EngineConfig, TaHDecodeEngine, Weights

    register(Architecture("Qwen3ForCausalLM",
                          lambda config, tensors, device, dtype: Weights.from_tensors(tensors, EngineConfig.from_config(config), device, dtype),
                          TaHDecodeEngine))


_zozosun()
_zedudra()
_qwen3()
