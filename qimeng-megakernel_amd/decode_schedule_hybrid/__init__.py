"""Route package of hybrid decoders: per-layer mixers (gated linear recurrence, wkv time mixing, latent attention) on a
hyper-connected residual stream, or (gated linear attention, softmax attention beside a gated delta rule) on a plain residual
that a stretch of layers may run over several times.  Exports the names every route package exports (``decode_schedule/__init__.py``)."""
from __future__ import annotations

import importlib

from .globs import Globals
from .model_config import HybridConfig, HybridShape, LayerShape

ModelConfig = HybridConfig

#: the kernel clears its own counters when the last workgroup retires
STATIC_MEGAKERNEL = True

_LAZY = {
    "instructions": ".instructions",
    "instruction_defs": ".instructions.instruction_defs",
    "scheduler": ".instructions.scheduler",
    "mk_kernel": ".mk_kernel",
    "weights": ".weights",
    "state": ".state",
}

__all__ = ["Globals", "ModelConfig", "HybridConfig", "HybridShape", "LayerShape", "STATIC_MEGAKERNEL", *_LAZY]


def __getattr__(name: str):
    target = _LAZY.get(name)
    if target is None:
        raise AttributeError(f"module {__name__!r} has no attribute {name!r}")
    return importlib.import_module(target, __name__)
