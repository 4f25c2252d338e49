"""Which route serves which model.

The counterpart of the reference's model registry (`qimeng_megakernel/models/LLM/registry.py:84-94, 238-262`): named
shapes for random-init workloads, and the family of a model folder by the ``architecture`` its ``config.json`` names.
"""
from __future__ import annotations

import dataclasses
import importlib
import json
from pathlib import Path
from typing import Any


@dataclasses.dataclass(frozen=True)
class Family:
    route: str      # route package: Globals, ModelConfig, scheduler, mk_kernel
    loop: str       # host loop module

    def module(self, name: str) -> Any:
        """``"route"`` or ``"loop"`` imported."""
        return importlib.import_module(f"{__package__}.{getattr(self, name)}")

    def mk_kernel(self) -> Any:
        return importlib.import_module(f"{__package__}.{self.route}.mk_kernel")


DENSE = Family("decode_schedule", "decode")
DENSE_BATCH = Family("decode_schedule_mb", "decode_batch")
MOE = Family("decode_schedule_moe", "decode_moe")
HYBRID = Family("decode_schedule_hybrid", "decode_hybrid")

#: model name -> (family at batch 1, module and attribute of its shape)
MODELS: dict[str, tuple[Family, str, str]] = {
    "llama-3.2-1b": (DENSE, "decode_schedule.model_config", "LLAMA_3_2_1B"),
    "qwen3-1.7b": (DENSE, "decode_schedule.model_config", "QWEN3_1_7B"),
    "qwen1.5-moe-a2.7b": (MOE, "decode_schedule_moe.model_config", "QWEN1_5_MOE_A2_7B"),
    "qwen3-30b-a3b": (MOE, "decode_schedule_moe.model_config", "QWEN3_30B_A3B"),
    "lusupel-1b": (HYBRID, "synthetic", "LUSUPEL_1B"),
    "lusupel-2b": (HYBRID, "synthetic", "LUSUPEL_2B"),
    "givopel-1b": (HYBRID, "synthetic", "GIVOPEL_1B"),
    "givopel-2b": (HYBRID, "synthetic", "GIVOPEL_2B"),
}

#: ``architecture`` of a model folder's config.json -> family
ARCHITECTURES: dict[str, Family] = {"Lusupel": HYBRID, "Givopel": HYBRID}


def shape_of(name: str) -> Any:
    _, module, attribute = MODELS[name]
    return getattr(importlib.import_module(f"{__package__}.{module}"), attribute)


def family_of(folder: Path | str) -> Family:
    """The family that serves a model folder."""
    with open(Path(folder) / "config.json") as f:
        config = json.load(f)
    name = config.get("architecture")
    if name not in ARCHITECTURES:
        raise ValueError(f"no family serves the architecture {name!r} (known: {', '.join(sorted(ARCHITECTURES))})")
    return ARCHITECTURES[name]
