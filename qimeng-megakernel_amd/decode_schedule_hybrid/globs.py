"""``Globals`` of the hybrid route: weights, per-slot states, buffers and the layer table the kernels read.

Unlike the routes of uniform layers, whose tensors are stacked over layers, every layer here has sizes of its own:
``layer_weights[i]`` / ``layer_state[i]`` hold the tensors of entry ``i`` of the shape (a layer, or a branch of one in one
of its passes: passes share weights and have states of their own) by the field names of ``QmkHybridLayer``
(``include/qmk_hybrid.h``), and ``build_globals`` writes their addresses into one table, kept on both sides.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Optional

import torch

from .model_config import HybridShape
from .weights import rope_tables

Tensor = torch.Tensor


@dataclass
class Globals:
    shape: HybridShape
    dtype: torch.dtype                               # element type of caches and prefill activations
    slots: int
    max_positions: int                               # tokens a request may hold
    portion_rows: int                                # tokens one prefill launch takes

    instructions: Optional[Tensor] = None            # int32 [queues, len, 32]
    instruction_splits: int = 0                      # parts the attention instructions cut the visible keys into
    barriers: Optional[Tensor] = None                # int32 [groups, 54, 48]
    position_id: int = 0
    slot: int = 0
    flip: int = 0

    embed_tokens: Optional[Tensor] = None            # bf16 [V, D]
    lm_head_norm_weights: Optional[Tensor] = None    # f32  [D]
    lm_head_weights: Optional[Tensor] = None         # bf16 [V, D]
    layer_weights: list[dict[str, Tensor]] = field(default_factory=list)
    layer_state: list[dict[str, Tensor]] = field(default_factory=list)

    token: Optional[Tensor] = None                   # int64 [1]: the token a decode step reads
    logits: Optional[Tensor] = None                  # f32 [V] of the last decode step

    @property
    def device(self) -> torch.device:
        return self.embed_tokens.device


def state_tensors(shape: HybridShape, i: int, *, slots: int, max_positions: int, portion_rows: int, dtype: torch.dtype,
                  device: torch.device | str) -> dict[str, Tensor]:
    """The per-slot state of entry ``i``.  The cache of a windowed attention is a ring: it holds the keys the window can
    still reach while a whole portion's rows are written, and no more."""
    l = shape.entries[i].shape

    def zeros(*size: int, dtype: torch.dtype = torch.float32) -> Tensor:
        return torch.zeros(*size, dtype=dtype, device=device)

    if l.type == "latent_attention":
        ring = min(max_positions, min(l.window, max_positions) - 1 + portion_rows)
        return {"cache": zeros(slots, ring, l.rank_s + l.rot_s, dtype=dtype)}
    if l.type == "attention":
        return {"cache": zeros(slots, max_positions, l.kv_heads, l.dim_s + l.v_s, dtype=dtype)}
    if l.type == "gla":
        return {"state": zeros(slots, l.heads, l.dim_s, l.v_s)}
    if l.type == "delta":
        return {"state": zeros(slots, l.heads, l.dim_s, l.v_s), "shift": zeros(slots, 2, l.taps - 1, l.conv_channels)}
    if l.type in ("join", "final"):
        return {}
    if l.type == "rglru":
        return {"state": zeros(slots, l.mix_width), "shift": zeros(slots, 2, max(l.taps - 1, 1), l.mix_width)[:, :, : l.taps - 1].contiguous()}
    return {"state": zeros(slots, l.heads, l.dim_s, l.dim_s), "shift": zeros(slots, 2, shape.width_s)}


def build_globals(shape: HybridShape, packed: dict[str, Any], *, dtype: torch.dtype = torch.bfloat16, slots: int = 1, max_positions: int,
                  portion_rows: int = 2048) -> Globals:
    """States, tables and buffers around the weights ``weights.pack`` made (on their device)."""
    if dtype not in (torch.bfloat16, torch.float32):
        raise TypeError(f"the hybrid route computes in bfloat16 or float32, not {dtype}")
    device = packed["embed"].device
    portion_rows = max(1, min(portion_rows, max_positions))
    g = Globals(shape=shape, dtype=dtype, slots=slots, max_positions=max_positions, portion_rows=portion_rows)
    g.embed_tokens, g.lm_head_weights, g.lm_head_norm_weights = packed["embed"], packed["head"], packed["final_norm"]
    tables: dict[tuple, tuple[Tensor, Tensor]] = {}
    for i, e in enumerate(shape.entries):
        l, w = e.shape, dict(packed["layers"][i])
        if l.type in ("latent_attention", "attention"):
            key = (l.rot_dim, l.rope_base, l.rope_scaling)
            if key not in tables:
                cos, sin = rope_tables(l.rot_dim, l.rope_base, max_positions, l.rope_scaling)
                tables[key] = (cos.to(device), sin.to(device))
            w["rope_cos"], w["rope_sin"] = tables[key]
        g.layer_weights.append(w)
        g.layer_state.append(state_tensors(shape, i, slots=slots, max_positions=max_positions, portion_rows=portion_rows, dtype=dtype, device=device))
    g.token = torch.zeros(1, dtype=torch.int64, device=device)
    g.logits = torch.zeros(shape.vocab_s, dtype=torch.float32, device=device)
    return g
