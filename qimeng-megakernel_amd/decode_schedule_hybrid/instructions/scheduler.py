"""Instruction queues of one hybrid decode step.

A layer is a chain of stages: input projections, the mixer's middle (recurrence; absorb, attend, value; wkv step), output
projection, and for a feed-forward up/gate and down; the LM head ends the step.  Each stage's output rows are cut into
blocks of equal size, about one per queue, and dealt to the queues from queue 0 on (the leaders of the per-XCD waits are
the first eight queues, so they take part in every stage).  All output and down projections are cut alike: a queue owns its
rows of the residual streams for the whole step, and the kernel relies on it.  One tensor serves every position: the split of the visible
keys over the parts of opcode 4 is worked out on the device.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Sequence

import torch

from ...instruction import INTS_PER_INSTRUCTION
from ..model_config import HybridShape
from . import instruction_defs as D

MI355X_QUEUES = 256
MAX_ROWS = 512             # rows of one instruction (pairs count as two)
MAX_OUT_ROWS = 64          # ... of an output projection: a thread per row and stream
MIN_ROWS = 4
KEYS_PER_PART = 64
MAX_PARTS = 32
ATTEND_COLUMNS = 128       # latent columns one attention instruction sums up
BARRIER_ROWS, BARRIER_SLOTS = 54, 48


def _ceil_div(a: int, b: int) -> int:
    return -(-a // b)


def cut(segments: Sequence[tuple[int, int]], queues: int, *, step: int = 2, most: int = MAX_ROWS) -> list[tuple[int, int, int]]:
    """``segments`` (sub, rows) -> blocks (sub, start, rows): equal block sizes, multiples of ``step``, no block over a
    segment's end, no more blocks than queues unless a block would exceed ``most`` rows."""
    total = sum(rows for _, rows in segments)
    size = max(_ceil_div(total, queues), min(MIN_ROWS, most))
    size = min(_ceil_div(size, step) * step, most)
    while sum(_ceil_div(rows, size) for _, rows in segments) > queues and size + step <= most:
        size += step
    return [(sub, start, min(size, rows - start)) for sub, rows in segments for start in range(0, rows, size)]


@dataclass
class HybridScheduler:
    shape: HybridShape
    queues: int = MI355X_QUEUES
    max_positions: int = 1 << 30

    def parts(self, layer: int) -> int:
        """Parts the visible keys of a latent attention are cut into."""
        reach = min(self.shape.layers[layer].window, self.max_positions)
        return max(1, min(MAX_PARTS, _ceil_div(reach, KEYS_PER_PART)))

    def max_parts(self) -> int:
        return max([self.parts(i) for i, l in enumerate(self.shape.layers) if l.type == "latent_attention"], default=1)

    def layer_stages(self, i: int) -> list[list[D.StageInstruction]]:
        l, q = self.shape.layers[i], self.queues
        stages: list[list[D.StageInstruction]] = []
        if l.type == "wkv":
            segments = [(s, l.mix_width) for s in range(4)] + [(4, l.rank_s)]
            stages.append([D.RMS_InProject(i, s, s * l.mix_width + a, n) for s, a, n in cut(segments, q)])
            stages[0][0].extra = 1
            stages.append([D.WkvStep(i, h, 0, 1) for h in range(l.heads)])
        else:
            stages.append([D.RMS_InProject(i, 0, a, n) for _, a, n in cut([(0, l.in_rows)], q)])
        if l.type == "rglru":
            stages.append([D.GatedRecurrence(i, b, a, n) for b, a, n in cut([(b, l.block_s) for b in range(l.blocks)], q, step=1, most=MAX_ROWS // 2)])
        elif l.type == "latent_attention":
            stages.append([D.LatentAbsorb(i, h, a, n) for h, a, n in cut([(h, l.rank_s) for h in range(l.heads)], q)])
            stages[-1][0].extra = 1
            parts = self.parts(i)
            stages.append([D.LatentAttendSplitKV(i, g, part, parts, extra=c) for g in range(_ceil_div(l.heads, 16)) for part in range(parts)
                           for c in range(_ceil_div(l.rank_s, ATTEND_COLUMNS))])
            stages.append([D.LatentValue(i, h, a, n, extra=parts) for h, a, n in cut([(h, l.v_s) for h in range(l.heads)], q)])
        D_s = self.shape.width_s
        stages.append([D.OutProject_Streams(i, 0, a, n) for _, a, n in cut([(0, D_s)], q, most=MAX_OUT_ROWS)])
        if l.ff:
            stages.append([D.RMS_UpGate_Gelu(i, 0, a, n) for _, a, n in cut([(0, l.ff_s)], q, most=MAX_ROWS // 2)])
            stages.append([D.OutProject_Streams(i, 1, a, n) for _, a, n in cut([(0, D_s)], q, most=MAX_OUT_ROWS)])
        return stages

    def stages(self) -> list[list[D.StageInstruction]]:
        out = [s for i in range(len(self.shape.layers)) for s in self.layer_stages(i)]
        last = len(self.shape.layers) - 1
        out.append([D.RMS_LMHead(last, 0, a, n) for _, a, n in cut([(0, self.shape.vocab_s)], self.queues)])
        for k, stage in enumerate(out):
            for ins in stage:
                if k:
                    ins.wait_stage, ins.wait_count = k - 1, len(out[k - 1])
                if k + 1 < len(out):
                    ins.arrive_stage = k
        return out

    def barrier_groups(self) -> int:
        return _ceil_div(len(self.stages()), 4)

    def instruction_queues(self) -> list[list[D.StageInstruction]]:
        queues: list[list[D.StageInstruction]] = [[] for _ in range(self.queues)]
        for stage in self.stages():
            for k, ins in enumerate(stage):
                queues[k % self.queues].append(ins)
        return queues


def tensorize(queues: Sequence[Sequence[Any]], device: torch.device | str) -> torch.Tensor:
    length = max(len(q) for q in queues)
    empty = [0] * INTS_PER_INSTRUCTION
    rows = [[ins.padded() for ins in q] + [empty] * (length - len(q)) for q in queues]
    return torch.tensor(rows, dtype=torch.int32, device=device)


def build(globs: Any, queues: int = MI355X_QUEUES) -> torch.Tensor:
    """Instruction tensor and counters of ``globs``' decode step."""
    scheduler = HybridScheduler(globs.shape, queues, globs.max_positions)
    globs.instructions = tensorize(scheduler.instruction_queues(), globs.device)
    globs.instruction_splits = scheduler.max_parts()
    globs.barriers = torch.zeros(scheduler.barrier_groups(), BARRIER_ROWS, BARRIER_SLOTS, dtype=torch.int32, device=globs.device)
    return globs.instructions
