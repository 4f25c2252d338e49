"""Instruction queues of one hybrid decode step.

A layer on residual streams is a chain of stages: input projections, the mixer's middle (recurrence; absorb, attend, value;
wkv step), output projection, and for a feed-forward up/gate and down.  A layer run on the plain residual, whose branches and
feed-forward read the same input, is three or four stages: all input projections and up/gate; state steps, attention and
low-rank output gates; merges, the output projections of the state branches and down; the output projections of the
attention.  (Without an attention the down projection runs beside the state steps, and the output projections follow.)  What a run leaves is added by
the stage that reads the residual next.  The LM head ends the step.  Each stage's output rows are cut into
blocks of equal size, about one per queue, and dealt to the queues from queue 0 on (the leaders of the per-XCD waits are
the first eight queues, so they take part in every stage).  All output and down projections are cut alike: a queue owns its
rows of the residual streams for the whole step, and the kernel relies on it (a plain residual has no such rows).  One tensor serves every position: the split of the visible
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
ATTEND_COLUMNS = 128       # latent or value columns one attention instruction sums up
STATE_COLUMNS = 64         # value columns of one state step: all key rows fit its threads' registers
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
        """Parts the visible keys of an attention are cut into; where other branches run in the same stage, no more than fit
        beside them (but at least eight)."""
        entry = self.shape.entries[layer]
        l, most = entry.shape, MAX_PARTS
        reach = min(l.window, self.max_positions) if l.type == "latent_attention" else self.max_positions
        if entry.branches > 1:
            beside = [e.shape for e in self.shape.entries[layer - entry.branch : layer - entry.branch + entry.branches] if e.type != "attention"]
            busy = sum(b.heads * _ceil_div(b.v_s, STATE_COLUMNS) for b in beside) + (self.gate_instructions if any(b.gate_rank for b in beside) else 0)
            most = min(MAX_PARTS, max(8, (self.queues - busy) // len(self.attention_groups(l))))
        return max(1, min(most, _ceil_div(reach, KEYS_PER_PART)))

    @property
    def gate_instructions(self) -> int:
        """Instructions the rows of a low-rank gate are cut into."""
        return max(1, self.queues // 8)

    @staticmethod
    def attention_groups(l: Any) -> list[tuple[int, int]]:
        """(key head and sixteen of its heads, value columns) of the instructions that make one part of an attention."""
        return [(g, c) for g in range(l.kv_heads * _ceil_div(l.heads // l.kv_heads, 16)) for c in range(_ceil_div(l.v_s, ATTEND_COLUMNS))]

    def max_parts(self) -> int:
        return max([self.parts(i) for i, e in enumerate(self.shape.entries) if e.type in ("latent_attention", "attention")], default=1)

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
            stages.append([D.AttendSplitKV(i, g, part, parts, extra=c) for g in range(_ceil_div(l.heads, 16)) for part in range(parts)
                           for c in range(_ceil_div(l.rank_s, ATTEND_COLUMNS))])
            stages.append([D.LatentValue(i, h, a, n, extra=parts) for h, a, n in cut([(h, l.v_s) for h in range(l.heads)], q)])
        D_s = self.shape.width_s
        stages.append([D.OutProject_Streams(i, 0, a, n) for _, a, n in cut([(0, D_s)], q, most=MAX_OUT_ROWS)])
        if l.ff:
            stages.append([D.RMS_UpGate_Gelu(i, 0, a, n) for _, a, n in cut([(0, l.ff_s)], q, most=MAX_ROWS // 2)])
            stages.append([D.OutProject_Streams(i, 1, a, n) for _, a, n in cut([(0, D_s)], q, most=MAX_OUT_ROWS)])
        return stages

    def _spread(self, parts: Sequence[tuple[int, Any]], busy: int = 0) -> list[D.StageInstruction]:
        """Row instructions of one stage, cut alike: ``parts`` are (rows, instruction of a start and a count); ``busy`` other
        instructions of the stage come before them."""
        queues = max(self.queues - busy, self.queues // 2, 1)
        return [parts[s][1](a, n) for s, a, n in cut([(k, rows) for k, (rows, _) in enumerate(parts)], queues)]

    def run_stages(self, first: int) -> list[list[D.StageInstruction]]:
        """Stages of the layer run whose branches start at entry ``first`` (plain residual)."""
        head = self.shape.entries[first]
        branches = {i: self.shape.entries[i].shape for i in range(first, first + head.branches)}
        width, ff = self.shape.width_s, self.shape.layers[head.layer].ff_s if head.ff else 0
        rows: list[tuple[int, Any]] = [(l.in_rows, lambda a, n, i=i: D.RMS_InProject(i, 0, a, n)) for i, l in branches.items()]
        down: list[tuple[int, Any]] = []
        if ff:
            rows.append((2 * ff, lambda a, n: D.RMS_UpGate_Gelu(first, 0, a // 2, n // 2)))
            down.append((width, lambda a, n: D.OutProject_Streams(first, 1, a, n)))
        stages = [self._spread(rows)]
        stages[0][0].extra = 1
        steps: list[D.StageInstruction] = []
        merges: list[D.StageInstruction] = []
        attend: list[D.StageInstruction] = []
        early: list[tuple[int, Any]] = []
        late: list[tuple[int, Any]] = []
        for i, l in branches.items():
            out = (width, lambda a, n, i=i: D.OutProject_Streams(i, 0, a, n))
            if l.type == "attention":
                parts = self.parts(i)
                attend += [D.AttendSplitKV(i, g, part, parts, extra=c) for part in range(parts) for g, c in self.attention_groups(l)]
                merges += [D.AttendMerge(i, h, 0, parts) for h in range(l.heads)]
                late.append(out)
            else:
                steps += [D.GatedStateStep(i, h, a, min(STATE_COLUMNS, l.v_s - a)) for h in range(l.heads) for a in range(0, l.v_s, STATE_COLUMNS)]
                if l.gate_rank:
                    steps += [D.OutputGate(i, 0, a, n) for _, a, n in cut([(0, l.mix_width)], self.gate_instructions)]
                early.append(out)
        if merges:
            stages += [steps + attend, merges + self._spread(early + down, len(merges)), self._spread(late)]
        else:
            stages += [steps + self._spread(down, len(steps)), self._spread(early)]
        return stages

    def stages(self) -> list[list[D.StageInstruction]]:
        out: list[list[D.StageInstruction]] = []
        last = len(self.shape.entries) - 1
        if not self.shape.plain:
            out = [s for i in range(len(self.shape.layers)) for s in self.layer_stages(i)]
        for i, e in enumerate(self.shape.entries if self.shape.plain else ()):
            if e.type == "join":
                out.append(self._spread([(self.shape.width_s, lambda a, n: D.JoinProject(i, 0, a, n))]))
            elif e.type != "final" and e.branch == 0:
                out += self.run_stages(i)
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
