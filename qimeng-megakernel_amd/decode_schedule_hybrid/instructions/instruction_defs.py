"""The opcodes of the hybrid decode route and their stage protocol.

Every instruction carries the same nine operands.  ``layer`` indexes the layer table; ``sub`` is the wkv input (r, k, v,
g, decay), the gate block, the head, the group of at most sixteen heads (of one key head, where there are several), or
0 / 1 for the output / down projection; ``start`` and ``count`` are output rows (pairs of rows for opcodes 2 and 8, part
number and number of parts for opcode 4).

A step is a chain of stages.  An instruction waits until ``wait_count`` arrivals are counted on ``wait_stage`` (-1: none)
and counts one arrival on ``arrive_stage``; the schedule's stages are all-to-all, so ``wait_count`` is the number of
instructions of the stage before.  Stage s is counted in group ``s // 4`` of ``barriers`` on counter row ``2 + s % 4`` of
the dense route's layout, one line per XCD.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import ClassVar

from ...instruction import Instruction


@dataclass
class NoOp(Instruction):
    OPCODE: ClassVar[int] = 0


@dataclass
class StageInstruction(Instruction):
    layer: int
    sub: int
    start: int
    count: int
    wait_stage: int = -1
    wait_count: int = 0
    arrive_stage: int = -1
    extra: int = 0


@dataclass
class RMS_InProject(StageInstruction):
    """Norm + the mixer's stacked input projections; convolution, rotation, gates where they act per output.
    ``extra`` = 1: also keeps the normed input for the next token (wkv), or the residual for its next reader (plain)."""
    OPCODE: ClassVar[int] = 1


@dataclass
class GatedRecurrence(StageInstruction):
    OPCODE: ClassVar[int] = 2


@dataclass
class LatentAbsorb(StageInstruction):
    """``extra`` = 1: also norms the latent and appends the cache row."""
    OPCODE: ClassVar[int] = 3


@dataclass
class AttendSplitKV(StageInstruction):
    """Over latents or over keys and values.  ``extra``: which 128 columns of the latent or value."""
    OPCODE: ClassVar[int] = 4


@dataclass
class LatentValue(StageInstruction):
    """``extra``: number of parts to merge."""
    OPCODE: ClassVar[int] = 5


@dataclass
class WkvStep(StageInstruction):
    OPCODE: ClassVar[int] = 6


@dataclass
class OutProject_Streams(StageInstruction):
    """On a plain residual the rows are left for the residual's next reader to add."""
    OPCODE: ClassVar[int] = 7


@dataclass
class RMS_UpGate_Gelu(StageInstruction):
    OPCODE: ClassVar[int] = 8


@dataclass
class RMS_LMHead(StageInstruction):
    OPCODE: ClassVar[int] = 9


@dataclass
class GatedStateStep(StageInstruction):
    """Value columns ``start`` .. of one head of a gated linear attention or gated delta rule: decays and recurrence.  The
    output projection norms the head and applies the gate."""
    OPCODE: ClassVar[int] = 10


@dataclass
class AttendMerge(StageInstruction):
    """Merge of ``count`` parts of one head and the output gate."""
    OPCODE: ClassVar[int] = 11


@dataclass
class JoinProject(StageInstruction):
    """Rows of the residual a pass of the loop starts from."""
    OPCODE: ClassVar[int] = 12


@dataclass
class OutputGate(StageInstruction):
    """Rows of a low-rank output gate."""
    OPCODE: ClassVar[int] = 13


INSTRUCTIONS = {c.OPCODE: c for c in (NoOp, RMS_InProject, GatedRecurrence, LatentAbsorb, AttendSplitKV, LatentValue, WkvStep,
                                      OutProject_Streams, RMS_UpGate_Gelu, RMS_LMHead, GatedStateStep, AttendMerge, JoinProject, OutputGate)}
