"""Load and call the hybrid route's library (``include/qmk_hybrid.h``) through its C ABI.

``get_mk`` returns the callable, ``call_mk(globs, mk)`` runs one decode step of ``globs.slot`` at ``globs.position_id``,
``HybridMegaKernel.prefill`` one portion of a prompt.  As in the other routes tensors cross the boundary as device
pointers, launches go onto torch's current stream, and there is no fallback: a missing library is an ``ImportError``, a
tensor off the GPU a ``ValueError``, a device-side error a ``RuntimeError``.
"""
from __future__ import annotations

import ctypes
from pathlib import Path
from typing import Any, Optional

import torch

from .globs import Globals
from .instructions import scheduler as _scheduler

_LIBRARY_NAME = "libqmk_hybrid.so"
_P, _I, _F = ctypes.c_void_p, ctypes.c_int32, ctypes.c_float
QMK_NORM_LAYER = QMK_ACT_SILU = 1      # include/qmk_hybrid.h
_ERRORS = {1: "null argument", 2: "struct_size does not match the library", 3: "dimension out of range", 4: "position outside the request's capacity",
           5: "more instruction queues than co-resident workgroups", 6: "no usable HIP device", 7: "kernel launch failed", 8: "unknown element type",
           9: "workspace too small", 32: "device: unknown opcode", 33: "device: instruction operand out of bounds",
           34: "device: counter wait ran out of polls"}

#: pointer fields of the layer table = keys of a layer's weight and state tensors
_LAYER_POINTERS = ("norm1", "norm2", "in_w", "in_b", "mid_w", "mid_b", "gate_w", "uk_w", "uv_w", "o_w", "mlp_w", "down_w", "vec0", "vec1", "vec2", "rope_cos",
                   "rope_sin", "hc", "next1", "next2", "out_norm", "cache", "state", "shift")


class QmkHybridLayer(ctypes.Structure):
    """Mirror of ``struct QmkHybridLayer`` (field order is the ABI)."""

    _fields_ = [(n, _I) for n in ("type", "has_mlp", "in_rows", "mix_width", "heads", "head_dim", "head_dim_true", "rot_dim", "rot_true", "q_stride",
                                  "v_dim", "rank", "rank_true", "window", "ring", "taps", "blocks", "block_dim", "ff")]
    _fields_ += [("scale", _F)]
    _fields_ += [(n, _I) for n in ("kv_heads", "v_true", "gate_rank", "norm", "act", "branch", "branches", "prev", "x_from", "x_to", "proj_at", "mix_at", "ff_at")]
    _fields_ += [(n, _F) for n in ("q_scale", "decay_scale", "out_scale")] + [(n, _P) for n in _LAYER_POINTERS]


class QmkHybridArgs(ctypes.Structure):
    """Mirror of ``struct QmkHybridArgs``."""

    _fields_ = [(n, ctypes.c_uint32) for n in ("struct_size", "dtype", "flags", "spin_limit")]
    _fields_ += [("layers", _P), ("layers_device", _P)]
    _fields_ += [(n, _I) for n in ("num_layers", "width", "width_true", "streams", "vocab", "vocab_rows", "slots", "slot", "position", "max_positions",
                                   "flip", "tokens", "num_want", "portion_rows")]
    _fields_ += [("eps", _F), ("logit_scale", _F), ("logit_softcap", _F), ("reserved0", _I)]
    _fields_ += [(n, _P) for n in ("embed", "final_norm", "head", "token_in", "token_out", "want", "logits", "layer_out", "workspace")]
    _fields_ += [("workspace_bytes", ctypes.c_uint64), ("instructions", _P), ("barriers", _P)]
    _fields_ += [(n, _I) for n in ("num_queues", "num_insts", "barrier_groups", "max_splits")]
    _fields_ += [("timeline", _P), ("stream", _P)]


def load_library(mk_dir: Path | None = None) -> ctypes.CDLL:
    root = (Path(__file__).resolve().parent.parent if mk_dir is None else Path(mk_dir)).resolve()
    dso = root / _LIBRARY_NAME
    if not dso.is_file():
        raise ImportError(f"missing prebuilt kernel {dso}; build it first (python -c 'import __graft_entry__ as g; g.build()')")
    try:
        lib = ctypes.CDLL(str(dso))
    except OSError as exc:
        raise ImportError(f"cannot load prebuilt kernel {dso}: {exc}") from exc
    for name in ("qmk_hybrid_decode_step", "qmk_hybrid_prefill"):
        getattr(lib, name).argtypes = [ctypes.POINTER(QmkHybridArgs)]
        getattr(lib, name).restype = ctypes.c_int
    for name in ("qmk_hybrid_decode_bytes", "qmk_hybrid_prefill_bytes"):
        getattr(lib, name).argtypes = [ctypes.POINTER(QmkHybridArgs)]
        getattr(lib, name).restype = ctypes.c_uint64
    lib.qmk_hybrid_status_fetch.argtypes = [_P, ctypes.POINTER(_I * 4)]
    lib.qmk_hybrid_status_fetch.restype = ctypes.c_int
    return lib


def layer_table(globs: Globals) -> ctypes.Array:
    """The layer table of ``globs``, one entry per entry of its shape: sizes from the shape, pointers from the tensors."""
    entries = globs.shape.entries
    table = (QmkHybridLayer * len(entries))()
    proj_at = mix_at = 0
    for i, entry in enumerate(entries):
        e, l = table[i], entry.shape
        e.type, e.has_mlp, e.ff = l.mixer, int(entry.ff > 0), globs.shape.layers[entry.layer].ff_s if entry.ff else 0
        if globs.shape.plain:   # a run's branches side by side in the buffers of a step, its feed-forward behind them
            if entry.branch == 0:
                proj_at = mix_at = 0
            e.norm, e.act = QMK_NORM_LAYER, QMK_ACT_SILU
            e.branch, e.branches, e.prev, e.x_from, e.x_to = entry.branch, entry.branches, entry.prev, entry.x_from, entry.x_to
            e.out_scale = 1.0 / entry.branches
            e.proj_at, e.mix_at = proj_at, mix_at
        if l.type not in ("join", "final"):
            e.in_rows, e.mix_width, e.heads, e.kv_heads = l.in_rows, l.mix_width, l.heads, l.kv_heads
            proj_at, mix_at = proj_at + l.in_rows + (l.mix_width if l.type == "delta" else 0), mix_at + l.mix_width
        if entry.ff and globs.shape.plain:
            e.ff_at = sum(b.shape.mix_width for b in entries[i : i + entry.branches])
        if l.type == "latent_attention":
            e.head_dim, e.rot_dim, e.rot_true, e.q_stride, e.v_dim = l.dim_s, l.rot_s, l.rot_dim, l.q_stride, l.v_s
            e.rank, e.rank_true, e.scale = l.rank_s, l.rank, l.scale
            e.window, e.ring = min(l.window, globs.max_positions), globs.layer_state[i]["cache"].shape[1]
        elif l.type == "attention":
            e.head_dim, e.rot_true, e.q_stride, e.v_dim, e.scale = l.dim_s, l.rot_dim, l.q_stride, l.v_s, l.scale
            e.window, e.ring = globs.max_positions, globs.layer_state[i]["cache"].shape[1]
        elif l.type in ("delta", "gla"):
            e.head_dim, e.v_dim, e.v_true, e.rank, e.gate_rank, e.taps = l.dim_s, l.v_s, l.v_dim, l.rank_s, l.gate_rank_s, l.taps
            e.q_scale, e.decay_scale = l.dim**-0.5, 1.0 / l.tau if l.tau else 0.0
        elif l.type == "rglru":
            e.taps, e.blocks, e.block_dim = l.taps, l.blocks, l.block_s
        elif l.type == "wkv":
            e.head_dim, e.head_dim_true, e.rank = l.dim_s, l.dim, l.rank_s
        tensors = {**globs.layer_weights[i], **globs.layer_state[i]}
        for name, t in tensors.items():
            if not t.is_contiguous() or t.data_ptr() % 16:
                raise ValueError(f"layer {i}: {name} must be contiguous and 16-byte aligned")
            setattr(e, name, t.data_ptr() if t.numel() else None)
    return table


class HybridMegaKernel:
    """The ``mk`` callable of this route, bound to one ``Globals`` at a time.

    ``mk(globs)``: one decode step.  ``mk.greedy_into(tokens, index)`` arms device-side sampling for the next step: it
    writes its greedy token there.  ``mk.read_from(tokens, index)`` makes the next step read its token there instead of
    ``globs.token``; a chain of both needs no host work between launches.  ``mk.prefill`` runs a portion."""

    def __init__(self, lib: ctypes.CDLL, *, spin_limit: int = 0):
        self._lib = lib
        self.spin_limit = int(spin_limit)
        self.timeline: Optional[torch.Tensor] = None
        self._key: tuple | None = None
        self._greedy: tuple[torch.Tensor, int] | None = None
        self._source: tuple[torch.Tensor, int] | None = None

    def _bind(self, g: Globals) -> None:
        if g.instructions is None:   # a step needs all its workgroups on the chip at once
            _scheduler.build(g, max(1, min(_scheduler.MI355X_QUEUES, int(self._lib.qmk_hybrid_max_queues()))))
        key = (id(g), g.instructions.data_ptr(), g.barriers.data_ptr())
        if key == self._key:
            return
        device = g.embed_tokens.device
        if device.type != "cuda":
            raise ValueError(f"the weights must live on the GPU, got {device}")
        self._globs, self._key = g, key
        self._table = layer_table(g)
        raw = torch.frombuffer(bytearray(bytes(self._table)), dtype=torch.uint8)
        self._table_device = raw.to(device)
        a = self._args = QmkHybridArgs()
        s = g.shape
        a.struct_size = ctypes.sizeof(QmkHybridArgs)
        a.dtype = 1 if g.dtype == torch.float32 else 0
        a.layers, a.layers_device = ctypes.addressof(self._table), self._table_device.data_ptr()
        a.num_layers, a.width, a.width_true, a.streams = len(s.entries), s.width_s, s.width, s.streams
        a.vocab, a.vocab_rows, a.eps, a.logit_scale, a.logit_softcap = s.vocab, s.vocab_s, s.eps, s.logit_scale, s.logit_softcap
        a.slots, a.max_positions, a.portion_rows = g.slots, g.max_positions, g.portion_rows
        a.embed, a.final_norm, a.head = g.embed_tokens.data_ptr(), g.lm_head_norm_weights.data_ptr(), g.lm_head_weights.data_ptr()
        a.instructions, a.barriers = g.instructions.data_ptr(), g.barriers.data_ptr()
        a.num_queues, a.num_insts, a.barrier_groups = g.instructions.shape[0], g.instructions.shape[1], g.barriers.shape[0]
        a.max_splits = g.instruction_splits
        sizes = [int(f(ctypes.byref(a))) for f in (self._lib.qmk_hybrid_decode_bytes, self._lib.qmk_hybrid_prefill_bytes)]
        if min(sizes) == 0:
            raise ValueError("the kernels do not support a size of this model (limits: qmk_hybrid_ops.h)")
        self._decode_ws, self._prefill_ws = (torch.zeros(n, dtype=torch.uint8, device=device) for n in sizes)

    def _raise(self, what: str, code: int) -> None:
        raise RuntimeError(f"{what} failed with {code}: {_ERRORS.get(code, 'unknown code')}")

    def greedy_into(self, tokens: torch.Tensor, index: int) -> None:
        self._greedy = self._token_slot(tokens, index)

    def read_from(self, tokens: torch.Tensor, index: int) -> None:
        self._source = self._token_slot(tokens, index)

    @staticmethod
    def _token_slot(tokens: torch.Tensor, index: int) -> tuple[torch.Tensor, int]:
        if tokens.dtype != torch.int64 or not tokens.is_contiguous() or tokens.device.type != "cuda":
            raise TypeError("tokens must be a contiguous int64 tensor on the GPU")
        if not 0 <= index < tokens.numel():
            raise IndexError(f"token index {index} outside a buffer of {tokens.numel()}")
        return tokens, index

    def __call__(self, g: Globals) -> None:
        self._bind(g)
        a = self._args
        a.slot, a.position, a.flip, a.spin_limit = g.slot, g.position_id, g.flip, self.spin_limit
        source, greedy, self._source, self._greedy = self._source, self._greedy, None, None
        a.token_in = g.token.data_ptr() if source is None else source[0].data_ptr() + 8 * source[1]
        a.token_out = None if greedy is None else greedy[0].data_ptr() + 8 * greedy[1]
        a.logits, a.tokens, a.num_want = g.logits.data_ptr(), 1, 0
        a.workspace, a.workspace_bytes = self._decode_ws.data_ptr(), self._decode_ws.numel()
        a.timeline = self.timeline.data_ptr() if self.timeline is not None else None
        a.stream = torch.cuda.current_stream(g.device).cuda_stream
        rc = int(self._lib.qmk_hybrid_decode_step(ctypes.byref(a)))
        if rc:
            self._raise("qmk_hybrid_decode_step", rc)

    def prefill(self, g: Globals, tokens: torch.Tensor, want: Optional[torch.Tensor] = None, *, layer_out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """One portion at ``g.position_id`` of ``g.slot``: ``tokens`` int64 on the GPU, ``want`` int32 places (or None).
        Returns the logits ``[len(want), storage vocabulary]``."""
        self._bind(g)
        n = 0 if want is None else int(want.numel())
        for name, t, dtype in (("tokens", tokens, torch.int64), ("want", want, torch.int32), ("layer_out", layer_out, torch.float32)):
            if t is not None and (t.dtype != dtype or not t.is_contiguous() or t.device != g.device):
                raise ValueError(f"{name} must be contiguous {dtype} on {g.device}")
        M = int(tokens.numel())
        if not 1 <= M <= g.portion_rows:
            raise ValueError(f"a portion holds 1..{g.portion_rows} tokens, got {M}")
        if layer_out is not None and tuple(layer_out.shape) != (g.shape.run_count, M, g.shape.width_s):
            raise ValueError("layer_out must be [layer runs, tokens, storage width]")
        logits = torch.empty(n, g.shape.vocab_s, dtype=torch.float32, device=g.device)
        a = self._args
        a.slot, a.position, a.flip, a.tokens, a.num_want = g.slot, g.position_id, g.flip, M, n
        a.token_in, a.token_out, a.want = tokens.data_ptr(), None, want.data_ptr() if n else None
        a.logits, a.layer_out = logits.data_ptr() if n else None, layer_out.data_ptr() if layer_out is not None else None
        a.workspace, a.workspace_bytes = self._prefill_ws.data_ptr(), self._prefill_ws.numel()
        a.stream = torch.cuda.current_stream(g.device).cuda_stream
        rc = int(self._lib.qmk_hybrid_prefill(ctypes.byref(a)))
        a.layer_out = None
        if rc:
            self._raise("qmk_hybrid_prefill", rc)
        return logits

    def check(self) -> None:
        """Synchronise and raise if a decode step reported a device-side error (its counters are then cleared)."""
        if self._key is None:
            return
        detail = (_I * 4)()
        code = int(self._lib.qmk_hybrid_status_fetch(_P(torch.cuda.current_stream(self._globs.device).cuda_stream), ctypes.byref(detail)))
        if code:
            self._globs.barriers.zero_()
            raise RuntimeError(f"hybrid megakernel error {code} ({_ERRORS.get(code, 'unknown code')}): workgroup={detail[0]} instruction={detail[1]} "
                               f"opcode={detail[2]} operand={detail[3]}")


_LIB_CACHE: dict[Any, ctypes.CDLL] = {}


def get_mk(mk_dir: Path | None = None, *, spin_limit: int = 0) -> HybridMegaKernel:
    if mk_dir not in _LIB_CACHE:
        _LIB_CACHE[mk_dir] = load_library(mk_dir)
    return HybridMegaKernel(_LIB_CACHE[mk_dir], spin_limit=spin_limit)


def call_mk(globs: Globals, mk: HybridMegaKernel) -> None:
    """One decode step (builds the instruction tensor on first use)."""
    mk(globs)
