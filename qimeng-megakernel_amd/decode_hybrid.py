"""Step function and host loop of the hybrid route.

``run_tokens`` feeds a request's next tokens — one, or a portion of a prompt — from the state earlier steps left, and
returns the logits asked for; ``decode`` is prefill + forced greedy decode with the timing of the other routes' loops
(`decode.py`).  A single token goes through the decode megakernel, several through the prefill kernels, in portions of at
most ``globs.portion_rows``.
"""
from __future__ import annotations

import time
from typing import Any, Sequence

import torch

from .decode_schedule_hybrid import mk_kernel as _mk_kernel
from .decode_schedule_hybrid.globs import Globals, build_globals
from .decode_schedule_hybrid.state import Request, RequestTable


def load(folder: Any, *, dtype: torch.dtype = torch.bfloat16, max_positions: int, slots: int = 1, device: torch.device | str = "cuda") -> Globals:
    """``Globals`` of a model folder (``config.json``, ``model.safetensors``)."""
    from .decode_schedule_hybrid import HybridConfig, weights

    shape, tensors = weights.read_checkpoint(folder)
    HybridConfig.set_shape(shape)
    return build_globals(shape, weights.pack(shape, tensors, device), dtype=dtype, slots=slots, max_positions=max_positions)


def _point_at(globs: Globals, request: Request) -> None:
    globs.slot, globs.position_id, globs.flip = request.slot, request.position, request.flip


def _advance(request: Request, tokens: int) -> None:
    request.position += tokens
    request.flip ^= 1


def run_tokens(globs: Globals, mk: Any, request: Request, tokens: Sequence[int] | torch.Tensor, want: Sequence[int] = ()) -> torch.Tensor:
    """Feed ``tokens``; logits fp32 ``[len(want), vocab]`` at the places ``want`` among them."""
    tokens = torch.as_tensor(tokens, dtype=torch.int64).to(globs.device)
    total, vocab = int(tokens.numel()), globs.shape.vocab
    if total == 0:
        raise ValueError("a step brings at least one token")
    if request.position + total > globs.max_positions:
        raise ValueError(f"{request.position + total} tokens do not fit a capacity of {globs.max_positions}")
    want = [int(w) for w in want]
    if any(not 0 <= w < total for w in want):
        raise IndexError("a wanted place lies outside the step's tokens")
    out = torch.empty(len(want), vocab, dtype=torch.float32, device=globs.device)
    for start in range(0, total, globs.portion_rows):
        part = tokens[start : start + globs.portion_rows]
        n = int(part.numel())
        rows = [k for k, w in enumerate(want) if start <= w < start + n]
        _point_at(globs, request)
        if n == 1:
            globs.token.copy_(part)
            _mk_kernel.call_mk(globs, mk)
            if rows:
                out[rows] = globs.logits[:vocab]
        else:
            places = sorted({want[k] - start for k in rows})
            logits = mk.prefill(globs, part.contiguous(), torch.tensor(places, dtype=torch.int32, device=globs.device) if places else None)
            for k in rows:
                out[k] = logits[places.index(want[k] - start), :vocab]
        _advance(request, n)
    return out


def generate_greedy_on_device(globs: Globals, mk: Any, request: Request, output_tokens: torch.Tensor, first: int, ntok: int, *,
                              events: list[tuple[torch.cuda.Event, torch.cuda.Event]] | None = None) -> int:
    """``ntok`` greedy steps with no host work between launches: step ``i`` reads ``output_tokens[first + i]`` and writes
    the token behind it."""
    for i in range(ntok):
        _point_at(globs, request)
        mk.read_from(output_tokens, first + i)
        mk.greedy_into(output_tokens, first + i + 1)
        if events is not None:
            events[i][0].record()
        _mk_kernel.call_mk(globs, mk)
        if events is not None:
            events[i][1].record()
        _advance(request, 1)
    return ntok


def decode(globs: Globals, prompt_ids: torch.Tensor, max_new_tokens: int, *, mk: Any = None, table: RequestTable | None = None, decode_time: bool = True,
           use_graph: bool = False, timed_steps: int | None = None) -> dict[str, Any]:
    """Prefill + forced greedy decode to exactly ``max_new_tokens`` tokens (no EOS stop).  ``use_graph``: the timed decode
    launches are captured into one HIP graph (positions are launch arguments, so the graph belongs to this request) and
    replayed.  ``timed_steps`` as in ``decode.decode``."""
    device, T = globs.device, int(prompt_ids.numel())
    if T < 1 or T + max_new_tokens > globs.max_positions:
        raise ValueError("the request does not fit the capacity")
    mk = mk or _mk_kernel.get_mk()
    table = table or RequestTable(globs)
    key = object()
    request = table.open(key)
    out = torch.zeros(T + max(max_new_tokens, 1), dtype=torch.long, device=device)
    out[:T] = prompt_ids.to(device)
    prefill_start, prefill_end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    prefill_start.record()
    logits = run_tokens(globs, mk, request, out[:T], [T - 1])
    prefill_end.record()
    out[T] = logits[0].argmax()
    total = max(max_new_tokens - 1, 0)
    ntok = total if timed_steps is None else max(0, min(int(timed_steps), total))
    lead = total - ntok
    generate_greedy_on_device(globs, mk, request, out, T, lead)
    graph = None
    if use_graph and ntok:
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):
            generate_greedy_on_device(globs, mk, request, out, T + lead, ntok)
    events = None
    if decode_time and graph is None:
        events = [(torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)) for _ in range(ntok)]
    loop_start, loop_end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    torch.cuda.synchronize(device)
    wall0 = time.perf_counter()
    loop_start.record()
    if graph is not None:
        graph.replay()
    else:
        generate_greedy_on_device(globs, mk, request, out, T + lead, ntok, events=events)
    loop_end.record()
    torch.cuda.synchronize(device)
    result: dict[str, Any] = {"generated_ids": out, "new_tokens": out[T:]}
    if decode_time and ntok:
        wall = time.perf_counter() - wall0
        gpu_s = loop_start.elapsed_time(loop_end) / 1e3
        per_step_ms = [a.elapsed_time(b) for a, b in events or []]
        kernel_s = sum(per_step_ms) / 1e3 if per_step_ms else float("inf")
        first = T + lead
        nbytes = sum(globs.shape.step_bytes(first + i + 1, globs.dtype.itemsize) for i in range(ntok))
        result["timing"] = {
            "prefill_gpu_s": prefill_start.elapsed_time(prefill_end) / 1e3, "decode_wall_s": wall, "decode_gpu_s": gpu_s, "mk_kernel_gpu_s": kernel_s,
            "effective_tok_s_wall": ntok / wall, "effective_tok_s_gpu": ntok / gpu_s, "kernel_tok_s": ntok / kernel_s,
            "kernel_steps": ntok, "kernel_ms_per_step": kernel_s * 1e3 / ntok, "first_timed_context": first + 1, "last_timed_context": first + ntok,
            "algorithmic_bytes": nbytes, "achieved_GBps": nbytes / kernel_s / 1e9, "per_step_ms": per_step_ms,
        }
    table.close(key)
    mk.check()
    return result
