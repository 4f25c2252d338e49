"""Checkpoint tensors of a hybrid decoder -> the storage the kernels stream.

Input: tensors by checkpoint name (``embed``, ``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.hc<q>.*``,
``final.norm``, ``head``), linear weights ``[out, in]``.  Output per layer: the input projections of a mixer stacked into
one matrix, matrices whose outputs meet element by element stored with their rows interleaved (gate/up, the two gates of
the recurrence), every block and head padded with zeros to its storage size.  bf16 matrices stay bf16 in every compute
mode; vectors become fp32 (both exactly).
"""
from __future__ import annotations

import json
from pathlib import Path
from typing import Mapping

import torch
import torch.nn.functional as F

from .model_config import HybridShape, LayerShape

Tensor = torch.Tensor


def read_checkpoint(folder: Path | str) -> tuple[HybridShape, dict[str, Tensor]]:
    """``config.json`` and ``model.safetensors`` of a model folder; every tensor the shape needs is there and fits."""
    from safetensors.torch import load_file

    folder = Path(folder)
    with open(folder / "config.json") as f:
        config = json.load(f)
    tensors = load_file(str(folder / "model.safetensors"))
    shape = HybridShape.from_config(config, {k: tuple(v.shape) for k, v in tensors.items()})
    check_tensors(shape, {k: tuple(v.shape) for k, v in tensors.items()})
    return shape, tensors


def tensor_shapes(shape: HybridShape) -> dict[str, tuple[int, ...]]:
    """Name -> shape of every checkpoint tensor of this model."""
    D, S = shape.width, shape.streams
    out: dict[str, tuple[int, ...]] = {"embed": (shape.vocab, D)}
    for i, l in enumerate(shape.layers):
        n = f"l{i}."
        m = n + "mix."
        out[n + "norm1"] = (D,)
        if l.ff:
            out[n + "norm2"] = (D,)
        if l.type == "rglru":
            W, b = l.lru_width, l.block
            out.update({m + "y": (W, D), m + "y.b": (W,), m + "x": (W, D), m + "x.b": (W,), m + "conv": (W, l.taps), m + "conv.b": (W,),
                        m + "ra": (l.blocks, b, b), m + "ra.b": (l.blocks, b), m + "ri": (l.blocks, b, b), m + "ri.b": (l.blocks, b),
                        m + "lam": (W,), m + "o": (D, W)})
        elif l.type == "latent_attention":
            H = l.heads
            out.update({m + "q": (H * (l.dim + l.rot_dim), D), m + "dkv": (l.rank + l.rot_dim, D), m + "dkv.norm": (l.rank,),
                        m + "uk": (H * l.dim, l.rank), m + "uv": (H * l.v_dim, l.rank), m + "g": (H * l.v_dim, D), m + "o": (D, H * l.v_dim)})
        else:
            N = l.heads * l.dim
            out.update({m + "mu." + s: (D,) for s in "rkvgw"})
            out.update({m + s: (N, D) for s in "rkvg"})
            out.update({m + "w1": (l.rank, D), m + "w2": (N, l.rank), m + "w0": (N,), m + "u": (l.heads, l.dim), m + "norm": (N,), m + "o": (D, N)})
        if l.ff:
            out.update({n + "mlp.gate": (l.ff, D), n + "mlp.up": (l.ff, D), n + "mlp.down": (D, l.ff)})
        for q in (1, 2) if l.ff else (1,):
            out.update({f"{n}hc{q}.in": (S,), f"{n}hc{q}.out": (S,), f"{n}hc{q}.mix": (S, S)})
    out["final.norm"] = (D,)
    out["head"] = (shape.vocab, D)
    return out


def check_tensors(shape: HybridShape, found: Mapping[str, tuple[int, ...]]) -> None:
    for name, want in tensor_shapes(shape).items():
        if name not in found:
            raise ValueError(f"the checkpoint has no tensor {name}")
        if tuple(found[name]) != want:
            raise ValueError(f"{name} has shape {tuple(found[name])}, the configuration says {want}")


def _pad(t: Tensor, *sizes: int) -> Tensor:
    """Zeros behind every dimension up to ``sizes``."""
    widths: list[int] = []
    for have, want in zip(reversed(t.shape), reversed(sizes)):
        widths += [0, want - have]
    return F.pad(t, widths) if any(widths) else t


def _rows(t: Tensor, groups: int, size: int, columns: int) -> Tensor:
    """[groups * n, c] -> [groups * size, columns]."""
    return _pad(t.reshape(groups, -1, t.shape[-1]), groups, size, columns).reshape(groups * size, columns)


def _columns(t: Tensor, rows: int, groups: int, size: int) -> Tensor:
    """[r, groups * n] -> [rows, groups * size]."""
    return _pad(t.reshape(t.shape[0], groups, -1), rows, groups, size).reshape(rows, groups * size)


def _vector(t: Tensor, groups: int, size: int) -> Tensor:
    return _pad(t.float().reshape(groups, -1), groups, size).reshape(-1)


def pack_layer(shape: HybridShape, i: int, w: Mapping[str, Tensor], device: torch.device | str) -> dict[str, Tensor]:
    l, D, Ds = shape.layers[i], shape.width, shape.width_s
    name = f"l{i}."

    def raw(key: str) -> Tensor:
        return w[name + key].to(device)

    def vec(key: str) -> Tensor:
        return _pad(raw(key).float(), Ds)

    p: dict[str, Tensor] = {"norm1": vec("norm1")}
    _PACK[l.type](l, Ds, lambda k: raw("mix." + k), p)
    if l.ff:
        gate, up = _pad(raw("mlp.gate"), l.ff_s, Ds), _pad(raw("mlp.up"), l.ff_s, Ds)
        p["norm2"] = vec("norm2")
        p["mlp_w"] = torch.stack((gate, up), dim=1).reshape(2 * l.ff_s, Ds)
        p["down_w"] = _pad(raw("mlp.down"), Ds, l.ff_s)
    p["hc"] = torch.cat([raw(f"hc{q}.{part}").float().reshape(-1) for q in ((1, 2) if l.ff else (1,)) for part in ("in", "out", "mix")])
    ones = torch.ones(shape.streams, device=device)

    def following(layer: int) -> Tensor:   # what reads the streams behind layer ``layer - 1``
        return w[f"l{layer}.hc1.in"].to(device).float() if layer < len(shape.layers) else ones

    p["next1"] = raw("hc2.in").float() if l.ff else following(i + 1)
    if l.ff:
        p["next2"] = following(i + 1)
    return {k: v.contiguous() for k, v in p.items()}


def _pack_rglru(l: LayerShape, Ds: int, raw, p: dict[str, Tensor]) -> None:
    B, n = l.blocks, l.block_s
    p["in_w"] = torch.cat([_rows(raw("y"), B, n, Ds), _rows(raw("x"), B, n, Ds)])
    p["in_b"] = torch.cat([_vector(raw("y.b"), B, n), _vector(raw("x.b"), B, n)])
    p["mid_w"] = torch.stack((_pad(raw("ra"), B, n, n), _pad(raw("ri"), B, n, n)), dim=2).reshape(B * 2 * n, n)
    p["mid_b"] = torch.stack((_vector(raw("ra.b"), B, n), _vector(raw("ri.b"), B, n)), dim=1).reshape(-1)
    p["vec0"] = _vector(-8.0 * F.softplus(raw("lam").double()).float(), B, n)
    p["vec1"] = _vector(raw("conv.b"), B, n)
    p["vec2"] = torch.stack([_vector(raw("conv")[:, j], B, n) for j in range(l.taps)])
    p["o_w"] = _columns(raw("o"), Ds, B, n)


def _pack_latent(l: LayerShape, Ds: int, raw, p: dict[str, Tensor]) -> None:
    H, dim, rot = l.heads, l.dim, l.rot_dim
    q = raw("q").reshape(H, dim + rot, -1)
    q = torch.cat([_pad(q[:, :dim], H, l.dim_s, Ds), _pad(q[:, dim:], H, l.q_stride - l.dim_s, Ds)], dim=1).reshape(H * l.q_stride, Ds)
    dkv = raw("dkv")
    p["in_w"] = torch.cat([q, _rows(raw("g"), H, l.v_s, Ds), _pad(dkv[: l.rank], l.rank_s, Ds), _pad(dkv[l.rank:], l.rot_s, Ds)])
    p["uk_w"] = _rows(raw("uk"), H, l.dim_s, l.rank_s)
    p["mid_w"] = p["uk_w"].reshape(H, l.dim_s, l.rank_s).transpose(1, 2).reshape(H * l.rank_s, l.dim_s)
    p["uv_w"] = _rows(raw("uv"), H, l.v_s, l.rank_s)
    p["vec0"] = _pad(raw("dkv.norm").float(), l.rank_s)
    p["o_w"] = _columns(raw("o"), Ds, H, l.v_s)


def _pack_wkv(l: LayerShape, Ds: int, raw, p: dict[str, Tensor]) -> None:
    H, n = l.heads, l.dim_s
    p["in_w"] = torch.cat([_rows(raw(s), H, n, Ds) for s in "rkvg"] + [_pad(raw("w1"), l.rank_s, Ds)])
    p["mid_w"] = _rows(raw("w2"), H, n, l.rank_s)
    p["mid_b"] = _vector(raw("w0"), H, n)
    p["vec0"] = _vector(raw("norm"), H, n)
    p["vec1"] = _pad(raw("u").float(), H, n).reshape(-1)
    p["vec2"] = torch.stack([_pad(raw("mu." + s).float(), Ds) for s in "rkvgw"])
    p["o_w"] = _columns(raw("o"), Ds, H, n)


_PACK = {"rglru": _pack_rglru, "latent_attention": _pack_latent, "wkv": _pack_wkv}


def pack(shape: HybridShape, tensors: Mapping[str, Tensor], device: torch.device | str) -> dict:
    """``{"embed", "head", "final_norm", "layers": [per-layer dict]}`` on ``device``."""
    bf16 = torch.bfloat16
    for name, t in tensors.items():
        if t.is_floating_point() and t.dtype != bf16:
            raise TypeError(f"{name} must be bfloat16, got {t.dtype}")
    return {
        "embed": _pad(tensors["embed"].to(device), shape.vocab_s, shape.width_s).contiguous(),
        "head": _pad(tensors["head"].to(device), shape.vocab_s, shape.width_s).contiguous(),
        "final_norm": _pad(tensors["final.norm"].to(device).float(), shape.width_s).contiguous(),
        "layers": [pack_layer(shape, i, tensors, device) for i in range(len(shape.layers))],
    }


def rope_tables(dims: int, base: float, positions: int) -> tuple[Tensor, Tensor]:
    """fp32 cos/sin of position x base^(-2i/dims), ``[positions, dims / 2]``, angles in fp64."""
    freq = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
    angle = torch.outer(torch.arange(positions, dtype=torch.float64), freq)
    return angle.cos().float().contiguous(), angle.sin().float().contiguous()
