"""Checkpoint tensors of a hybrid decoder -> the storage the kernels stream.

Input: tensors by checkpoint name (``embed``, ``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.hc<q>.*``,
``final.norm``, ``head``; a looped model also ``loop.in``, a mixer of two branches ``l<i>.mix.left.*`` and
``l<i>.mix.right.*``), linear weights ``[out, in]``.  Output per entry of ``HybridShape.entries`` (a looped layer's passes
share theirs): the input projections of a mixer stacked into one matrix, matrices whose outputs meet element by element
stored with their rows interleaved (gate/up, the two gates of the recurrence), every block and head padded with zeros to
its storage size.  bf16 matrices stay bf16 in every compute
mode; vectors become fp32 (both exactly).
"""
from __future__ import annotations

import json
import math
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
    if shape.loop is not None:
        out["loop.in"] = (D, 2 * D)
    for i, l in enumerate(shape.layers):
        n = f"l{i}."
        m = n + "mix."
        out[n + "norm1"] = (D,)
        if l.ff and not shape.plain:
            out[n + "norm2"] = (D,)
        if l.type == "gla":
            out.update(_gla_shapes(l, m, D))
        elif l.type == "parallel":
            out.update(_attention_shapes(l.branches[0], m + "left.", D))
            out.update(_delta_shapes(l.branches[1], m + "right.", D))
            out.update({m + "left.out": (D,), m + "right.out": (D,)})
        elif l.type == "rglru":
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
        for q in () if shape.plain else (1, 2) if l.ff else (1,):
            out.update({f"{n}hc{q}.in": (S,), f"{n}hc{q}.out": (S,), f"{n}hc{q}.mix": (S, S)})
    out["final.norm"] = (D,)
    out["head"] = (shape.vocab, D)
    return out


def _attention_shapes(l: LayerShape, m: str, D: int) -> dict[str, tuple[int, ...]]:
    H, G = l.heads, l.kv_heads
    return {m + "q": (H * l.dim, D), m + "k": (G * l.dim, D), m + "v": (G * l.v_dim, D), m + "g": (H * l.v_dim, D), m + "o": (D, H * l.v_dim)}


def _delta_shapes(l: LayerShape, m: str, D: int) -> dict[str, tuple[int, ...]]:
    H, G = l.heads, l.kv_heads
    out: dict[str, tuple[int, ...]] = {}
    for name, rows in (("q", G * l.dim), ("k", G * l.dim), ("v", H * l.v_dim)):
        out[m + name] = (rows, D)
        out[m + name + ".conv"] = (rows, l.taps)
    out.update({m + "b": (H, D), m + "A_log": (H,), m + "norm": (l.v_dim,), m + "a1": (l.rank, D), m + "a2": (H * l.dim, l.rank),
                m + "dt_bias": (H * l.dim,), m + "g1": (l.gate_rank, D), m + "g2": (H * l.v_dim, l.gate_rank), m + "o": (D, H * l.v_dim)})
    return out


def _gla_shapes(l: LayerShape, m: str, D: int) -> dict[str, tuple[int, ...]]:
    H = l.heads
    return {m + "q": (H * l.dim, D), m + "k": (H * l.dim, D), m + "v": (H * l.v_dim, D), m + "g": (H * l.v_dim, D), m + "o": (D, H * l.v_dim),
            m + "norm": (l.v_dim,), m + "a1": (l.rank, D), m + "a2": (H * l.dim, l.rank), m + "a2.b": (H * l.dim,)}


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


def _pack_attention(l: LayerShape, Ds: int, raw, p: dict[str, Tensor]) -> None:
    H, G = l.heads, l.kv_heads
    p["in_w"] = torch.cat([_rows(raw("q"), H, l.q_stride, Ds), _rows(raw("k"), G, l.dim_s, Ds), _rows(raw("v"), G, l.v_s, Ds), _rows(raw("g"), H, l.v_s, Ds)])
    p["o_w"] = _columns(raw("o"), Ds, H, l.v_s)


def _pack_delta(l: LayerShape, Ds: int, raw, p: dict[str, Tensor]) -> None:
    H, G = l.heads, l.kv_heads
    parts = (("q", G, l.dim_s), ("k", G, l.dim_s), ("v", H, l.v_s))
    p["in_w"] = torch.cat([_rows(raw(name), n, size, Ds) for name, n, size in parts]
                          + [_pad(raw("a1"), l.rank_s, Ds), _pad(raw("g1"), l.gate_rank_s, Ds), _pad(raw("b"), l.heads_s, Ds)])
    p["mid_w"] = _rows(raw("a2"), H, l.dim_s, l.rank_s)
    p["gate_w"] = _rows(raw("g2"), H, l.v_s, l.gate_rank_s)
    p["mid_b"] = _vector(raw("dt_bias"), H, l.dim_s)
    p["vec0"] = _pad(raw("norm").float(), l.v_s)
    p["vec1"] = _pad(-torch.exp(raw("A_log").double()).float(), l.heads_s)
    p["vec2"] = torch.stack([torch.cat([_vector(raw(name + ".conv")[:, j], n, size) for name, n, size in parts]) for j in range(l.taps)])
    p["o_w"] = _columns(raw("o"), Ds, H, l.v_s)


def _pack_gla(l: LayerShape, Ds: int, raw, p: dict[str, Tensor]) -> None:
    H = l.heads
    p["in_w"] = torch.cat([_rows(raw("q"), H, l.dim_s, Ds), _rows(raw("k"), H, l.dim_s, Ds), _rows(raw("v"), H, l.v_s, Ds), _rows(raw("g"), H, l.v_s, Ds),
                           _pad(raw("a1"), l.rank_s, Ds)])
    p["mid_w"] = _rows(raw("a2"), H, l.dim_s, l.rank_s)
    p["mid_b"] = _vector(raw("a2.b"), H, l.dim_s)
    p["vec0"] = _pad(raw("norm").float(), l.v_s)
    p["o_w"] = _columns(raw("o"), Ds, H, l.v_s)


_PACK_BRANCH = {"attention": _pack_attention, "delta": _pack_delta, "gla": _pack_gla}


def pack_branches(shape: HybridShape, i: int, w: Mapping[str, Tensor], device: torch.device | str) -> list[dict[str, Tensor]]:
    """One dict per branch of layer ``i`` of a plain residual; norm and feed-forward are the first one's."""
    l, Ds, name = shape.layers[i], shape.width_s, f"l{i}."

    def raw(key: str) -> Tensor:
        return w[name + key].to(device)

    out = []
    for side, part in (("left.", l.branches[0]), ("right.", l.branches[1])) if l.branches else (("", l),):
        p: dict[str, Tensor] = {}
        _PACK_BRANCH[part.type](part, Ds, lambda k: raw("mix." + side + k), p)
        if l.branches:
            p["out_norm"] = _pad(raw(f"mix.{side}out").float(), Ds)
        out.append(p)
    out[0]["norm1"] = _pad(raw("norm1").float(), Ds)
    if l.ff:
        out[0]["mlp_w"] = torch.stack((_pad(raw("mlp.gate"), l.ff_s, Ds), _pad(raw("mlp.up"), l.ff_s, Ds)), dim=1).reshape(2 * l.ff_s, Ds)
        out[0]["down_w"] = _pad(raw("mlp.down"), Ds, l.ff_s)
    return [{k: v.contiguous() for k, v in p.items()} for p in out]


def _pack_plain(shape: HybridShape, tensors: Mapping[str, Tensor], device: torch.device | str) -> list[dict[str, Tensor]]:
    layers = [pack_branches(shape, i, tensors, device) for i in range(len(shape.layers))]
    model = {"final": {"norm1": _pad(tensors["final.norm"].to(device).float(), shape.width_s)}}
    if shape.loop is not None:
        model["join"] = {"in_w": _columns(tensors["loop.in"].to(device), shape.width_s, 2, shape.width_s).contiguous()}
    return [model[e.type] if e.layer < 0 else layers[e.layer][e.branch] for e in shape.entries]


_PACK = {"rglru": _pack_rglru, "latent_attention": _pack_latent, "wkv": _pack_wkv}


def pack(shape: HybridShape, tensors: Mapping[str, Tensor], device: torch.device | str) -> dict:
    """``{"embed", "head", "final_norm", "layers": [dict per entry of the shape]}`` on ``device``."""
    bf16 = torch.bfloat16
    for name, t in tensors.items():
        if t.is_floating_point() and t.dtype != bf16:
            raise TypeError(f"{name} must be bfloat16, got {t.dtype}")
    return {
        "embed": _pad(tensors["embed"].to(device), shape.vocab_s, shape.width_s).contiguous(),
        "head": _pad(tensors["head"].to(device), shape.vocab_s, shape.width_s).contiguous(),
        "final_norm": _pad(tensors["final.norm"].to(device).float(), shape.width_s).contiguous(),
        "layers": _pack_plain(shape, tensors, device) if shape.plain else [pack_layer(shape, i, tensors, device) for i in range(len(shape.layers))],
    }


def rope_frequencies(dims: int, base: float, scaling: tuple[float, float, float, float] | None = None) -> tuple[Tensor, float]:
    """Angle per position of every pair (fp64) and the factor on cos and sin.  ``scaling`` (factor, original, fast, slow) is
    YaRN's: pairs that turn less than ``slow`` times in ``original`` positions are interpolated by ``factor``, those that turn
    more than ``fast`` times are not, with a linear ramp over the pair number between them."""
    freq = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / max(dims, 1))
    if scaling is None:
        return freq, 1.0
    factor, original, fast, slow = scaling
    low, high = (dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base)) for turns in (fast, slow))
    low, high = max(math.floor(low), 0), min(math.ceil(high), dims - 1)
    ramp = ((torch.arange(dims // 2, dtype=torch.float64) - low) / max(high - low, 0.001)).clamp(0.0, 1.0)
    return freq / factor * ramp + freq * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rope_tables(dims: int, base: float, positions: int, scaling: tuple[float, float, float, float] | None = None) -> tuple[Tensor, Tensor]:
    """fp32 cos/sin of position x frequency, ``[positions, dims / 2]``, angles in fp64."""
    freq, magnitude = rope_frequencies(dims, base, scaling)
    angle = torch.outer(torch.arange(positions, dtype=torch.float64), freq)
    return (angle.cos() * magnitude).float().contiguous(), (angle.sin() * magnitude).float().contiguous()
