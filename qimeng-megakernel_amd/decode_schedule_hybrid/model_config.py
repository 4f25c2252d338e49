"""Model shape of the hybrid route: a list of layers, each with its own mixer and sizes.

``HybridShape.from_config`` reads a model folder's ``config.json`` (architecture ``Lusupel``):
``width``, ``vocab``, ``streams``, ``norm.eps`` and ``layers``, each ``{type, mixer, mlp}``.  Nothing but these keys
enters a computation; storage sizes (``*_s`` properties) are the true sizes rounded up to what the kernels read.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Mapping

ARCHITECTURE = "Lusupel"
MIXERS = ("rglru", "latent_attention", "wkv")   # place = the kernels' mixer number


def storage(n: int, multiple: int = 16) -> int:
    """Storage size of ``n`` elements: rows start on 16-byte boundaries, a lane owns four neighbouring outputs."""
    return (n + multiple - 1) // multiple * multiple


@dataclasses.dataclass(frozen=True)
class LayerShape:
    type: str
    ff: int = 0                 # 0: no feed-forward
    # rglru
    lru_width: int = 0
    blocks: int = 0
    taps: int = 0
    # latent_attention; ``heads`` and ``dim`` also wkv
    heads: int = 0
    dim: int = 0
    rot_dim: int = 0
    v_dim: int = 0
    rank: int = 0               # latent size; wkv: rank of the decay's first matrix (from the weights)
    window: int = 0
    rope_base: float = 0.0
    scale: float = 0.0

    @property
    def mixer(self) -> int:
        return MIXERS.index(self.type)

    @property
    def block(self) -> int:
        return self.lru_width // self.blocks

    @property
    def block_s(self) -> int:
        return storage(self.block)

    @property
    def dim_s(self) -> int:
        return storage(self.dim)

    @property
    def rot_s(self) -> int:
        return storage(self.rot_dim)

    @property
    def v_s(self) -> int:
        return storage(self.v_dim)

    @property
    def rank_s(self) -> int:
        return storage(self.rank)

    @property
    def ff_s(self) -> int:
        return storage(self.ff)

    @property
    def q_stride(self) -> int:
        return storage(self.dim_s + self.rot_s, 32)

    @property
    def mix_width(self) -> int:
        """Storage width of what the mixer hands to its output projection."""
        if self.type == "rglru":
            return self.blocks * self.block_s
        return self.heads * (self.v_s if self.type == "latent_attention" else self.dim_s)

    @property
    def in_rows(self) -> int:
        if self.type == "rglru":
            return 2 * self.mix_width
        if self.type == "latent_attention":
            return self.heads * (self.q_stride + self.v_s) + self.rank_s + self.rot_s
        return 4 * self.mix_width + self.rank_s

    def weight_count(self, width: int) -> int:
        """Matrix elements one token has to stream (norms, biases and taps aside)."""
        if self.type == "rglru":
            n = 3 * self.lru_width * width + 2 * self.lru_width * self.block
        elif self.type == "latent_attention":
            n = width * (self.heads * (self.dim + self.rot_dim + 2 * self.v_dim) + self.rank + self.rot_dim) + self.heads * self.rank * (self.dim + self.v_dim)
        else:
            n = 5 * self.heads * self.dim * width + self.rank * (width + self.heads * self.dim)
        return n + 3 * self.ff * width


@dataclasses.dataclass(frozen=True)
class HybridShape:
    layers: tuple[LayerShape, ...]
    width: int
    vocab: int
    streams: int
    eps: float

    @property
    def width_s(self) -> int:
        return storage(self.width)

    @property
    def vocab_s(self) -> int:
        return storage(self.vocab)

    @classmethod
    def from_config(cls, config: Mapping[str, Any], tensor_shapes: Mapping[str, tuple[int, ...]] | None = None) -> "HybridShape":
        """``tensor_shapes`` names the checkpoint's tensors: it gives the one size that no key names, the decay's rank."""
        layers = []
        for i, entry in enumerate(config["layers"]):
            kind, m, mlp = entry["type"], entry["mixer"], entry.get("mlp")
            if kind not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp.get('kind')!r}")
            kw: dict[str, Any] = dict(type=kind, ff=int(mlp["ff"]) if mlp is not None else 0)
            if kind == "rglru":
                kw.update(lru_width=int(m["width"]), blocks=int(m["blocks"]), taps=int(m["conv"]))
                if kw["lru_width"] % kw["blocks"]:
                    raise ValueError(f"layer {i}: {kw['blocks']} blocks do not divide a width of {kw['lru_width']}")
            elif kind == "latent_attention":
                rot = m["rot"]
                if int(rot["dims"]) != int(m["rot_dim"]) or int(rot["dims"]) % 2:
                    raise ValueError(f"layer {i}: rotated dimensions {rot['dims']} of a rotated part of {m['rot_dim']}")
                kw.update(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), v_dim=int(m["vdim"]), rank=int(m["kv_rank"]),
                          window=int(m["mask"]["size"]), rope_base=float(rot["base"]), scale=float(m["scale"]))
            else:
                rank = m.get("rank")
                if rank is None:
                    name = f"l{i}.mix.w1"
                    if tensor_shapes is None or name not in tensor_shapes:
                        raise ValueError(f"layer {i}: the decay's rank is the size of {name}, which is not at hand")
                    rank = tensor_shapes[name][0]
                kw.update(heads=int(m["heads"]), dim=int(m["dim"]), rank=int(rank))
            layers.append(LayerShape(**kw))
        return cls(layers=tuple(layers), width=int(config["width"]), vocab=int(config["vocab"]), streams=int(config["streams"]),
                   eps=float(config["norm"]["eps"]))

    def to_config(self) -> dict[str, Any]:
        """The ``config.json`` of this shape."""
        layers = []
        for l in self.layers:
            if l.type == "rglru":
                mixer: dict[str, Any] = {"width": l.lru_width, "blocks": l.blocks, "conv": l.taps}
            elif l.type == "latent_attention":
                mixer = {"heads": l.heads, "dim": l.dim, "rot_dim": l.rot_dim, "vdim": l.v_dim, "kv_rank": l.rank, "mask": {"size": l.window},
                         "rot": {"base": l.rope_base, "dims": l.rot_dim}, "scale": l.scale}
            else:
                mixer = {"heads": l.heads, "dim": l.dim}
            layers.append({"type": l.type, "mixer": mixer, "mlp": {"kind": "dense", "ff": l.ff} if l.ff else None})
        return {"architecture": ARCHITECTURE, "layers": layers, "norm": {"eps": self.eps}, "streams": self.streams, "vocab": self.vocab,
                "width": self.width}

    def weight_bytes_per_token(self) -> int:
        """bf16 bytes of the matrices one decode step streams."""
        return 2 * (sum(l.weight_count(self.width) for l in self.layers) + self.vocab * self.width)

    def step_bytes(self, context_len: int, element_bytes: int = 2) -> int:
        """Algorithmic HBM bytes of one decode step: weights, visible cache rows read and one written, recurrent states
        read and written."""
        n = self.weight_bytes_per_token()
        for l in self.layers:
            if l.type == "latent_attention":
                n += (min(context_len, l.window) + 1) * (l.rank + l.rot_dim) * element_bytes
            elif l.type == "rglru":
                n += 8 * l.lru_width * l.taps
            else:
                n += 8 * (l.heads * l.dim * l.dim + self.width)
        return n

    def prefill_flops(self, tokens: int, position: int = 0) -> float:
        """Multiply-adds x 2 of a prompt's matrix products and visible score/value pairs (no LM head)."""
        flops = 2.0 * tokens * sum(l.weight_count(self.width) for l in self.layers)
        for l in self.layers:
            if l.type == "latent_attention":
                pairs = sum(min(position + t + 1, l.window) for t in range(tokens))
                flops += 2.0 * pairs * l.heads * (l.dim + l.rot_dim + l.v_dim)
            elif l.type == "wkv":
                flops += 6.0 * tokens * l.heads * l.dim * l.dim
        return flops


class HybridConfig:
    """The route's current shape, kept the way the other routes keep theirs (``LlamaConfig``)."""

    _shape: HybridShape | None = None

    @classmethod
    def shape(cls) -> HybridShape:
        if cls._shape is None:
            raise RuntimeError("no hybrid shape is set")
        return cls._shape

    @classmethod
    def set_shape(cls, shape: HybridShape) -> None:
        cls._shape = shape

    @classmethod
    def update_from_dict(cls, config: Mapping[str, Any], tensor_shapes: Mapping[str, tuple[int, ...]] | None = None) -> None:
        cls.set_shape(HybridShape.from_config(config, tensor_shapes))
