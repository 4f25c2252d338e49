"""Model shape of the hybrid route: a list of layers, each with its own mixer and sizes.

``HybridShape.from_config`` reads a model folder's ``config.json``.  Both designs name ``width``, ``vocab``, ``norm.eps``
and ``layers``, each ``{type, mixer, mlp}``; ``Lusupel`` adds ``streams``, ``Givopel`` ``loop``, ``logit_scale`` and
``logit_softcap``.  Nothing but these keys enters a computation; storage sizes (``*_s`` properties) are the true sizes
rounded up to what the kernels read.

What the kernels run is ``HybridShape.entries``: the layers in the order they run, one entry per mixer.  A ``Lusupel``
layer is one entry.  A ``Givopel`` layer run is one entry per branch of its mixer (branches read the same normed input),
the passes of a loop are entries of their own with the same weights, and joining the embedding at the start of a pass and
the model's norm are entries too.
"""
from __future__ import annotations

import dataclasses
import functools
from typing import Any, Mapping

ARCHITECTURE = "Lusupel"
LOOPED_ARCHITECTURE = "Givopel"
#: place = the kernels' entry type.  The first three work on residual streams, the others on a plain residual.
MIXERS = ("rglru", "latent_attention", "wkv", "gla", "attention", "delta", "join", "final")
STREAM_MIXERS = MIXERS[:3]


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
    # attention (also heads, dim, v_dim, scale, rope_base, and rot_dim: how many dimensions of a head are rotated), delta
    # (also heads, dim, v_dim, taps, rank), gla (also heads, dim, v_dim, rank)
    kv_heads: int = 0
    rope_scaling: tuple[float, float, float, float] | None = None    # factor, original, fast, slow
    gate_rank: int = 0          # delta: rank of the output gate
    tau: float = 0.0
    branches: tuple["LayerShape", ...] = ()    # parallel: the mixers side by side

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
    def gate_rank_s(self) -> int:
        return storage(self.gate_rank)

    @property
    def heads_s(self) -> int:
        return storage(self.heads)

    @property
    def conv_channels(self) -> int:
        """delta: channels of the short convolution (q, k, v)."""
        return 2 * self.kv_heads * self.dim_s + self.heads * self.v_s

    @property
    def ff_s(self) -> int:
        return storage(self.ff)

    @property
    def q_stride(self) -> int:
        return storage(self.dim_s + (0 if self.type == "attention" else self.rot_s), 32)

    @property
    def mix_width(self) -> int:
        """Storage width of what the mixer hands to its output projection."""
        if self.type == "rglru":
            return self.blocks * self.block_s
        return self.heads * (self.dim_s if self.type == "wkv" else self.v_s)

    @property
    def in_rows(self) -> int:
        if self.type == "rglru":
            return 2 * self.mix_width
        if self.type == "latent_attention":
            return self.heads * (self.q_stride + self.v_s) + self.rank_s + self.rot_s
        if self.type == "attention":
            return self.heads * (self.q_stride + self.v_s) + self.kv_heads * (self.dim_s + self.v_s)
        if self.type == "delta":
            return self.conv_channels + self.rank_s + self.gate_rank_s + self.heads_s
        if self.type == "gla":
            return 2 * self.heads * (self.dim_s + self.v_s) + self.rank_s
        return 4 * self.mix_width + self.rank_s

    def weight_count(self, width: int) -> int:
        """Matrix elements one token has to stream (norms, biases and taps aside)."""
        if self.type == "parallel":
            n = sum(b.weight_count(width) for b in self.branches)
        elif self.type == "attention":
            n = width * (self.heads * (self.dim + 2 * self.v_dim) + self.kv_heads * (self.dim + self.v_dim))
        elif self.type == "delta":
            n = (width * (2 * self.kv_heads * self.dim + 2 * self.heads * self.v_dim + self.rank + self.gate_rank + self.heads)
                 + self.heads * (self.rank * self.dim + self.gate_rank * self.v_dim))
        elif self.type == "gla":
            n = width * (self.heads * (2 * self.dim + 3 * self.v_dim) + self.rank) + self.heads * self.dim * self.rank
        elif self.type == "rglru":
            n = 3 * self.lru_width * width + 2 * self.lru_width * self.block
        elif self.type == "latent_attention":
            n = width * (self.heads * (self.dim + self.rot_dim + 2 * self.v_dim) + self.rank + self.rot_dim) + self.heads * self.rank * (self.dim + self.v_dim)
        else:
            n = 5 * self.heads * self.dim * width + self.rank * (width + self.heads * self.dim)
        return n + 3 * self.ff * width


@dataclasses.dataclass(frozen=True)
class Entry:
    """One entry of the kernels' table.  ``prev``: on the plain residual, the first entry of the layer run whose outputs are
    still to be added when this entry reads the residual (-1: none).  ``x_from`` / ``x_to``: the copy of the residual it
    reads (-1: the token's embedding) and the one it leaves."""

    layer: int                  # index of the layer whose weights it uses (-1: the model's)
    shape: LayerShape
    ff: int = 0                 # feed-forward that runs with this entry
    branch: int = 0
    branches: int = 1
    prev: int = -1
    x_from: int = -1
    x_to: int = 0
    last: bool = False          # the layer run's last entry

    @property
    def type(self) -> str:
        return self.shape.type


@dataclasses.dataclass(frozen=True)
class HybridShape:
    layers: tuple[LayerShape, ...]
    width: int
    vocab: int
    streams: int                # copies of the residual behind hyper-connections; 0: a plain residual, parallel sublayers
    eps: float
    loop: tuple[int, int, int] | None = None    # start, stop, times
    logit_scale: float = 1.0
    logit_softcap: float = 0.0                  # 0: none

    @property
    def width_s(self) -> int:
        return storage(self.width)

    @property
    def vocab_s(self) -> int:
        return storage(self.vocab)

    @property
    def plain(self) -> bool:
        return self.streams == 0

    def layer_runs(self) -> list[tuple[int, bool]]:
        """(layer, does a pass of the loop start with it) in the order they run."""
        n = len(self.layers)
        start, stop, times = self.loop or (n, n, 0)
        body = [(i, i == start) for i in range(start, stop)]
        return [(i, False) for i in range(start)] + body * times + [(i, False) for i in range(stop, n)]

    @functools.cached_property
    def entries(self) -> tuple[Entry, ...]:
        if not self.plain:
            return tuple(Entry(i, l, ff=l.ff, last=True) for i, l in enumerate(self.layers))
        out: list[Entry] = []
        state = {"prev": -1, "x": -1}

        def reads() -> dict[str, int]:      # every reader leaves the residual in the copy it did not read
            kw = dict(prev=state["prev"], x_from=state["x"], x_to=1 if state["x"] == 0 else 0)
            state["prev"], state["x"] = -1, kw["x_to"]
            return kw

        for i, enters in self.layer_runs():
            l = self.layers[i]
            if enters:
                out.append(Entry(-1, LayerShape("join"), **reads()))
            kw, first = reads(), len(out)
            parts = l.branches or (l,)
            for b, part in enumerate(parts):
                out.append(Entry(i, part, ff=l.ff if b == 0 else 0, branch=b, branches=len(parts), last=b + 1 == len(parts), **kw))
            state["prev"] = first
        out.append(Entry(-1, LayerShape("final"), **reads()))
        return tuple(out)

    @property
    def run_count(self) -> int:
        """Layer runs of one step."""
        return len(self.layer_runs())

    @classmethod
    def from_config(cls, config: Mapping[str, Any], tensor_shapes: Mapping[str, tuple[int, ...]] | None = None) -> "HybridShape":
        """``tensor_shapes`` names the checkpoint's tensors: it gives the sizes that no key names, the ranks of decays and
        gates."""
        plain = config.get("architecture") == LOOPED_ARCHITECTURE

        def rank(m: Mapping[str, Any], key: str, name: str) -> int:
            if m.get(key) is not None:
                return int(m[key])
            if tensor_shapes is None or name not in tensor_shapes:
                raise ValueError(f"a rank is the size of {name}, which is not at hand")
            return int(tensor_shapes[name][0])

        layers = []
        for i, entry in enumerate(config["layers"]):
            kind, m, mlp = entry["type"], entry["mixer"], entry.get("mlp")
            if kind not in (("gla", "parallel") if plain else STREAM_MIXERS):
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
            elif kind == "wkv":
                kw.update(heads=int(m["heads"]), dim=int(m["dim"]), rank=rank(m, "rank", f"l{i}.mix.w1"))
            elif kind == "gla":
                kw.update(heads=int(m["heads"]), kv_heads=int(m["heads"]), dim=int(m["dim"]), v_dim=int(m["vdim"]), tau=float(m["tau"]),
                          rank=rank(m, "rank", f"l{i}.mix.a1"))
            else:
                a, d = m["left"], m["right"]
                rot, scaling = a["rot"], a["rot"].get("scaling")
                if not 0 <= int(rot["dims"]) <= int(a["dim"]) or int(rot["dims"]) % 2:
                    raise ValueError(f"layer {i}: {rot['dims']} rotated dimensions of heads of {a['dim']}")
                for part in (a, d):
                    if int(part["heads"]) % int(part["kv_heads"]):
                        raise ValueError(f"layer {i}: {part['kv_heads']} key/value heads do not divide {part['heads']} heads")
                kw["branches"] = (
                    LayerShape("attention", heads=int(a["heads"]), kv_heads=int(a["kv_heads"]), dim=int(a["dim"]), v_dim=int(a["vdim"]),
                               rot_dim=int(rot["dims"]), rope_base=float(rot["base"]), scale=float(a["scale"]),
                               rope_scaling=None if scaling is None else tuple(float(scaling[k]) for k in ("factor", "original", "fast", "slow"))),
                    LayerShape("delta", heads=int(d["heads"]), kv_heads=int(d["kv_heads"]), dim=int(d["dim"]), v_dim=int(d["vdim"]), taps=int(d["conv"]),
                               rank=rank(d, "rank", f"l{i}.mix.right.a1"), gate_rank=rank(d, "gate_rank", f"l{i}.mix.right.g1")))
            layers.append(LayerShape(**kw))
        kw = {}
        if plain:
            loop, cap = config.get("loop"), config.get("logit_softcap")
            if loop is not None:
                kw["loop"] = start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
                if not (0 <= start < stop <= len(layers) and times >= 1):
                    raise ValueError(f"a loop of layers {start}..{stop - 1} run {times} times in a model of {len(layers)} layers")
            scale = config.get("logit_scale")
            kw.update(logit_scale=1.0 if scale is None else float(scale), logit_softcap=0.0 if cap is None else float(cap))
        return cls(layers=tuple(layers), width=int(config["width"]), vocab=int(config["vocab"]), streams=0 if plain else int(config["streams"]),
                   eps=float(config["norm"]["eps"]), **kw)

    def to_config(self) -> dict[str, Any]:
        """The ``config.json`` of this shape."""
        layers = []
        for l in self.layers:
            if l.type == "rglru":
                mixer: dict[str, Any] = {"width": l.lru_width, "blocks": l.blocks, "conv": l.taps}
            elif l.type == "latent_attention":
                mixer = {"heads": l.heads, "dim": l.dim, "rot_dim": l.rot_dim, "vdim": l.v_dim, "kv_rank": l.rank, "mask": {"size": l.window},
                         "rot": {"base": l.rope_base, "dims": l.rot_dim}, "scale": l.scale}
            elif l.type == "wkv":
                mixer = {"heads": l.heads, "dim": l.dim}
            elif l.type == "gla":
                mixer = {"heads": l.heads, "dim": l.dim, "vdim": l.v_dim, "tau": l.tau}
            else:
                a, d = l.branches
                rot: dict[str, Any] = {"base": a.rope_base, "dims": a.rot_dim}
                if a.rope_scaling is not None:
                    rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), a.rope_scaling))
                mixer = {"left": {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.v_dim, "scale": a.scale, "rot": rot},
                         "right": {"heads": d.heads, "kv_heads": d.kv_heads, "dim": d.dim, "vdim": d.v_dim, "conv": d.taps}}
            layers.append({"type": l.type, "mixer": mixer, "mlp": {"kind": "dense", "ff": l.ff} if l.ff else None})
        out = {"architecture": ARCHITECTURE, "layers": layers, "norm": {"eps": self.eps}, "vocab": self.vocab, "width": self.width}
        if self.plain:
            out.update(architecture=LOOPED_ARCHITECTURE, logit_scale=self.logit_scale)
            if self.loop is not None:
                out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
            if self.logit_softcap:
                out["logit_softcap"] = self.logit_softcap
        else:
            out["streams"] = self.streams
        return out

    def _run_weights(self) -> int:
        """Matrix elements of all layer runs of one step (a looped layer's once per pass)."""
        joins = sum(e.type == "join" for e in self.entries)
        return sum(self.layers[i].weight_count(self.width) for i, _ in self.layer_runs()) + joins * 2 * self.width * self.width

    def weight_bytes_per_token(self) -> int:
        """bf16 bytes of the matrices one decode step streams."""
        return 2 * (self._run_weights() + self.vocab * self.width)

    def step_bytes(self, context_len: int, element_bytes: int = 2) -> int:
        """Algorithmic HBM bytes of one decode step: weights, visible cache rows read and one written, recurrent states
        read and written."""
        n = self.weight_bytes_per_token()
        for e in self.entries:
            l = e.shape
            if l.type == "latent_attention":
                n += (min(context_len, l.window) + 1) * (l.rank + l.rot_dim) * element_bytes
            elif l.type == "attention":
                n += (context_len + 1) * l.kv_heads * (l.dim + l.v_dim) * element_bytes
            elif l.type == "rglru":
                n += 8 * l.lru_width * l.taps
            elif l.type == "wkv":
                n += 8 * (l.heads * l.dim * l.dim + self.width)
            elif l.type in ("gla", "delta"):
                n += 8 * l.heads * l.dim * l.v_dim
                if l.type == "delta":
                    n += 8 * (l.taps - 1) * (2 * l.kv_heads * l.dim + l.heads * l.v_dim)
        return n

    def prefill_flops(self, tokens: int, position: int = 0) -> float:
        """Multiply-adds x 2 of a prompt's matrix products and visible score/value pairs (no LM head)."""
        flops = 2.0 * tokens * self._run_weights()
        for e in self.entries:
            l = e.shape
            if l.type == "latent_attention":
                pairs = sum(min(position + t + 1, l.window) for t in range(tokens))
                flops += 2.0 * pairs * l.heads * (l.dim + l.rot_dim + l.v_dim)
            elif l.type == "attention":
                flops += 2.0 * (tokens * position + tokens * (tokens + 1) / 2) * l.heads * (l.dim + l.v_dim)
            elif l.type == "wkv":
                flops += 6.0 * tokens * l.heads * l.dim * l.dim
            elif l.type in ("gla", "delta"):
                flops += (6.0 if l.type == "gla" else 8.0) * tokens * l.heads * l.dim * l.v_dim
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
