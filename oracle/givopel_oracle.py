"""Plain restatement of the Givopel decoder (gated linear attention, rotary softmax attention beside a gated delta rule,
parallel feed-forward, a looped stretch of layers): the checker of the hybrid route's second design.

One function per mechanism, written from its equations; nothing is fast and nothing is shared with the product path.
``forward`` runs one whole sequence with literal loops over tokens, so there is no state to carry and nothing to get wrong
about portions.  x [T, D] residual, h [T, D] a sublayer's input, weights ``W`` [out, in].
"""
from __future__ import annotations

import math
from typing import Any, Mapping, Optional

import torch

Tensor = torch.Tensor


def layer_norm(x: Tensor, weight: Tensor, eps: float) -> Tensor:
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight


def rms_norm(x: Tensor, weight: Tensor, eps: float) -> Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def silu(z: Tensor) -> Tensor:
    return z / (1.0 + torch.exp(-z))


def unit(x: Tensor) -> Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def short_conv(x: Tensor, taps: Tensor) -> Tensor:
    """x [T, C], taps [C, n] (last column: the current token), zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x)
    for j in range(n):
        back = n - 1 - j
        if back < T:
            y[back:] += taps[:, j] * x[: T - back]
    return y


def pair_frequencies(dims: int, base: float, scaling: Optional[Mapping[str, float]]) -> tuple[Tensor, float]:
    """Angle per position of every pair, and what cos and sin are multiplied with (both fp64).

    With ``scaling``: pairs that turn fewer than ``slow`` times within ``original`` positions are slowed by ``factor``,
    pairs that turn more than ``fast`` times are left, a ramp over the pair's number in between."""
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    if scaling is None:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def where(turns: float) -> float:
        return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(where(float(scaling["fast"]))), 0)
    hi = min(math.ceil(where(float(scaling["slow"]))), dims - 1)
    out = []
    for i in range(dims // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f[i] / factor * ramp + f[i] * (1.0 - ramp))
    return torch.stack(out), 0.1 * math.log(factor) + 1.0


def rotate_pairs(x: Tensor, freq: Tensor, magnitude: float) -> Tensor:
    """x [T, H, d]: the first 2 len(freq) dimensions as neighbouring pairs, turned by position * freq."""
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=torch.float64)
    for i in range(len(freq)):
        c, s = (torch.cos(pos * freq[i]) * magnitude).to(x.dtype)[:, None], (torch.sin(pos * freq[i]) * magnitude).to(x.dtype)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def causal_attention(q: Tensor, k: Tensor, v: Tensor, scale: float) -> Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, e]: head h reads key/value head h // (H / G) at every position up to its own."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    hidden = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        s = s.masked_fill(hidden, -math.inf)
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        out.append((p / p.sum(-1, keepdim=True)) @ v[:, g])
    return torch.stack(out, dim=1)


def attention_branch(h: Tensor, w: Mapping[str, Tensor], cfg: Mapping[str, Any]) -> Tensor:
    T, H, G, d, e = h.shape[0], cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    freq, magnitude = pair_frequencies(int(cfg["rot"]["dims"]), float(cfg["rot"]["base"]), cfg["rot"].get("scaling"))
    q = rotate_pairs((h @ w["q"].T).view(T, H, d), freq, magnitude)
    k = rotate_pairs((h @ w["k"].T).view(T, G, d), freq, magnitude)
    o = causal_attention(q, k, (h @ w["v"].T).view(T, G, e), float(cfg["scale"])).reshape(T, H * e)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def delta_rule(q: Tensor, k: Tensor, v: Tensor, g: Tensor, beta: Tensor) -> Tensor:
    """q, k, g [T, H, d], v [T, H, e], beta [T, H]: S decays by key channel, then moves by beta towards S^T k = v, then
    answers q."""
    T, H, d = q.shape
    s = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(T):
        s = g[t][:, :, None] * s
        u = beta[t][:, None] * (v[t] - (s * k[t][:, :, None]).sum(1))
        s = s + k[t][:, :, None] * u[:, None, :]
        out.append((s * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def delta_branch(h: Tensor, w: Mapping[str, Tensor], cfg: Mapping[str, Any], eps: float) -> Tensor:
    T, H, G, d, e = h.shape[0], cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q, k, v = (silu(short_conv(h @ w[n].T, w[n + ".conv"])) for n in "qkv")
    each = torch.arange(H) // (H // G)
    q, k = unit(q.view(T, G, d))[:, each] * d ** -0.5, unit(k.view(T, G, d))[:, each]
    beta = torch.sigmoid(h @ w["b"].T)
    rate = torch.nn.functional.softplus((h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]).view(T, H, d)
    g = torch.exp(-torch.exp(w["A_log"])[None, :, None] * rate)
    o = rms_norm(delta_rule(q, k, v.view(T, H, e), g, beta), w["norm"], eps).reshape(T, H * e)
    return (o * torch.sigmoid((h @ w["g1"].T) @ w["g2"].T)) @ w["o"].T


def mixer_parallel(h: Tensor, w: Mapping[str, Tensor], cfg: Mapping[str, Any], eps: float) -> Tensor:
    left = attention_branch(h, _group(w, "left."), cfg["left"])
    right = delta_branch(h, _group(w, "right."), cfg["right"], eps)
    return 0.5 * (rms_norm(left, w["left.out"], eps) + rms_norm(right, w["right.out"], eps))


def decayed_sum(q: Tensor, k: Tensor, v: Tensor, alpha: Tensor) -> Tensor:
    """S = diag(alpha) S + k v^T, then S^T q; all [T, H, .]."""
    s = torch.zeros(q.shape[1], q.shape[2], v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        s = alpha[t][:, :, None] * s + k[t][:, :, None] * v[t][:, None, :]
        out.append((s * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def mixer_gla(h: Tensor, w: Mapping[str, Tensor], cfg: Mapping[str, Any], eps: float) -> Tensor:
    T, H, d, e = h.shape[0], cfg["heads"], cfg["dim"], cfg["vdim"]
    q, k, v = (h @ w["q"].T).view(T, H, d) * d ** -0.5, (h @ w["k"].T).view(T, H, d), (h @ w["v"].T).view(T, H, e)
    z = ((h @ w["a1"].T) @ w["a2"].T + w["a2.b"]).view(T, H, d)
    alpha = torch.exp(torch.nn.functional.logsigmoid(z) / float(cfg["tau"]))
    o = rms_norm(decayed_sum(q, k, v, alpha), w["norm"], eps).reshape(T, H * e)
    return (o * silu(h @ w["g"].T)) @ w["o"].T


def dense_mlp(h: Tensor, w: Mapping[str, Tensor]) -> Tensor:
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def soft_cap(z: Tensor, cap: Optional[float]) -> Tensor:
    return z if cap is None else cap * torch.tanh(z / cap)


def loop_input(x: Tensor, x0: Tensor, w: Tensor) -> Tensor:
    return torch.cat([x, x0], dim=-1) @ w.T


def schedule(layers: int, loop: Optional[Mapping[str, int]]) -> list[tuple[int, bool]]:
    """(layer, does a pass of the loop start before it) in the order they run."""
    if loop is None:
        return [(i, False) for i in range(layers)]
    start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    runs = [(i, False) for i in range(start)]
    for _ in range(times):
        runs += [(i, i == start) for i in range(start, stop)]
    return runs + [(i, False) for i in range(stop, layers)]


MIXERS = {"gla": mixer_gla, "parallel": mixer_parallel}


def _group(w: Mapping[str, Tensor], prefix: str) -> dict[str, Tensor]:
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def forward(config: Mapping[str, Any], weights: Mapping[str, Tensor], tokens: Tensor, *, dtype: torch.dtype = torch.float32,
            layer_outputs: Optional[list[Tensor]] = None) -> Tensor:
    """Logits [T, vocab] of one whole sequence.  ``layer_outputs`` receives the residual behind every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items() if v.is_floating_point()}
    eps = float(config["norm"]["eps"])
    x0 = x = w["embed"][tokens.long()]
    for i, enters in schedule(len(config["layers"]), config.get("loop")):
        layer, name = config["layers"][i], f"l{i}."
        if enters:
            x = loop_input(x, x0, w["loop.in"])
        h = layer_norm(x, w[name + "norm1"], eps)
        y = MIXERS[layer["type"]](h, _group(w, name + "mix."), layer["mixer"], eps)
        if layer["mlp"] is not None:
            y = y + dense_mlp(h, _group(w, name + "mlp."))
        x = x + y
        if layer_outputs is not None:
            layer_outputs.append(x)
    z = layer_norm(x, w["final.norm"], eps) @ w["head"].T * float(config.get("logit_scale") or 1.0)
    return soft_cap(z, config.get("logit_softcap"))
