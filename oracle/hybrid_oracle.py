"""Plain fp32/fp64 restatement of the hybrid decoder (recurrent and latent-attention mixers on a hyper-connected
residual): the checker of the hybrid route.

One function per mechanism, written from its equations; nothing here is fast and nothing is shared with the
product path.  ``forward`` runs one whole sequence; the loops over tokens are literal, so there is no state to
carry and nothing to get wrong about portions.

Notation: x [T, streams, D] residual streams, h [T, D] a mixer's input, weights ``W`` [out, in].
"""
from __future__ import annotations

import math
from typing import Any, Callable, Mapping

import torch

Tensor = torch.Tensor


def rms_norm(x: Tensor, eps: float, weight: Tensor | None = None) -> Tensor:
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def gelu_tanh(z: Tensor) -> Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z * z * z)))


def silu(z: Tensor) -> Tensor:
    return z / (1.0 + torch.exp(-z))


def causal_conv(x: Tensor, taps: Tensor, bias: Tensor) -> Tensor:
    """x [T, C], taps [C, n] (last column: the current token), zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        acc = bias.clone()
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                acc = acc + taps[:, j] * x[s]
        y[t] = acc
    return y


def block_diagonal(u: Tensor, weight: Tensor, bias: Tensor) -> Tensor:
    """u [T, C] in ``blocks`` equal parts, weight [blocks, n, n] ([out, in]), bias [blocks, n]."""
    blocks, n = weight.shape[0], weight.shape[1]
    parts = [u[:, b * n:(b + 1) * n] @ weight[b].T + bias[b] for b in range(blocks)]
    return torch.cat(parts, dim=1)


def linear_recurrent_unit(u: Tensor, r: Tensor, i: Tensor, lam: Tensor) -> Tensor:
    """S_t = a S_{t-1} + sqrt(1 - a^2) i u with log a = -8 r softplus(lam); every S_t [T, C]."""
    log_a = -8.0 * r * torch.nn.functional.softplus(lam)
    a = torch.exp(log_a)
    b = torch.sqrt(-torch.expm1(2.0 * log_a)) * i * u
    s = torch.zeros_like(u[0])
    out = []
    for t in range(u.shape[0]):
        s = a[t] * s + b[t]
        out.append(s)
    return torch.stack(out)


def mixer_rglru(h: Tensor, w: Mapping[str, Tensor], cfg: Mapping[str, Any], eps: float) -> Tensor:
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = causal_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    r = torch.sigmoid(block_diagonal(u, w["ra"], w["ra.b"]))
    i = torch.sigmoid(block_diagonal(u, w["ri"], w["ri.b"]))
    return (linear_recurrent_unit(u, r, i, w["lam"]) * y) @ w["o"].T


def rotate_pairs(x: Tensor, positions: Tensor, base: float) -> Tensor:
    """x [T, ..., d]: the pair (2i, 2i+1) turned by position * base^(-2i/d)."""
    d = x.shape[-1]
    out = x.clone()
    for i in range(d // 2):
        angle = positions.double() * base ** (-2.0 * i / d)
        c, s = torch.cos(angle).to(x.dtype), torch.sin(angle).to(x.dtype)
        while c.dim() < x.dim() - 1:
            c, s = c[..., None], s[..., None]
        a, b = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = a * c - b * s
        out[..., 2 * i + 1] = b * c + a * s
    return out


def windowed_softmax_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, window: int) -> Tensor:
    """q, k [T, H, d], v [T, H, e]: query i sees keys j with 0 <= i - j < window."""
    T = q.shape[0]
    pos = torch.arange(T)
    dist = pos[:, None] - pos[None, :]
    seen = (dist >= 0) & (dist < window)
    out = []
    for head in range(q.shape[1]):
        s = (q[:, head] @ k[:, head].T) * scale
        s = torch.where(seen, s, torch.full_like(s, -math.inf))
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        out.append((p / p.sum(-1, keepdim=True)) @ v[:, head])
    return torch.stack(out, dim=1)


def mixer_latent_attention(h: Tensor, w: Mapping[str, Tensor], cfg: Mapping[str, Any], eps: float) -> Tensor:
    T = h.shape[0]
    H, dim, rot, vdim, rank = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"]
    base, pos = float(cfg["rot"]["base"]), torch.arange(T)
    q = (h @ w["q"].T).view(T, H, dim + rot)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :rank], eps, w["dkv.norm"])
    k_rot = rotate_pairs(down[:, rank:], pos, base)
    k_nope = (c @ w["uk"].T).view(T, H, dim)
    v = (c @ w["uv"].T).view(T, H, vdim)
    q = torch.cat([q[..., :dim], rotate_pairs(q[..., dim:], pos, base)], dim=-1)
    k = torch.cat([k_nope, k_rot[:, None, :].expand(T, H, rot)], dim=-1)
    o = windowed_softmax_attention(q, k, v, float(cfg["scale"]), int(cfg["mask"]["size"])).reshape(T, H * vdim)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def token_shift(h: Tensor, mu: Tensor) -> Tensor:
    """h_t + (h_{t-1} - h_t) mu, with zeros before the first token."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mu


def wkv_recurrence(r: Tensor, k: Tensor, v: Tensor, decay: Tensor, bonus: Tensor) -> Tensor:
    """r, k, v, decay [T, H, n], bonus [H, n]: o_t = (S + diag(bonus) k v^T)^T r, then S = diag(decay) S + k v^T."""
    T, H, n = r.shape
    s = torch.zeros(H, n, n, dtype=r.dtype)
    out = []
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out.append(((s + bonus[:, :, None] * kv) * r[t][:, :, None]).sum(1))
        s = decay[t][:, :, None] * s + kv
    return torch.stack(out)


def mixer_wkv(h: Tensor, w: Mapping[str, Tensor], cfg: Mapping[str, Any], eps: float) -> Tensor:
    T, H, n = h.shape[0], cfg["heads"], cfg["dim"]
    mix = {s: token_shift(h, w["mu." + s]) for s in "rkvgw"}
    r, k, v = ((mix[s] @ w[s].T).view(T, H, n) for s in "rkv")
    gate = silu(mix["g"] @ w["g"].T)
    decay = torch.exp(-torch.exp(torch.tanh(mix["w"] @ w["w1"].T) @ w["w2"].T + w["w0"])).view(T, H, n)
    o = rms_norm(wkv_recurrence(r, k, v, decay, w["u"]), eps).reshape(T, H * n)
    return (o * w["norm"] * gate) @ w["o"].T


def dense_mlp(h: Tensor, w: Mapping[str, Tensor]) -> Tensor:
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def hyper_connection(x: Tensor, w_in: Tensor, w_mix: Tensor, w_out: Tensor, sublayer: Callable[[Tensor], Tensor]) -> Tensor:
    """x [T, streams, D] -> the streams behind one sublayer; ``w_mix`` is indexed [from, to]."""
    y = sublayer(torch.einsum("s,tsd->td", w_in, x))
    return torch.einsum("su,tsd->tud", w_mix, x) + w_out[None, :, None] * y[:, None, :]


MIXERS = {"rglru": mixer_rglru, "latent_attention": mixer_latent_attention, "wkv": mixer_wkv}


def forward(config: Mapping[str, Any], weights: Mapping[str, Tensor], tokens: Tensor, *, dtype: torch.dtype = torch.float32,
            layer_outputs: list[Tensor] | None = None) -> Tensor:
    """Logits [T, vocab] of one whole sequence.  ``layer_outputs`` receives the summed streams behind every layer."""
    w = {k: v.to(dtype) for k, v in weights.items() if v.is_floating_point()}
    eps = float(config["norm"]["eps"])

    def group(prefix: str) -> dict[str, Tensor]:
        return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}

    x = w["embed"][tokens.long()][:, None, :].repeat(1, int(config["streams"]), 1)
    for i, layer in enumerate(config["layers"]):
        name = f"l{i}."
        mix, mlp, cfg = group(name + "mix."), group(name + "mlp."), layer["mixer"]
        mixer = MIXERS[layer["type"]]

        def hc(q: int, x: Tensor, sublayer: Callable[[Tensor], Tensor]) -> Tensor:
            norm = w[f"{name}norm{q}"]
            g = group(f"{name}hc{q}.")
            return hyper_connection(x, g["in"], g["mix"], g["out"], lambda u: sublayer(rms_norm(u, eps, norm)))

        x = hc(1, x, lambda h: mixer(h, mix, cfg, eps))
        if layer["mlp"] is not None:
            x = hc(2, x, lambda h: dense_mlp(h, mlp))
        if layer_outputs is not None:
            layer_outputs.append(x.sum(1))
    return rms_norm(x.sum(1), eps, w["final.norm"]) @ w["head"].T
