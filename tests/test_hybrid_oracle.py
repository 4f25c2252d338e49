"""The plain hybrid implementation against closed forms and torch's own operations, mechanism by mechanism (CPU)."""
import math

import pytest
import torch

import hybrid_oracle as O
from qimeng_megakernel_amd import synthetic

F64 = torch.float64


def rnd(*size, seed=0):
    return torch.randn(*size, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_rms_norm_has_eps_inside_the_root():
    x = torch.tensor([[3.0, 4.0]], dtype=F64)
    assert torch.allclose(O.rms_norm(x, 3.5), x / 4.0)


def test_gelu_is_torchs_tanh_form():
    z = rnd(200) * 4
    assert torch.allclose(O.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_convolution_is_causal_and_ends_at_the_current_token(taps):
    x, w, b = rnd(9, 3), rnd(3, taps, seed=1), rnd(3, seed=2)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (taps - 1, 0)), w[:, None], b, groups=3)[0].T
    assert torch.allclose(O.causal_conv(x, w, b), want)


def test_linear_recurrence_is_a_weighted_sum_of_the_past():
    T, C = 7, 3
    u, r, i, lam = rnd(T, C), torch.rand(T, C, dtype=F64), torch.rand(T, C, dtype=F64), rnd(C, seed=3)
    a = torch.exp(-8 * r * torch.nn.functional.softplus(lam))
    b = torch.sqrt(1 - a * a) * i * u
    got = O.linear_recurrent_unit(u, r, i, lam)
    for t in range(T):
        want = sum(b[s] * torch.prod(a[s + 1:t + 1], dim=0) for s in range(t + 1))
        assert torch.allclose(got[t], want)


def test_rotation_keeps_norms_and_depends_on_distance():
    q, k = rnd(1, 6), rnd(1, 6, seed=1)
    dot = lambda p, s: (O.rotate_pairs(q, torch.tensor([p]), 100.0) * O.rotate_pairs(k, torch.tensor([s]), 100.0)).sum()
    assert torch.allclose(dot(11, 4), dot(107, 100))
    assert not torch.allclose(dot(11, 4), dot(12, 4))
    angle = 5 * 100.0 ** (-2 / 6)
    got = O.rotate_pairs(torch.tensor([[0.0, 0, 1, 0, 0, 0]], dtype=F64), torch.tensor([5]), 100.0)
    assert torch.allclose(got, torch.tensor([[0, 0, math.cos(angle), math.sin(angle), 0, 0]], dtype=F64))


@pytest.mark.parametrize("window", [1, 3, 50])
def test_window_counts_the_query_itself(window):
    T = 8
    q, k, v = rnd(T, 2, 4), rnd(T, 2, 4, seed=1), rnd(T, 2, 3, seed=2)
    got = O.windowed_softmax_attention(q, k, v, 0.7, window)
    for i in range(T):
        lo = max(0, i - window + 1)
        for h in range(2):
            p = torch.softmax(0.7 * k[lo:i + 1, h] @ q[i, h], dim=0)
            assert torch.allclose(got[i, h], p @ v[lo:i + 1, h])


def test_wkv_is_a_decayed_sum_with_a_bonus_for_the_current_token():
    T, H, n = 6, 2, 3
    r, k, v, u = rnd(T, H, n), rnd(T, H, n, seed=1), rnd(T, H, n, seed=2), rnd(H, n, seed=3)
    w = torch.rand(T, H, n, dtype=F64)
    got = O.wkv_recurrence(r, k, v, w, u)
    for t in range(T):
        for h in range(H):
            want = (r[t, h] * u[h] * k[t, h]).sum() * v[t, h]
            for s in range(t):
                want = want + (r[t, h] * torch.prod(w[s + 1:t, h], dim=0) * k[s, h]).sum() * v[s, h]
            assert torch.allclose(got[t, h], want)


def test_token_shift_starts_from_zeros():
    h, mu = rnd(3, 4), torch.rand(4, dtype=F64)
    got = O.token_shift(h, mu)
    assert torch.allclose(got[0], h[0] * (1 - mu)) and torch.allclose(got[2], h[2] + (h[1] - h[2]) * mu)


def test_hyper_connection_is_a_residual_sum_for_one_stream_and_unit_weights():
    x, one = rnd(4, 1, 5), torch.ones(1, dtype=F64)
    got = O.hyper_connection(x, one, torch.ones(1, 1, dtype=F64), one, lambda u: u * u)
    assert torch.allclose(got, x + x * x)


def test_hyper_connection_mixes_from_row_to_column():
    x = rnd(2, 2, 3)
    mix = torch.tensor([[0.0, 2.0], [0.0, 0.0]], dtype=F64)          # stream 0 goes to stream 1, doubled
    got = O.hyper_connection(x, torch.zeros(2, dtype=F64), mix, torch.zeros(2, dtype=F64), lambda u: u)
    assert torch.allclose(got[:, 1], 2 * x[:, 0]) and torch.all(got[:, 0] == 0)


def test_a_prefix_has_the_logits_of_the_whole():
    shape = synthetic.hybrid_shape("rwa", width=24, vocab=50, streams=2, ff={"r": 20}, heads=2, dim=8, rot_dim=4, v_dim=6, rank=10, window=4,
                                   lru_width=24, blocks=3, taps=3, wkv_heads=2, wkv_dim=6, wkv_rank=5)
    w = synthetic.random_hybrid_weights(shape, 3)
    tokens = torch.randint(0, 50, (11,), generator=torch.Generator().manual_seed(1))
    whole = O.forward(shape.to_config(), w, tokens, dtype=F64)
    assert torch.allclose(O.forward(shape.to_config(), w, tokens[:7], dtype=F64), whole[:7])


def _planted():
    """Mistakes that a kernel could make, planted in the plain implementation."""
    norm, rot, att, wkv, lru, hyper, conv = (O.rms_norm, O.rotate_pairs, O.windowed_softmax_attention, O.wkv_recurrence, O.linear_recurrent_unit,
                                             O.hyper_connection, O.causal_conv)
    return {
        "window one longer": ("windowed_softmax_attention", lambda q, k, v, s, w: att(q, k, v, s, w + 1)),
        "window one shorter": ("windowed_softmax_attention", lambda q, k, v, s, w: att(q, k, v, s, w - 1)),
        "rotation one position off on one side": ("rotate_pairs", lambda x, p, b: rot(x, p + (x.dim() == 3), b)),
        "halves instead of pairs": ("rotate_pairs", lambda x, p, b: torch.cat([rot(x[..., ::2], p, b), x[..., 1::2]], -1)),
        "no bonus": ("wkv_recurrence", lambda r, k, v, d, u: wkv(r, k, v, d, torch.zeros_like(u))),
        "decay before the key": ("wkv_recurrence", lambda r, k, v, d, u: wkv(r, k, v, torch.cat([d[1:], d[-1:]]), u)),
        "recurrence forgets at token 20": ("linear_recurrent_unit", lambda u, r, i, lam: torch.cat([lru(u[:20], r[:20], i[:20], lam), lru(u[20:], r[20:], i[20:], lam)])),
        "wkv forgets at token 20": ("wkv_recurrence", lambda r, k, v, d, u: torch.cat([wkv(r[:20], k[:20], v[:20], d[:20], u), wkv(r[20:], k[20:], v[20:], d[20:], u)])),
        "convolution forgets at token 20": ("causal_conv", lambda x, w, b: torch.cat([conv(x[:20], w, b), conv(x[20:], w, b)])),
        "no shift": ("token_shift", lambda h, mu: h),
        "mix transposed": ("hyper_connection", lambda x, i, m, o, f: hyper(x, i, m.T, o, f)),
        "eps outside the root": ("rms_norm", lambda x, eps, weight=None: norm(x, 0.0, weight) if eps < 1e-4 else norm(x, eps / 2, weight)),
    }


@pytest.mark.parametrize("mistake", sorted(_planted()))
def test_the_gpu_tests_sizes_show_a_planted_mistake(mistake, monkeypatch):
    """Each mistake moves the logits of the GPU tests' models well beyond what those tests allow in fp32."""
    from test_gpu_hybrid import SHAPES, TOL, error, tokens_of

    worst = 0.0
    for name in ("odd", "one_stream", "many_heads"):
        shape = SHAPES[name]
        w = synthetic.random_hybrid_weights(shape, 0)
        tokens = torch.tensor(tokens_of(shape, 80))
        want = O.forward(shape.to_config(), w, tokens, dtype=F64)
        with monkeypatch.context() as m:
            m.setattr(O, *_planted()[mistake])
            got = O.forward(shape.to_config(), w, tokens, dtype=F64)
        worst = max(worst, error(got, want))
    assert worst > 20 * TOL[torch.float32], worst
