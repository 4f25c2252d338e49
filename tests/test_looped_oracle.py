"""The plain Givopel implementation against closed forms and torch's own operations, mechanism by mechanism (CPU), and against
planted mistakes: what the GPU tests' sizes would show."""
import math

import pytest
import torch

import givopel_oracle as O
from qimeng_megakernel_amd import synthetic
from qimeng_megakernel_amd.decode_schedule_hybrid import weights

F64 = torch.float64


def rnd(*size, seed=0):
    return torch.randn(*size, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_layer_norm_is_torchs_without_bias():
    x, w = rnd(4, 7) + 3, rnd(7, seed=1)
    assert torch.allclose(O.layer_norm(x, w, 1e-3), torch.nn.functional.layer_norm(x, (7,), w, None, 1e-3))


def test_rms_norm_has_eps_inside_the_root():
    assert torch.allclose(O.rms_norm(torch.tensor([[3.0, 4.0]], dtype=F64), torch.ones(2, dtype=F64), 3.5), torch.tensor([[0.75, 1.0]], dtype=F64))


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_convolution_is_causal_and_ends_at_the_current_token(taps):
    x, w = rnd(9, 3), rnd(3, taps, seed=1)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (taps - 1, 0)), w[:, None], groups=3)[0].T
    assert torch.allclose(O.short_conv(x, w), want)


def test_unscaled_frequencies_fall_geometrically():
    f, m = O.pair_frequencies(6, 100.0, None)
    assert m == 1.0 and torch.allclose(f, torch.tensor([1.0, 100 ** (-1 / 3), 100 ** (-2 / 3)], dtype=F64))


def test_scaling_leaves_fast_pairs_and_slows_slow_ones():
    scaling = {"factor": 4.0, "original": 1000.0, "fast": 30.0, "slow": 2.0}
    f, m = O.pair_frequencies(32, 10000.0, scaling)
    plain, _ = O.pair_frequencies(32, 10000.0, None)
    turns = 1000.0 * plain / (2 * math.pi)
    assert m == pytest.approx(1 + 0.1 * math.log(4))
    assert torch.allclose(f[turns > 60], plain[turns > 60]) and torch.allclose(f[turns < 1], plain[turns < 1] / 4)
    assert torch.all(f[1:] <= f[:-1]) and torch.all(f <= plain) and torch.all(f >= plain / 4)


@pytest.mark.parametrize("scaling", [None, (8.0, 300.0, 20.0, 1.5), (2.0, 4096.0, 32.0, 1.0), (3.0, 6.0, 0.5, 0.4), (2.0, 64.0, 1.0, 1.0)])
def test_the_products_tables_hold_the_same_angles(scaling):
    named = None if scaling is None else dict(zip(("factor", "original", "fast", "slow"), scaling))
    f, m = O.pair_frequencies(20, 777.0, named)
    cos, sin = weights.rope_tables(20, 777.0, 50, scaling)
    x = rnd(50, 1, 24)
    got = O.rotate_pairs(x, f, m)[:, 0]
    c, s = cos.double(), sin.double()
    assert torch.allclose(got[:, :20:2], x[:, 0, :20:2] * c - x[:, 0, 1:20:2] * s, atol=1e-5)
    assert torch.allclose(got[:, 1:20:2], x[:, 0, 1:20:2] * c + x[:, 0, :20:2] * s, atol=1e-5)
    assert torch.equal(got[:, 20:], x[:, 0, 20:])


def test_rotation_depends_on_distance():
    f, _ = O.pair_frequencies(6, 100.0, None)
    q, k = rnd(1, 1, 6).expand(120, 1, 6), rnd(1, 1, 6, seed=1).expand(120, 1, 6)
    rq, rk = O.rotate_pairs(q, f, 1.0)[:, 0], O.rotate_pairs(k, f, 1.0)[:, 0]
    assert torch.allclose(rq[11] @ rk[4], rq[107] @ rk[100]) and not torch.allclose(rq[11] @ rk[4], rq[12] @ rk[4])


def test_grouped_causal_attention():
    q, k, v = rnd(7, 6, 4), rnd(7, 2, 4, seed=1), rnd(7, 2, 3, seed=2)
    got = O.causal_attention(q, k, v, 0.7)
    for i in range(7):
        for h in range(6):
            p = torch.softmax(0.7 * k[: i + 1, h // 3] @ q[i, h], dim=0)
            assert torch.allclose(got[i, h], p @ v[: i + 1, h // 3])


def test_decayed_sum_is_a_weighted_sum_of_the_past_and_the_present():
    q, k, v, a = rnd(6, 2, 3), rnd(6, 2, 3, seed=1), rnd(6, 2, 4, seed=2), torch.rand(6, 2, 3, dtype=F64)
    got = O.decayed_sum(q, k, v, a)
    for t in range(6):
        want = sum((q[t, 1] * torch.prod(a[s + 1:t + 1, 1], dim=0) * k[s, 1]).sum() * v[s, 1] for s in range(t + 1))
        assert torch.allclose(got[t, 1], want)


def test_delta_rule_with_full_steps_returns_what_was_written_last():
    T = 5
    k = O.unit(rnd(T, 1, 4))
    v, ones = rnd(T, 1, 3, seed=1), torch.ones(T, 1, 4, dtype=F64)
    got = O.delta_rule(k, k, v, ones, torch.ones(T, 1, dtype=F64))      # asked with its own key
    assert torch.allclose(got, v, atol=1e-6)


def test_delta_rule_is_the_decayed_sum_for_orthogonal_keys():
    k = torch.eye(4, dtype=F64)[:, None]
    q, v, g, beta = rnd(4, 1, 4), rnd(4, 1, 3, seed=1), torch.rand(4, 1, 4, dtype=F64), torch.rand(4, 1, dtype=F64)
    assert torch.allclose(O.delta_rule(q, k, v, g, beta), O.decayed_sum(q, k, v * beta[..., None], g))


def test_chunks_with_a_triangular_system_are_the_delta_rule():
    """The form the prefill kernels compute, over one chunk from a state that is not zero."""
    C, d, e = 8, 5, 3
    q, k, v = rnd(C, 1, d), O.unit(rnd(C, 1, d, seed=1)), rnd(C, 1, e, seed=2)
    g, beta = torch.rand(C, 1, d, dtype=F64), torch.rand(C, 1, dtype=F64)
    lead = rnd(3, 1, d, seed=3)
    want = O.delta_rule(torch.cat([lead, q]), torch.cat([O.unit(lead), k]), torch.cat([rnd(3, 1, e, seed=4), v]),
                        torch.cat([torch.rand(3, 1, d, dtype=F64, generator=torch.Generator().manual_seed(5)), g]), torch.cat([torch.ones(3, 1, dtype=F64), beta]))[3:]
    state = torch.zeros(d, e, dtype=F64)
    lk, lv = O.unit(lead)[:, 0], rnd(3, 1, e, seed=4)[:, 0]
    lg = torch.rand(3, 1, d, dtype=F64, generator=torch.Generator().manual_seed(5))[:, 0]
    for t in range(3):
        state = lg[t][:, None] * state
        state = state + lk[t][:, None] * (lv[t] - state.T @ lk[t])[None]
    q, k, v, g, beta = q[:, 0], k[:, 0], v[:, 0], g[:, 0], beta[:, 0]
    cum = torch.cumprod(g, 0)
    a, b = torch.zeros(C, C, dtype=F64), torch.zeros(C, C, dtype=F64)
    for t in range(C):
        for s in range(t + 1):
            decayed = k[s] * torch.prod(g[s + 1:t + 1], dim=0)
            b[t, s] = q[t] @ decayed
            if s < t:
                a[t, s] = k[t] @ decayed
    u = torch.linalg.solve(torch.eye(C, dtype=F64) + beta[:, None] * a, beta[:, None] * (v - (cum * k) @ state))
    assert torch.allclose((cum * q) @ state + b @ u, want[:, 0])


def test_a_loop_runs_its_layers_again_with_the_embedding_joined_each_time():
    assert O.schedule(4, {"start": 1, "stop": 3, "times": 2}) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    shape = synthetic.looped_shape("pgp", width=16, vocab=9, loop=(1, 3, 2), heads=2, kv_heads=1, dim=4, v_dim=4, delta_heads=1, delta_kv_heads=1, delta_dim=4,
                                   delta_v_dim=4, delta_rank=2, gate_rank=2, gla_heads=1, gla_dim=4, gla_v_dim=4, gla_rank=2)
    assert shape.layer_runs() == O.schedule(3, shape.to_config()["loop"])


def test_soft_cap():
    assert float(O.soft_cap(torch.tensor(100.0), 5.0)) == pytest.approx(5.0) and float(O.soft_cap(torch.tensor(0.01), 5.0)) == pytest.approx(0.01, rel=1e-4)


def test_a_prefix_has_the_logits_of_the_whole():
    from test_gpu_looped import SHAPES, tokens_of

    shape = SHAPES["odd"]
    w = synthetic.random_hybrid_weights(shape, 3)
    tokens = torch.tensor(tokens_of(shape, 11))
    whole = O.forward(shape.to_config(), w, tokens, dtype=F64)
    assert torch.allclose(O.forward(shape.to_config(), w, tokens[:7], dtype=F64), whole[:7])


def _planted():
    """Mistakes that a kernel could make, planted in the plain implementation."""
    ln, rms, conv, rot, att = O.layer_norm, O.rms_norm, O.short_conv, O.rotate_pairs, O.causal_attention
    delta, gla, join, freq, cap, unit = O.delta_rule, O.decayed_sum, O.loop_input, O.pair_frequencies, O.soft_cap, O.unit
    ones = torch.ones_like
    return {
        "mean not taken off": ("layer_norm", lambda x, w, eps: rms(x, w, eps)),
        "eps half as large": ("layer_norm", lambda x, w, eps: ln(x, w, eps / 2)),
        "no rotation scaling": ("pair_frequencies", lambda d, b, s: freq(d, b, None)),
        "no magnitude": ("pair_frequencies", lambda d, b, s: (freq(d, b, s)[0], 1.0)),
        "ramp ends early": ("pair_frequencies", lambda d, b, s: freq(d, b, s if s is None else {**s, "slow": 3 * s["slow"]})),
        "ramp starts early": ("pair_frequencies", lambda d, b, s: freq(d, b, s if s is None else {**s, "fast": 10 * s["fast"]})),
        "halves instead of pairs": ("rotate_pairs", lambda x, f, m: torch.cat([rot(torch.stack(x[..., : 2 * len(f)].chunk(2, -1), -1).flatten(-2), f, m),
                                                                              x[..., 2 * len(f):]], -1)),
        "all dimensions pass": ("rotate_pairs", lambda x, f, m: x),
        "first key unseen": ("causal_attention", lambda q, k, v, s: torch.cat([att(q, k, v, s)[:1], att(q[1:], k[1:], v[1:], s)])),
        "key heads interleaved": ("causal_attention", lambda q, k, v, s: att(q, k.flip(1), v.flip(1), s)),
        "scale of the dimension": ("causal_attention", lambda q, k, v, s: att(q, k, v, q.shape[-1] ** -0.5)),
        "state forgotten at token 20": ("delta_rule", lambda q, k, v, g, b: torch.cat([delta(q[:20], k[:20], v[:20], g[:20], b[:20]), delta(q[20:], k[20:], v[20:], g[20:], b[20:])])),
        "read before the write": ("delta_rule", lambda q, k, v, g, b: delta(q, k, v, g, b) - (q * k).sum(-1, keepdim=True) * b[..., None] * v),
        "correction before the decay": ("delta_rule", lambda q, k, v, g, b: delta(q, k, v, torch.cat([g[1:], g[-1:]]), b)),
        "full steps": ("delta_rule", lambda q, k, v, g, b: delta(q, k, v, g, ones(b))),
        "no decay": ("delta_rule", lambda q, k, v, g, b: delta(q, k, v, ones(g), b)),
        "no correction": ("delta_rule", lambda q, k, v, g, b: gla(q, k, v * b[..., None], g)),
        "keys not unit vectors": ("unit", lambda x: x * 0.9),
        "gla state forgotten at token 20": ("decayed_sum", lambda q, k, v, a: torch.cat([gla(q[:20], k[:20], v[:20], a[:20]), gla(q[20:], k[20:], v[20:], a[20:])])),
        "gla decay late": ("decayed_sum", lambda q, k, v, a: gla(q, k, v, torch.cat([a[1:], a[-1:]]))),
        "tau left out": ("decayed_sum", lambda q, k, v, a: gla(q, k, v, a ** 1.1)),
        "convolution forgets at token 20": ("short_conv", lambda x, w: torch.cat([conv(x[:20], w), conv(x[20:], w)])),
        "convolution backwards": ("short_conv", lambda x, w: conv(x, w.flip(1))),
        "embedding not joined": ("loop_input", lambda x, x0, w: join(x, torch.zeros_like(x0), w)),
        "join swapped": ("loop_input", lambda x, x0, w: join(x0, x, w)),
        "no cap": ("soft_cap", lambda z, c: z),
    }


@pytest.mark.parametrize("mistake", sorted(_planted()))
def test_the_gpu_tests_sizes_show_a_planted_mistake(mistake, monkeypatch):
    """Each mistake moves the logits of the GPU tests' models well beyond what those tests allow in fp32."""
    from test_gpu_looped import SHAPES, TOL, error, tokens_of

    worst = 0.0
    for name in ("odd", "from_the_start", "many_heads"):
        shape = SHAPES[name]
        w = synthetic.random_hybrid_weights(shape, 0)
        tokens = torch.tensor(tokens_of(shape, 60))
        want = O.forward(shape.to_config(), w, tokens, dtype=F64)
        with monkeypatch.context() as m:
            m.setattr(O, *_planted()[mistake])
            got = O.forward(shape.to_config(), w, tokens, dtype=F64)
        worst = max(worst, error(got, want))
    assert worst > 10 * TOL[torch.float32], worst
