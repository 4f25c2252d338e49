"""The hybrid route on the GPU against the plain implementation (oracle/hybrid_oracle.py), through the C ABI.

fp32 is compared at rounding level, so a wrong key, decay or edge anywhere shows; bf16 at bf16's.
"""
import functools
import json

import pytest
import torch

import hybrid_oracle as O
from qimeng_megakernel_amd import decode_hybrid, synthetic
from qimeng_megakernel_amd.decode_schedule_hybrid import mk_kernel, weights
from qimeng_megakernel_amd.decode_schedule_hybrid.globs import build_globals
from qimeng_megakernel_amd.decode_schedule_hybrid.instructions import scheduler
from qimeng_megakernel_amd.decode_schedule_hybrid.state import RequestTable

pytestmark = pytest.mark.gpu

DEVICE = "cuda:0"
TOL = {torch.float32: 2e-5, torch.bfloat16: 4e-2}
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])

#: sizes off and on the storage multiples, one stream to many, every mixer with and without a feed-forward
SHAPES = {
    "odd": synthetic.hybrid_shape("rawar", width=52, vocab=77, streams=2, ff={"r": 36, "w": 20}, heads=3, dim=20, rot_dim=10, v_dim=12, rank=28, window=9,
                                  lru_width=60, blocks=5, taps=3, wkv_heads=3, wkv_dim=12, wkv_rank=7, scale=0.31, rope_base=50.0),
    "one_stream": synthetic.hybrid_shape("wra", width=64, vocab=130, streams=1, ff={"a": 48}, heads=1, dim=16, rot_dim=16, v_dim=32, rank=16, window=33,
                                         lru_width=32, blocks=1, taps=1, wkv_heads=1, wkv_dim=16, wkv_rank=16, eps=1e-3),
    "many_heads": synthetic.hybrid_shape("aw", width=160, vocab=512, streams=8, ff={"a": 96, "w": 80}, heads=18, dim=32, rot_dim=8, v_dim=24, rank=48, window=70,
                                         wkv_heads=5, wkv_dim=40, wkv_rank=12),
    "wide": synthetic.hybrid_shape("raw", width=640, vocab=1000, streams=4, ff={"r": 1100, "a": 520}, heads=4, dim=128, rot_dim=64, v_dim=128, rank=256,
                                   window=100, lru_width=512, blocks=2, taps=4, wkv_heads=4, wkv_dim=64, wkv_rank=32),
    "large_heads": synthetic.hybrid_shape("aw", width=96, vocab=64, streams=3, heads=2, dim=160, rot_dim=32, v_dim=200, rank=80, window=21, wkv_heads=2,
                                          wkv_dim=136, wkv_rank=24),
    "long_taps": synthetic.hybrid_shape("rr", width=48, vocab=96, streams=2, lru_width=96, blocks=2, taps=7),
}


@functools.lru_cache(maxsize=None)
def model(name, seed=0):
    shape = SHAPES[name]
    return shape, synthetic.random_hybrid_weights(shape, seed)


def on_gpu(shape, w, dtype, *, max_positions=160, slots=1, portion_rows=64):
    return build_globals(shape, weights.pack(shape, w, DEVICE), dtype=dtype, slots=slots, max_positions=max_positions, portion_rows=portion_rows)


def tokens_of(shape, n, seed=0):
    return torch.randint(0, shape.vocab, (n,), generator=torch.Generator().manual_seed(seed + 17)).tolist()


def run(g, mk, tokens, cuts, table=None, key="x", close=True):
    """Logits [len(tokens), vocab] with the prompt cut into portions of the given sizes."""
    table = table or RequestTable(g)
    request, out, at = table.get(key), [], 0
    for n in cuts:
        out.append(decode_hybrid.run_tokens(g, mk, request, tokens[at:at + n], range(n)))
        at += n
    assert at == len(tokens)
    mk.check()
    if close:
        table.close(key)
    return torch.cat(out).double().cpu()


def error(got, want):
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()).max())


@functools.lru_cache(maxsize=None)
def expected(name, n, seed=0):
    shape, w = model(name)
    return O.forward(shape.to_config(), w, torch.tensor(tokens_of(shape, n, seed)), dtype=torch.float64)


def check(name, dtype, n, cuts, **kw):
    shape, w = model(name)
    got = run(on_gpu(shape, w, dtype, **kw), mk_kernel.get_mk(), tokens_of(shape, n), cuts)
    err = error(got, expected(name, n))
    assert err < TOL[dtype], f"{name}: {err:.3g}"


@BOTH
@pytest.mark.parametrize("name", sorted(SHAPES))
def test_whole_prompt(name, dtype):
    check(name, dtype, 130, [130], portion_rows=160)


@BOTH
@pytest.mark.parametrize("name", sorted(SHAPES))
def test_token_by_token(name, dtype):
    check(name, dtype, 60, [1] * 60)


@BOTH
@pytest.mark.parametrize("cuts", [[2] * 40, [3, 1, 2, 61, 1, 1, 11], [31, 33, 16], [77, 2, 1]], ids=["twos", "mixed", "tiles", "tail"])
@pytest.mark.parametrize("name", ["odd", "many_heads", "wide"])
def test_portions(name, dtype, cuts):
    check(name, dtype, 80, cuts, portion_rows=96)


def test_portions_longer_than_a_launch_takes():
    check("odd", torch.float32, 110, [70, 40], portion_rows=16)      # the cache is a ring of 24 rows


def test_long_decoding_over_a_small_ring():
    check("odd", torch.float32, 400, [5] + [1] * 395, max_positions=400, portion_rows=8)


def test_decode_and_prefill_leave_the_same_state():
    shape, w = model("wide")
    mk, tokens = mk_kernel.get_mk(), tokens_of(shape, 40)
    states = []
    for cuts in ([40], [1] * 40):
        g = on_gpu(shape, w, torch.float32)
        table = RequestTable(g)
        run(g, mk, tokens, cuts, table=table, close=False)
        flip = table.live["x"].flip
        states.append([{k: (t[0] if k != "shift" else t[0, flip]).clone() for k, t in s.items()} for s in g.layer_state])
    for a, b in zip(*states):
        for k in a:
            n = 40 if k == "cache" else None
            assert torch.allclose(a[k][:n], b[k][:n], rtol=1e-4, atol=1e-5), k


@pytest.mark.parametrize("pattern,kw", [
    ("r", dict(lru_width=48, blocks=3, taps=4)), ("r", dict(lru_width=40, blocks=1, taps=2)), ("r", dict(lru_width=96, blocks=2, taps=16)),
    ("a", dict(heads=2, dim=24, rot_dim=4, v_dim=40, rank=20, window=7)), ("a", dict(heads=17, dim=8, rot_dim=24, v_dim=8, rank=36, window=40)),
    ("w", dict(wkv_heads=2, wkv_dim=20, wkv_rank=3)), ("w", dict(wkv_heads=1, wkv_dim=250, wkv_rank=40)),
])
@pytest.mark.parametrize("ff", [0, 56])
def test_each_mechanism_alone(pattern, kw, ff):
    """One layer; the streams behind it as well as the logits."""
    shape = synthetic.hybrid_shape(pattern, width=40, vocab=61, streams=3, ff={pattern: ff}, **kw)
    w = synthetic.random_hybrid_weights(shape, 4)
    tokens = tokens_of(shape, 50)
    layers = []
    want = O.forward(shape.to_config(), w, torch.tensor(tokens), dtype=torch.float64, layer_outputs=layers)
    g, mk = on_gpu(shape, w, torch.float32), mk_kernel.get_mk()
    assert error(run(g, mk, tokens, [1] * 50), want) < TOL[torch.float32]
    request = RequestTable(g).open("y")
    g.slot, g.position_id, g.flip = request.slot, 0, 0
    out = torch.zeros(1, 50, shape.width_s, device=DEVICE)
    logits = mk.prefill(g, torch.tensor(tokens, device=DEVICE), torch.arange(50, dtype=torch.int32, device=DEVICE), layer_out=out)
    assert error(logits[:, : shape.vocab].double().cpu(), want) < TOL[torch.float32]
    assert error(out[0, :, : shape.width].double().cpu(), layers[0]) < TOL[torch.float32]
    assert torch.all(out[0, :, shape.width:] == 0)


def pointed_model(window, heads=2):
    """One latent attention layer in which token 1 asks and token 0 answers: the asker's score for the answerer stands far
    above all others, whatever lies between them."""
    shape = synthetic.hybrid_shape("a", width=32, vocab=40, streams=2, heads=heads, dim=16, rot_dim=8, v_dim=16, rank=16, window=window, scale=1.0)
    w = synthetic.random_hybrid_weights(shape, 9)
    w["embed"][:, :2] = 0
    w["embed"][0] = 0
    w["embed"][0, 0] = 4.0
    w["embed"][1] = 0
    w["embed"][1, 1] = 4.0
    w["l0.norm1"] = torch.ones_like(w["l0.norm1"])
    q = w["l0.mix.q"].view(heads, 24, 32)
    q.mul_(0.02)
    q[:, :16, 1] = 0
    q[:, 0, 1] = 3.0
    dkv = w["l0.mix.dkv"]
    dkv[:16, 0] = 0
    dkv[0, :] *= 0.02
    dkv[0, 0] = 3.0
    w["l0.mix.dkv.norm"] = torch.ones_like(w["l0.mix.dkv.norm"])
    uk = w["l0.mix.uk"].view(heads, 16, 16)
    uk[:, 0] = 0
    uk[:, 0, 0] = 2.0
    w["l0.mix.uv"] *= 3.0
    return shape, w


@pytest.mark.parametrize("window", [2, 5, 32, 33, 64, 65, 100])
def test_keys_just_inside_and_just_outside_the_window(window):
    shape, w = pointed_model(window)
    config, mk = shape.to_config(), mk_kernel.get_mk()
    g = on_gpu(shape, w, torch.float32, max_positions=240, portion_rows=48)
    filler = torch.randint(2, 40, (230,), generator=torch.Generator().manual_seed(2)).tolist()
    for ask in (window + 3, 130, 200):
        rows = {}
        for distance in (window - 1, window):
            tokens = filler[: ask + 1]
            tokens[ask - distance], tokens[ask] = 0, 1
            want = O.forward(config, w, torch.tensor(tokens), dtype=torch.float64)
            rows[distance] = want[ask]
            for cuts in ([ask + 1], [ask, 1], [max(1, ask - distance), ask + 1 - max(1, ask - distance)], [ask - 1, 2], [ask - 2, 1, 1, 1]):
                got = run(g, mk, tokens, cuts)
                assert error(got[ask:], want[ask:]) < TOL[torch.float32], (ask, distance, cuts)
        apart = error(rows[window - 1][None], rows[window][None])
        assert apart > 0.1, f"the edge would not show ({apart:.3g})"


def test_the_first_token_is_seen_while_the_window_reaches_it():
    shape, w = pointed_model(12)
    mk, g = mk_kernel.get_mk(), on_gpu(shape, w, torch.float32)
    tokens = [0] + [1] * 20
    want = O.forward(shape.to_config(), w, torch.tensor(tokens), dtype=torch.float64)
    assert error(want[11:12], want[12:13]) > 0.1
    for cuts in ([21], [1] * 21, [2, 9, 1, 1, 8]):
        assert error(run(g, mk, tokens, cuts), want) < TOL[torch.float32]


@BOTH
def test_slots_and_cache_rows_used_again(dtype):
    """Unequal requests side by side in two slots, finished and replaced while others live, against each alone."""
    shape, w = model("odd")
    mk, g = mk_kernel.get_mk(), on_gpu(shape, w, dtype, slots=2, portion_rows=16)
    table, n = RequestTable(g), {"a": 41, "b": 17, "c": 60, "d": 3}
    got = {k: [] for k in n}
    tokens = {k: tokens_of(shape, v, seed=ord(k)) for k, v in n.items()}
    at = dict.fromkeys(n, 0)

    def feed(key, count):
        part = tokens[key][at[key]: at[key] + count]
        got[key].append(decode_hybrid.run_tokens(g, mk, table.get(key), part, range(len(part))))
        at[key] += len(part)
        if at[key] == n[key]:
            table.close(key)

    for key, count in (("a", 20), ("b", 9), ("a", 1), ("b", 1), ("b", 7), ("c", 2), ("a", 20), ("c", 30), ("d", 2), ("c", 1), ("d", 1), ("c", 27)):
        feed(key, count)
    mk.check()
    assert not table.live
    for key in n:
        want = O.forward(shape.to_config(), w, torch.tensor(tokens[key]), dtype=torch.float64)
        assert error(torch.cat(got[key]).double().cpu(), want) < TOL[dtype], key


@BOTH
def test_cutting_changes_only_rounding(dtype):
    shape, w = model("wide")
    mk, tokens = mk_kernel.get_mk(), tokens_of(shape, 70)
    g = on_gpu(shape, w, dtype, portion_rows=96)
    whole = run(g, mk, tokens, [70])
    for cuts in ([1] * 70, [2] * 35, [33, 37], [69, 1]):
        assert error(run(g, mk, tokens, cuts), whole) < TOL[dtype]


@pytest.mark.parametrize("queues", [256, 64, 5])
def test_any_number_of_queues(queues):
    shape, w = model("many_heads")
    mk, g = mk_kernel.get_mk(), on_gpu(shape, w, torch.float32)
    scheduler.build(g, queues)
    assert error(run(g, mk, tokens_of(shape, 20), [4] + [1] * 16), expected("many_heads", 20)) < TOL[torch.float32]


def test_wanted_rows_in_any_order():
    shape, w = model("odd")
    mk, g = mk_kernel.get_mk(), on_gpu(shape, w, torch.float32, portion_rows=16)
    request = RequestTable(g).open(0)
    got = decode_hybrid.run_tokens(g, mk, request, tokens_of(shape, 50), [49, 3, 17, 3]).double().cpu()
    assert error(got, expected("odd", 50)[[49, 3, 17, 3]]) < TOL[torch.float32]


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_greedy_generation(name):
    """The framework's own loop: prefill, device-side sampling, launches or one HIP graph."""
    shape, w = model(name)
    mk, prompt = mk_kernel.get_mk(), torch.tensor(tokens_of(shape, 12))
    g = on_gpu(shape, w, torch.float32, slots=2)
    tokens = prompt.tolist()
    for _ in range(20):
        tokens.append(int(O.forward(shape.to_config(), w, torch.tensor(tokens), dtype=torch.float64)[-1].argmax()))
    out = decode_hybrid.decode(g, prompt, 20, mk=mk)
    assert out["generated_ids"].tolist() == tokens
    assert out["timing"]["kernel_steps"] == 19
    graph = decode_hybrid.decode(g, prompt, 20, mk=mk, use_graph=True)
    assert graph["new_tokens"].tolist() == tokens[12:]
    late = decode_hybrid.decode(g, prompt, 20, mk=mk, timed_steps=5)
    assert late["new_tokens"].tolist() == tokens[12:] and late["timing"]["kernel_steps"] == 5


def test_a_captured_step_replays():
    """A captured decode step, replayed from the same state with eager work in between, gives the eager result every time."""
    shape, w = model("odd")
    mk, g = mk_kernel.get_mk(), on_gpu(shape, w, torch.float32)
    request = RequestTable(g).open(0)
    decode_hybrid.run_tokens(g, mk, request, tokens_of(shape, 9))
    g.slot, g.position_id, g.flip = request.slot, request.position, request.flip
    g.token.fill_(5)
    saved = [{k: t.clone() for k, t in s.items()} for s in g.layer_state]

    def restore():
        for have, kept in zip(g.layer_state, saved):
            for k in have:
                have[k].copy_(kept[k])

    mk(g)
    want = g.logits.clone()
    restore()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        mk(g)
    for _ in range(4):
        restore()
        g.logits.fill_(7.0)
        graph.replay()
        torch.cuda.synchronize()
        assert torch.equal(g.logits, want)
    mk.check()


def test_a_failed_step_is_reported_and_the_next_request_runs():
    """A poll budget of one is not enough for a step's waits; every workgroup still retires."""
    shape, w = model("wide")
    g, tokens = on_gpu(shape, w, torch.float32), tokens_of(shape, 10)
    hurried = mk_kernel.get_mk(spin_limit=1)
    table = RequestTable(g)
    decode_hybrid.run_tokens(g, hurried, table.open("x"), tokens[:1], [0])
    with pytest.raises(RuntimeError, match="ran out of polls"):
        hurried.check()
    table.close("x")
    mk = mk_kernel.get_mk()
    assert error(run(g, mk, tokens, [1] * 10, table=table), expected("wide", 10)) < TOL[torch.float32]


def test_malformed_instructions_are_rejected():
    shape, w = model("odd")
    g, mk = on_gpu(shape, w, torch.float32), mk_kernel.get_mk()
    scheduler.build(g)
    good = g.instructions.clone()
    for word, value, message in ((0, 77, "unknown opcode"), (1, 99, "out of bounds"), (4, 4000, "out of bounds"), (3, -2, "out of bounds")):
        g.instructions.zero_()
        g.instructions[0, 0] = good[0, 0]
        g.instructions[0, 0, word] = value
        mk(g)
        with pytest.raises(RuntimeError, match=message):
            mk.check()


def test_positions_outside_the_capacity_are_refused():
    shape, w = model("odd")
    g, mk = on_gpu(shape, w, torch.float32, max_positions=16), mk_kernel.get_mk()
    g.position_id = 16
    with pytest.raises(RuntimeError, match="position"):
        mk(g)
    g.position_id = 12
    with pytest.raises(RuntimeError, match="position"):
        mk.prefill(g, torch.zeros(5, dtype=torch.int64, device=DEVICE))


@BOTH
def test_a_model_folder_is_served(tmp_path, dtype):
    from safetensors.torch import save_file

    shape, w = model("odd")
    (tmp_path / "config.json").write_text(json.dumps(shape.to_config()))
    save_file(w, str(tmp_path / "model.safetensors"))
    g = decode_hybrid.load(tmp_path, dtype=dtype, max_positions=64)
    assert error(run(g, mk_kernel.get_mk(), tokens_of(shape, 30), [25, 1, 4]), expected("odd", 30)) < TOL[dtype]


def test_trace_runner(tmp_path):
    import subprocess
    import sys

    import numpy as np
    from safetensors.torch import save_file
    from __graft_entry__ import ROOT

    shape, w = model("odd")
    (tmp_path / "config.json").write_text(json.dumps(shape.to_config()))
    save_file(w, str(tmp_path / "model.safetensors"))
    out = tmp_path / "out"
    out.mkdir()
    tokens = tokens_of(shape, 30)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:20], "want": [4, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[20:21], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": tokens[21:], "want": [8]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": tokens[:1], "want": [0]}], "end": ["b"]}]
    done = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(out), "--max-tokens", "64"],
                          input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [x for x in done.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(4)]
    want = expected("odd", 30)
    for name, rows in (("0", [4, 19]), ("2", [29]), ("3", [0])):
        got = torch.from_numpy(np.fromfile(out / f"{name}.f32", dtype="<f4").reshape(len(rows), -1).copy()).double()
        assert error(got, want[rows]) < TOL[torch.float32]
    assert not (out / "1.f32").exists()
