"""The hybrid route's plain-residual design (Givopel) on the GPU against the plain implementation (oracle/givopel_oracle.py).

fp32 is compared at rounding level, so a wrong key, decay, step size or edge anywhere shows; bf16 at bf16's.
"""
import functools
import json

import pytest
import torch

import givopel_oracle as O
from qimeng_megakernel_amd import decode_hybrid, synthetic
from qimeng_megakernel_amd.decode_schedule_hybrid import mk_kernel, weights
from qimeng_megakernel_amd.decode_schedule_hybrid.globs import build_globals
from qimeng_megakernel_amd.decode_schedule_hybrid.instructions import scheduler
from qimeng_megakernel_amd.decode_schedule_hybrid.state import RequestTable

pytestmark = pytest.mark.gpu

DEVICE = "cuda:0"
TOL = {torch.float32: 4e-5, torch.bfloat16: 8e-2}
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])

#: sizes off and on the storage multiples, grouped heads everywhere, loops at either end, with and without feed-forwards
SHAPES = {
    "odd": synthetic.looped_shape("pgp", width=52, vocab=77, ff={"p": 36}, loop=(1, 3, 2), logit_scale=0.7, logit_softcap=4.0, heads=6, kv_heads=2, dim=20,
                                  v_dim=12, rot_dim=10, rope_base=50.0, rope_scaling=(3.0, 40.0, 2.0, 0.7), scale=0.31, delta_heads=6, delta_kv_heads=3,
                                  delta_dim=12, delta_v_dim=20, taps=4, delta_rank=7, gate_rank=5, gla_heads=3, gla_dim=20, gla_v_dim=28, gla_rank=9, tau=5.0),
    "from_the_start": synthetic.looped_shape("gp", width=64, vocab=130, ff={"g": 48, "p": 16}, loop=(0, 2, 3), heads=2, kv_heads=2, dim=32, v_dim=16, rot_dim=32,
                                             delta_heads=2, delta_kv_heads=1, delta_dim=16, delta_v_dim=16, taps=1, delta_rank=16, gate_rank=16, gla_heads=1,
                                             gla_dim=16, gla_v_dim=16, gla_rank=16, tau=1.0, eps=1e-3, logit_scale=3.0, logit_softcap=9.0),
    "no_loop": synthetic.looped_shape("gpg", width=80, vocab=96, ff={"p": 100}, heads=5, kv_heads=1, dim=24, v_dim=40, rot_dim=0, delta_heads=4, delta_kv_heads=4,
                                      delta_dim=36, delta_v_dim=8, taps=2, delta_rank=20, gate_rank=33, gla_heads=2, gla_dim=70, gla_v_dim=30, gla_rank=3, tau=8.0),
    "many_heads": synthetic.looped_shape("pg", width=160, vocab=512, ff={"p": 96, "g": 80}, loop=(0, 1, 2), heads=36, kv_heads=2, dim=16, v_dim=24, rot_dim=8,
                                         delta_heads=18, delta_kv_heads=9, delta_dim=32, delta_v_dim=24, taps=3, delta_rank=12, gate_rank=40, gla_heads=7,
                                         gla_dim=24, gla_v_dim=16, gla_rank=12, tau=2.0, rope_scaling=(2.0, 64.0, 4.0, 1.0)),
    "wide": synthetic.looped_shape("pgp", width=640, vocab=1000, ff={"p": 1100, "g": 520}, loop=(1, 2, 2), heads=8, kv_heads=4, dim=128, v_dim=128, rot_dim=64,
                                   delta_heads=4, delta_kv_heads=2, delta_dim=128, delta_v_dim=128, taps=4, delta_rank=64, gate_rank=64, gla_heads=4, gla_dim=64,
                                   gla_v_dim=128, gla_rank=16, logit_softcap=20.0),
    "large_heads": synthetic.looped_shape("pg", width=96, vocab=64, loop=(0, 2, 1), heads=2, kv_heads=1, dim=200, v_dim=250, rot_dim=36, delta_heads=2,
                                          delta_kv_heads=2, delta_dim=250, delta_v_dim=136, taps=7, delta_rank=24, gate_rank=8, gla_heads=2, gla_dim=136,
                                          gla_v_dim=250, gla_rank=24),
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
@pytest.mark.parametrize("cuts", [[2] * 40, [3, 1, 2, 61, 1, 1, 11], [31, 33, 16], [77, 2, 1], [16, 17, 15, 32]], ids=["twos", "mixed", "tiles", "tail", "chunks"])
@pytest.mark.parametrize("name", ["odd", "from_the_start", "many_heads", "wide"])
def test_portions(name, dtype, cuts):
    check(name, dtype, 80, cuts, portion_rows=96)


def test_portions_longer_than_a_launch_takes():
    check("odd", torch.float32, 110, [70, 40], portion_rows=16)


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_long_decoding(name):
    check(name, torch.float32, 300, [5] + [1] * 295, max_positions=300, portion_rows=8)


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
            assert torch.allclose(a[k][:n], b[k][:n], rtol=1e-3, atol=2e-5), k


PARTS = {
    "gla": ("g", dict(gla_heads=2, gla_dim=24, gla_v_dim=40, gla_rank=20, tau=3.0)),
    "gla, one head": ("g", dict(gla_heads=1, gla_dim=256, gla_v_dim=16, gla_rank=33, tau=16.0)),
    "parallel": ("p", dict(heads=4, kv_heads=2, dim=24, v_dim=40, rot_dim=4, delta_heads=2, delta_kv_heads=1, delta_dim=20, delta_v_dim=12, taps=3, delta_rank=4,
                           gate_rank=6)),
    "parallel, many taps": ("p", dict(heads=17, kv_heads=17, dim=8, v_dim=8, rot_dim=8, delta_heads=3, delta_kv_heads=3, delta_dim=40, delta_v_dim=24, taps=16,
                                      delta_rank=17, gate_rank=1)),
}


@pytest.mark.parametrize("part", sorted(PARTS))
@pytest.mark.parametrize("ff", [0, 56])
@pytest.mark.parametrize("loop", [None, (0, 1, 2)])
def test_each_mechanism_alone(part, ff, loop):
    """One layer; the residual behind every run of it as well as the logits."""
    pattern, kw = PARTS[part]
    shape = synthetic.looped_shape(pattern, width=40, vocab=61, ff={pattern: ff}, loop=loop, **kw)
    w = synthetic.random_hybrid_weights(shape, 4)
    tokens = tokens_of(shape, 50)
    layers = []
    want = O.forward(shape.to_config(), w, torch.tensor(tokens), dtype=torch.float64, layer_outputs=layers)
    g, mk = on_gpu(shape, w, torch.float32), mk_kernel.get_mk()
    assert error(run(g, mk, tokens, [1] * 50), want) < TOL[torch.float32]
    request = RequestTable(g).open("y")
    g.slot, g.position_id, g.flip = request.slot, 0, 0
    out = torch.zeros(shape.run_count, 50, shape.width_s, device=DEVICE)
    logits = mk.prefill(g, torch.tensor(tokens, device=DEVICE), torch.arange(50, dtype=torch.int32, device=DEVICE), layer_out=out)
    assert error(logits[:, : shape.vocab].double().cpu(), want) < TOL[torch.float32]
    assert len(layers) == shape.run_count
    for k, layer in enumerate(layers):
        assert error(out[k, :, : shape.width].double().cpu(), layer) < TOL[torch.float32]
    assert torch.all(out[:, :, shape.width:] == 0)


def pointed_model(heads=4, kv_heads=2):
    """One layer in whose attention token 1 asks and token 0 answers: the asker's score for the answerer stands far above all
    others, whatever lies between them."""
    shape = synthetic.looped_shape("p", width=48, vocab=40, heads=heads, kv_heads=kv_heads, dim=16, v_dim=16, rot_dim=8, scale=1.0, delta_heads=2,
                                   delta_kv_heads=1, delta_dim=16, delta_v_dim=16, taps=2, delta_rank=4, gate_rank=4)
    w = synthetic.random_hybrid_weights(shape, 9)
    w["embed"][:, :4] = 0
    w["embed"][0, :2] = torch.tensor([12.0, -12.0])     # the mean the norm takes off stays where it is
    w["embed"][1, 2:4] = torch.tensor([12.0, -12.0])
    w["l0.norm1"] = torch.ones_like(w["l0.norm1"])
    for name, n, column in (("q", heads, 2), ("k", kv_heads, 0)):
        m = w[f"l0.mix.left.{name}"].view(n, 16, 48)
        m.mul_(0.02)
        m[:, 12, column], m[:, 12, column + 1] = 1.5, -1.5      # a dimension that is not rotated
    w["l0.mix.left.v"] *= 3.0
    return shape, w


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
def test_a_far_key_is_found_wherever_it_is(dtype):
    """The key at the edges of tiles, parts, chunks and portions, near and far, from a prompt and from a decoded token."""
    shape, w = pointed_model()
    config, mk = shape.to_config(), mk_kernel.get_mk()
    g = on_gpu(shape, w, dtype, max_positions=420, portion_rows=128)
    filler = torch.randint(2, 40, (400,), generator=torch.Generator().manual_seed(2)).tolist()
    blank = {ask: O.forward(config, w, torch.tensor(filler[:ask] + [1]), dtype=torch.float64)[ask:] for ask in (130, 399)}
    for ask in (130, 399):
        for at in (0, 1, 15, 16, 31, 32, 63, 64, 127, 128, ask - 1):
            tokens = filler[:ask] + [1]
            tokens[at] = 0
            want = O.forward(config, w, torch.tensor(tokens), dtype=torch.float64)[ask:]
            assert error(blank[ask], want) > 0.1, "the key would not show"
            for cuts in ([ask + 1], [ask, 1], [max(at, 1), ask + 1 - max(at, 1)], [ask - 1, 2]):
                assert error(run(g, mk, tokens, cuts)[ask:], want) < TOL[dtype], (ask, at, cuts)


def test_the_current_token_is_seen_and_written():
    """The newest key of the attention and the newest write of the delta rule enter a token's own output."""
    shape, w = pointed_model()
    w["embed"][1, :2] = torch.tensor([12.0, -12.0])      # token 1 answers itself
    mk, g = mk_kernel.get_mk(), on_gpu(shape, w, torch.float32)
    tokens = [5, 9, 1, 7, 1, 1, 3]
    want = O.forward(shape.to_config(), w, torch.tensor(tokens), dtype=torch.float64)
    for cuts in ([7], [1] * 7, [2, 1, 4]):
        assert error(run(g, mk, tokens, cuts), want) < TOL[torch.float32]


@pytest.mark.parametrize("strength", [0.0, 30.0], ids=["hardly any decay", "decays that underflow"])
def test_extreme_decays(strength):
    """Decays near one over hundreds of tokens, and so strong that the products over a chunk underflow."""
    shape, w = model("odd")
    w = dict(w)
    for name in list(w):
        if name.endswith("A_log"):
            w[name] = torch.full_like(w[name], -9.0 if strength == 0 else 3.5)
        if name.endswith("dt_bias"):
            w[name] = torch.full_like(w[name], strength)
        if name.endswith("a2.b"):
            w[name] = torch.full_like(w[name], 12.0 if strength == 0 else -8.0 * strength)
    mk, g = mk_kernel.get_mk(), on_gpu(shape, w, torch.float32, max_positions=300, portion_rows=256)
    tokens = tokens_of(shape, 220)
    want = O.forward(shape.to_config(), w, torch.tensor(tokens), dtype=torch.float64)
    for cuts in ([220], [200] + [1] * 20, [2] * 10 + [99, 101]):
        assert error(run(g, mk, tokens, cuts), want) < 2 * TOL[torch.float32]


def test_the_same_key_over_and_over():
    """Repeated tokens: the delta rule's keys in a chunk are parallel, its triangular system as far from diagonal as it gets."""
    shape, w = model("odd")
    mk, g = mk_kernel.get_mk(), on_gpu(shape, w, torch.float32)
    tokens = [3] * 70 + [5, 3] * 20
    want = O.forward(shape.to_config(), w, torch.tensor(tokens), dtype=torch.float64)
    rounding = error(O.forward(shape.to_config(), w, torch.tensor(tokens), dtype=torch.float32).double(), want)     # above the usual here
    for cuts in ([64, 46], [1] * 110):
        assert error(run(g, mk, tokens, cuts), want) < max(TOL[torch.float32], 4 * rounding)


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


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_greedy_generation(name):
    """The framework's own loop: prefill, device-side sampling, launches or one HIP graph (replayed by the loop itself)."""
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


def test_a_captured_step_replays():
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


def test_malformed_instructions_are_rejected():
    shape, w = model("odd")
    g, mk = on_gpu(shape, w, torch.float32), mk_kernel.get_mk()
    scheduler.build(g)
    stages = scheduler.HybridScheduler(shape, 256, g.max_positions).stages()
    kinds = {ins.opcode(): ins for stage in reversed(stages) for ins in stage}
    for opcode, field, value in ((10, "sub", 99), (10, "layer", 0), (11, "count", 4000), (11, "sub", -1), (12, "start", 4000), (4, "sub", 50), (4, "start", 99),
                                 (7, "start", 4000), (1, "start", 4000)):
        words = kinds[opcode].padded()
        ins = type(kinds[opcode])(**{**vars(kinds[opcode]), field: value, "wait_stage": -1})
        assert ins.padded() != words
        g.instructions.zero_()
        g.instructions[0, 0] = torch.tensor(ins.padded(), dtype=torch.int32)
        mk(g)
        with pytest.raises(RuntimeError, match="out of bounds"):
            mk.check()


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
