"""Host side of the hybrid route's plain-residual design without a GPU: configuration, table, weight storage, queues, states."""
import ctypes
import json

import pytest
import torch
from safetensors.torch import save_file

from __graft_entry__ import HYBRID_LIBRARY, build_library
from qimeng_megakernel_amd import instruction, registry, synthetic
from qimeng_megakernel_amd.decode_schedule_hybrid import HybridShape, mk_kernel, weights
from qimeng_megakernel_amd.decode_schedule_hybrid.globs import build_globals
from qimeng_megakernel_amd.decode_schedule_hybrid.instructions import instruction_defs as D
from qimeng_megakernel_amd.decode_schedule_hybrid.instructions import scheduler as S
from qimeng_megakernel_amd.decode_schedule_hybrid.state import RequestTable


def odd_shape(pattern="pgp", **kw):
    """Sizes off every storage multiple."""
    args = dict(width=52, vocab=77, ff={"p": 36}, loop=(1, 3, 2), logit_scale=0.7, logit_softcap=4.0, heads=6, kv_heads=2, dim=20, v_dim=12, rot_dim=10,
                rope_base=50.0, rope_scaling=(3.0, 40.0, 6.0, 0.7), scale=0.31, delta_heads=6, delta_kv_heads=3, delta_dim=12, delta_v_dim=20, taps=4,
                delta_rank=7, gate_rank=5, gla_heads=3, gla_dim=20, gla_v_dim=28, gla_rank=9, tau=5.0)
    args.update(kw)
    return synthetic.looped_shape(pattern, **args)


def on_cpu(shape, **kw):
    return build_globals(shape, weights.pack(shape, synthetic.random_hybrid_weights(shape, 0), "cpu"), **kw)


def test_configuration_round_trip(tmp_path):
    shape = odd_shape()
    w = synthetic.random_hybrid_weights(shape, 0)
    (tmp_path / "config.json").write_text(json.dumps(shape.to_config()))
    save_file(w, str(tmp_path / "model.safetensors"))
    read, tensors = weights.read_checkpoint(tmp_path)
    assert read == shape and set(tensors) == set(weights.tensor_shapes(shape))
    assert registry.family_of(tmp_path) is registry.HYBRID
    del w["l0.mix.right.g2"]
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l0.mix.right.g2"):
        weights.read_checkpoint(tmp_path)


def test_every_size_and_constant_comes_from_the_configuration():
    shape = odd_shape()
    config = shape.to_config()
    ranks = {"l0.mix.right.a1": (3, 52), "l0.mix.right.g1": (4, 52), "l1.mix.a1": (6, 52), "l2.mix.right.a1": (8, 52), "l2.mix.right.g1": (11, 52)}
    left, right = config["layers"][2]["mixer"]["left"], config["layers"][2]["mixer"]["right"]
    left.update(scale=0.9, heads=4, vdim=9)
    left["rot"].update(base=33.0, dims=4)
    left["rot"]["scaling"]["slow"] = 0.1
    right.update(conv=2, heads=3)
    config["layers"][1]["mixer"]["tau"] = 2.5
    config["layers"][2]["mlp"] = None
    config.update(loop={"start": 0, "stop": 1, "times": 4}, logit_scale=5.0, logit_softcap=None)
    config["norm"]["eps"] = 1e-2
    got = HybridShape.from_config(config, ranks)
    a, d = got.layers[2].branches
    assert (a.scale, a.heads, a.v_dim, a.rope_base, a.rot_dim, a.rope_scaling) == (0.9, 4, 9, 33.0, 4, (3.0, 40.0, 6.0, 0.1))
    assert (d.taps, d.heads, d.rank, d.gate_rank) == (2, 3, 8, 11) and got.layers[0].branches[1].gate_rank == 4
    assert (got.layers[1].tau, got.layers[1].rank, got.layers[2].ff, got.layers[0].ff) == (2.5, 6, 0, 36)
    assert (got.loop, got.logit_scale, got.logit_softcap, got.eps) == ((0, 1, 4), 5.0, 0.0, 1e-2)
    del config["loop"], config["logit_scale"], left["rot"]["scaling"]
    got = HybridShape.from_config(config, ranks)
    assert got.loop is None and got.logit_scale == 1.0 and got.layers[2].branches[0].rope_scaling is None


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="rglru"), "unknown mixer"),
    (lambda c: c["loop"].update(stop=9), "a loop of layers"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "do not divide"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=64), "rotated dimensions"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "unknown feed-forward"),
])
def test_bad_configurations_are_refused(change, message):
    config = odd_shape().to_config()
    change(config)
    with pytest.raises(ValueError, match=message):
        HybridShape.from_config(config, {f"l{i}.mix.{n}": (5, 52) for i in range(3) for n in ("a1", "right.a1", "right.g1")})


def test_entries_follow_the_loop_and_hand_the_residual_on():
    entries = odd_shape().entries
    assert [e.type for e in entries] == ["attention", "delta", "join", "gla", "attention", "delta", "join", "gla", "attention", "delta", "final"]
    assert [e.layer for e in entries] == [0, 0, -1, 1, 2, 2, -1, 1, 2, 2, -1]
    readers = [e for e in entries if e.branch == 0]
    assert [e.prev for e in readers] == [-1, 0, -1, 3, 4, -1, 7, 8]
    assert readers[0].x_from == -1
    for before, after in zip(readers, readers[1:]):
        assert after.x_from == before.x_to != after.x_to
    assert [e.ff for e in entries] == [36, 0, 0, 0, 36, 0, 0, 0, 36, 0, 0]


def test_passes_share_weights_and_have_states_of_their_own():
    g = on_cpu(odd_shape(), max_positions=16)
    for key in ("in_w", "o_w"):
        assert g.layer_weights[3][key].data_ptr() == g.layer_weights[7][key].data_ptr()
    assert g.layer_state[3]["state"].data_ptr() != g.layer_state[7]["state"].data_ptr()
    assert g.layer_state[4]["cache"].data_ptr() != g.layer_state[8]["cache"].data_ptr()
    assert g.layer_state[4]["cache"].shape == (1, 16, 2, 48) and g.layer_state[5]["shift"].shape == (1, 2, 3, 2 * 3 * 16 + 6 * 32)


def test_slots_are_handed_out_cleared():
    g = on_cpu(odd_shape(), max_positions=32, slots=2)
    table = RequestTable(g)
    a, b = table.open("a"), table.open("b")
    for s in g.layer_state:
        for t in s.values():
            t.fill_(3.0)
    table.close("a")
    c = table.get("c")
    assert c.slot == a.slot
    for s in g.layer_state:
        for name in ("state", "shift"):
            if name in s:
                assert torch.all(s[name][c.slot] == 0) and torch.all(s[name][b.slot] == 3.0)


def test_stored_matrices_compute_what_the_checkpoint_says():
    """Every stored matrix applied to padded vectors gives the checkpoint's product, in the rows the kernels expect, and zeros
    in the padding."""
    shape = odd_shape()
    w = synthetic.random_hybrid_weights(shape, 5)
    p = weights.pack(shape, w, "cpu")["layers"]
    gen = torch.Generator().manual_seed(0)
    h = torch.randn(shape.width, generator=gen, dtype=torch.float64)
    hp = torch.zeros(shape.width_s, dtype=torch.float64)
    hp[: shape.width] = h
    f = {k: v.double() for k, v in w.items()}

    def rows(entry, sizes):
        out, at = p[entry]["in_w"].double() @ hp, 0
        for name, n, size, true in sizes:
            part = out[at: at + n * size].view(n, size)
            want = (f[name] @ h).view(n, true) if n > 1 else (f[name] @ h)[None]
            assert torch.allclose(part[:, :true], want) and torch.all(part[:, true:] == 0), name
            at += n * size
        assert at == out.numel()

    rows(0, [("l0.mix.left.q", 6, 32, 20), ("l0.mix.left.k", 2, 32, 20), ("l0.mix.left.v", 2, 16, 12), ("l0.mix.left.g", 6, 16, 12)])
    rows(1, [("l0.mix.right.q", 3, 16, 12), ("l0.mix.right.k", 3, 16, 12), ("l0.mix.right.v", 6, 32, 20), ("l0.mix.right.a1", 1, 16, 7), ("l0.mix.right.g1", 1, 16, 5),
             ("l0.mix.right.b", 1, 16, 6)])
    rows(3, [("l1.mix.q", 3, 32, 20), ("l1.mix.k", 3, 32, 20), ("l1.mix.v", 3, 32, 28), ("l1.mix.g", 3, 32, 28), ("l1.mix.a1", 1, 16, 9)])
    d = p[1]
    assert torch.equal(d["mid_w"].view(6, 16, 16)[:, :12, :7].double(), f["l0.mix.right.a2"].view(6, 12, 7))
    assert torch.equal(d["gate_w"].view(6, 32, 16)[:, :20, :5].double(), f["l0.mix.right.g2"].view(6, 20, 5))
    assert torch.allclose(d["vec1"][:6].double(), -torch.exp(f["l0.mix.right.A_log"]))
    taps = d["vec2"].view(4, -1).double()
    assert torch.equal(taps[:, :48].view(4, 3, 16)[:, :, :12], f["l0.mix.right.q.conv"].T.reshape(4, 3, 12))
    assert torch.equal(taps[:, 96:].view(4, 6, 32)[:, :, :20], f["l0.mix.right.v.conv"].T.reshape(4, 6, 20))
    o = p[1]["o_w"].view(64, 6, 32).double()
    assert torch.equal(o[:52, :, :20], f["l0.mix.right.o"].view(52, 6, 20)) and torch.all(o[:, :, 20:] == 0)
    join = p[2]["in_w"].double()
    x0 = torch.zeros_like(hp)
    x0[: shape.width] = torch.randn(shape.width, generator=gen, dtype=torch.float64)
    assert torch.allclose((join @ torch.cat([hp, x0]))[: shape.width], f["loop.in"] @ torch.cat([h, x0[: shape.width]]))
    assert torch.equal(p[-1]["norm1"][: shape.width].double(), f["final.norm"])


@pytest.mark.parametrize("queues", [256, 24, 3])
@pytest.mark.parametrize("pattern,kw", [("pgp", {}), ("g", dict(loop=None)), ("pp", dict(loop=(0, 1, 3), heads=40, kv_heads=2, v_dim=150)), ("ggp", dict(ff={"g": 52}))])
def test_schedule_covers_every_row_once(queues, pattern, kw):
    shape = odd_shape(pattern, **kw)
    sched = S.HybridScheduler(shape, queues, 500)
    stages = sched.stages()
    for k, stage in enumerate(stages):
        assert stage
        for ins in stage:
            assert ins.wait_stage == k - 1 and ins.arrive_stage == (k if k + 1 < len(stages) else -1)
            assert ins.wait_count == (len(stages[k - 1]) if k else 0)
            assert instruction.decode_words(ins.padded(), D.INSTRUCTIONS) == ins
    done: dict = {}
    for ins in (i for stage in stages for i in stage):
        code = ins.opcode()
        if code == 4:
            done.setdefault((code, ins.layer, ins.sub, ins.extra), []).append(ins.start)
            assert ins.count == sched.parts(ins.layer) <= S.MAX_PARTS
        elif code == 11:
            done.setdefault((code, ins.layer), []).append(ins.sub)
        else:
            done.setdefault((code, ins.layer, ins.sub), []).extend(range(ins.start, ins.start + ins.count))
            assert ins.count * (2 if code == 8 else 1) <= S.MAX_ROWS
    want: dict = {}
    for i, e in enumerate(shape.entries):
        l, width = e.shape, shape.width_s
        if e.type == "join":
            want[12, i, 0] = width
        elif e.type == "final":
            want[9, i, 0] = shape.vocab_s
        else:
            want[1, i, 0], want[7, i, 0] = l.in_rows, width
            if e.ff:
                want[8, i, 0], want[7, i, 1] = shape.layers[e.layer].ff_s, width
            if e.type == "attention":
                want[11, i] = l.heads
                for g, c in sched.attention_groups(l):
                    want[4, i, g, c] = sched.parts(i)
            else:
                want.update({(10, i, h): l.v_s for h in range(l.heads)})
                if e.type == "delta":
                    want[13, i, 0] = l.mix_width
    assert {k: sorted(v) for k, v in done.items()} == {k: list(range(n)) for k, n in want.items()}


def test_one_instruction_of_a_run_keeps_the_residual():
    shape = odd_shape()
    stages = S.HybridScheduler(shape, 16).stages()
    kept = [i.layer for s in stages for i in s if i.opcode() == 1 and i.extra]
    assert kept == [0, 3, 4, 7, 8]


def test_bytes_and_operations_count_every_pass():
    once, twice = odd_shape(loop=(1, 3, 1)), odd_shape(loop=(1, 3, 2))
    assert twice.run_count == once.run_count + 2
    body = 2 * (sum(once.layers[i].weight_count(52) for i in (1, 2)) + 2 * 52 * 52)
    assert twice.weight_bytes_per_token() - once.weight_bytes_per_token() == body
    assert twice.step_bytes(100) > once.step_bytes(100) + body and twice.prefill_flops(10) > once.prefill_flops(10)


@pytest.fixture(scope="module")
def lib():
    if not HYBRID_LIBRARY.is_file():
        build_library(HYBRID_LIBRARY)
    return mk_kernel.load_library()


@pytest.mark.parametrize("field,value", [("prev", 9), ("x_from", 2), ("x_to", -1), ("branch", 1), ("branches", 3), ("type", 2), ("proj_at", 3), ("head_dim", 8),
                                         ("kv_heads", 5), ("v_dim", 512), ("q_stride", 16)])
def test_tables_that_do_not_fit_are_refused(lib, field, value):
    shape = odd_shape()
    g = on_cpu(shape, max_positions=32)
    table = mk_kernel.layer_table(g)
    a = mk_kernel.QmkHybridArgs()
    a.layers, a.struct_size = ctypes.addressof(table), ctypes.sizeof(a)
    a.num_layers, a.width, a.width_true, a.streams, a.vocab, a.vocab_rows = len(shape.entries), shape.width_s, shape.width, 0, shape.vocab, shape.vocab_s
    a.eps, a.max_positions, a.portion_rows, a.max_splits = shape.eps, 32, 8, 1
    assert lib.qmk_hybrid_decode_bytes(ctypes.byref(a)) > 0 and lib.qmk_hybrid_prefill_bytes(ctypes.byref(a)) > 0
    setattr(table[4], field, value)
    assert lib.qmk_hybrid_decode_bytes(ctypes.byref(a)) == 0 and lib.qmk_hybrid_prefill_bytes(ctypes.byref(a)) == 0
