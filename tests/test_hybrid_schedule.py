"""Host side of the hybrid route without a GPU: configuration, weight storage, instruction queues, slots, C ABI."""
import ctypes
import json
import subprocess
import sys

import pytest
import torch
from safetensors.torch import save_file

import hybrid_oracle as O
from __graft_entry__ import HYBRID_LIBRARY, ROOT, build_library
from qimeng_megakernel_amd import decode_hybrid, instruction, registry, synthetic
from qimeng_megakernel_amd.decode_schedule_hybrid import HybridShape, mk_kernel, weights
from qimeng_megakernel_amd.decode_schedule_hybrid.globs import build_globals
from qimeng_megakernel_amd.decode_schedule_hybrid.instructions import instruction_defs as D
from qimeng_megakernel_amd.decode_schedule_hybrid.instructions import scheduler as S
from qimeng_megakernel_amd.decode_schedule_hybrid.state import RequestTable

HEADER = ROOT / "include" / "qmk_hybrid.h"


def odd_shape(**kw):
    """Sizes off every storage multiple."""
    args = dict(width=52, vocab=77, streams=2, ff={"r": 36, "a": 20}, heads=3, dim=20, rot_dim=10, v_dim=12, rank=28, window=9, lru_width=60, blocks=5,
                taps=3, wkv_heads=3, wkv_dim=12, wkv_rank=7)
    args.update(kw)
    return synthetic.hybrid_shape(args.pop("pattern", "raw"), **args)


def write_model(folder, shape, seed=0):
    w = synthetic.random_hybrid_weights(shape, seed)
    folder.mkdir(exist_ok=True)
    (folder / "config.json").write_text(json.dumps(shape.to_config()))
    save_file(w, str(folder / "model.safetensors"))
    return w


def test_configuration_round_trip(tmp_path):
    shape = odd_shape()
    write_model(tmp_path / "m", shape)
    read, tensors = weights.read_checkpoint(tmp_path / "m")
    assert read == shape
    assert set(tensors) == set(weights.tensor_shapes(shape))
    assert registry.family_of(tmp_path / "m") is registry.HYBRID


def test_every_size_comes_from_the_configuration(tmp_path):
    config = odd_shape().to_config()
    config["layers"][1]["mixer"]["mask"]["size"] = 5
    config["layers"][1]["mixer"]["scale"] = 0.3
    config["layers"][1]["mixer"]["rot"]["base"] = 77.0
    config["norm"]["eps"] = 1e-3
    shape = HybridShape.from_config(config, {"l2.mix.w1": (7, 52)})
    assert (shape.layers[1].window, shape.layers[1].scale, shape.layers[1].rope_base, shape.eps) == (5, 0.3, 77.0, 1e-3)
    assert shape.layers[2].ff == 0 and shape.layers[0].ff == 36


def test_bad_checkpoints_are_refused(tmp_path):
    shape = odd_shape()
    w = write_model(tmp_path / "m", shape)
    del w["l1.mix.uk"]
    save_file(w, str(tmp_path / "m" / "model.safetensors"))
    with pytest.raises(ValueError, match="l1.mix.uk"):
        weights.read_checkpoint(tmp_path / "m")
    (tmp_path / "m" / "config.json").write_text(json.dumps({"architecture": "Other"}))
    with pytest.raises(ValueError, match="Other"):
        registry.family_of(tmp_path / "m")
    with pytest.raises(ValueError, match="unknown mixer"):
        HybridShape.from_config({**shape.to_config(), "layers": [{"type": "conv", "mixer": {}, "mlp": None}]})


def test_registered_shapes_resolve():
    for name, (family, _, _) in registry.MODELS.items():
        assert registry.shape_of(name) is not None
        assert family.mk_kernel() is not None and family.module("loop") is not None


def test_stored_matrices_compute_what_the_checkpoint_says():
    """Every stored matrix applied to padded vectors gives the checkpoint's product, in the rows the kernels expect, and
    zeros in the padding."""
    shape = odd_shape()
    w = synthetic.random_hybrid_weights(shape, 5)
    p = weights.pack(shape, w, "cpu")
    gen = torch.Generator().manual_seed(0)
    h = torch.randn(shape.width, generator=gen, dtype=torch.float64)
    hp = torch.zeros(shape.width_s, dtype=torch.float64)
    hp[: shape.width] = h
    f = {k: v.double() for k, v in w.items()}

    r, l = p["layers"][0], shape.layers[0]
    got = (r["in_w"].double() @ hp + r["in_b"].double()).view(2, l.blocks, l.block_s)
    for k, name in enumerate("yx"):
        want = (f[f"l0.mix.{name}"] @ h + f[f"l0.mix.{name}.b"]).view(l.blocks, l.block)
        assert torch.allclose(got[k, :, : l.block], want) and torch.all(got[k, :, l.block:] == 0)
    gates = r["mid_w"].view(l.blocks, l.block_s, 2, l.block_s).double()
    for k, name in enumerate(("ra", "ri")):
        assert torch.equal(gates[:, : l.block, k, : l.block], f[f"l0.mix.{name}"])
        assert torch.equal(r["mid_b"].view(l.blocks, l.block_s, 2)[:, : l.block, k].double(), f[f"l0.mix.{name}.b"])
    mlp = r["mlp_w"].view(l.ff_s, 2, shape.width_s).double()
    assert torch.equal(mlp[: l.ff, 0, : shape.width], f["l0.mlp.gate"]) and torch.equal(mlp[: l.ff, 1, : shape.width], f["l0.mlp.up"])
    assert torch.all(mlp[l.ff:] == 0) and torch.equal(r["down_w"][: shape.width, : l.ff].double(), f["l0.mlp.down"])

    a, l = p["layers"][1], shape.layers[1]
    rows = a["in_w"].double() @ hp
    q, rest = rows[: l.heads * l.q_stride].view(l.heads, l.q_stride), rows[l.heads * l.q_stride:]
    want = (f["l1.mix.q"] @ h).view(l.heads, -1)
    assert torch.allclose(q[:, : l.dim], want[:, : l.dim]) and torch.allclose(q[:, l.dim_s: l.dim_s + l.rot_dim], want[:, l.dim:])
    gate, latent = rest[: l.heads * l.v_s].view(l.heads, l.v_s), rest[l.heads * l.v_s:]
    assert torch.allclose(gate[:, : l.v_dim], (f["l1.mix.g"] @ h).view(l.heads, -1))
    down = f["l1.mix.dkv"] @ h
    assert torch.allclose(latent[: l.rank], down[: l.rank]) and torch.allclose(latent[l.rank_s: l.rank_s + l.rot_dim], down[l.rank:])
    absorb = a["mid_w"].view(l.heads, l.rank_s, l.dim_s).double()
    assert torch.equal(absorb[:, : l.rank, : l.dim], f["l1.mix.uk"].view(l.heads, l.dim, l.rank).transpose(1, 2))

    k, l = p["layers"][2], shape.layers[2]
    rows = (k["in_w"].double() @ hp)
    for i, name in enumerate("rkvg"):
        got = rows[i * l.mix_width: (i + 1) * l.mix_width].view(l.heads, l.dim_s)
        assert torch.allclose(got[:, : l.dim], (f[f"l2.mix.{name}"] @ h).view(l.heads, -1)) and torch.all(got[:, l.dim:] == 0)
    assert torch.allclose(rows[4 * l.mix_width:][: l.rank], f["l2.mix.w1"] @ h)
    assert torch.equal(k["next1"], torch.ones(shape.streams)) and torch.equal(a["next2"].double(), f["l2.hc1.in"])


@pytest.mark.parametrize("queues", [256, 24, 3])
@pytest.mark.parametrize("pattern", ["raw", "w", "aar"])
def test_schedule_covers_every_row_once(queues, pattern):
    shape = odd_shape(pattern=pattern)
    sched = S.HybridScheduler(shape, queues)
    stages = sched.stages()
    assert sched.barrier_groups() == -(-len(stages) // 4)
    covered: dict = {}
    for k, stage in enumerate(stages):
        kinds = {(type(i), i.layer) for i in stage}
        assert len(kinds) == 1, "a stage holds one kind of instruction"
        for ins in stage:
            assert ins.wait_stage == k - 1 and ins.arrive_stage == (k if k + 1 < len(stages) else -1)
            assert ins.wait_count == (len(stages[k - 1]) if k else 0)
            assert instruction.decode_words(ins.padded(), D.INSTRUCTIONS) == ins
            if ins.opcode() not in (4, 6):
                key = (k, ins.sub)
                covered.setdefault(key, []).extend(range(ins.start, ins.start + ins.count))
                assert ins.count * (2 if ins.opcode() in (2, 8) else 1) <= S.MAX_ROWS
    for rows in covered.values():
        first = min(rows)
        assert sorted(rows) == list(range(first, first + len(rows)))
    last = covered[(len(stages) - 1, 0)]
    assert sorted(last) == list(range(shape.vocab_s))
    lanes = sched.instruction_queues()
    assert sum(len(q) for q in lanes) == sum(len(s) for s in stages)
    assert all([i.wait_stage for i in q] == sorted(i.wait_stage for i in q) for q in lanes), "a queue runs its stages in order"


@pytest.mark.parametrize("queues", [256, 24, 3])
def test_a_queue_owns_its_rows_of_the_streams(queues):
    owner: dict = {}
    for q, column in enumerate(S.HybridScheduler(odd_shape(width=300, ff={"r": 36, "a": 20, "w": 52}), queues).instruction_queues()):
        for ins in column:
            if ins.opcode() == 7:
                assert ins.count <= S.MAX_OUT_ROWS
                for row in range(ins.start, ins.start + ins.count):
                    assert owner.setdefault(row, q) == q
    assert sorted(owner) == list(range(304))


def test_one_leading_instruction_keeps_shared_rows():
    stages = S.HybridScheduler(odd_shape(pattern="aw"), 16).stages()
    assert sum(i.extra for s in stages for i in s if i.opcode() == 3) == 1
    assert [i.extra for s in stages for i in s if i.opcode() == 1 and i.layer == 1].count(1) == 1


def test_the_cache_is_a_ring_of_window_and_portion():
    shape = odd_shape(pattern="a", window=9)
    packed = weights.pack(shape, synthetic.random_hybrid_weights(shape, 0), "cpu")
    assert build_globals(shape, packed, max_positions=1000, portion_rows=16).layer_state[0]["cache"].shape[1] == 9 - 1 + 16
    assert build_globals(shape, packed, max_positions=12, portion_rows=16).layer_state[0]["cache"].shape[1] == 12
    assert build_globals(shape, packed, max_positions=12, dtype=torch.float32).layer_state[0]["cache"].dtype == torch.float32


def test_slots_are_handed_out_cleared():
    shape = odd_shape()
    g = build_globals(shape, weights.pack(shape, synthetic.random_hybrid_weights(shape, 0), "cpu"), max_positions=32, slots=2)
    table = RequestTable(g)
    a, b = table.open("a"), table.open("b")
    assert {a.slot, b.slot} == {0, 1}
    with pytest.raises(RuntimeError):
        table.open("c")
    g.layer_state[0]["state"].fill_(3.0)
    g.layer_state[2]["shift"].fill_(3.0)
    a.position, a.flip = 5, 1
    table.close("a")
    c = table.get("c")
    assert (c.slot, c.position, c.flip) == (a.slot, 0, 0)
    assert torch.all(g.layer_state[0]["state"][c.slot] == 0) and torch.all(g.layer_state[2]["shift"][c.slot] == 0)
    assert torch.all(g.layer_state[0]["state"][b.slot] == 3.0)


def test_step_arguments_are_checked_on_the_host():
    shape = odd_shape()
    g = build_globals(shape, weights.pack(shape, synthetic.random_hybrid_weights(shape, 0), "cpu"), max_positions=8)
    request = RequestTable(g).open("a")
    for tokens, want, error in (([], [], ValueError), ([1] * 9, [], ValueError), ([1, 2], [2], IndexError)):
        with pytest.raises(error):
            decode_hybrid.run_tokens(g, None, request, tokens, want)


@pytest.fixture(scope="module")
def lib():
    if not HYBRID_LIBRARY.is_file():
        build_library(HYBRID_LIBRARY)
    return mk_kernel.load_library()


@pytest.mark.parametrize("struct,mirror", [("QmkHybridLayer", mk_kernel.QmkHybridLayer), ("QmkHybridArgs", mk_kernel.QmkHybridArgs)])
def test_struct_layout_matches_header(tmp_path, struct, mirror):
    fields = [name for name, _ in mirror._fields_]
    lines = ['#include <stdio.h>', '#include <stddef.h>', f'#include "{HEADER}"', "int main(void) {", f'  printf("%zu\\n", sizeof({struct}));']
    lines += [f'  printf("%zu\\n", offsetof({struct}, {f}));' for f in fields] + ["  return 0;", "}"]
    (tmp_path / "layout.c").write_text("\n".join(lines))
    subprocess.run(["gcc", "-std=c99", "-Wall", "-Werror", "-o", str(tmp_path / "layout"), str(tmp_path / "layout.c")], check=True)
    out = [int(x) for x in subprocess.run([str(tmp_path / "layout")], check=True, capture_output=True, text=True).stdout.split()]
    assert out == [ctypes.sizeof(mirror)] + [getattr(mirror, f).offset for f in fields]


def test_argument_errors_come_back_as_codes(lib):
    a = mk_kernel.QmkHybridArgs()
    assert lib.qmk_hybrid_decode_step(ctypes.byref(a)) == 1 and lib.qmk_hybrid_prefill(ctypes.byref(a)) == 1
    shape = odd_shape()
    g = build_globals(shape, weights.pack(shape, synthetic.random_hybrid_weights(shape, 0), "cpu"), max_positions=32)
    table = mk_kernel.layer_table(g)
    a.layers = ctypes.addressof(table)
    assert lib.qmk_hybrid_decode_step(ctypes.byref(a)) == 2
    a.struct_size = ctypes.sizeof(a)
    a.num_layers, a.width, a.width_true, a.streams, a.vocab, a.vocab_rows = len(shape.layers), shape.width_s, shape.width, shape.streams, shape.vocab, shape.vocab_s
    a.eps, a.max_positions, a.portion_rows, a.max_splits = shape.eps, 32, 8, 1
    assert lib.qmk_hybrid_decode_bytes(ctypes.byref(a)) > 0 and lib.qmk_hybrid_prefill_bytes(ctypes.byref(a)) > 0
    a.streams = 9
    assert lib.qmk_hybrid_decode_bytes(ctypes.byref(a)) == 0
    a.streams = shape.streams
    table[1].rank = 8
    assert lib.qmk_hybrid_prefill_bytes(ctypes.byref(a)) == 0


def test_a_missing_library_is_an_import_error(tmp_path):
    with pytest.raises(ImportError, match="build it first"):
        mk_kernel.load_library(tmp_path)


def test_trace_runner_explains_itself():
    out = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--help"], capture_output=True, text=True)
    assert out.returncode == 0 and "--max-tokens" in out.stdout
