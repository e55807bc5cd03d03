"""Pikadra without a GPU: the configuration reader and writer, the checkpoint reader, the registry, the order of layer runs, the host
side of a step, and the float64 oracle (``oracle/pikadra_oracle.py``) against itself -- a prompt at once, token by token, and in
portions must agree, and every mechanism must matter."""
import copy
import ctypes
import json
import math
import os
import subprocess

import pytest
import torch

from oracle import pikadra_oracle as O
from promptcache_amd.model import weights as W
from promptcache_amd.model.config import PikadraLayer, PikadraShape, architecture_of

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64


def small_shape():
    mla = dict(scale=0.5, rot_base=700.0)
    return PikadraShape(vocab_size=53, hidden_size=36, norm_eps=1e-5, embed_scale=5.5, loop_start=1, loop_stop=3, loop_times=3,
                        logit_scale=1.7, logit_softcap=9.0, layers=[
        PikadraLayer(heads=3, dim=10, rot_dim=6, vdim=7, kv_rank=14, q_rank=11, rot_dims=6, ff_kind="moe", experts=5, top=2, expert_ff=9,
                     shared_ff=8, **mla),
        PikadraLayer(heads=2, dim=5, rot_dim=4, vdim=12, kv_rank=9, q_rank=20, rot_dims=4, **mla),
        PikadraLayer(heads=1, dim=8, rot_dim=2, vdim=8, kv_rank=6, q_rank=5, rot_dims=2, ff_kind="dense", ff=15, **mla),
        PikadraLayer(heads=4, dim=6, rot_dim=8, vdim=5, kv_rank=16, q_rank=8, rot_dims=8, ff_kind="moe", experts=3, top=3, expert_ff=10, **mla),
    ])


def toks(n, vocab, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def changed(s, **kw):
    s2 = copy.deepcopy(s)
    for k, v in kw.items():
        setattr(s2, k, v)
    return s2


# ---- configuration, checkpoint, registry ---------------------------------------------------------------------------------------------
def test_configuration_round_trip_and_what_is_left_out():
    s = small_shape()
    c = json.loads(json.dumps(s.to_config()))
    assert PikadraShape.from_config(c).to_config() == c
    # what a configuration leaves out does not exist: no loop, no cap, no feed-forward, no shared expert, no rotated part
    for k in ("loop", "logit_softcap"):
        c.pop(k)
    c["layers"][0]["mlp"].pop("shared")
    c["layers"][2]["mlp"] = None
    c["layers"][2]["mixer"] = {"heads": 2, "dim": 4, "vdim": 4, "kv_rank": 6, "q_rank": 3, "scale": 0.25}
    t = PikadraShape.from_config(c)
    assert (t.loop_times, t.logit_softcap, t.layers[0].shared_ff, t.layers[2].ff_kind) == (0, 0.0, 0, "")
    assert (t.layers[2].rot_dim, t.layers[2].rot_dims) == (0, 0) and [i for i, _ in t.runs()] == [0, 1, 2, 3]
    assert "loop.in" not in W.pikadra_weight_shapes(t) and "l2.mlp.gate" not in W.pikadra_weight_shapes(t)
    with pytest.raises(ValueError):
        PikadraShape.from_config(dict(c, architecture="Other"))
    with pytest.raises(ValueError):
        PikadraShape.from_config(dict(c, loop={"start": 2, "stop": 5, "times": 2}))
    bad = json.loads(json.dumps(c))
    bad["layers"][0]["mlp"]["router"]["top"] = 6
    with pytest.raises(ValueError):
        PikadraShape.from_config(bad)
    c["layers"][0]["type"] = "unknown"
    with pytest.raises(ValueError):
        PikadraShape.from_config(c)


@pytest.mark.parametrize("loop", [(0, 4, 2), (1, 3, 3), (3, 4, 1), (0, 1, 4), None])
def test_order_of_layer_runs(loop):
    s = small_shape()
    s.loop_start, s.loop_stop, s.loop_times = loop or (0, 0, 0)
    s.check()
    want = []
    if loop:
        a, b, n = loop
        want += [(i, -1) for i in range(a)]
        for t in range(n):
            want += [(a, t)] + [(i, -1) for i in range(a + 1, b)]
        want += [(i, -1) for i in range(b, 4)]
    else:
        want = [(i, -1) for i in range(4)]
    assert s.runs() == want and O.layer_runs(s) == want
    assert PikadraShape.from_config(json.loads(json.dumps(s.to_config()))).runs() == want


def test_checkpoint_directory_reader_and_registry(tmp_path):
    from safetensors.torch import save_file
    s = small_shape()
    w = W.make_pikadra_weights(s, seed=1)
    shapes = W.pikadra_weight_shapes(s)
    assert set(w) == set(shapes) and all(tuple(w[k].shape) == tuple(v) for k, v in shapes.items())
    assert shapes["loop.in"] == (36, 72) and shapes["loop.step"] == (3, 36) and shapes["l0.mlp.shared.sg"] == (1, 36)
    (tmp_path / "config.json").write_text(json.dumps(s.to_config()))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    assert architecture_of(str(tmp_path)) == "pikadra"
    from promptcache_amd.model import ADAPTERS
    assert ADAPTERS["pikadra"].__name__ == "Pikadra"
    got = W.load_pikadra_safetensors(str(tmp_path), PikadraShape.from_dir(str(tmp_path)))
    assert all(torch.equal(got[k], w[k]) for k in w)
    bad = dict(w)
    bad["l1.mix.uq"] = bad["l1.mix.uq"][:-1]
    save_file({k: v.contiguous() for k, v in bad.items()}, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError):
        W.load_pikadra_safetensors(str(tmp_path), s)
    bad.pop("l1.mix.uq")
    save_file({k: v.contiguous() for k, v in bad.items()}, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError):
        W.load_pikadra_safetensors(str(tmp_path), s)


def test_frequency_table_of_the_model_is_the_oracles_rotation():
    from promptcache_amd.model.fivesun_hip import rotary_frequencies
    for base, dims in ((10000.0, 64), (350.0, 6), (2e6, 18)):
        fr, mag = rotary_frequencies(base, dims)
        x = torch.zeros(1, dims, dtype=F64)
        x[0, :dims // 2] = 1.0                                 # (1, 0) pairs: the turned pair is (cos, sin) of the angle
        pos = torch.tensor([12345])
        y = O.rotate_halves(x, pos, base, dims)[0]
        want = [12345 * f for f in fr]
        assert mag == 1.0 and all(math.isclose(float(y[i]), math.cos(a), abs_tol=1e-9) for i, a in enumerate(want))
        assert all(math.isclose(float(y[dims // 2 + i]), math.sin(a), abs_tol=1e-9) for i, a in enumerate(want))


def test_rows_of_a_step_are_laid_out_and_checked():
    from promptcache_amd.model.kv_arena import SlotArena
    from promptcache_amd.model.slot_model import StepRows
    ar = SlotArena([(1, 4)], 3, 8, "cpu", torch.float32)
    a, b = ar.alloc(), ar.alloc()
    ar.lengths[b] = 5
    st = StepRows(ar, [b, a], [[7, 8], [1, 2, 3]], [[1], [0, 2]], 9)
    assert st.counts == [2, 3] and st.starts == [5, 0] and st.row0.tolist() == [0, 2, 5] and st.ids.tolist() == [7, 8, 1, 2, 3]
    assert st.row_slot.tolist() == [b, b, a, a, a] and st.row_pos.tolist() == [5, 6, 0, 1, 2] and st.want_rows.tolist() == [1, 2, 4]
    assert StepRows(ar, [a], [[1, 2]], None, 9).want_rows.tolist() == [1]
    StepRows(ar, [b], [[1] * 6], None, 9)                     # 5 + 6 positions: the rows grow
    assert ar.cap >= 11
    for bad in (([a, a], [[1], [2]], None), ([a], [[]], None), ([a], [[9]], None), ([a], [[-1]], None), ([a], [[1]], [[1]]), ([a], [[1], [2]], None)):
        with pytest.raises(ValueError):
            StepRows(ar, bad[0], bad[1], bad[2], 9)


# ---- the oracle's own mechanisms --------------------------------------------------------------------------------------------------------
def test_rotation_in_halves_depends_on_distance_only_and_leaves_the_rest():
    g = torch.Generator().manual_seed(2)
    q, k = torch.randn(1, 9, generator=g, dtype=F64), torch.randn(1, 9, generator=g, dtype=F64)

    def dot(i, j):
        return float((O.rotate_halves(q, torch.tensor([i]), 50.0, 6) * O.rotate_halves(k, torch.tensor([j]), 50.0, 6)).sum())
    assert math.isclose(dot(7, 3), dot(104, 100), rel_tol=1e-9) and abs(dot(7, 3) - dot(7, 4)) > 1e-6
    y = O.rotate_halves(q, torch.tensor([11]), 50.0, 6)
    assert torch.equal(y[:, 6:], q[:, 6:]) and math.isclose(float(y.pow(2).sum()), float(q.pow(2).sum()))
    assert torch.equal(O.rotate_halves(q, torch.tensor([0]), 50.0, 6), q)
    # column 0 turns with column 3 by exactly one radian per position
    assert math.isclose(float(y[0, 0]), float(q[0, 0] * math.cos(11.0) - q[0, 3] * math.sin(11.0)), rel_tol=1e-12)


def test_attention_sees_itself_and_before_and_a_sink_takes_weight_without_a_value():
    q, k, v = torch.zeros(2, 3, dtype=F64), torch.zeros(4, 3, dtype=F64), torch.tensor([[1.0], [2.0], [4.0], [100.0]], dtype=F64)
    out = O.attend(q, k, v, [0, 2], 1.0)
    assert torch.allclose(out, torch.tensor([[1.0], [7.0 / 3.0]], dtype=F64))
    out = O.attend(q, k, v, [0, 2], 1.0, sink=torch.tensor(0.0, dtype=F64))
    assert torch.allclose(out, torch.tensor([[0.5], [7.0 / 4.0]], dtype=F64))
    # the sink is not scaled with the scores
    out = O.attend(q, k, v, [0], 7.0, sink=torch.tensor(math.log(3.0), dtype=F64))
    assert math.isclose(float(out[0]), 0.25)


def test_router_weights_are_the_scores_as_they_are():
    g = torch.Generator().manual_seed(5)
    h = torch.randn(7, 6, generator=g, dtype=F64)
    p = {"r.router": torch.randn(9, 6, generator=g, dtype=F64)}
    idx, w = O.route(h, p, "r.", 3)
    s = torch.softmax(h @ p["r.router"].T, dim=-1)
    for t in range(7):
        order = sorted(range(9), key=lambda e: -float(s[t, e]))[:3]
        assert idx[t].tolist() == order and torch.equal(w[t], s[t, order]) and float(w[t].sum()) < 1.0


@pytest.mark.parametrize("seed", [0, 1])
def test_oracle_prompt_equals_token_by_token_and_portions_and_every_mechanism_matters(seed):
    s = small_shape()
    p = O.to_f64(W.make_pikadra_weights(s, seed=seed))
    t = toks(23, s.vocab_size, seed)
    whole, streams = O.forward(s, p, t, return_streams=True)
    assert whole.shape == (23, s.vocab_size) and streams.shape == (8, 23, 36) and bool(torch.isfinite(whole).all())
    assert float(whole.abs().max()) < s.logit_softcap
    for cuts in ([1] * 23, [2, 2, 5, 1, 13], [22, 1]):
        assert float((O.forward_in_portions(s, p, t, cuts) - whole).abs().max()) < 1e-10
    moved = lambda s2, p2=p: float((O.forward(s2, p2, t)[-1] - whole[-1]).abs().max())
    assert moved(changed(s, embed_scale=5.0)) > 1e-4 and moved(changed(s, loop_times=2)) > 1e-4 and moved(changed(s, logit_scale=1.6)) > 1e-3
    assert moved(changed(s, logit_softcap=0.0)) > 1e-3
    for name in p:                                             # no tensor is idle
        if ".mlp.e" in name or name == "embed":
            continue
        p2 = dict(p)
        p2[name] = p[name] + 0.5 * torch.randn(p[name].shape, generator=torch.Generator().manual_seed(7), dtype=F64)
        assert moved(s, p2) > 1e-6, name


def test_passes_of_the_loop_keep_memories_of_their_own():
    """A pass that read another pass's latents would still be causal and still agree with itself in portions; here the carried memories of
    the passes are swapped, which must show."""
    s = small_shape()
    p = O.to_f64(W.make_pikadra_weights(s, seed=3))
    t = toks(12, s.vocab_size, 3)
    carry = [None] * 8
    O.forward(s, p, t[:9], carry=carry)
    good = O.forward(s, p, t[9:], pos0=9, carry=list(carry))
    runs = O.layer_runs(s)
    a, b = [r for r, (i, _) in enumerate(runs) if i == 1][:2]
    carry[a], carry[b] = carry[b], carry[a]
    assert float((O.forward(s, p, t[9:], pos0=9, carry=carry) - good).abs().max()) > 1e-4


# ---- the library's argument checks ----------------------------------------------------------------------------------------------------------
def test_new_struct_layouts_match_the_header(tmp_path):
    from promptcache_amd import _blocks
    structs = (("pcb_linear_args", _blocks.LinearArgs), ("pcb_post_norm_args", _blocks.PostNormArgs), ("pcb_head_prep_args", _blocks.HeadPrepArgs),
               ("pcb_attn_prompt_args", _blocks.AttnPromptArgs), ("pcb_attn_latent_args", _blocks.AttnLatentArgs))
    body = ['#include <stdio.h>', '#include <stddef.h>', f'#include "{ROOT}/include/promptcache_blocks.h"', 'int main(void) {']
    for st, cls in structs:
        body.append(f'  printf("{st} %zu\\n", sizeof({st}));')
        for f, _ in cls._fields_:
            body.append(f'  printf("{st}.{f} %zu\\n", offsetof({st}, {f}));')
    body += ['  return 0;', '}']
    src, exe = tmp_path / "layout.c", tmp_path / "layout"
    src.write_text("\n".join(body))
    subprocess.check_call(["gcc", "-std=c99", "-Wall", "-Werror", str(src), "-o", str(exe)])
    got = dict(line.rsplit(" ", 1) for line in subprocess.check_output([str(exe)], text=True).strip().splitlines())
    for st, cls in structs:
        assert int(got[st]) == ctypes.sizeof(cls), st
        for name, _ in cls._fields_:
            assert int(got[f"{st}.{name}"]) == getattr(cls, name).offset, (st, name)


def test_blocks_reject_bad_arguments_on_the_host():
    """The library checks its arguments before it launches anything, so these calls need no GPU."""
    from promptcache_amd import _blocks as b
    assert os.path.exists(b.lib_path()), "run __graft_entry__.build() first"
    lb = b.load(build_missing=False)
    err = lb.pcb_last_error_string

    def prompt(**kw):
        a = b.AttnPromptArgs(struct_bytes=ctypes.sizeof(b.AttnPromptArgs), ldq=48, n_tiles=1, tile_rows=64, k_row_stride=48, k_head_stride=24,
                             v_row_stride=48, v_head_stride=24, H=2, Hkv=2, dim=24, vdim=24, scale=1.0, ldo=48)
        for k, v in kw.items():
            setattr(a, k, v)
        return lb.pcb_attn_prompt(ctypes.byref(a), None)
    assert prompt() == -2001 and b"null pointer" in err()
    assert prompt(dim=300, ldq=600) == -2001 and b"up to 256" in err()
    assert prompt(tail_dim=24) == -2001 and b"bad sizes" in err()
    assert prompt(Hkv=3) == -2001 and prompt(ldo=40) == -2001
    assert prompt(tile_rows=32) == -2001 and b"64 rows" in err()
    assert prompt(tile_rows=128, dtype=b.F32) == -2001 and b"64 rows" in err()
    assert prompt(struct_bytes=8) == -2001 and b"struct size" in err()
    assert prompt(n_tiles=0) == 0

    def latent(**kw):
        a = b.AttnLatentArgs(struct_bytes=ctypes.sizeof(b.AttnLatentArgs), ldq=60, n_rows=1, slot_stride=300, row_stride=30, H=2, dim=30, vdim=20,
                             scale=1.0, ldo=40)
        for k, v in kw.items():
            setattr(a, k, v)
        return lb.pcb_attn_latent(ctypes.byref(a), None)
    assert latent() == -2001 and b"null pointer" in err()
    assert latent(vdim=31, ldo=62) == -2001 and b"bad sizes" in err()
    assert latent(dim=800, ldq=1600, row_stride=800) == -2001 and latent(row_stride=29) == -2001
    assert latent(n_rows=0) == 0

    def linear(**kw):
        a = b.LinearArgs(struct_bytes=ctypes.sizeof(b.LinearArgs), ldx=8, ldw=8, M=2, N=4, K=8, ldy=4, x=16, w=16, y=16)
        for k, v in kw.items():
            setattr(a, k, v)
        return lb.pcb_linear(ctypes.byref(a), None)
    assert linear(n_batch=2, bias=16) == -2001 and b"batch" in err()
    assert linear(n_batch=2, n_groups=2, group_off=16) == -2001 and b"batch" in err()
    assert linear(row_gate=16, ld_row_gate=1) == -2001 and b"gate per row" in err()
    assert linear(split_n=2, y2=16, y2_f32=1, head_stride2=1) == -2001 and b"split destination" in err()
    p = b.PostNormArgs(struct_bytes=ctypes.sizeof(b.PostNormArgs), x=16, eps=1e-6, n_rows=2, width=8, y_scale=1.0, pair=16)
    assert lb.pcb_post_norm(ctypes.byref(p), None) == -2001 and b"pairs" in err()
