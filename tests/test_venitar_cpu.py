"""Venitar without a GPU: the configuration reader and writer, the checkpoint reader, the registry, the order of layer runs, and the
float64 oracle (``oracle/venitar_oracle.py``) against itself -- a prompt at once, token by token, and in portions must agree, every
mechanism must matter, and each mechanism has a closed form somewhere that it must meet."""
import copy
import ctypes
import json
import math
import os
import subprocess

import pytest
import torch

from oracle import venitar_oracle as O
from promptcache_amd.model import weights as W
from promptcache_amd.model.config import VenitarAttention, VenitarDelta, VenitarLayer, VenitarRetention, VenitarRot, VenitarShape, architecture_of

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64


def small_shape():
    yarn = (3.0, 40.0, 20.0, 1.5)
    return VenitarShape(vocab_size=47, hidden_size=28, norm_eps=1e-5, embed_scale=6.5, loop_start=1, loop_stop=3, loop_times=3, layers=[
        VenitarLayer("retention", mix=VenitarRetention(3, 6, 5, [0.5, 0.9, 1.0], VenitarRot(300.0, 4)), ff=17),
        VenitarLayer("attention", mix=VenitarAttention(4, 2, 8, 8, 0.6, block=5, rot=VenitarRot(90.0, 6))),
        VenitarLayer("parallel", left=VenitarAttention(6, 3, 6, 9, 0.5, window=4, rot=VenitarRot(800.0, 6, yarn)),
                     right=VenitarDelta(4, 2, 5, 7, 3, 6, 4), left_scale=0.7, right_scale=-1.3, ff=11),
        VenitarLayer("attention", mix=VenitarAttention(2, 1, 4, 4, 1.0)),
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
    assert VenitarShape.from_config(c).to_config() == c
    # what a configuration leaves out does not exist: no loop, no mask, no rotation, no scaling, no feed-forward, one key head per query head
    c.pop("loop")
    c["layers"][0]["mlp"] = None
    c["layers"][0]["mixer"].pop("rot")
    c["layers"][1]["mixer"].pop("mask")
    c["layers"][1]["mixer"].pop("kv_heads")
    c["layers"][2]["mixer"]["left"]["rot"].pop("scaling")
    t = VenitarShape.from_config(c)
    assert (t.loop_times, t.layers[0].ff, t.layers[0].mix.rot.dims, t.layers[1].mix.block, t.layers[1].mix.kv_heads) == (0, 0, 0, 0, 4)
    assert t.layers[2].left.rot.scaling is None and t.layers[2].left.window == 4 and [i for i, _ in t.runs()] == [0, 1, 2, 3]
    assert "l0.norm2" not in W.venitar_weight_shapes(t) and "l0.mlp.up" not in W.venitar_weight_shapes(t)
    for edit in (lambda d: d.update(architecture="Other"), lambda d: d.update(loop={"start": 2, "stop": 5, "times": 2}),
                 lambda d: d["layers"][0].update(type="unknown"), lambda d: d["layers"][0]["mixer"].update(decay=[0.5, 0.5]),
                 lambda d: d["layers"][0]["mixer"].update(decay=[0.5, 0.5, 1.5]), lambda d: d["layers"][1]["mixer"].update(vdim=9),
                 lambda d: d["layers"][1]["mixer"]["rot"].update(dims=10), lambda d: d["layers"][1]["mixer"]["rot"].update(dims=3),
                 lambda d: d["layers"][2]["mixer"]["left"].update(kv_heads=4), lambda d: d["layers"][2]["mixer"]["right"].update(kv_heads=3),
                 lambda d: d["layers"][2]["mixer"]["right"].update(conv=0), lambda d: d["layers"][2]["mlp"].update(kind="moe")):
        bad = json.loads(json.dumps(c))
        edit(bad)
        with pytest.raises(ValueError):
            VenitarShape.from_config(bad)


@pytest.mark.parametrize("loop", [(0, 4, 2), (1, 3, 3), (3, 4, 1), (0, 1, 4), None])
def test_order_of_layer_runs(loop):
    s = small_shape()
    s.loop_start, s.loop_stop, s.loop_times = loop or (0, 0, 0)
    s.check()
    want = []
    if loop:
        a, b, n = loop
        want += [(i, False) for i in range(a)]
        for t in range(n):
            want += [(a, t > 0)] + [(i, False) for i in range(a + 1, b)]
        want += [(i, False) for i in range(b, 4)]
    else:
        want = [(i, False) for i in range(4)]
    assert s.runs() == want and O.layer_runs(s) == want
    assert VenitarShape.from_config(json.loads(json.dumps(s.to_config()))).runs() == want


def test_checkpoint_directory_reader_and_registry(tmp_path):
    from safetensors.torch import save_file
    s = small_shape()
    w = W.make_venitar_weights(s, seed=1)
    shapes = W.venitar_weight_shapes(s)
    assert set(w) == set(shapes) and all(tuple(w[k].shape) == tuple(v) for k, v in shapes.items())
    assert shapes["l2.mix.right.a2"] == (20, 6) and shapes["l2.mix.right.v.conv"] == (28, 3) and shapes["l2.mix.left.v.b"] == (27,)
    assert shapes["l1.mix.k.norm"] == (8,) and "l1.mix.v" not in shapes and "head" not in shapes
    (tmp_path / "config.json").write_text(json.dumps(s.to_config()))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    assert architecture_of(str(tmp_path)) == "venitar"
    from promptcache_amd.model import ADAPTERS
    assert ADAPTERS["venitar"].__name__ == "Venitar"
    fresh = VenitarShape.from_dir(str(tmp_path))
    assert (fresh.layers[2].right.a_rank, fresh.layers[2].right.g_rank) == (0, 0)
    got = W.load_venitar_safetensors(str(tmp_path), fresh)
    assert (fresh.layers[2].right.a_rank, fresh.layers[2].right.g_rank) == (6, 4)      # the low ranks are tensor shapes
    assert all(torch.equal(got[k], w[k]) for k in w)
    bad = dict(w)
    bad["l1.mix.q"] = bad["l1.mix.q"][:-1]
    save_file({k: v.contiguous() for k, v in bad.items()}, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError):
        W.load_venitar_safetensors(str(tmp_path), s)
    bad.pop("l1.mix.q")
    save_file({k: v.contiguous() for k, v in bad.items()}, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError):
        W.load_venitar_safetensors(str(tmp_path), s)


@pytest.mark.parametrize("base,dims,scaling", [(10000.0, 64, None), (350.0, 6, None), (500.0, 20, (2.5, 60.0, 16.0, 1.0)), (2e6, 48, (8.0, 4096.0, 32.0, 1.0)),
                                               (5e5, 12, (1.0, 100.0, 8.0, 2.0)), (1e4, 8, (4.0, 10.0, 1.0, 1.0)), (1e4, 8, (4.0, 3.0, 30.0, 20.0))])
def test_frequency_table_of_the_model_is_the_oracles_rotation(base, dims, scaling):
    from promptcache_amd.model.fivesun_hip import rotary_frequencies
    fr, mag = rotary_frequencies(base, dims, *(scaling or ()))
    x = torch.zeros(1, 1, dims + 2, dtype=F64)
    x[0, 0, :dims // 2] = 1.0                                  # (1, 0) pairs: the turned pair is mag (cos, sin) of the angle
    x[0, 0, dims:] = 5.0
    y = O.rotate(x, torch.tensor([12345]), VenitarRot(base, dims, scaling))[0, 0]
    assert (mag == 1.0) == (scaling is None or scaling[0] == 1.0)
    for i, f in enumerate(fr):
        assert math.isclose(float(y[i]), mag * math.cos(12345 * f), abs_tol=1e-9)
        assert math.isclose(float(y[dims // 2 + i]), mag * math.sin(12345 * f), abs_tol=1e-9)
    assert torch.equal(y[dims:], x[0, 0, dims:])


def test_frequency_ramp_keeps_fast_pairs_and_slows_slow_ones():
    base, dims, factor, original = 10000.0, 32, 4.0, 2048.0
    plain = O.plain_frequencies(base, dims)
    fr, mag = O.ramped_frequencies(base, dims, factor, original, 32.0, 1.0)
    turns = [original * f / (2 * math.pi) for f in plain]
    lo = max(i for i, t in enumerate(turns) if t > 32.0)
    hi = min(i for i, t in enumerate(turns) if t < 1.0)
    assert all(fr[i] == plain[i] for i in range(lo)) and all(math.isclose(fr[i], plain[i] / factor) for i in range(hi + 1, dims // 2))
    assert all(plain[i] / factor < fr[i] < plain[i] for i in range(lo + 2, hi - 1)) and math.isclose(mag, 1.0 + 0.1 * math.log(4.0))


# ---- the oracle's own mechanisms --------------------------------------------------------------------------------------------------------
def test_rotation_depends_on_distance_only():
    g = torch.Generator().manual_seed(2)
    q, k = torch.randn(1, 1, 9, generator=g, dtype=F64), torch.randn(1, 1, 9, generator=g, dtype=F64)
    rot = VenitarRot(50.0, 6)

    def dot(i, j):
        return float((O.rotate(q, torch.tensor([i]), rot) * O.rotate(k, torch.tensor([j]), rot)).sum())
    assert math.isclose(dot(7, 3), dot(104, 100), rel_tol=1e-9) and abs(dot(7, 3) - dot(7, 4)) > 1e-6
    y = O.rotate(q, torch.tensor([11]), rot)
    # column 0 turns with column 3 by exactly one radian per position
    assert math.isclose(float(y[0, 0, 0]), float(q[0, 0, 0] * math.cos(11.0) - q[0, 0, 3] * math.sin(11.0)), rel_tol=1e-12)


def test_visible_keys_and_the_sink():
    assert O.visible(7, block=4) == [4, 5, 6, 7] and O.visible(8, block=4) == [8] and O.visible(3, block=1) == [3]
    assert O.visible(7, window=3) == [5, 6, 7] and O.visible(1, window=3) == [0, 1] and O.visible(2) == [0, 1, 2]
    q, k, v = torch.zeros(2, 3, dtype=F64), torch.zeros(4, 3, dtype=F64), torch.tensor([[1.0], [2.0], [4.0], [100.0]], dtype=F64)
    assert torch.allclose(O.attend(q, k, v, [0, 2], 1.0), torch.tensor([[1.0], [7.0 / 3.0]], dtype=F64))
    assert torch.allclose(O.attend(q, k, v, [0, 2], 1.0, sink=True), torch.tensor([[0.5], [7.0 / 4.0]], dtype=F64))
    # a very quiet key against the sink: its weight is e^s / (1 + e^s), not renormalised away
    k2 = torch.full((1, 3), -10.0, dtype=F64)
    out = O.attend(torch.ones(1, 3, dtype=F64), k2, torch.ones(1, 1, dtype=F64), [0], 1.0, sink=True)
    assert math.isclose(float(out), math.exp(-30.0) / (1 + math.exp(-30.0)), rel_tol=1e-9)


def test_retention_is_a_decayed_sum_over_the_past():
    g = torch.Generator().manual_seed(4)
    q, k, v = (torch.randn(9, d, generator=g, dtype=F64) for d in (4, 4, 3))
    out, S = O.retain(q, k, v, 0.8, torch.zeros(4, 3, dtype=F64))
    for t in range(9):
        want = sum(0.8 ** (t - j) * float(q[t] @ k[j]) * v[j] for j in range(t + 1))
        assert torch.allclose(out[t], want)
    assert torch.allclose(S, sum(0.8 ** (8 - j) * torch.outer(k[j], v[j]) for j in range(9)))


def test_delta_rule_overwrites_what_a_key_reads():
    """With step size one and no forgetting, a unit key reads back the value written last, and orthogonal keys do not disturb each
    other; the read-out sees the token's own write; a decay scales the rows of its own key channel."""
    e = torch.eye(4, dtype=F64)
    v = torch.tensor([[1.0, 2.0], [3.0, -1.0], [7.0, 0.5]], dtype=F64)
    ones = torch.ones(3, 4, dtype=F64)
    k = torch.stack([e[0], e[1], e[0]])
    out, S = O.delta_rule(k, k, v, torch.ones(3, dtype=F64), ones, torch.zeros(4, 2, dtype=F64))
    assert torch.allclose(out, v) and torch.allclose(S[0], v[2]) and torch.allclose(S[1], v[1])
    out, _ = O.delta_rule(k, k, v, torch.full((3,), 0.25, dtype=F64), ones, torch.zeros(4, 2, dtype=F64))
    assert torch.allclose(out[2], 0.25 * v[0] + 0.25 * (v[2] - 0.25 * v[0]))
    g = ones.clone()
    g[2, 1] = 0.5
    _, S = O.delta_rule(k, k, v, torch.ones(3, dtype=F64), g, torch.zeros(4, 2, dtype=F64))
    assert torch.allclose(S[1], 0.5 * v[1]) and torch.allclose(S[0], v[2])


def test_short_convolution_looks_back_over_portions():
    g = torch.Generator().manual_seed(6)
    x, w = torch.randn(7, 2, generator=g, dtype=F64), torch.randn(2, 3, generator=g, dtype=F64)
    y, keep = O.short_convolution(x, w, None)
    assert torch.allclose(y[0], w[:, 2] * x[0]) and torch.allclose(y[4], w[:, 0] * x[2] + w[:, 1] * x[3] + w[:, 2] * x[4])
    a, past = O.short_convolution(x[:1], w, None)
    b, past = O.short_convolution(x[1:], w, past)
    assert torch.allclose(torch.cat([a, b]), y) and torch.equal(past, x[5:]) and torch.equal(keep, x[5:])


@pytest.mark.parametrize("seed", [0, 1])
def test_oracle_prompt_equals_token_by_token_and_portions_and_every_mechanism_matters(seed):
    s = small_shape()
    p = O.to_f64(W.make_venitar_weights(s, seed=seed))
    t = toks(23, s.vocab_size, seed)
    whole, streams = O.forward(s, p, t, return_streams=True)
    assert whole.shape == (23, s.vocab_size) and streams.shape == (8, 23, 28) and bool(torch.isfinite(whole).all())
    for cuts in ([1] * 23, [2, 2, 5, 1, 13], [22, 1]):
        assert float((O.forward_in_portions(s, p, t, cuts) - whole).abs().max()) < 1e-10
    moved = lambda s2, p2=p: float((O.forward(s2, p2, t)[-1] - whole[-1]).abs().max())
    assert moved(changed(s, embed_scale=5.0)) > 1e-4 and moved(changed(s, loop_times=2)) > 1e-4

    def edit(f):
        s2 = copy.deepcopy(s)
        f(s2.layers)
        return s2
    for f in (lambda ls: setattr(ls[0].mix, "decay", [0.5, 0.9, 0.95]), lambda ls: setattr(ls[0].mix.rot, "dims", 6), lambda ls: setattr(ls[1].mix, "block", 6),
              lambda ls: setattr(ls[1].mix, "scale", 0.5), lambda ls: setattr(ls[2].left, "window", 5), lambda ls: setattr(ls[2].left.rot, "scaling", None),
              lambda ls: setattr(ls[2], "left_scale", 0.8), lambda ls: setattr(ls[2], "right_scale", 1.0), lambda ls: setattr(ls[3].mix, "block", 20)):
        assert moved(edit(f)) > 1e-6
    for name in p:                                             # no tensor is idle
        if name == "embed":
            continue
        p2 = dict(p)
        p2[name] = p[name] + 0.5 * torch.randn(p[name].shape, generator=torch.Generator().manual_seed(7), dtype=F64)
        assert moved(s, p2) > 1e-6, name


def test_passes_of_the_loop_keep_memories_of_their_own():
    """A pass that read another pass's memories would still be causal and still agree with itself in portions; here the carried memories
    of two passes are swapped, which must show."""
    s = small_shape()
    p = O.to_f64(W.make_venitar_weights(s, seed=3))
    t = toks(12, s.vocab_size, 3)
    carry = [None] * 8
    O.forward(s, p, t[:9], carry=carry)
    good = O.forward(s, p, t[9:], pos0=9, carry=list(carry))
    for layer in (1, 2):
        swapped = list(carry)
        a, b = [r for r, (i, _) in enumerate(O.layer_runs(s)) if i == layer][:2]
        swapped[a], swapped[b] = swapped[b], swapped[a]
        assert float((O.forward(s, p, t[9:], pos0=9, carry=swapped) - good).abs().max()) > 1e-5


# ---- the library's argument checks ----------------------------------------------------------------------------------------------------------
def test_new_struct_layouts_match_the_header(tmp_path):
    from promptcache_amd import _blocks
    structs = (("pcb_rec_args", _blocks.RecArgs), ("pcb_attn_rows_args", _blocks.AttnRowsArgs), ("pcb_attn_prompt_args", _blocks.AttnPromptArgs),
               ("pcb_head_prep_args", _blocks.HeadPrepArgs), ("pcb_post_norm_args", _blocks.PostNormArgs))
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

    def rec(fn, **kw):
        a = b.RecArgs(struct_bytes=ctypes.sizeof(b.RecArgs), ldq=24, ldk=24, ldv=24, decay=16, n_reqs=1, n_chunks=2, slot_stride=300, H=2, Hk=2, dim=12,
                      vdim=12, ldo=24, ldy=24, scratch_floats=10 ** 6)
        for k, v in kw.items():
            setattr(a, k, v)
        return getattr(lb, fn)(ctypes.byref(a), None)
    for fn in ("pcb_rec_prompt", "pcb_rec_step"):
        assert rec(fn) == -2001 and b"null pointer" in err()
        assert rec(fn, dim=257, ldq=600, ldk=600) == -2001 and b"up to 256" in err()
        assert rec(fn, Hk=3) == -2001 and rec(fn, slot_stride=200) == -2001 and rec(fn, ldv=20) == -2001
        assert rec(fn, decay=None) == -2001 and b"one of them" in err()
        assert rec(fn, ld=16, ldld=24) == -2001 and b"one of them" in err()
        assert rec(fn, decay=None, ld=16, ldld=20) == -2001 and b"too short" in err()
        assert rec(fn, beta=16, ldbeta=1) == -2001 and b"too short" in err()
        assert rec(fn, rot=16, rot_dims=7) == -2001 and rec(fn, rot_dims=4) == -2001 and b"pairs" in err()
        assert rec(fn, struct_bytes=8) == -2001 and b"struct size" in err()
        assert rec(fn, n_reqs=0) == 0
    assert rec("pcb_rec_prompt", scratch_floats=10) == -2001 and b"scratch" in err()
    assert rec("pcb_rec_prompt", n_reqs=3) == -2001
    assert rec("pcb_rec_step", vdim=1024, ldv=4096, ldy=4096, slot_stride=10 ** 6) == -2001 and b"registers" in err()
    assert rec("pcb_rec_step", ldy=20) == -2001 and rec("pcb_rec_step", gate=16, ldg=20) == -2001 and b"too short" in err()
    assert b.rec_step_fits(128, 128) and b.rec_step_fits(256, 256) and b.rec_step_fits(5, 7) and not b.rec_step_fits(256, 512) and not b.rec_step_fits(300, 8)
    assert b.rec_scratch(0, 2, 12) == 0 and b.rec_scratch(3, 2, 12) == 3 * 2 * (4 * 784 + 512)

    def rows(**kw):
        a = b.AttnRowsArgs(struct_bytes=ctypes.sizeof(b.AttnRowsArgs), ldq=80, n_rows=1, k_slot_stride=300, k_head_stride=30, k_row_stride=30, v_slot_stride=300,
                           v_head_stride=30, v_row_stride=30, H=4, Hkv=2, dim=20, vdim=10, scale=1.0, ldo=40)
        for k, v in kw.items():
            setattr(a, k, v)
        return lb.pcb_attn_rows(ctypes.byref(a), None)
    assert rows() == -2001 and b"null pointer" in err()
    assert rows(dim=300, ldq=1200, k_row_stride=300) == -2001 and b"up to 256" in err()
    assert rows(Hkv=3) == -2001 and rows(ldo=39) == -2001 and rows(k_row_stride=19) == -2001 and rows(v_row_stride=9) == -2001
    assert rows(n_rows=0) == 0

    def prompt(**kw):
        a = b.AttnPromptArgs(struct_bytes=ctypes.sizeof(b.AttnPromptArgs), ldq=48, n_tiles=1, tile_rows=64, k_row_stride=48, k_head_stride=24,
                             v_row_stride=48, v_head_stride=24, H=2, Hkv=2, dim=24, vdim=24, scale=1.0, ldo=48, q=16, tiles=16, k=16, v=16, out=16)
        for k, v in kw.items():
            setattr(a, k, v)
        return lb.pcb_attn_prompt(ctypes.byref(a), None)
    assert prompt(slots=1, tail_dim=4, k_tail=16, tail_row_stride=4) == -2001 and b"no shared part" in err()
    assert prompt(gate=16, ldg=2, gate_cols=1) == -2001 and b"null pointer" in err()
    assert lb.pcb_rot_table(None, None, 1.0, None, 1, 4, None) == -2001 and lb.pcb_rot_table(None, None, 1.0, None, 1, 600, None) == -2001
    assert lb.pcb_rot_table(None, None, 1.0, None, 0, 4, None) == 0
    assert lb.pcb_conv_step(None, 8, None, None, b.F32, 1, None, 1, None, 24, None, 8, 8, 4, None) == -2001 and b"null pointer" in err()
    assert lb.pcb_conv_step(None, 8, None, None, b.F32, 1, None, 1, None, 24, None, 8, 8, 17, None) == -2001 and b"16" in err()
