"""Venitar on the GPU against the plain float64 oracle (``oracle/venitar_oracle.py``): every new or extended building-block kernel alone --
with inputs built so that a far key, a key block's or chunk's border, a window's or block's edge, the sink or a strong decay decides the
result --, then the model through its arena: prompts, token-by-token decoding, portions down to two tokens, unequal batches, reused slots
and states, loops of every extent, long decoding through captured graphs, and greedy generation through the engines and the trace runner.
float32 runs are held to float32 accuracy; bfloat16 runs to what bf16 operands allow."""
import json
import os
import subprocess

import pytest
import torch

from oracle import venitar_oracle as O
from promptcache_amd.model import weights as W
from promptcache_amd.model.config import VenitarAttention, VenitarDelta, VenitarLayer, VenitarRetention, VenitarRot, VenitarShape

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda:0"
F64 = torch.float64
DTYPES = [torch.float32, torch.bfloat16]


def rel(got, want):
    got, want = got.detach().to("cpu", F64), want.detach().to("cpu", F64)
    return float((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt().clamp_min(1e-30))


def tol(dtype, f32=2e-5, bf16=2e-2):
    return f32 if dtype == torch.float32 else bf16


def close(got, want, dtype, f32=3e-5, bf16=4e-2):
    """Logits row by row.  float32: every row within float32 accuracy.  bfloat16: a head whose output is next to nothing is scaled up by its
    unit-RMS norm, rounding included (a first token whose query is almost orthogonal to its key), so rows are judged together: the median
    row within ``bf16``, at most one row in ten (or one) beyond three times that."""
    got, want = got.detach().to("cpu", F64), want.detach().to("cpu", F64)
    err = (got - want).pow(2).mean(dim=-1).sqrt() / want.pow(2).mean(dim=-1).sqrt().clamp_min(1e-30)
    if dtype == torch.float32:
        return bool(err.max() < f32)
    return bool(err.median() <= bf16) and int((err > 3 * bf16).sum()) <= max(1, err.numel() // 10)


def B():
    from promptcache_amd import _blocks
    return _blocks


def rnd(*shape, dtype=torch.float32, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (scale * torch.randn(*shape, generator=g)).to(dtype).to(DEV)


def f64(t):
    return t.detach().to("cpu", F64)


def dev_i32(rows):
    return torch.tensor(rows, dtype=torch.int32, device=DEV).reshape(-1)


YARN = (4.0, 300.0, 24.0, 1.0)


def ret(heads, dim, vdim, rot=None, ff=0, base=4000.0, decay=None):
    decay = decay or [1.0 - 0.3 ** (1 + 1.7 * h / max(1, heads - 1)) for h in range(heads)]
    return VenitarLayer("retention", mix=VenitarRetention(heads, dim, vdim, decay, VenitarRot(base, dim if rot is None else rot)), ff=ff)


def att(heads, kv, dim, block, rot=None, ff=0, sharp=2.5, base=3000.0):
    """``sharp``: the factor on the usual score scale, so that single keys carry weight among many."""
    return VenitarLayer("attention", mix=VenitarAttention(heads, kv, dim, dim, sharp * dim ** -0.5, block=block, rot=VenitarRot(base, dim if rot is None else rot)), ff=ff)


def par(left, right, window, rot=None, yarn=YARN, conv=4, ranks=(12, 20), scales=(0.7, 1.4), ff=0, sharp=2.5):
    h, kv, d, dv = left
    dims = d - d % 2 if rot is None else rot
    return VenitarLayer("parallel", left=VenitarAttention(h, kv, d, dv, sharp * d ** -0.5, window=window, rot=VenitarRot(2000.0, dims, yarn if dims else None)),
                        right=VenitarDelta(right[0], right[1], right[2], right[3], conv, *ranks), left_scale=scales[0], right_scale=scales[1], ff=ff)


# ---- shapes: layers differ from one another, come in different orders, and no size is a round one -------------------------------
def shape_mixed():
    return VenitarShape(vocab_size=170, hidden_size=104, norm_eps=1e-5, embed_scale=8.0, loop_start=1, loop_stop=3, loop_times=2, layers=[
        ret(3, 24, 40, rot=16, ff=72), att(6, 2, 40, 33, rot=24, ff=48), par((8, 2, 24, 48), (6, 3, 40, 24), 21, rot=16, ff=56), att(2, 2, 16, 70), ret(5, 16, 8),
        par((3, 3, 32, 16), (2, 2, 16, 72), 50, yarn=None, conv=2, scales=(1.3, 0.4))])


def shape_odd():
    """Sizes that are no multiple of a 16-byte chunk in either element type; one head, a layer without rotation, masks of one position and
    none at all, a single tap, a decay of one, a weight of nothing and a negative one, a loop over the whole stack."""
    return VenitarShape(vocab_size=77, hidden_size=50, norm_eps=1e-6, embed_scale=1.0, loop_start=0, loop_stop=4, loop_times=3, layers=[
        par((3, 1, 7, 5), (1, 1, 9, 3), 1, conv=1, ranks=(5, 3), scales=(0.0, 0.9), ff=15), ret(3, 10, 7, rot=0, decay=[1.0, 0.3, 0.6], ff=9),
        att(5, 1, 6, 1, rot=4), par((2, 2, 10, 13), (3, 1, 5, 6), 0, rot=2, conv=5, ranks=(1, 7), scales=(0.8, -1.1))])


def shape_wide():
    """Enough columns to reach the wider kernel instantiations: states of 128, 200 and 256 key columns, heads of 129 .. 256 columns, twenty
    query heads on one key head (a full group of sixteen and a rest); no loop."""
    return VenitarShape(vocab_size=300, hidden_size=128, norm_eps=1e-6, embed_scale=11.3, layers=[
        ret(2, 128, 128, ff=136), att(20, 1, 128, 64), par((2, 1, 192, 200), (2, 2, 200, 48), 40, ff=64), ret(1, 256, 520, rot=64), att(2, 1, 256, 0),
        par((4, 4, 64, 64), (4, 2, 64, 128), 33, conv=3)])


SHAPES = {"mixed": shape_mixed, "odd": shape_odd, "wide": shape_wide}
_models = {}


def model(name, dtype, seed=11):
    from promptcache_amd.model.venitar_hip import VenitarHIP
    key = (name, dtype, seed)
    if key not in _models:
        s = SHAPES[name]()
        w = W.make_venitar_weights(s, seed=seed)
        _models[key] = (s, w, VenitarHIP(s, w, device=DEV, dtype=dtype))
    return _models[key]


def toks(n, vocab, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def run_alone(m, tokens, cuts=None):
    """One request on a fresh arena, its tokens cut into the given portions; logits of every token."""
    ar = m.new_arena(1, 8)
    s = ar.alloc()
    cuts = cuts or [len(tokens)]
    assert sum(cuts) == len(tokens)
    out, at = [], 0
    for c in cuts:
        out.append(m.forward_rows(ar, [s], [tokens[at:at + c]], [list(range(c))]))
        at += c
    return torch.cat(out)


_oracle = {}


def oracle(s, w, tokens):
    """(logits, streams), remembered: several tests and both element types ask for the same ones."""
    key = (s.to_config().__repr__(), tuple(tokens), float(w["final.norm"].float().sum()))
    if key not in _oracle:
        _oracle[key] = O.forward(s, O.to_f64(w), tokens, return_streams=True)
    return _oracle[key]


# =====================================================================================================================================
# building blocks alone
# =====================================================================================================================================
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,rot,scaling", [(14, 8, None), (13, 6, YARN), (70, 70, None), (150, 128, (2.0, 5000.0, 30.0, 1.0))])
def test_rotation_tables_serve_head_preparation(dtype, D, rot, scaling):
    """Tabled turns (positions in the hundreds of thousands, where a 32-bit angle would have lost its low bits) against the oracle, and the
    same rows prepared with the table and with positions and frequencies; a row count on both sides of the few-row launch shape."""
    from promptcache_amd.model.fivesun_hip import rotary_frequencies
    H, b = 7, B()
    for T in (6, 80):
        pos = ([0, 1, 31, 250001, 7, 999983] * 20)[:T]
        P, gain = rnd(T, H * D, dtype=dtype, seed=1), 1 + 0.1 * rnd(D, seed=2)
        fr, mag = rotary_frequencies(700.0, rot, *(scaling or ()))
        fr = torch.from_numpy(fr).to(DEV)
        table = torch.empty(T, rot, device=DEV)
        b.rot_table(dev_i32(pos), fr, mag, table, T)
        want = O.rotate(O.unit_rms(f64(P).view(T, H, D), 1e-5) * f64(gain), torch.tensor(pos), VenitarRot(700.0, rot, scaling)).reshape(T, -1)
        outs = []
        for kw in (dict(table=table), dict(pos=dev_i32(pos), freqs=fr, rot_mag=mag)):
            out = torch.zeros(T, H * D, dtype=dtype, device=DEV)
            b.head_prep([b.head_seg(P, H * D, H, D, out, norm=True, gain=gain, rot_dims=rot, ld_dst=H * D)], T, dtype, eps=1e-5, rot_half=True, **kw)
            assert rel(out, want) < tol(dtype, 2e-6, 5e-3)
            outs.append(out)
        assert torch.equal(outs[0], outs[1])


@pytest.mark.parametrize("dtype", DTYPES)
def test_residual_step_with_another_addend(dtype):
    T, W_, b = 7, 300, B()
    x0, y, add, gain = rnd(T, W_, seed=1, scale=3.0), rnd(T, W_, seed=2), rnd(T, W_, seed=3), 1 + 0.1 * rnd(W_, seed=5)
    for yy in (y, None):
        new = f64(x0) + (-1.5 * f64(yy) if yy is not None else 0.0) + f64(add)
        x, out = x0.clone(), torch.empty(T, W_, dtype=dtype, device=DEV)
        b.post_norm(x, y=yy, y_scale=-1.5, add=add, gain=gain, out=out, eps=1e-5)
        assert rel(x, new) < 1e-6 and rel(out, O.unit_rms(new, 1e-5) * f64(gain)) < tol(dtype, 1e-6, 5e-3)
        rows = dev_i32([5, 0, 5])
        x, out3 = x0.clone(), torch.empty(3, W_, dtype=dtype, device=DEV)
        b.post_norm(x, y=yy, y_scale=-1.5, add=add, gain=gain, out=out3, rows=rows, eps=1e-5)
        assert torch.equal(x, x0) and torch.equal(out3, out[rows.long()])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps,pad", [(6, 1, 0), (600, 2, 2), (514, 3, 0), (40, 4, 6), (41, 4, 0), (1100, 4, 0), (30, 5, 1), (10, 16, 0)])
def test_short_convolutions_over_portions_single_tokens_and_reused_slots(dtype, C, taps, pad):
    """Requests of unequal lengths fed in portions -- prompts that end inside a run of rows, two tokens, one token through the step that
    moves the state itself -- on slots whose old inputs are garbage."""
    b = B()
    w = rnd(C, taps, dtype=dtype, seed=1, scale=taps ** -0.5)
    lens = {0: 37, 1: 9, 2: 1, 3: 20}
    x = {k: rnd(n, C, dtype=dtype, seed=10 + k) for k, n in lens.items()}
    want = {k: O.silu(O.short_convolution(f64(x[k]), f64(w), None)[0]) for k in lens}
    state = torch.full((5, taps - 1, C), 1e3, dtype=dtype, device=DEV)
    slot, at, got = {0: 3, 1: 0, 2: 4, 3: 1}, {k: 0 for k in lens}, {k: [] for k in lens}
    N = C + pad
    for portion in ({0: 19, 1: 2, 2: 1}, {0: 2, 1: 1}, {0: 1, 1: 1}, {0: 1}, {0: 13, 1: 4, 3: 17}, {0: 1, 1: 1, 3: 1}, {3: 2}):
        X = torch.full((sum(portion.values()), N), 7.0, dtype=dtype, device=DEV)
        meta, reqs, row = [], [], 0
        for k, n in portion.items():
            X[row:row + n, :C] = x[k][at[k]:at[k] + n]
            meta += [(slot[k], at[k] + i, i, 0) for i in range(n)]
            reqs.append((slot[k], at[k], n, row))
            row += n
        out = torch.empty(row, C, dtype=dtype, device=DEV)
        if all(n == 1 for n in portion.values()):
            b.conv_step(X, N, w, None, True, dev_i32(reqs), len(reqs), state, out)
        else:
            b.causal_conv(X, N, w, None, True, dev_i32(meta), state, out, row)
            if taps > 1:
                b.conv_state_update(X, N, dev_i32(reqs), len(reqs), state)
        row = 0
        for k, n in portion.items():
            got[k].append(out[row:row + n])
            row += n
            at[k] += n
    assert at == lens
    for k in lens:
        assert rel(torch.cat(got[k]), want[k]) < tol(dtype, 2e-6, 6e-3), k


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,group", [(1, 520), (1, 24), (3, 520), (5, 24), (2, 7), (1, 7), (4, 128), (2, 200), (3, 36)])
@pytest.mark.parametrize("with_gain", [True, False])
def test_output_norm_of_every_head_with_and_without_a_gain(dtype, heads, group, with_gain):
    """One head is a head too: its norm does not hang on a gain.  Into a column block of a wider matrix."""
    b, T, N = B(), 9, heads * group
    x, gate = rnd(T, N, seed=1, scale=3.0), rnd(T, N + 8, dtype=dtype, seed=2).sigmoid()
    gain = 1 + 0.2 * rnd(N, seed=3) if with_gain else None
    out = torch.full((T, N + 12), 7.0, dtype=dtype, device=DEV)
    b.gated_norm(x, gain, gate[:, 8:], N + 8, out[:, 4:], 1e-5, T, group=group, ldo=N + 12)
    want = O.unit_rms(f64(x).view(T, heads, group), 1e-5).reshape(T, N) * (f64(gain) if with_gain else 1.0) * f64(gate)[:, 8:]
    assert rel(out[:, 4:4 + N], want) < tol(dtype, 1e-6, 5e-3)
    assert bool((out[:, :4] == 7.0).all()) and bool((out[:, 4 + N:] == 7.0).all())


# ---- recurrences with a matrix state -----------------------------------------------------------------------------------------------------
class Rec:
    """One recurrence's inputs for several requests, its float64 result, and a way to feed any portions of them to the kernels."""

    def __init__(self, dtype, H, Hk, D, Dv, lens, *, delta, rows, rot=0, unit=False, z=0.0, zs=1.0, seed=0, decay=None, edit=None):
        self.b, self.dtype, self.dims, self.lens, self.delta, self.rows, self.rot, self.unit = B(), dtype, (H, Hk, D, Dv), lens, delta, rows, rot, unit
        T = sum(lens)
        self.q, self.k, self.v = (rnd(T, n + 3, dtype=dtype, seed=seed + i) for i, n in ((1, Hk * D), (2, Hk * D), (3, H * Dv)))
        self.ld = rnd(T, H * D + 2, seed=seed + 4, scale=zs) + z
        self.coef = -torch.exp(0.5 * rnd(H, seed=seed + 5))
        self.beta = rnd(T, H + 1, seed=seed + 6, scale=1.5)
        self.decay = torch.tensor(decay or [0.3 ** (1.0 / (1 + 3 * h)) for h in range(H)], device=DEV)
        self.gate, self.gain = rnd(T, H * Dv + 1, dtype=dtype, seed=seed + 7).sigmoid(), 1 + 0.2 * rnd(Dv, seed=seed + 8)
        self.qs, self.ks = 0.7, D ** -0.5
        if edit:
            edit(self)
        self.first = [sum(lens[:i]) for i in range(len(lens))]
        self.freqs = torch.tensor([300.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F64, device=DEV) if rot else None
        self.state = torch.full((len(lens) + 2, H, D, Dv), float("nan"), device=DEV)
        self.slot = [len(lens) + 1 - i for i in range(len(lens))]
        self.at, self.o, self.y = [0] * len(lens), [[] for _ in lens], [[] for _ in lens]
        self.want()

    def want(self):
        H, Hk, D, Dv = self.dims
        self.wo, self.wS = [], []
        for f, n in zip(self.first, self.lens):
            sl = slice(f, f + n)
            q, k = f64(self.q)[sl, :Hk * D].view(n, Hk, D), f64(self.k)[sl, :Hk * D].view(n, Hk, D)
            if self.unit:
                q, k = O.unit_length(q), O.unit_length(k)
            pos, rt = torch.arange(n), VenitarRot(300.0, self.rot)
            q, k = O.rotate(q, pos, rt) * self.qs, O.rotate(k, pos, rt) * self.ks
            v = f64(self.v)[sl, :H * Dv].view(n, H, Dv)
            out, S1 = torch.zeros(n, H, Dv, dtype=F64), torch.zeros(H, D, Dv, dtype=F64)
            for h in range(H):
                kh, qh, S = k[:, h // (H // Hk)], q[:, h // (H // Hk)], torch.zeros(D, Dv, dtype=F64)
                if self.rows:
                    z = f64(self.ld)[sl, h * D:(h + 1) * D]
                    g = torch.exp(f64(self.coef)[h] * torch.nn.functional.softplus(z, threshold=1e9))
                else:
                    g = f64(self.decay)[h].expand(n, D)
                if self.delta:
                    out[:, h], S1[h] = O.delta_rule(qh, kh, v[:, h], torch.sigmoid(f64(self.beta)[sl, h]), g, S)
                else:
                    for t in range(n):
                        S = g[t].unsqueeze(1) * S + torch.outer(kh[t], v[t, h])
                        out[t, h] = S.T @ qh[t]
                    S1[h] = S
            self.wo.append(out)
            self.wS.append(S1)

    def feed(self, portion, step=False):
        """``portion``: request -> its next tokens; ``step``: through the one-token kernel."""
        b, (H, Hk, D, Dv) = self.b, self.dims
        rows = torch.cat([torch.arange(self.first[r] + self.at[r], self.first[r] + self.at[r] + n) for r, n in portion.items()]).to(DEV)
        T = rows.numel()
        q, k, v, ld, beta, gate = (t[rows].contiguous() for t in (self.q, self.k, self.v, self.ld, self.beta, self.gate))
        reqs, chunks, chunk0, pos, row = [], [], [], [], 0
        for r, n in portion.items():
            reqs.append((self.slot[r], self.at[r], n, row))
            chunk0.append(len(chunks))
            chunks += [(row + i, min(16, n - i), 0, 0) for i in range(0, n, 16)]
            pos += list(range(self.at[r], self.at[r] + n))
            row += n
        kw = dict(q_scale=self.qs, k_scale=self.ks, unit_norm=self.unit)
        if self.rot:
            table = torch.empty(T, self.rot, device=DEV)
            b.rot_table(dev_i32(pos), self.freqs, 1.0, table, T)
            kw.update(rot=table, rot_dims=self.rot)
        kw.update(dict(ld=ld, ldld=H * D + 2, ld_coef=self.coef, ld_softplus=True) if self.rows else dict(decay=self.decay))
        if self.delta:
            kw.update(beta=beta, ldbeta=H + 1)
        lds_ = (Hk * D + 3, Hk * D + 3, H * Dv + 3)
        if step:
            y = torch.full((T, H * Dv + 2), 9.0, dtype=self.dtype, device=DEV)
            b.rec_step(q, k, v, lds_, dev_i32(reqs), len(reqs), self.state, H, Hk, D, Dv, y, H * Dv + 2, eps=1e-5, gain=self.gain, gate=gate, ldg=H * Dv + 1, **kw)
            assert bool((y[:, H * Dv:] == 9.0).all())
            out = y[:, :H * Dv]
        else:
            scratch = torch.full((b.rec_scratch(len(chunks), H, D),), float("nan"), device=DEV)
            out = torch.full((T, H * Dv), float("nan"), device=DEV)
            b.rec_prompt(q, k, v, lds_, dev_i32(reqs), len(reqs), dev_i32(chunks), dev_i32(chunk0), len(chunks), self.state, H, Hk, D, Dv, scratch, out, **kw)
        row = 0
        for r, n in portion.items():
            part = out[row:row + n].view(n, H, Dv)
            (self.y if step else self.o)[r].append((self.at[r], part))
            self.at[r] += n
            row += n

    def check(self, f32=2e-5, bf16=2e-2, eps=1e-5):
        """Everything that came out so far against the float64 result."""
        H, Hk, D, Dv = self.dims
        for r, n in enumerate(self.lens):
            for t0, part in self.o[r]:
                assert bool(torch.isfinite(part).all())
                assert rel(part, self.wo[r][t0:t0 + part.shape[0]]) < f32, (r, t0, rel(part, self.wo[r][t0:t0 + part.shape[0]]))
            for t0, part in self.y[r]:
                w = O.unit_rms(self.wo[r][t0:t0 + 1], eps) * f64(self.gain) * f64(self.gate)[self.first[r] + t0, :H * Dv].view(1, H, Dv)
                assert rel(part, w) < tol(self.dtype, 2 * f32, bf16), (r, t0, rel(part, w))
            if self.at[r] == n:
                assert rel(self.state[self.slot[r]], self.wS[r]) < f32


MODES = [dict(delta=False, rows=False), dict(delta=False, rows=True), dict(delta=True, rows=False, unit=True), dict(delta=True, rows=True, unit=True)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mode", range(4))
@pytest.mark.parametrize("H,Hk,D,Dv,rot", [(3, 3, 24, 40, 16), (4, 2, 64, 64, 0), (2, 2, 65, 17, 10), (2, 1, 128, 128, 128), (3, 1, 5, 7, 2), (1, 1, 200, 48, 0),
                                           (2, 2, 256, 96, 64), (1, 1, 16, 1, 16), (1, 1, 1, 20, 0), (2, 2, 96, 528, 0)])
def test_matrix_states_in_chunks_and_steps(dtype, mode, H, Hk, D, Dv, rot):
    """Whole prompts of unequal lengths in one launch, continued by portions of two tokens, of a chunk and a bit, and -- for heads that fit
    -- by one-token steps, on slots whose old states are not numbers."""
    r = Rec(dtype, H, Hk, D, Dv, [45, 1, 17, 16, 60], rot=rot, z=-2.0, **MODES[mode])
    r.feed({0: 20, 1: 1, 2: 15, 3: 16})
    r.feed({0: 2, 2: 2, 4: 33})
    r.feed({4: 2})
    if r.b.rec_step_fits(D, Dv):
        r.feed({0: 1, 4: 1}, step=True)
        r.feed({4: 1}, step=True)
    else:
        r.feed({0: 1, 4: 1})
        r.feed({4: 1})
    r.feed({0: 22, 4: 22})
    r.check()


@pytest.mark.parametrize("mode", [1, 3])
@pytest.mark.parametrize("z,zs", [(6.0, 8.0), (-12.0, 1.0), (40.0, 5.0), (0.0, 30.0)])
def test_strong_and_weak_decays_inside_a_chunk(mode, z, zs):
    """Channels that forget everything from one token to the next beside channels that forget nothing: factors of the decays over a chunk
    would leave the range of 32-bit floats on both sides, their products must not."""
    r = Rec(torch.float32, 2, 2, 48, 32, [70], z=z, zs=zs, **MODES[mode])
    r.feed({0: 50})
    for _ in range(3):
        r.feed({0: 1}, step=True)
    r.feed({0: 17})
    r.check()


@pytest.mark.parametrize("mode", range(4))
def test_tokens_one_by_one_equal_chunks(mode):
    """The one-token kernel from the first token on against chunks of every fill, and both against the float64 result."""
    lens = [40]
    whole = Rec(torch.float32, 3, 3, 36, 28, lens, rot=12, z=-1.0, **MODES[mode])
    whole.feed({0: 40})
    single = Rec(torch.float32, 3, 3, 36, 28, lens, rot=12, z=-1.0, **MODES[mode])
    for _ in range(40):
        single.feed({0: 1}, step=True)
    whole.check()
    single.check()
    for cut in (1, 2, 7, 15, 16, 17, 31):
        r = Rec(torch.float32, 3, 3, 36, 28, lens, rot=12, z=-1.0, **MODES[mode])
        r.feed({0: cut})
        r.feed({0: 40 - cut})
        r.check()
        assert rel(r.state[r.slot[0]], whole.state[whole.slot[0]]) < 1e-5


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_state_remembers_one_far_token(dtype):
    """Decay one: the read-out hundreds of tokens later is the value that one loud key wrote; decay nothing: only the token itself."""
    D, Dv, n, loud = 20, 12, 700, 3

    def edit(r):
        r.k.mul_(1e-4)
        r.q.mul_(1e-4)
        r.k[loud, :2 * D] = 0.0
        r.k[loud, 0] = r.k[loud, D] = 30.0
        r.q[650:, 0] = r.q[650:, D] = 1.0
        r.v[loud] = 5.0
        r.qs = r.ks = 1.0
    r = Rec(dtype, 2, 2, D, Dv, [n], delta=False, rows=False, decay=[1.0, 0.0], edit=edit)
    r.feed({0: 640})
    r.feed({0: 40})
    for _ in range(20):
        r.feed({0: 1}, step=True)
    r.check(f32=5e-5)
    got = torch.cat([p for t0, p in r.o[0] if t0 >= 640])[10:]
    assert float((got[:, 0] - 150.0).abs().max()) < 0.5 and float(got[:, 1].abs().max()) < 1.0


@pytest.mark.parametrize("dtype", DTYPES)
def test_delta_rule_overwrites_across_chunks_and_steps(dtype):
    """Unit keys on two axes, step size one, no forgetting: a query on an axis reads the value that its key wrote LAST, however many chunks
    ago, and the other axis's writes do not disturb it."""
    D, Dv, n = 16, 8, 90

    def edit(r):
        r.k.zero_(), r.q.zero_()
        r.k[:, 1] = 1.0                                        # every token writes on axis 1 ...
        r.k[[2, 40], :D] = 0.0
        r.k[[2, 40], 0] = 3.0                                  # ... but two, which write on axis 0
        r.q[:, 0] = 2.0
        r.v[2, :Dv], r.v[40, :Dv] = 5.0, -7.0
        r.beta.fill_(60.0)
        r.ld.fill_(-80.0)
        r.qs = r.ks = 1.0
    r = Rec(dtype, 1, 1, D, Dv, [n], edit=edit, **MODES[3])
    r.feed({0: 33})
    r.feed({0: 40})
    for _ in range(17):
        r.feed({0: 1}, step=True)
    r.check()
    got = torch.cat([p for _, p in r.o[0]])[:, 0]
    assert float((got[2:40] - 5.0).abs().max()) < 1e-3 and float((got[40:] + 7.0).abs().max()) < 1e-3 and float(got[:2].abs().max()) < 1e-4


# ---- attention over a slot's cached rows --------------------------------------------------------------------------------------------------
def cached_case(kind, dtype, reqs, H, Hkv, D, Dv, scale, *, window=0, block=0, sink=None, gate=None, splits=1, tile=64, loud=None, seed=0):
    """``reqs``: (slot, position of the first query, queries).  Keys and values interleave in one plane of three slots; what lies behind a
    slot's newest key is not a number.  ``gate``: None, "cols" or "head".  -> (got [rows, H, Dv], want)."""
    b, T = B(), sum(n for _, _, n in reqs)
    cap = 32 * (max(p + n - 1 for _, p, n in reqs) // 32 + 1)
    RW = D + Dv
    plane = rnd(3, Hkv, cap, RW, dtype=dtype, seed=seed + 1)
    q = rnd(T, H * D + 8, dtype=dtype, seed=seed + 2)
    gw = H * Dv if gate == "cols" else H
    G = rnd(T, gw + 8, dtype=dtype, seed=seed + 3).sigmoid() if gate else None
    if loud:
        loud(q[:, :H * D].view(T, H, D), plane)
    for s in range(3):
        top = max([p + n - 1 for s_, p, n in reqs if s_ == s], default=-1)
        plane[s, :, top + 1:] = float("nan")
    ldo = H * Dv + (7 if Dv % 2 else 8)
    out = torch.full((T, ldo), float("nan"), dtype=dtype, device=DEV)
    values = plane.view(-1)[D:]
    ss, hs = Hkv * cap * RW, cap * RW
    kw = dict(ldo=ldo, ldq=H * D + 8, window=window, block=block, sink=sink, gate=G[:, 8:] if gate else None, ldg=gw + 8)
    row, tiles = 0, []
    for s, p, n in reqs:
        step = 1 if kind == "rows" else tile
        tiles += [(s, p + i, min(step, n - i), row + i) for i in range(0, n, step)]
        row += n
    if kind == "rows":
        part = torch.empty(b.attn_softmax_part(T, H, splits, Dv), device=DEV) if splits > 1 else None
        b.attn_rows(q, dev_i32(tiles), T, plane, (ss, hs, RW), values, (ss, hs, RW), H, Hkv, D, Dv, scale, out, gate_per_head=gate == "head", n_splits=splits,
                    part=part, **kw)
    else:
        b.attn_prompt(q, dev_i32(tiles), len(tiles), tile, plane, (RW, hs, ss), values, (RW, hs, ss), H, Hkv, D, Dv, scale, out, gate_cols=gate == "cols", **kw)
    assert bool(torch.isnan(out[:, H * Dv:].float()).all())
    want, row = torch.zeros(T, H, Dv, dtype=F64), 0
    for s, p, n in reqs:
        for i in range(n):
            js = O.visible(p + i, block, window)
            for h in range(H):
                kv = f64(plane[s, h // (H // Hkv)])[js]
                sc = (kv[:, :D] @ f64(q)[row, h * D:(h + 1) * D]) * scale
                top = sc.max() if sink is None else torch.maximum(sc.max(), f64(sink)[h])
                e = torch.exp(sc - top)
                den = e.sum() + (torch.exp(f64(sink)[h] - top) if sink is not None else 0.0)
                want[row, h] = (e / den) @ kv[:, D:]
            row += 1
    if gate:
        g = f64(G)[:, 8:]
        want *= g.view(T, H, Dv) if gate == "cols" else g.view(T, H, 1)
    return out[:, :H * Dv].reshape(T, H, Dv), want


KINDS = [("rows", torch.float32, 1, 1), ("rows", torch.float32, 5, 1), ("rows", torch.bfloat16, 1, 1), ("rows", torch.bfloat16, 64, 1),
         ("prompt", torch.float32, 1, 64), ("prompt", torch.bfloat16, 1, 64), ("prompt", torch.bfloat16, 1, 128)]


@pytest.mark.parametrize("kind,dtype,splits,tile", KINDS)
@pytest.mark.parametrize("H,Hkv,D,Dv", [(6, 2, 40, 40), (20, 1, 64, 64), (4, 4, 128, 128), (17, 1, 24, 136), (2, 2, 200, 56), (3, 1, 7, 9), (2, 1, 256, 256)])
def test_attention_over_cached_rows(kind, dtype, splits, tile, H, Hkv, D, Dv):
    """Several slots in one launch, from a first token to rows deep in a sequence; windows, blocks, sinks and both kinds of gate."""
    reqs = [(0, 0, 3), (2, 61, 6), (1, 250, 70)] if kind == "prompt" else [(0, 0, 3), (2, 61, 6), (1, 250, 2)]
    sink = rnd(H, seed=9, scale=2.0)
    for kw in (dict(sink=sink, block=50), dict(gate="cols", window=70), dict(sink=sink, gate="head"), dict(window=33, block=64)):
        got, want = cached_case(kind, dtype, reqs, H, Hkv, D, Dv, 2.0 * D ** -0.5, splits=splits, tile=tile, **kw)
        assert rel(got, want) < tol(dtype, 1e-5, 1e-2), kw


@pytest.mark.parametrize("kind,dtype,splits,tile", KINDS)
@pytest.mark.parametrize("mask", ["window", "block"])
@pytest.mark.parametrize("size", [1, 31, 32, 64, 100])
def test_one_loud_key_just_inside_and_just_outside_every_edge(kind, dtype, splits, tile, mask, size):
    """Every key is quiet but one whose score towers over the rest: rows up to the mask's edge return its value, the next must not."""
    H, D, Dv = 4, 16, 24
    spot = 130
    first = spot // size * size if mask == "block" else spot                  # the first and last rows that see the spot
    last = first + size - 1 if mask == "block" else spot + size - 1

    def make(q, plane):
        q.mul_(0.05)
        plane[..., :D].mul_(0.05)
        q[:, :, 3] = 2.0
        plane[:, :, spot, 3] = 30.0
        plane[:, :, spot, D:] = 5.0
    rows = sorted({spot - 1, spot, last, last + 1, (spot + last) // 2})
    reqs = [(0, spot - 1, last + 2 - (spot - 1))] if kind == "prompt" else [(i % 3, p, 1) for i, p in enumerate(rows)]
    got, want = cached_case(kind, dtype, reqs, H, 2, D, Dv, 1.0, splits=splits, tile=tile, loud=make, **{mask: size})
    assert rel(got, want) < tol(dtype, 1e-5, 1e-2)
    where = {p: (p - (spot - 1) if kind == "prompt" else i) for i, p in enumerate(rows)}
    for p, r in where.items():
        hit = float((got[r].float() - 5.0).abs().max()) < 0.05
        assert hit == (spot <= p <= last), (p, spot, last)


@pytest.mark.parametrize("kind,dtype,splits,tile", KINDS)
def test_far_keys_at_key_block_borders_and_the_sink(kind, dtype, splits, tile):
    """One loud key per column: the first of the sequence, the last and first of key blocks, and recent ones; each row listens to one of
    them, hundreds of positions away.  A sink of score zero halves what an equally quiet key gets and does nothing to a loud one."""
    spots, p0, n = [0, 1, 31, 32, 63, 64, 127, 128, 300], 640, 40 if kind == "prompt" else 12

    def make(q, plane):
        q.mul_(0.02)
        plane[..., :16].mul_(0.02)
        for i, s in enumerate(spots):
            plane[:, :, s, i] = 25.0
            plane[:, :, s, 16:] = float(i + 1)
        for r in range(q.shape[0]):
            q[r, :, (r * 7) % len(spots)] = 2.0
    zero = torch.zeros(2, device=DEV)
    for sink in (None, zero):
        got, want = cached_case(kind, dtype, [(1, p0, n)], 2, 1, 16, 8, 1.0, splits=splits, tile=tile, loud=make, sink=sink)
        assert rel(got, want) < tol(dtype, 1e-5, 1e-2)
        for r in range(n):
            i = (r * 7) % len(spots)
            assert float((got[r].float() - (i + 1)).abs().max()) < 0.05 * (i + 1), r

    def lone(q, plane):
        q.zero_()
        plane[..., 16:] = 8.0
    got, _ = cached_case(kind, dtype, [(0, 0, 4)], 2, 1, 16, 8, 1.0, splits=splits, tile=tile, loud=lone, sink=zero)
    for r in range(4):                                         # r + 1 keys and the sink share the weight
        assert float((got[r].float() - 8.0 * (r + 1) / (r + 2)).abs().max()) < tol(dtype, 1e-4, 3e-2)


# =====================================================================================================================================
# the model through its arena
# =====================================================================================================================================
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("by_rows", [False, True])
@pytest.mark.parametrize("name", list(SHAPES))
def test_whole_prompt_against_the_oracle_layer_by_layer(name, dtype, by_rows):
    """Both forms of the attention: tiles of neighbouring queries, and every row by itself."""
    s, w, m = model(name, dtype)
    tokens = toks(115, s.vocab_size, seed=3)
    want, want_streams = oracle(s, w, tokens)
    m.PROMPT_ROWS = 10 ** 9 if by_rows else 1
    try:
        ar = m.new_arena(1, 120)
        logits, streams = m.forward_rows(ar, [ar.alloc()], [tokens], [list(range(len(tokens)))], return_streams=True)
    finally:
        del m.PROMPT_ROWS
    runs = s.runs()
    assert streams.shape[0] == len(runs)
    for r, (i, _) in enumerate(runs):
        assert close(streams[r], want_streams[r], dtype), f"run {r} (layer {i})"
    assert close(logits, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(SHAPES))
def test_prompt_equals_token_by_token_decoding_and_any_portions(name, dtype):
    s, w, m = model(name, dtype)
    n = 72
    tokens = toks(n, s.vocab_size, seed=5)
    whole = run_alone(m, tokens)
    for cuts in ([1] * n, [2] * (n // 2), [33, 2, 2, 19, 16], [16, 16, 16, 24], [1, 71], [40] + [1] * 32, [15, 57], [64, 8], [3] * 24):
        assert close(run_alone(m, tokens, cuts), whole, dtype, 2e-5), cuts
    assert close(whole, oracle(s, w, tokens)[0], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("graphs", [True, False])
def test_unequal_batches_and_reused_slots(dtype, graphs):
    """Requests of different lengths step together -- prompts, short portions and decoded tokens side by side --, some end, newcomers take
    their slots (the previous owner's rows, states and last inputs still lie there), the rest go on: every request's logits equal those
    it gets alone."""
    s, w, m = model("mixed", dtype)
    m.use_graphs = graphs
    try:
        prompts = {k: toks(n, s.vocab_size, seed=20 + k) for k, n in enumerate([61, 3, 38, 1, 47])}
        alone = {k: run_alone(m, p) for k, p in prompts.items()}
        ar = m.new_arena(2, 16)
        got = {k: [] for k in prompts}
        slots, at = {}, {k: 0 for k in prompts}

        def step(parts):
            for k in parts:
                if k not in slots:
                    slots[k] = ar.alloc()
            ks = list(parts)
            out = m.forward_rows(ar, [slots[k] for k in ks], [prompts[k][at[k]:at[k] + parts[k]] for k in ks], [list(range(parts[k])) for k in ks])
            o = 0
            for k in ks:
                got[k].append(out[o:o + parts[k]])
                o += parts[k]
                at[k] += parts[k]
                if at[k] == len(prompts[k]):
                    ar.free(slots.pop(k))
        step({0: 50, 1: 2, 2: 20})
        step({0: 1, 1: 1, 2: 1})                              # request 1 ends here
        step({0: 1, 2: 1, 3: 1})                              # 3 arrives on 1's slot and ends at once (a first token among decoded ones)
        step({2: 16, 4: 30, 0: 1})                            # 4 arrives on that slot again; 2 ends
        while any(at[k] < len(prompts[k]) for k in (0, 4)):
            step({k: 1 for k in (0, 4) if at[k] < len(prompts[k])})
        for k in prompts:
            assert close(torch.cat(got[k]), alone[k], dtype, 2e-5), k
    finally:
        m.use_graphs = True


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_through_graphs_and_a_growing_arena(dtype):
    """A short prompt, then 190 tokens one by one on an arena that starts too small: the planes move (captured steps are recaptured), and
    the decoded positions pass window edges, block edges and key blocks."""
    s, w, m = model("mixed", dtype)
    tokens = toks(200, s.vocab_size, seed=9)
    ar = m.new_arena(1, 24)
    slot = ar.alloc()
    out = [m.forward_rows(ar, [slot], [tokens[:10]], [list(range(10))])]
    for t_ in tokens[10:]:
        out.append(m.forward_rows(ar, [slot], [[t_]], [[0]]))
    assert ar.cap >= 200
    assert close(torch.cat(out), oracle(s, w, tokens)[0], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_positions_in_a_long_prompt_and_after_it(dtype):
    """600 tokens with sharp scores and slow decays: tiles deep in the sequence, a short portion far behind a long cache, and decoded
    tokens after it."""
    from promptcache_amd.model.venitar_hip import VenitarHIP
    s = VenitarShape(vocab_size=90, hidden_size=48, norm_eps=1e-6, embed_scale=6.9, loop_start=0, loop_stop=1, loop_times=2, layers=[
        att(4, 2, 16, 0, sharp=5.0, ff=32), ret(2, 16, 24, decay=[0.999, 1.0]), par((4, 1, 24, 16), (2, 1, 16, 24), 500, sharp=5.0), att(2, 1, 24, 512, sharp=5.0)])
    w = W.make_venitar_weights(s, seed=4)
    m = VenitarHIP(s, w, device=DEV, dtype=dtype)
    tokens = toks(600, s.vocab_size, seed=2)
    want = oracle(s, w, tokens)[0]
    ar = m.new_arena(1, 640)
    slot = ar.alloc()
    got = [m.forward_rows(ar, [slot], [tokens[:540]], [list(range(540))]), m.forward_rows(ar, [slot], [tokens[540:592]], [list(range(52))])]
    got += [m.forward_rows(ar, [slot], [[t_]], [[0]]) for t_ in tokens[592:]]
    assert close(torch.cat(got), want, dtype, 1e-4, 6e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["attention", "retention", "parallel"])
def test_one_early_token_decides_far_logits(dtype, kind):
    """Two prompts that differ in their second token only: logits hundreds of positions later differ, and both agree with the oracle
    about it, in a prompt and decoded -- through sharp scores, through a state that forgets nothing, through both halves."""
    from promptcache_amd.model.venitar_hip import VenitarHIP
    lay = {"attention": att(2, 1, 16, 0, rot=0, sharp=12.0, ff=24), "retention": ret(2, 12, 16, rot=2, decay=[1.0, 0.9999], base=1e9),
           "parallel": par((2, 2, 16, 16), (2, 2, 12, 16), 0, rot=0, sharp=12.0)}[kind]
    s = VenitarShape(vocab_size=40, hidden_size=32, norm_eps=1e-6, embed_scale=5.0, layers=[lay])
    w = W.make_venitar_weights(s, seed=6)
    if kind == "parallel":
        w["l0.mix.right.dt_bias"].fill_(-12.0)
    p6 = O.to_f64(w)
    rest = [t % 39 for t in toks(420, 40, seed=8)]
    m = VenitarHIP(s, w, device=DEV, dtype=dtype)
    a, b_ = [3, 39] + rest, [3, 5] + rest
    wa, wb = O.forward(s, p6, a)[-30:], O.forward(s, p6, b_)[-30:]
    gap = rel(wa, wb)
    ga, gb = run_alone(m, a)[-30:], run_alone(m, b_)[-30:]
    da = run_alone(m, a, [400] + [1] * 22)[-22:]
    assert gap > 1e-4
    if dtype == torch.float32:
        assert abs(rel(ga, gb) - gap) < 0.05 * gap + 1e-6
    assert close(ga, wa, dtype) and close(gb, wb, dtype) and close(da, wa[-22:], dtype)


@pytest.mark.parametrize("loop", [(0, 1, 1), (0, 3, 1), (2, 3, 4), (0, 3, 2), (1, 2, 3), None])
def test_loops_of_every_extent(loop):
    """float32, whole and decoded: a loop at the front, at the end, over everything, over one layer, run once, or none at all."""
    from promptcache_amd.model.venitar_hip import VenitarHIP
    a, b_, n = loop or (0, 0, 0)
    s = VenitarShape(vocab_size=60, hidden_size=40, norm_eps=1e-5, embed_scale=4.4, loop_start=a, loop_stop=b_, loop_times=n, layers=[
        ret(2, 12, 8, ff=24), att(3, 1, 8, 9, ff=16), par((2, 1, 16, 10), (2, 2, 12, 20), 13)])
    w = W.make_venitar_weights(s, seed=13)
    m = VenitarHIP(s, w, device=DEV, dtype=torch.float32)
    tokens = toks(41, s.vocab_size, seed=1)
    want, streams = oracle(s, w, tokens)
    ar = m.new_arena(1, 48)
    assert len(ar.planes) == 3 + (b_ - a) * (n - 1 if n else 0)
    got, gs = m.forward_rows(ar, [ar.alloc()], [tokens], [list(range(41))], return_streams=True)
    assert close(got, want, torch.float32) and rel(gs, streams) < 2e-5
    assert close(run_alone(m, tokens, [20] + [1] * 21), want, torch.float32)


def test_same_rows_same_values_whatever_the_company():
    """float32: a request's logits next to other requests, and on another slot, agree with those it gets alone to summation order."""
    s, w, m = model("wide", torch.float32)
    a, b_, c = toks(50, s.vocab_size, 1), toks(9, s.vocab_size, 2), toks(23, s.vocab_size, 3)
    alone = run_alone(m, a)
    ar = m.new_arena(3, 64)
    s0, s1, s2 = ar.alloc(), ar.alloc(), ar.alloc()
    out = m.forward_rows(ar, [s0, s2, s1], [b_, a, c], [[0], list(range(50)), []])
    assert rel(out[1:], alone) < 3e-6


@pytest.mark.parametrize("dtype", DTYPES)
def test_captured_steps_replay_what_eager_steps_compute(dtype):
    """Graph replays interleaved with eager work and other batch sizes: every replay against the eager result of the same step."""
    s, w, m = model("mixed", dtype)
    tokens = [toks(40, s.vocab_size, seed=50 + k) for k in range(3)]
    arenas = []
    for graphs in (True, False):
        ar = m.new_arena(3, 64)
        arenas.append((graphs, ar, [ar.alloc() for _ in range(3)]))
    try:
        for k in range(20):
            live = [0, 1, 2] if k % 3 else [0, 2]
            outs = []
            for graphs, ar, slots in arenas:
                m.use_graphs = graphs
                outs.append(m.forward_rows(ar, [slots[i] for i in live], [[tokens[i][ar.lengths[slots[i]]]] for i in live]))
                torch.randn(64, 64, device=DEV).sum()
                torch.cuda.synchronize()
            assert rel(outs[0], outs[1]) < 1e-6, k
    finally:
        m.use_graphs = True


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_batch_engine(dtype):
    from promptcache_amd import BatchEngine, GenerationParameters
    from promptcache_amd.model import Venitar
    s = shape_mixed()
    w = W.make_venitar_weights(s, seed=11)
    lm = Venitar(shape=s, weights=w, device=DEV, dtype=dtype)
    prompts = [toks(n, s.vocab_size, seed=40 + n) for n in (12, 3, 30)]
    eng = BatchEngine(lm, max_tokens=80)                      # (a budget that does not hold all three at once)
    params = GenerationParameters(temperature=0.0, max_new_tokens=12, stop_token_ids=[])
    got = eng.generate(prompts, params)
    p6 = O.to_f64(w)
    for prompt, out in zip(prompts, got):
        assert len(out) == 12
        logits = O.forward(s, p6, list(prompt) + out)[len(prompt) - 1:-1]
        for k, tok in enumerate(out):                         # every generated token is the oracle's choice given the same history,
            best = int(logits[k].argmax())                    # unless the oracle's two best are closer than the format resolves
            if tok != best:
                assert float(logits[k][best] - logits[k][tok]) < (1e-4 if dtype == torch.float32 else 0.2), (k, tok, best)


def random_shape(rng):
    """Sizes, layer order, loop and constants drawn at random."""
    width = rng.choice([64, 72, 96, 160, 200, 264])
    layers = []
    for _ in range(rng.randrange(1, 6)):
        kind, ff = rng.choice(["retention", "attention", "parallel"]), rng.choice([0, 32, 56, 2 * width])
        if kind == "retention":
            h, d = rng.choice([1, 2, 4, 7]), rng.choice([8, 16, 24, 48, 96])
            layers.append(ret(h, d, rng.choice([8, 16, 40, 80]), rot=rng.choice([0, 4, d]), ff=ff, base=rng.choice([500.0, 10000.0, 1e6]),
                              decay=[rng.choice([0.4, 0.9, 0.99, 0.9995]) for _ in range(h)]))
        elif kind == "attention":
            kv, d = rng.choice([1, 2, 3]), rng.choice([8, 16, 32, 80])
            layers.append(att(kv * rng.choice([1, 2, 6, 18]), kv, d, rng.choice([0, 1, 7, 16, 50, 64]), rot=rng.choice([0, 4, d]), ff=ff, sharp=rng.choice([1.0, 3.0])))
        else:
            kv, d, rk = rng.choice([1, 2]), rng.choice([8, 24, 64]), rng.choice([1, 2, 3])
            layers.append(par((kv * rng.choice([1, 3, 4]), kv, d, rng.choice([8, 24, 72])), (rk * rng.choice([1, 2]), rk, rng.choice([8, 16, 40, 72]), rng.choice([8, 24, 64])),
                              rng.choice([0, 1, 5, 32, 60]), rot=rng.choice([0, 4, d]), yarn=rng.choice([None, YARN, (2.0, 64.0, 16.0, 1.0)]), conv=rng.choice([1, 2, 3, 4, 6]),
                              ranks=(rng.choice([4, 16, 30]), rng.choice([8, 12])), scales=(rng.choice([0.5, 1.0, -0.8]), rng.choice([0.3, 1.0, 1.5])), ff=ff))
    s = VenitarShape(vocab_size=rng.randrange(50, 900), hidden_size=width, norm_eps=rng.choice([1e-5, 1e-6]), embed_scale=rng.choice([1.0, 9.5]), layers=layers)
    if rng.random() < 0.75:
        s.loop_start = rng.randrange(len(layers))
        s.loop_stop = rng.randrange(s.loop_start + 1, len(layers) + 1)
        s.loop_times = rng.randrange(1, 4)
    return s


@pytest.mark.parametrize("seed", range(10))
def test_random_configurations_whole_decoded_and_in_company(seed):
    import random
    from promptcache_amd.model.venitar_hip import VenitarHIP
    rng = random.Random(3000 + seed)
    s = random_shape(rng)
    ranks = [(l.right.a_rank, l.right.g_rank) if l.kind == "parallel" else None for l in s.layers]
    s = VenitarShape.from_config(json.loads(json.dumps(s.to_config())))
    for l, r in zip(s.layers, ranks):
        if r:
            l.right.a_rank, l.right.g_rank = r
    w = W.make_venitar_weights(s, seed=seed)
    n = rng.randrange(90, 200)
    a, b_ = toks(n, s.vocab_size, seed), toks(rng.randrange(1, 70), s.vocab_size, seed + 1)
    want_a, want_b = oracle(s, w, a)[0], oracle(s, w, b_)[0]
    for dtype in DTYPES:
        m = VenitarHIP(s, w, device=DEV, dtype=dtype)
        assert close(run_alone(m, a), want_a, dtype, 1e-4, 8e-2), s.to_config()
        ar = m.new_arena(1, 16)
        sa, sb = ar.alloc(), ar.alloc()
        cut = n - 20
        out = [m.forward_rows(ar, [sb, sa], [b_, a[:cut]], [list(range(len(b_))), list(range(cut))])]
        out += [m.forward_rows(ar, [sa], [[t_]], [[0]]) for t_ in a[cut:]]
        got = torch.cat(out)
        assert close(got[len(b_):], want_a, dtype, 1e-4, 8e-2) and close(got[:len(b_)], want_b, dtype, 1e-4, 8e-2), s.to_config()


def test_single_request_engine_and_the_adapters_call():
    """GenerationEngine drives the model through the adapters' ``model(input_ids, past_key_values)`` call; a padded batch through
    that call gives each row its own logits."""
    from promptcache_amd import BatchEngine, GenerationEngine, GenerationParameters
    from promptcache_amd.model import Venitar
    s = shape_mixed()
    w = W.make_venitar_weights(s, seed=21)
    lm = Venitar(shape=s, weights=w, device=DEV, dtype=torch.float32)
    assert lm.get_cache_shape() == (8, 2, 40)
    prompts = [toks(13, s.vocab_size, 30), toks(5, s.vocab_size, 31)]
    params = GenerationParameters(temperature=0.0, max_new_tokens=6, stop_token_ids=[])
    want = BatchEngine(lm).generate(prompts, params)
    out = None
    for out in GenerationEngine(lm).generate(prompts[0], list(range(13)), params):
        pass
    assert out is not None and lm.decode(want[0]) == out.new_text
    ids, mask = torch.zeros((2, 13), dtype=torch.long), torch.zeros((2, 13), dtype=torch.long)
    ids[0, :13], mask[0, :13] = torch.tensor(prompts[0]), 1
    ids[1, :5], mask[1, :5] = torch.tensor(prompts[1]), 1
    res = lm(input_ids=ids, attention_mask=mask, past_key_values=None, use_cache=True)
    p6 = O.to_f64(w)
    assert rel(res.logits[0], O.forward(s, p6, prompts[0])) < 3e-5 and rel(res.logits[1, :5], O.forward(s, p6, prompts[1])) < 3e-5
    assert int(res.logits[0, 12].argmax()) == want[0][0] and int(res.logits[1, 4].argmax()) == want[1][0]


def test_what_the_kernels_do_not_hold_is_refused():
    from promptcache_amd.model.venitar_hip import VenitarHIP
    for bad in (ret(1, 260, 8), att(1, 1, 258, 0), par((1, 1, 8, 300), (1, 1, 8, 8), 4), par((1, 1, 8, 8), (1, 1, 300, 8), 4), par((1, 1, 8, 8), (1, 1, 8, 8), 4, conv=17)):
        s = VenitarShape(vocab_size=20, hidden_size=16, norm_eps=1e-6, layers=[bad])
        with pytest.raises(ValueError):
            VenitarHIP(s, W.make_venitar_weights(s), device=DEV)
    s = shape_odd()
    with pytest.raises(ValueError):
        VenitarHIP(s, W.make_venitar_weights(s), device=DEV, dtype=torch.float16)


def test_checkpoint_directory_command_line_and_trace_runner(tmp_path):
    """config.json + model.safetensors written from a shape, found by the registry, and replayed by bin/trace_run in both formats."""
    import numpy as np
    from safetensors.torch import save_file
    from promptcache_amd.model import load_language_model
    s = shape_odd()
    w = W.make_venitar_weights(s, seed=3)
    d = tmp_path / "ckpt"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(s.to_config()))
    save_file({k: v.contiguous() for k, v in w.items()}, str(d / "model.safetensors"))
    lm = load_language_model(str(d), dtype=torch.float32)
    assert type(lm).__name__ == "Venitar" and lm.hf_model.config.to_config() == s.to_config()
    a, b_ = toks(21, s.vocab_size, 1), toks(6, s.vocab_size, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:15], "want": [0, 14]}, {"id": "b", "tokens": b_[:5], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[15:16], "want": [0]}, {"id": "b", "tokens": b_[5:], "want": [0]}], "end": ["b"]}] + \
            [{"step": 2 + k, "entries": [{"id": "a", "tokens": [a[16 + k]], "want": [0] if k % 2 else []}], "end": ["a"] if k == 4 else []}
             for k in range(5)]
    wa, wb = oracle(s, w, a)[0], oracle(s, w, b_)[0]
    want = {0: wa[[0, 14]], 1: torch.stack([wa[15], wb[5]]), 3: wa[17:18], 5: wa[19:20]}
    env = dict(os.environ, PYTHONPATH=os.pathsep.join([ROOT, os.path.join(ROOT, "prompt-cache_amd")]))
    for fmt, t in (("float32", 3e-5), ("bfloat16", 8e-2)):
        out = tmp_path / fmt
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(d), "--dtype", fmt, "--out", str(out), "--max-tokens", "40"],
                           input="\n".join(json.dumps(x) for x in steps) + "\n", capture_output=True, text=True, env=env, timeout=600)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {k}" for k in range(7)]
        assert sorted(os.listdir(out)) == ["0.f32", "1.f32", "3.f32", "5.f32"]
        for k, wv in want.items():
            got = torch.from_numpy(np.fromfile(out / f"{k}.f32", dtype="<f4").reshape(-1, s.vocab_size))
            assert rel(got, wv) < t, (fmt, k)
