"""Pikadra on the GPU against the plain float64 oracle (``oracle/pikadra_oracle.py``): every new or extended building-block kernel alone --
with inputs built so that a far key, a tile's or key block's border, a window's edge or a sink decides the result --, then the model
through its arena: prompts in both forms of the attention, token-by-token decoding, portions down to two tokens, unequal batches, reused
slots, loops of every extent, long decoding through captured graphs, and greedy generation through the engines and the trace runner.
float32 runs are held to float32 accuracy; bfloat16 runs to what bf16 operands allow."""
import json
import os
import subprocess

import pytest
import torch

from oracle import pikadra_oracle as O
from promptcache_amd.model import weights as W
from promptcache_amd.model.config import PikadraLayer, PikadraShape

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


def close(got, want, dtype, f32=3e-5, bf16=3e-2):
    """Logits row by row.  float32: every row within float32 accuracy.  bfloat16: where two router scores of the float64 oracle lie closer
    than bf16 operands resolve, a token may take another expert than the oracle's, so rows are judged together: the median row within
    ``bf16``, at most one row in ten (or one) beyond three times that."""
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


def mla(heads, dim, rot, vdim, rank, qrank, sharp=2.5, base=3000.0, **ff):
    """``sharp``: the factor on the usual score scale, so that single keys carry weight among hundreds."""
    return PikadraLayer(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=rank, q_rank=qrank, scale=sharp * (dim + rot) ** -0.5,
                        rot_base=base, rot_dims=rot, **ff)


MOE = dict(ff_kind="moe", experts=6, top=3, expert_ff=24, shared_ff=40)
BARE = dict(ff_kind="moe", experts=5, top=1, expert_ff=32)
DENSE = dict(ff_kind="dense", ff=72)


# ---- shapes: layers differ from one another, come in different orders, and no size is a round one -------------------------------
def shape_mixed():
    return PikadraShape(vocab_size=170, hidden_size=104, norm_eps=1e-5, embed_scale=8.0, loop_start=1, loop_stop=3, loop_times=2, logit_scale=2.5,
                        logit_softcap=14.0, layers=[
        mla(5, 24, 8, 40, 48, 56, **MOE), mla(3, 40, 16, 24, 32, 40, **DENSE), mla(6, 16, 32, 16, 80, 24, **BARE), mla(2, 32, 8, 48, 40, 64)])


def shape_odd():
    """Sizes that are no multiple of a 16-byte chunk in either element type; one head, one expert, a layer without a rotated part, one
    without a feed-forward, no cap, a loop over the whole stack."""
    return PikadraShape(vocab_size=77, hidden_size=50, norm_eps=1e-6, embed_scale=1.0, loop_start=0, loop_stop=4, loop_times=3, logit_scale=1.0,
                        logit_softcap=0.0, layers=[
        mla(1, 10, 6, 7, 13, 9, **DENSE), mla(3, 6, 2, 10, 22, 15, ff_kind="moe", experts=1, top=1, expert_ff=14, shared_ff=6),
        mla(2, 9, 0, 5, 11, 30), mla(4, 7, 10, 6, 18, 7, ff_kind="moe", experts=7, top=7, expert_ff=10)])


def shape_wide():
    """Enough columns to reach the wider kernel instantiations: a latent of hundreds of columns, heads of 192 and of more than 200 key
    columns, 17 and 20 heads (a full group of sixteen and a rest), heads too wide for rebuilt keys; no loop."""
    return PikadraShape(vocab_size=300, hidden_size=128, norm_eps=1e-6, embed_scale=11.3, logit_scale=0.7, logit_softcap=30.0, layers=[
        mla(17, 128, 64, 64, 512, 96, **DENSE), mla(4, 144, 64, 200, 200, 48, **MOE), mla(20, 48, 32, 40, 320, 80, **BARE),
        mla(2, 240, 48, 72, 96, 64, **DENSE)])


SHAPES = {"mixed": shape_mixed, "odd": shape_odd, "wide": shape_wide}
_models = {}


def model(name, dtype, seed=11):
    from promptcache_amd.model.pikadra_hip import PikadraHIP
    key = (name, dtype, seed)
    if key not in _models:
        s = SHAPES[name]()
        w = W.make_pikadra_weights(s, seed=seed)
        _models[key] = (s, w, PikadraHIP(s, w, device=DEV, dtype=dtype))
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
@pytest.mark.parametrize("D,off,rot", [(14, 4, 8), (13, 0, 6), (70, 0, 70), (150, 22, 128), (9, 2, 0)])
def test_rotation_in_halves_with_norm_and_in_place(dtype, D, off, rot):
    """Halves of the rotated range turn together; the columns around it pass; positions in the hundreds of thousands, where an angle taken
    in 32-bit would have lost its low bits; the same result when a segment works in place."""
    H, b = 3, B()
    pos = [0, 1, 31, 250001, 7, 999983]
    T, N = len(pos), H * D + 5
    P, gain = rnd(T, N, dtype=dtype, seed=1), 1 + 0.1 * rnd(D, seed=2)
    fr = torch.tensor([700.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F64, device=DEV) if rot else None

    def turned(x):
        x = x.clone()
        x[..., off:off + rot] = O.rotate_halves(x[..., off:off + rot], torch.tensor(pos), 700.0, rot)
        return x
    x6 = f64(P)[:, 2:2 + H * D].view(T, H, D)
    out = torch.zeros(T, H * D, dtype=dtype, device=DEV)
    kw = dict(pos=dev_i32(pos), freqs=fr, eps=1e-5, rot_half=True)
    b.head_prep([b.head_seg(P[:, 2:], N, H, D, out, norm=True, gain=gain, rot_off=off, rot_dims=rot, ld_dst=H * D)], T, dtype, **kw)
    assert rel(out, turned(O.rms(x6, 1e-5) * f64(gain)).reshape(T, -1)) < tol(dtype, 2e-6, 5e-3)
    Q = P.clone()
    b.head_prep([b.head_seg(Q[:, 2:], N, H, D, Q, rot_off=off, rot_dims=rot, ld_dst=N, dst_offset=2)], T, dtype, **kw)
    assert rel(Q[:, 2:2 + H * D], turned(x6).reshape(T, -1)) < tol(dtype, 2e-6, 5e-3)
    assert torch.equal(Q[:, :2], P[:, :2]) and torch.equal(Q[:, 2 + H * D:], P[:, 2 + H * D:])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K,N,ld_pad", [(1, 40, 24, 0), (9, 37, 50, 3), (70, 64, 80, 8), (150, 96, 72, 0)])
def test_batched_projections_of_head_by_head_rows(dtype, M, K, N, ld_pad):
    """Every head's columns through a matrix of its own, into a column block of a wider matrix; with row tables only those rows move."""
    H, b = 5, B()
    ldx, ldy = H * K + ld_pad, H * N + 2 * ld_pad + 1
    x, w = rnd(M + 4, ldx, dtype=dtype, seed=1), rnd(H, N, K, dtype=dtype, seed=2, scale=K ** -0.5)
    y = torch.full((M + 4, ldy), 7.0, dtype=dtype, device=DEV)
    b.linear(x, w, y, M=M, n_batch=H, ldx=ldx, x_batch_stride=K, ldy=ldy, y_batch_stride=N)
    want = torch.stack([f64(x)[:, h * K:(h + 1) * K] @ f64(w)[h].T for h in range(H)], dim=1).reshape(M + 4, -1)
    assert rel(y[:M, :H * N], want[:M]) < tol(dtype, 2e-6, 5e-3)
    assert bool((y[M:] == 7.0).all()) and bool((y[:, H * N:] == 7.0).all())
    rows = [r for r in range(M + 4) if r % 3 == 1]
    y.fill_(7.0)
    b.linear(x, w, y, M=len(rows), row_src=dev_i32(rows), row_dst=dev_i32(rows), n_batch=H, ldx=ldx, x_batch_stride=K, ldy=ldy, y_batch_stride=N)
    assert rel(y[rows, :H * N], want[rows]) < tol(dtype, 2e-6, 5e-3)
    others = [r for r in range(M + 4) if r not in rows]
    assert bool((y[others] == 7.0).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [3, 40, 150])
def test_gate_per_row_and_fp32_split_columns(dtype, M):
    K, N, b = 56, 88, B()
    x, wg, wu = rnd(M, K, dtype=dtype, seed=1), rnd(N, K, dtype=dtype, seed=2, scale=0.3), rnd(N, K, dtype=dtype, seed=3, scale=0.3)
    gates = rnd(M, 9, dtype=dtype, seed=4).sigmoid()
    y = torch.zeros(M, N + 30, dtype=dtype, device=DEV)
    b.linear(x, wg, y[:, 30:], M=M, epilogue=b.EPI_SILU_MUL, w2=wu, row_gate=gates[:, 5:], ld_row_gate=9, ldy=N + 30)
    want = O.silu(f64(x) @ f64(wg).T) * (f64(x) @ f64(wu).T) * f64(gates)[:, 5:6]
    assert rel(y[:, 30:], want) < tol(dtype, 2e-6, 6e-3) and float(y[:, :30].float().abs().max()) == 0.0
    # the last columns of a projection as fp32 rows: router logits that no rounding to E may touch; the activation stays with the others
    z, lg = torch.empty(M, N - 20, dtype=dtype, device=DEV), torch.zeros(M, 24, device=DEV)
    b.linear(x, wg, z, M=M, act_split=10, act2=b.ACT_SIGMOID, split_n=N - 20, y2=lg, y2_f32=True, head_stride2=24)
    full = f64(x) @ f64(wg).T
    assert rel(lg[:, :20], full[:, N - 20:]) < 2e-6 and float(lg[:, 20:].abs().max()) == 0.0
    want = torch.cat([full[:, :10], torch.sigmoid(full[:, 10:N - 20])], dim=1)
    assert rel(z, want) < tol(dtype, 2e-6, 5e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W_", [50, 1500])
def test_residual_step_takes_experts_and_leaves_the_stream_as_it_is(dtype, W_):
    T, top, eps, b = 7, 3, 1e-5, B()
    x0, y, pair, pw = rnd(T, W_, seed=1, scale=3.0), rnd(T, W_, seed=2), rnd(T * top, W_, seed=3), rnd(T * top, seed=4)
    gain = 1 + 0.1 * rnd(W_, seed=5)
    mix = (f64(pw).view(T, top, 1) * f64(pair).view(T, top, W_)).sum(dim=1)
    for yy in (y, None):
        new = f64(x0) + mix + (f64(yy) if yy is not None else 0.0)
        x, out = x0.clone(), torch.empty(T, W_, dtype=dtype, device=DEV)
        b.post_norm(x, y=yy, pair=pair, pair_weight=pw, pair_top=top, gain=gain, out=out, eps=eps)
        assert rel(x, new) < 1e-6 and rel(out, O.rms(new, eps) * f64(gain)) < tol(dtype, 1e-6, 5e-3)
        rows = dev_i32([5, 0, 5])
        x, out3 = x0.clone(), torch.empty(3, W_, dtype=dtype, device=DEV)
        b.post_norm(x, y=yy, pair=pair, pair_weight=pw, pair_top=top, gain=gain, out=out3, rows=rows, eps=eps)
        assert torch.equal(x, x0) and torch.equal(out3, out[rows.long()])
    # without a gain: the stream itself as E, into a column block of a wider matrix
    both = torch.full((T, 2 * W_), 3.0, dtype=dtype, device=DEV)
    x = x0.clone()
    b.post_norm(x, y=y, out=both[:, W_:], ldo=2 * W_)
    assert torch.equal(both[:, W_:], x.to(dtype)) and bool((both[:, :W_] == 3.0).all()) and rel(x, f64(x0) + f64(y)) < 1e-7


def matmul32(x, w):
    return torch.matmul(x.float(), w.float().t().contiguous())


@pytest.mark.parametrize("M,N", [(2048, 2048), (2000, 2300), (1000, 3300), (300, 1100), (130, 80), (40, 200), (29, 264)])
@pytest.mark.parametrize("K", [8, 72, 200, 1032])
def test_many_row_projections_at_every_tile_shape_and_their_edges(M, N, K):
    """bf16 panels that travel to LDS by themselves: k ranges that end inside a stage (and before the ring is full), row and column counts
    that end inside a tile, grids that select each tile size; bias, an activation split inside a tile, gated units, rows gathered and
    scattered, the scaled accumulation."""
    b, bf = B(), torch.bfloat16
    x, w, w2 = (rnd(r, K, dtype=bf, seed=i, scale=K ** -0.25) for i, r in ((1, M), (2, N), (3, N)))
    bias, bias2 = rnd(N, dtype=bf, seed=4), rnd(N, dtype=bf, seed=5)
    z = matmul32(x, w) + bias.float()
    y32, y16 = torch.zeros(M, N, device=DEV), torch.zeros(M, N + 4, dtype=bf, device=DEV)
    b.linear(x, w, y32, M=M, bias=bias)
    assert rel(y32, z) < 2e-6
    cut = N // 2 + 3
    b.linear(x, w, y16, M=M, bias=bias, act=b.ACT_SILU, act_split=cut, act2=b.ACT_SIGMOID, ldy=N + 4)
    want = torch.cat([z[:, :cut] * torch.sigmoid(z[:, :cut]), torch.sigmoid(z[:, cut:])], dim=1)
    assert rel(y16[:, :N], want) < 4e-3 and float(y16[:, N:].float().abs().max()) == 0.0
    g = torch.zeros(M, N, dtype=bf, device=DEV)
    for act, f in ((b.ACT_NONE, torch.nn.functional.silu), (b.ACT_RELU, torch.relu), (b.ACT_GELU_TANH, lambda t: torch.nn.functional.gelu(t, approximate="tanh"))):
        b.linear(x, w, g, M=M, epilogue=b.EPI_SILU_MUL, w2=w2, bias=bias, bias2=bias2, act=act)
        assert rel(g, f(z) * (matmul32(x, w2) + bias2.float())) < 4e-3
    perm = torch.randperm(M, generator=torch.Generator().manual_seed(6)).to(torch.int32).to(DEV)
    y32.zero_()
    b.linear(x, w, y32, M=M, bias=bias, row_src=perm, row_dst=perm)
    assert rel(y32, z) < 2e-6
    base, cs = rnd(M, N, seed=7), rnd(N, seed=8)
    b.linear(x, w, y32, M=M, bias=bias, epilogue=b.EPI_SCALE_ADD, base=base, col_scale=cs)
    assert rel(y32, base + cs * z) < 2e-6


@pytest.mark.parametrize("K", [64, 136])
def test_many_row_projections_of_experts_and_split_destinations(K):
    """Groups of unequal sizes (one empty, one of a single row) in a launch that takes the large tiles, and the three-way split store."""
    b, bf, N = B(), torch.bfloat16, 264
    sizes = [300, 0, 1, 130, 513]
    M = sum(sizes)
    x, w = rnd(M, K, dtype=bf, seed=1), rnd(len(sizes), N, K, dtype=bf, seed=2, scale=K ** -0.5)
    off = dev_i32([0] + [sum(sizes[:i + 1]) for i in range(len(sizes))])
    src = torch.randperm(M, generator=torch.Generator().manual_seed(3))
    y = torch.zeros(M, N, device=DEV)
    b.linear(x, w, y, M=M, row_src=src.to(torch.int32).to(DEV), group_off=off, n_groups=len(sizes))
    want, at = [], 0
    for g, n in enumerate(sizes):
        want.append(matmul32(x[src.to(DEV)[at:at + n]], w[g]))
        at += n
    assert rel(y, torch.cat(want)) < 2e-6
    # columns: 100 to rows, 84 to a cache of 3 heads kept row by row, 80 to one kept column by column
    W1, R, cap = w[0], 500, 512
    y1, y2 = torch.zeros(R, 100, dtype=bf, device=DEV), torch.zeros(3, cap, 28, dtype=bf, device=DEV)
    y3 = torch.zeros(80, cap, dtype=bf, device=DEV)
    pos = torch.randperm(cap, generator=torch.Generator().manual_seed(4))[:R].to(DEV)
    b.linear(x, W1, y1, M=R, act=b.ACT_RELU2, split_n=100, y2=y2, row_off2=pos * 28, head_dim2=28, head_stride2=cap * 28, split_n3=184, y3=y3,
             row_off3=pos.clone(), col_stride3=cap)
    z = matmul32(x[:R], W1)
    assert rel(y1, torch.relu(z[:, :100]) ** 2) < 5e-3
    assert rel(y2[:, pos].permute(1, 0, 2).reshape(R, 84), z[:, 100:184]) < 5e-3 and rel(y3[:, pos].T, z[:, 184:]) < 5e-3


def test_router_scores_are_not_renormalised():
    b, T, n, top = B(), 9, 11, 4
    z = rnd(T, n, seed=3, scale=2.0)
    ex, wt = torch.zeros(T * top, dtype=torch.int32, device=DEV), torch.zeros(T * top, device=DEV)
    b.router_select(z, top, ex, wt, T, score_fn=b.SCORE_SOFTMAX, renorm=False)
    s = torch.softmax(f64(z), dim=-1)
    val, idx = torch.sort(s, dim=-1, descending=True, stable=True)
    assert ex.view(T, top).cpu().tolist() == idx[:, :top].tolist() and rel(wt.view(T, top), val[:, :top]) < 1e-6


# ---- attention of prompt rows -------------------------------------------------------------------------------------------------------------
def prompt_case(dtype, reqs, H, Hkv, D, R, Dv, scale, tile, *, window=0, sink=None, gated=False, seed=0, loud=None, table=True):
    """``reqs``: (new tokens, tokens before them) per request.  Keys and values of a request lie from a row of their own on, 32 rows apart at
    least; the shared key columns in rows the table points at, in another order.  ``loud`` (position, query column, value): edits before
    the launch.  -> (got [rows, H, Dv], want)."""
    b = B()
    T, base, tiles, row = sum(n for n, _ in reqs), 0, [], 0
    bases = []
    for n, before in reqs:
        bases.append(base)
        tiles += [(base, before + q, min(tile, n - q), row + q) for q in range(0, n, tile)]
        base += -(-(n + before) // 32) * 32
        row += n
    NK = Hkv * (D + Dv)
    q = rnd(T, H * (D + R), dtype=dtype, seed=seed + 1)
    kv = rnd(base, NK, dtype=dtype, seed=seed + 2)
    tail = rnd(base + 3, R + 5, dtype=dtype, seed=seed + 3) if R else None
    perm = torch.randperm(base, generator=torch.Generator().manual_seed(seed)) if table else torch.arange(base)
    gate = rnd(T, H + 2, dtype=dtype, seed=seed + 4).sigmoid() if gated else None
    if loud:
        loud(q, kv, tail, perm, bases)
    ldo = H * Dv + 7 if Dv % 2 else H * Dv + 8
    out = torch.full((T, ldo), float("nan"), dtype=dtype, device=DEV)
    b.attn_prompt(q, dev_i32(tiles), len(tiles), tile, kv, (NK, D), kv[:, Hkv * D:], (NK, Dv), H, Hkv, D + R, Dv, scale, out, ldo=ldo,
                  k_tail=tail[:, 5:] if R else None, tail_row_stride=R + 5, tail_rows=perm.to(torch.int32).to(DEV) if (R and table) else None,
                  tail_dim=R, window=window, sink=sink, gate=gate[:, 2:] if gated else None, ldg=H + 2)
    want, row = torch.zeros(T, H, Dv, dtype=F64), 0
    q6, kv6 = f64(q).view(T, H, D + R), f64(kv)
    for (n, before), ba in zip(reqs, bases):
        m = n + before
        for h in range(H):
            g = h // (H // Hkv)
            k = kv6[ba:ba + m, g * D:(g + 1) * D]
            if R:
                k = torch.cat([k, f64(tail)[perm[ba:ba + m], 5:]], dim=1)
            v = kv6[ba:ba + m, Hkv * D + g * Dv:Hkv * D + (g + 1) * Dv]
            for i in range(n):
                p = before + i
                lo = max(0, p - window + 1) if window else 0
                want[row + i, h] = O.attend(q6[row + i:row + i + 1, h], k[lo:p + 1], v[lo:p + 1], [p - lo], scale,
                                            f64(sink)[h] if sink is not None else None)[0]
        row += n
    if gated:
        want *= f64(gate)[:, 2:].unsqueeze(-1)
    assert bool(torch.isnan(out[:, H * Dv:].float()).all())
    return out[:, :H * Dv].reshape(T, H, Dv), want


TILES = [(torch.float32, 64), (torch.bfloat16, 64), (torch.bfloat16, 128)]


@pytest.mark.parametrize("dtype,tile", TILES)
@pytest.mark.parametrize("H,Hkv,D,R,Dv", [(2, 2, 24, 8, 40), (4, 2, 64, 0, 64), (3, 3, 40, 56, 104), (2, 2, 128, 64, 128), (1, 1, 144, 96, 200),
                                          (2, 2, 9, 6, 7), (2, 1, 10, 0, 5), (2, 2, 20, 12, 36)])
def test_prompt_attention_over_rebuilt_rows(dtype, tile, H, Hkv, D, R, Dv):
    """Several requests in one launch, from a fresh prompt of one token to portions that continue behind others; sinks and gates."""
    reqs = [(70, 0), (1, 0), (33, 95), (130, 3), (2, 31)]
    sink = rnd(H, seed=9, scale=2.0)
    got, want = prompt_case(dtype, reqs, H, Hkv, D, R, Dv, 2.0 * (D + R) ** -0.5, tile, sink=sink, gated=True)
    assert rel(got, want) < tol(dtype, 1e-5, 1e-2)


@pytest.mark.parametrize("dtype,tile", TILES)
@pytest.mark.parametrize("window", [1, 31, 64, 100])
def test_prompt_attention_windows_and_one_loud_key_at_their_edge(dtype, tile, window):
    """Every key is quiet but one whose score towers over the rest: queries up to window - 1 positions behind it return its value, the next
    one must not.  The shared columns carry the loudness of one head, the head's own columns that of the other."""
    loud = 40

    def make(q, kv, tail, perm, bases):
        q.mul_(0.05); kv[:, :2 * 16].mul_(0.05); tail.mul_(0.05)
        q.view(-1, 2, 24)[:, 0, 3] = 2.0                       # head 0 listens to its own column 3, head 1 to shared column 1
        q.view(-1, 2, 24)[:, 1, 17] = 2.0
        kv[bases[0] + loud, 3] = 30.0
        tail[perm[bases[0] + loud], 5 + 1] = 30.0
        kv[bases[0] + loud, 32:] = 5.0
    got, want = prompt_case(dtype, [(200, 0)], 2, 2, 16, 8, 12, 1.0, tile, window=window, loud=make)
    assert rel(got, want) < tol(dtype, 1e-5, 1e-2)
    for p in (loud, loud + window - 1):
        assert float((got[p].float() - 5.0).abs().max()) < 0.05, p
    if loud > 0:
        assert float((got[loud - 1].float() - 5.0).abs().min()) > 1.0
    assert float((got[loud + window].float() - 5.0).abs().min()) > 1.0


@pytest.mark.parametrize("dtype,tile", TILES)
@pytest.mark.parametrize("table", [True, False])
def test_prompt_attention_far_keys_at_block_borders_and_sinks(dtype, tile, table):
    """One loud key per query row group: the first key of the sequence, the last and first keys of key blocks (31, 32, 63, 64), the query's
    own; each query listens to one of them through a column of its own, among hundreds of quiet keys."""
    spots, n = [0, 1, 31, 32, 63, 64, 127, 128, 300], 420

    def make(q, kv, tail, perm, bases):
        q.mul_(0.02); kv[:, :16].mul_(0.02); tail.mul_(0.02)
        for i, s in enumerate(spots):
            kv[bases[0] + s, i] = 25.0
            kv[bases[0] + s, 16:] = float(i + 1)
        for r in range(q.shape[0]):
            q[r, (r * 7) % len(spots)] = 2.0
    got, want = prompt_case(dtype, [(n, 0)], 1, 1, 16, 4, 8, 1.0, tile, loud=make, table=table)
    assert rel(got, want) < tol(dtype, 1e-5, 1e-2)
    for r in range(301, n):
        i = (r * 7) % len(spots)
        assert float((got[r].float() - (i + 1)).abs().max()) < 0.05 * (i + 1), r
    # a sink that outweighs even the loud keys, and one that is nothing
    for val, check in ((80.0, lambda g: float(g[301:].float().abs().max()) < 1e-3), (-80.0, lambda g: rel(g, want) < tol(dtype, 1e-5, 1e-2))):
        g2, _ = prompt_case(dtype, [(n, 0)], 1, 1, 16, 4, 8, 1.0, tile, loud=make, table=table, sink=torch.tensor([val], device=DEV))
        assert check(g2)


# ---- attention of single rows over the latent -------------------------------------------------------------------------------------------------
def latent_case(dtype, rows, H, D, Dv, scale, *, window=0, sink=None, gated=False, splits=1, loud=None, seed=0):
    """``rows``: (slot, position) per query row; every slot's keys exist up to the largest position asked of it."""
    b = B()
    cap = 32 * (max(p for _, p in rows) // 32 + 1)
    cache = rnd(3, cap, D, dtype=dtype, seed=seed + 1)
    q = rnd(len(rows), H * D, dtype=dtype, seed=seed + 2)
    gate = rnd(len(rows), H + 3, dtype=dtype, seed=seed + 3).sigmoid() if gated else None
    if loud:
        loud(q, cache)
    for s in range(3):                                        # what lies behind the newest key need not be numbers
        top = max([p for s_, p in rows if s_ == s], default=-1)
        cache[s, top + 1:] = float("nan")
    out = torch.full((len(rows), H * Dv), float("nan"), dtype=dtype, device=DEV)
    part = torch.empty(b.attn_softmax_part(len(rows), H, splits, Dv), device=DEV) if splits > 1 else None
    tiles = dev_i32([(s, p, 1, r) for r, (s, p) in enumerate(rows)])
    b.attn_latent(q, tiles, len(rows), cache, cap * D, D, H, D, Dv, scale, out, window=window, sink=sink, gate=gate, ldg=H + 3, n_splits=splits,
                  part=part)
    want = torch.zeros(len(rows), H, Dv, dtype=F64)
    for r, (s, p) in enumerate(rows):
        lo = max(0, p - window + 1) if window else 0
        k = f64(cache[s, lo:p + 1])
        for h in range(H):
            want[r, h] = O.attend(f64(q[r:r + 1, h * D:(h + 1) * D]), k, k[:, :Dv], [p - lo], scale, f64(sink)[h] if sink is not None else None)[0]
    if gated:
        want *= f64(gate)[:, :H].unsqueeze(-1)
    return out.view(len(rows), H, Dv), want


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("splits", [1, 5, 64])
@pytest.mark.parametrize("H,D,Dv", [(3, 40, 24), (16, 112, 112), (20, 256, 192), (17, 330, 300), (2, 576, 512), (1, 700, 400), (5, 13, 9)])
def test_latent_attention_of_single_rows(dtype, splits, H, D, Dv):
    rows = [(0, 0), (1, 5), (0, 63), (2, 64), (0, 65), (1, 200), (2, 333)]
    sink = rnd(H, seed=4, scale=2.0)
    got, want = latent_case(dtype, rows, H, D, Dv, 2.0 * D ** -0.5, sink=sink, gated=True, splits=splits)
    assert rel(got, want) < tol(dtype, 1e-5, 1e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("splits", [1, 7])
@pytest.mark.parametrize("window", [0, 1, 32, 70])
def test_latent_attention_loud_keys_far_away_and_at_the_windows_edge(dtype, splits, window):
    H, D, Dv, loud = 18, 24, 16, 130

    def make(q, cache):
        q.mul_(0.05); cache.mul_(0.05)
        q.view(-1, H, D)[:, :, 20] = 2.0
        cache[:, loud, 20] = 30.0
        cache[:, loud, :Dv] = 5.0
    inside = loud + window - 1 if window else 900
    rows = [(0, loud), (1, inside), (2, loud - 1)] + ([(0, loud + window)] if window else [])
    got, want = latent_case(dtype, rows, H, D, Dv, 1.0, window=window, splits=splits, loud=make)
    assert rel(got, want) < tol(dtype, 1e-5, 1e-2)
    assert float((got[:2].float() - 5.0).abs().max()) < 0.05 and float((got[2:].float() - 5.0).abs().min()) > 1.0
    sink = torch.full((H,), -80.0, device=DEV)
    sink[3] = 90.0                                             # one head's sink outweighs even the loud key
    got, _ = latent_case(dtype, rows, H, D, Dv, 1.0, window=window, splits=splits, loud=make, sink=sink)
    assert float(got[:, 3].float().abs().max()) < 1e-3 and float((got[0, 4].float() - 5.0).abs().max()) < 0.05


# =====================================================================================================================================
# the model through its arena
# =====================================================================================================================================
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("folded", [False, True])
@pytest.mark.parametrize("name", list(SHAPES))
def test_whole_prompt_against_the_oracle_layer_by_layer(name, dtype, folded):
    """Both forms of the attention: keys and values rebuilt for the prompt, and queries folded into the latent's space."""
    s, w, m = model(name, dtype)
    tokens = toks(75, s.vocab_size, seed=3)
    want, want_streams = oracle(s, w, tokens)
    m.PROMPT_ROWS = 10 ** 9 if folded else 1
    try:
        ar = m.new_arena(1, 80)
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
    n = 70
    tokens = toks(n, s.vocab_size, seed=5)
    whole = run_alone(m, tokens)
    for cuts in ([1] * n, [2] * (n // 2), [33, 2, 2, 17, 16], [16, 16, 16, 22], [1, 69], [40] + [1] * 30, [15, 55], [64, 6]):
        assert close(run_alone(m, tokens, cuts), whole, dtype, 1e-5), cuts
    assert close(whole, oracle(s, w, tokens)[0], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("graphs", [True, False])
def test_unequal_batches_and_reused_slots(dtype, graphs):
    """Requests of different lengths step together -- prompts, short portions and decoded tokens side by side --, some end, newcomers take
    their slots (the previous owner's latents still lie there), the rest go on: every request's logits equal those it gets alone."""
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
        step({0: 1, 2: 1, 3: 1})                              # 3 arrives on 1's slot and ends at once
        step({2: 16, 4: 30, 0: 1})                            # 4 arrives on that slot again; 2 ends
        while any(at[k] < len(prompts[k]) for k in (0, 4)):
            step({k: 1 for k in (0, 4) if at[k] < len(prompts[k])})
        for k in prompts:
            assert close(torch.cat(got[k]), alone[k], dtype, 1e-5), k
    finally:
        m.use_graphs = True


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_through_graphs_and_a_growing_arena(dtype):
    """A short prompt, then 150 tokens one by one on an arena that starts too small: the planes move (captured steps are recaptured), and
    the decoded positions pass several borders of the kernel's key blocks."""
    s, w, m = model("mixed", dtype)
    tokens = toks(160, s.vocab_size, seed=9)
    ar = m.new_arena(1, 24)
    slot = ar.alloc()
    out = [m.forward_rows(ar, [slot], [tokens[:10]], [list(range(10))])]
    for t_ in tokens[10:]:
        out.append(m.forward_rows(ar, [slot], [[t_]], [[0]]))
    assert ar.cap >= 160
    assert close(torch.cat(out), oracle(s, w, tokens)[0], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_positions_in_a_long_prompt_and_after_it(dtype):
    """600 tokens with sharp scores: tiles deep in the sequence, a short portion far behind a long cache (which folds its queries although it
    brings many tokens), and decoded tokens after it."""
    from promptcache_amd.model.pikadra_hip import PikadraHIP
    s = PikadraShape(vocab_size=90, hidden_size=48, norm_eps=1e-6, embed_scale=6.9, loop_start=0, loop_stop=1, loop_times=2, logit_scale=1.4,
                     logit_softcap=11.0, layers=[mla(4, 16, 8, 8, 24, 20, sharp=5.0, ff_kind="dense", ff=32), mla(2, 24, 4, 16, 40, 12, sharp=5.0)])
    w = W.make_pikadra_weights(s, seed=4)
    m = PikadraHIP(s, w, device=DEV, dtype=dtype)
    tokens = toks(600, s.vocab_size, seed=2)
    want = oracle(s, w, tokens)[0]
    for ratio in (64, 8):
        m.REBUILD_RATIO = ratio
        ar = m.new_arena(1, 640)
        slot = ar.alloc()
        got = [m.forward_rows(ar, [slot], [tokens[:540]], [list(range(540))]), m.forward_rows(ar, [slot], [tokens[540:592]], [list(range(52))])]
        got += [m.forward_rows(ar, [slot], [[t_]], [[0]]) for t_ in tokens[592:]]
        assert close(torch.cat(got), want, dtype, 5e-5), ratio


@pytest.mark.parametrize("dtype", DTYPES)
def test_one_early_token_decides_far_logits(dtype):
    """Two prompts that differ in their second token only, through a layer with sharp scores: logits hundreds of positions later differ, and
    both agree with the oracle about it, in a prompt and decoded."""
    from promptcache_amd.model.pikadra_hip import PikadraHIP
    s = PikadraShape(vocab_size=40, hidden_size=32, norm_eps=1e-6, embed_scale=5.0, logit_scale=3.0, logit_softcap=25.0,
                     layers=[mla(2, 16, 0, 16, 24, 16, sharp=20.0, ff_kind="dense", ff=24)])
    w = W.make_pikadra_weights(s, seed=6)
    w["l0.mix.sink"].zero_()
    p6 = O.to_f64(w)
    rest = [t % 39 for t in toks(420, 40, seed=8)]
    m = PikadraHIP(s, w, device=DEV, dtype=dtype)
    a, b_ = [3, 39] + rest, [3, 5] + rest
    wa, wb = O.forward(s, p6, a)[-30:], O.forward(s, p6, b_)[-30:]
    gap = rel(wa, wb)
    ga, gb = run_alone(m, a)[-30:], run_alone(m, b_)[-30:]
    da = run_alone(m, a, [400] + [1] * 22)[-22:]
    assert gap > 1e-2
    if dtype == torch.float32:
        assert abs(rel(ga, gb) - gap) < 0.05 * gap + 1e-6
    assert close(ga, wa, dtype) and close(gb, wb, dtype) and close(da, wa[-22:], dtype)


@pytest.mark.parametrize("loop", [(0, 1, 1), (0, 3, 1), (2, 3, 4), (0, 3, 2), (1, 2, 3), None])
def test_loops_of_every_extent(loop):
    """float32, whole and decoded: a loop at the front, at the end, over everything, over one layer, run once, or none at all."""
    from promptcache_amd.model.pikadra_hip import PikadraHIP
    a, b_, n = loop or (0, 0, 0)
    s = PikadraShape(vocab_size=60, hidden_size=40, norm_eps=1e-5, embed_scale=4.4, loop_start=a, loop_stop=b_, loop_times=n, logit_scale=1.3,
                     logit_softcap=7.0, layers=[mla(2, 12, 4, 8, 16, 12, **DENSE), mla(3, 8, 8, 12, 24, 8, **BARE), mla(1, 16, 2, 10, 12, 20)])
    w = W.make_pikadra_weights(s, seed=13)
    m = PikadraHIP(s, w, device=DEV, dtype=torch.float32)
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
    from promptcache_amd.model import Pikadra
    s = shape_mixed()
    w = W.make_pikadra_weights(s, seed=11)
    lm = Pikadra(shape=s, weights=w, device=DEV, dtype=dtype)
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
                assert float(logits[k][best] - logits[k][tok]) < (1e-4 if dtype == torch.float32 else 0.3), (k, tok, best)


def random_shape(rng):
    """Sizes, layer order, loop and constants drawn at random."""
    width = rng.choice([64, 72, 96, 160, 200, 256])
    layers = []
    for _ in range(rng.randrange(1, 6)):
        kind = rng.choice(["", "dense", "moe", "moe"])
        ff = {}
        if kind == "dense":
            ff = dict(ff_kind="dense", ff=rng.choice([32, 56, 2 * width]))
        elif kind == "moe":
            n = rng.choice([1, 2, 5, 8, 16])
            ff = dict(ff_kind="moe", experts=n, top=rng.randrange(1, min(n, 4) + 1), expert_ff=rng.choice([16, 40, 64]), shared_ff=rng.choice([0, 24, 80]))
        layers.append(mla(rng.choice([1, 2, 4, 7, 12, 18]), rng.choice([8, 16, 32, 48, 96]), rng.choice([2, 4, 8, 32, 64]), rng.choice([8, 16, 40, 80]),
                          rng.choice([16, 40, 96, 200, 256]), rng.choice([12, 40, 112, 200]), sharp=rng.choice([1.0, 3.0]),
                          base=rng.choice([500.0, 10000.0, 1e6]), **ff))
    s = PikadraShape(vocab_size=rng.randrange(50, 900), hidden_size=width, norm_eps=rng.choice([1e-5, 1e-6]), embed_scale=rng.choice([1.0, 9.5]),
                     logit_scale=rng.choice([0.5, 1.0, 3.0]), logit_softcap=rng.choice([0.0, 8.0, 40.0]), layers=layers)
    if rng.random() < 0.75:
        s.loop_start = rng.randrange(len(layers))
        s.loop_stop = rng.randrange(s.loop_start + 1, len(layers) + 1)
        s.loop_times = rng.randrange(1, 4)
    return s


@pytest.mark.parametrize("seed", range(8))
def test_random_configurations_whole_decoded_and_in_company(seed):
    import random
    from promptcache_amd.model.pikadra_hip import PikadraHIP
    rng = random.Random(2000 + seed)
    s = PikadraShape.from_config(json.loads(json.dumps(random_shape(rng).to_config())))
    w = W.make_pikadra_weights(s, seed=seed)
    n = rng.randrange(90, 200)
    a, b_ = toks(n, s.vocab_size, seed), toks(rng.randrange(1, 70), s.vocab_size, seed + 1)
    want_a, want_b = oracle(s, w, a)[0], oracle(s, w, b_)[0]
    for dtype in DTYPES:
        m = PikadraHIP(s, w, device=DEV, dtype=dtype)
        assert close(run_alone(m, a), want_a, dtype, 5e-5, 4e-2), s.to_config()
        ar = m.new_arena(1, 16)
        sa, sb = ar.alloc(), ar.alloc()
        cut = n - 20
        out = [m.forward_rows(ar, [sb, sa], [b_, a[:cut]], [list(range(len(b_))), list(range(cut))])]
        out += [m.forward_rows(ar, [sa], [[t_]], [[0]]) for t_ in a[cut:]]
        got = torch.cat(out)
        assert close(got[len(b_):], want_a, dtype, 5e-5, 4e-2) and close(got[:len(b_)], want_b, dtype, 5e-5, 4e-2), s.to_config()


def test_single_request_engine_and_the_adapters_call():
    """GenerationEngine drives the model through the adapters' ``model(input_ids, past_key_values)`` call; a padded batch through
    that call gives each row its own logits."""
    from promptcache_amd import BatchEngine, GenerationEngine, GenerationParameters
    from promptcache_amd.model import Pikadra
    s = shape_mixed()
    w = W.make_pikadra_weights(s, seed=21)
    lm = Pikadra(shape=s, weights=w, device=DEV, dtype=torch.float32)
    assert lm.get_cache_shape() == (6, 1, 56)
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
    from promptcache_amd.model.pikadra_hip import PikadraHIP
    for bad in (mla(1, 8, 8, 8, 520, 8), mla(1, 8, 300, 8, 500, 8)):
        s = PikadraShape(vocab_size=20, hidden_size=16, norm_eps=1e-6, layers=[bad])
        with pytest.raises(ValueError):
            PikadraHIP(s, W.make_pikadra_weights(s), device=DEV)
    s = shape_odd()
    with pytest.raises(ValueError):
        PikadraHIP(s, W.make_pikadra_weights(s), device=DEV, dtype=torch.float16)


def test_checkpoint_directory_command_line_and_trace_runner(tmp_path):
    """config.json + model.safetensors written from a shape, found by the registry, and replayed by bin/trace_run in both formats."""
    import numpy as np
    from safetensors.torch import save_file
    from promptcache_amd.model import load_language_model
    s = shape_odd()
    w = W.make_pikadra_weights(s, seed=3)
    d = tmp_path / "ckpt"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(s.to_config()))
    save_file({k: v.contiguous() for k, v in w.items()}, str(d / "model.safetensors"))
    lm = load_language_model(str(d), dtype=torch.float32)
    assert type(lm).__name__ == "Pikadra" and lm.hf_model.config.to_config() == s.to_config()
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
