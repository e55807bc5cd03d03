"""Plain, slow statement of the Venitar design in float64 torch on the CPU: one function per mechanism, written from the
equations and sharing nothing with the product path (``promptcache_amd/model/venitar_hip.py`` and its kernels).

Notation: n tokens of one sequence at positions pos0 .. pos0 + n - 1; ``p`` a dict of float64 tensors keyed like the checkpoint.
Attention walks an explicit list of visible keys per query; recurrences and convolutions are literal loops over tokens.  ``carry`` is
what a sequence leaves behind for its next tokens, one entry per layer RUN (a looped layer runs several times, each time with
memories of its own).
"""
from __future__ import annotations

import math

import torch

F = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def unit_length(x, eps=1e-6):
    return x / torch.sqrt(x.pow(2).sum(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


# ---- rotary positions ---------------------------------------------------------------------------------------------------------------
def plain_frequencies(base, dims):
    return [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]


def ramped_frequencies(base, dims, factor, original, fast, slow):
    """YaRN: pairs that turn more than ``fast`` times within ``original`` positions keep their frequency, those below ``slow`` turns are
    slowed by ``factor``, with a linear ramp over the pair index in between.  -> (frequencies, factor on cos and sin)."""
    def index_of(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(index_of(fast)), 0)
    hi = min(math.ceil(index_of(slow)), dims - 1)
    out = []
    for i, f in enumerate(plain_frequencies(base, dims)):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * r + f * (1.0 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, positions, rot):
    """x [n, heads, D]: columns i and i + dims/2 turn together by position * f_i; columns from ``dims`` on stay."""
    if not rot.dims:
        return x
    freqs, mag = (plain_frequencies(rot.base, rot.dims), 1.0) if not rot.scaling else ramped_frequencies(rot.base, rot.dims, *rot.scaling)
    out, half = x.clone(), rot.dims // 2
    for i, f in enumerate(freqs):
        a = (positions.to(F) * f).view(-1, 1)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = mag * (u * torch.cos(a) - v * torch.sin(a))
        out[..., i + half] = mag * (v * torch.cos(a) + u * torch.sin(a))
    return out


# ---- softmax attention -----------------------------------------------------------------------------------------------------------------
def visible(i, block=0, window=0):
    """Positions the query at position i sees."""
    return [j for j in range(i + 1) if (not block or i // block == j // block) and (not window or i - j < window)]


def attend(q, k, v, qpos, scale, block=0, window=0, sink=False):
    """One head: q [n, D] at positions qpos, k [m, D], v [m, Dv] at positions 0 .. m - 1.  ``sink``: one more exp(0) in the
    denominator."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F)
    for r, i in enumerate(qpos):
        js = visible(i, block, window)
        s = (k[js] @ q[r]) * scale
        top = max(float(s.max()), 0.0) if sink else float(s.max())
        e = torch.exp(s - top)
        out[r] = (e / (e.sum() + (math.exp(-top) if sink else 0.0))) @ v[js]
    return out


def heads_attend(q, k, v, pos, a, **kw):
    n, per = q.shape[0], a.heads // a.kv_heads
    out = torch.zeros(n, a.heads, v.shape[2], dtype=F)
    for h in range(a.heads):
        out[:, h] = attend(q[:, h], k[:, h // per], v[:, h // per], pos.tolist(), a.scale, **kw)
    return out


def join_past(past, *new):
    return new if past is None else tuple(torch.cat([o, x]) for o, x in zip(past, new))


def block_attention(h, p, pre, a, eps, pos0, past):
    """The ``attention`` mixer.  -> (result [n, W], (keys, values) so far)."""
    n = h.shape[0]
    pos = torch.arange(pos0, pos0 + n)
    q, k = (h @ p[pre + "q"].T).view(n, a.heads, a.dim), (h @ p[pre + "k"].T).view(n, a.kv_heads, a.dim)
    v = k
    q = rotate(unit_rms(q, eps) * p[pre + "q.norm"], pos, a.rot)
    k = rotate(unit_rms(k, eps) * p[pre + "k.norm"], pos, a.rot)
    past = join_past(past, k, v)
    out = heads_attend(q, past[0], past[1], pos, a, block=a.block, sink=True)
    return out.reshape(n, -1) @ p[pre + "o"].T, past


def gated_window_attention(h, p, pre, a, eps, pos0, past):
    """The left half of a ``parallel`` mixer."""
    n = h.shape[0]
    pos = torch.arange(pos0, pos0 + n)
    q, k, v = ((h @ p[pre + t].T + p[pre + t + ".b"]) for t in ("q", "k", "v"))
    q = rotate(q.view(n, a.heads, a.dim), pos, a.rot)
    k = rotate(k.view(n, a.kv_heads, a.dim), pos, a.rot)
    past = join_past(past, k, v.view(n, a.kv_heads, a.vdim))
    out = heads_attend(q, past[0], past[1], pos, a, window=a.window)
    return (out.reshape(n, -1) * torch.sigmoid(h @ p[pre + "g"].T)) @ p[pre + "o"].T, past


# ---- recurrences ------------------------------------------------------------------------------------------------------------------------
def retain(q, k, v, decay, S):
    """One head: S <- decay S + k v^T, o = S^T q, token by token.  -> (o [n, Dv], S)."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F)
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out, S


def retention(h, p, pre, m, eps, pos0, S):
    """-> (result [n, W], states [heads, dim, vdim])."""
    n = h.shape[0]
    pos = torch.arange(pos0, pos0 + n)
    q = rotate((h @ p[pre + "q"].T).view(n, m.heads, m.dim), pos, m.rot)
    k = rotate((h @ p[pre + "k"].T).view(n, m.heads, m.dim), pos, m.rot) * m.dim ** -0.5
    v = (h @ p[pre + "v"].T).view(n, m.heads, m.vdim)
    S = torch.zeros(m.heads, m.dim, m.vdim, dtype=F) if S is None else S.clone()
    out = torch.zeros(n, m.heads, m.vdim, dtype=F)
    for hd in range(m.heads):
        out[:, hd], S[hd] = retain(q[:, hd], k[:, hd], v[:, hd], m.decay[hd], S[hd])
    out = unit_rms(out, eps).reshape(n, -1) * silu(h @ p[pre + "g"].T)
    return out @ p[pre + "o"].T, S


def short_convolution(x, w, past):
    """x [n, C], w [C, taps] (last column: the current token), past [taps - 1, C] or None (zeros).  -> (out [n, C], last inputs)."""
    taps = w.shape[1]
    if past is None:
        past = torch.zeros(taps - 1, x.shape[1], dtype=F)
    full = torch.cat([past, x])
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            out[t] += w[:, j] * full[t + j]
    return out, full[full.shape[0] - (taps - 1):]


def delta_rule(q, k, v, beta, g, S):
    """One head: forget (g [n, dim] scales the state's rows), correct what the key reads towards the value, then read.
    -> (o [n, Dv], S)."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F)
    for t in range(q.shape[0]):
        S = g[t].unsqueeze(1) * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out, S


def log_decays(h, p, pre, b):
    """-e^A softplus(low-rank projection + bias), [n, heads, dim]."""
    z = (h @ p[pre + "a1"].T) @ p[pre + "a2"].T + p[pre + "dt_bias"]
    return -torch.exp(p[pre + "A_log"]).view(1, -1, 1) * torch.nn.functional.softplus(z, threshold=1e9).view(-1, b.heads, b.dim)


def gated_delta(h, p, pre, b, eps, past):
    """The right half of a ``parallel`` mixer.  -> (result [n, W], (three convolutions' last inputs, states))."""
    n, per = h.shape[0], b.heads // b.kv_heads
    convs, S = past if past is not None else ((None,) * 3, torch.zeros(b.heads, b.dim, b.vdim, dtype=F))
    qkv, left = [], []
    for t, old in zip(("q", "k", "v"), convs):
        y, keep = short_convolution(h @ p[pre + t].T, p[pre + t + ".conv"], old)
        qkv.append(silu(y))
        left.append(keep)
    q = unit_length(qkv[0].view(n, b.kv_heads, b.dim)) * b.dim ** -0.5
    k = unit_length(qkv[1].view(n, b.kv_heads, b.dim))
    v = qkv[2].view(n, b.heads, b.vdim)
    beta = torch.sigmoid(h @ p[pre + "b"].T)
    g = torch.exp(log_decays(h, p, pre, b))
    S = S.clone()
    out = torch.zeros(n, b.heads, b.vdim, dtype=F)
    for hd in range(b.heads):
        out[:, hd], S[hd] = delta_rule(q[:, hd // per], k[:, hd // per], v[:, hd], beta[:, hd], g[:, hd], S[hd])
    gate = torch.sigmoid((h @ p[pre + "g1"].T) @ p[pre + "g2"].T)
    out = (unit_rms(out, eps) * p[pre + "norm"]).reshape(n, -1) * gate
    return out @ p[pre + "o"].T, (tuple(left), S)


def mixer(h, p, pre, lay, eps, pos0, past):
    if lay.kind == "retention":
        return retention(h, p, pre, lay.mix, eps, pos0, past)
    if lay.kind == "attention":
        return block_attention(h, p, pre, lay.mix, eps, pos0, past)
    past = (None, None) if past is None else past
    yl, pl = gated_window_attention(h, p, pre + "left.", lay.left, eps, pos0, past[0])
    yr, pr = gated_delta(h, p, pre + "right.", lay.right, eps, past[1])
    return lay.left_scale * yl + lay.right_scale * yr, (pl, pr)


# ---- the stack ----------------------------------------------------------------------------------------------------------------------------
def feed_forward(h, p, pre):
    return torch.relu(h @ p[pre + "up"].T).pow(2) @ p[pre + "down"].T


def layer_runs(cfg):
    """The order in which layers run: (layer, whether the embedding output is added to the stream right before)."""
    n = len(cfg.layers)
    if not cfg.loop_times:
        return [(i, False) for i in range(n)]
    runs = [(i, False) for i in range(cfg.loop_start)]
    for t in range(cfg.loop_times):
        for i in range(cfg.loop_start, cfg.loop_stop):
            runs.append((i, i == cfg.loop_start and t >= 1))
    return runs + [(i, False) for i in range(cfg.loop_stop, n)]


def layer(x, p, i, lay, eps, pos0, past):
    y, past = mixer(unit_rms(x, eps) * p[f"l{i}.norm1"], p, f"l{i}.mix.", lay, eps, pos0, past)
    x = x + y
    if lay.ff:
        x = x + feed_forward(unit_rms(x, eps) * p[f"l{i}.norm2"], p, f"l{i}.mlp.")
    return x, past


def forward(cfg, p, tokens, pos0=0, carry=None, return_streams=False):
    """Logits [n, vocab] of ``tokens`` at positions pos0 .. ; ``carry`` (a list with one entry per layer run, updated in place) holds
    what earlier calls left.  ``return_streams``: also the residual stream after every layer run [runs, n, width]."""
    runs = layer_runs(cfg)
    carry = [None] * len(runs) if carry is None else carry
    x0 = p["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg.embed_scale
    x, streams = x0, []
    for r, (i, joins) in enumerate(runs):
        if joins:
            x = x + x0
        x, carry[r] = layer(x, p, i, cfg.layers[i], cfg.norm_eps, pos0, carry[r])
        streams.append(x)
    logits = (unit_rms(x, cfg.norm_eps) * p["final.norm"]) @ p["embed"].T
    return (logits, torch.stack(streams)) if return_streams else logits


def forward_in_portions(cfg, p, tokens, cuts):
    """The same sequence fed in portions of the given sizes, each continuing from what the ones before left."""
    carry, out, at = [None] * len(layer_runs(cfg)), [], 0
    for c in cuts:
        out.append(forward(cfg, p, tokens[at:at + c], pos0=at, carry=carry))
        at += c
    return torch.cat(out)


def to_f64(weights):
    return {k: v.to(F) for k, v in weights.items()}
