"""Plain, slow statement of the Pikadra design in float64 torch on the CPU: one function per mechanism, written from the
equations and sharing nothing with the product path (``promptcache_amd/model/pikadra_hip.py`` and its kernels).

Notation: n tokens of one sequence at positions pos0 .. pos0 + n - 1; ``p`` a dict of float64 tensors keyed like the checkpoint;
``lay`` a ``config.PikadraLayer``.  Attention rebuilds every head's keys and values from the latents and walks an explicit list of
visible keys; experts are applied token by token.  ``carry`` is what a sequence leaves behind for its next tokens: per layer RUN
(a looped layer runs several times, each time with a memory of its own) the latents and rotated key parts so far.
"""
from __future__ import annotations

import torch

F = torch.float64


def rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def zero_centred_norm(x, w, eps):
    """Unit RMS times (1 + w): a gain stored as its distance from one."""
    return rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


# ---- rotary positions ---------------------------------------------------------------------------------------------------------------
def rotate_halves(x, positions, base, dims):
    """x [n, ..., D]: column i turns with column i + dims/2 (i < dims/2) by position * base^(-2i/dims); columns from ``dims`` on stay."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        a = positions.to(F) * (float(base) ** (-2.0 * i / dims))
        a = a.view(-1, *([1] * (x.dim() - 2)))
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


# ---- attention ------------------------------------------------------------------------------------------------------------------------
def attend(q, k, v, qpos, scale, sink=None):
    """One head.  q [n, D] at positions qpos; k [m, D], v [m, Dv] at positions 0 .. m-1; every key at or before the query is seen.
    ``sink``: the denominator has one more term exp(sink)."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F)
    for r, i in enumerate(qpos):
        s = (k[:i + 1] @ q[r]) * scale
        top = s.max() if sink is None else torch.maximum(s.max(), sink)
        e = torch.exp(s - top)
        den = e.sum() if sink is None else e.sum() + torch.exp(sink - top)
        out[r] = (e / den) @ v[:i + 1]
    return out


def latent_attention(h, p, pre, lay, eps, pos0, past):
    """-> (result [n, W], (latents, rotated key parts) so far)."""
    n = h.shape[0]
    H, D, R, Dv, C = lay.heads, lay.dim, lay.rot_dim, lay.vdim, lay.kv_rank
    pos = torch.arange(pos0, pos0 + n)
    c_q = rms(h @ p[pre + "dq"].T, eps) * p[pre + "dq.norm"]
    q = (c_q @ p[pre + "uq"].T).view(n, H, D + R)
    down = h @ p[pre + "dkv"].T
    c = rms(down[:, :C], eps) * p[pre + "dkv.norm"]
    kr = rotate_halves(down[:, C:], pos, lay.rot_base, lay.rot_dims)
    if past is not None:
        c, kr = torch.cat([past[0], c]), torch.cat([past[1], kr])
    k = (c @ p[pre + "uk"].T).view(-1, H, D)
    v = (c @ p[pre + "uv"].T).view(-1, H, Dv)
    gate = torch.sigmoid(h @ p[pre + "g"].T)
    out = torch.zeros(n, H, Dv, dtype=F)
    for hd in range(H):
        qh = torch.cat([q[:, hd, :D], rotate_halves(q[:, hd, D:], pos, lay.rot_base, lay.rot_dims)], dim=1)
        kh = torch.cat([k[:, hd], kr], dim=1)
        out[:, hd] = attend(qh, kh, v[:, hd], pos.tolist(), lay.scale, p[pre + "sink"][hd]) * gate[:, hd:hd + 1]
    return out.reshape(n, H * Dv) @ p[pre + "o"].T, (c, kr)


# ---- feed-forwards ----------------------------------------------------------------------------------------------------------------------
def gated_unit(h, p, pre):
    return (silu(h @ p[pre + "gate"].T) * (h @ p[pre + "up"].T)) @ p[pre + "down"].T


def route(h, p, pre, top):
    """Per token the ``top`` outputs with the largest softmax scores, and those scores as they are."""
    s = torch.softmax(h @ p[pre + "router"].T, dim=-1)
    val, idx = torch.sort(s, dim=-1, descending=True, stable=True)
    return idx[:, :top], val[:, :top]


def mixture(h, p, pre, lay):
    idx, w = route(h, p, pre, lay.top)
    out = torch.zeros(h.shape[0], h.shape[1], dtype=F)
    for t in range(h.shape[0]):
        for k in range(lay.top):
            out[t] += w[t, k] * gated_unit(h[t:t + 1], p, f"{pre}e{int(idx[t, k])}.")[0]
    if lay.shared_ff:
        out = out + torch.sigmoid(h @ p[pre + "shared.sg"].T) * gated_unit(h, p, pre + "shared.")
    return out


def feed_forward(h, p, pre, lay):
    return gated_unit(h, p, pre) if lay.ff_kind == "dense" else mixture(h, p, pre, lay)


# ---- the stack ----------------------------------------------------------------------------------------------------------------------------
def layer_runs(cfg):
    """The order in which layers run: (layer, number of the pass that starts right before it, or -1)."""
    n = len(cfg.layers)
    if not cfg.loop_times:
        return [(i, -1) for i in range(n)]
    body = list(range(cfg.loop_start, cfg.loop_stop))
    runs = [(i, -1) for i in range(cfg.loop_start)]
    for t in range(cfg.loop_times):
        runs += [(i, t if i == cfg.loop_start else -1) for i in body]
    return runs + [(i, -1) for i in range(cfg.loop_stop, n)]


def parallel_layer(x, p, i, lay, eps, pos0, past):
    """x + (mixer(h) + feed-forward(h)), both reading h = norm(x).  -> (x, what the mixer leaves for the next tokens)."""
    h = zero_centred_norm(x, p[f"l{i}.norm1"], eps)
    y, past = latent_attention(h, p, f"l{i}.mix.", lay, eps, pos0, past)
    if lay.ff_kind:
        y = y + feed_forward(h, p, f"l{i}.mlp.", lay)
    return x + y, past


def enter_pass(x, x0, p, t):
    """What happens to the stream right before pass ``t`` of the loop: W [x; x0] + step_t."""
    return torch.cat([x, x0], dim=-1) @ p["loop.in"].T + p["loop.step"][t]


def output_logits(x, p, cfg):
    z = (zero_centred_norm(x, p["final.norm"], cfg.norm_eps) @ p["embed"].T) * cfg.logit_scale
    return cfg.logit_softcap * torch.tanh(z / cfg.logit_softcap) if cfg.logit_softcap else z


def forward(cfg, p, tokens, pos0=0, carry=None, return_streams=False):
    """Logits [n, vocab] of ``tokens`` at positions pos0 .. ; ``carry`` (a list with one entry per layer run, updated in place) holds
    what earlier calls left.  ``return_streams``: also the residual stream after every layer run [runs, n, width]."""
    runs = layer_runs(cfg)
    carry = [None] * len(runs) if carry is None else carry
    x0 = p["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg.embed_scale
    x, streams = x0, []
    for r, (i, starts) in enumerate(runs):
        if starts >= 0:
            x = enter_pass(x, x0, p, starts)
        x, carry[r] = parallel_layer(x, p, i, cfg.layers[i], cfg.norm_eps, pos0, carry[r])
        streams.append(x)
    logits = output_logits(x, p, cfg)
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
