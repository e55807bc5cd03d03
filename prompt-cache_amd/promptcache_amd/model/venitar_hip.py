"""Venitar forward pass on MI355X (``config.VenitarShape`` says what the design is).

Like the other flat-row models this one keeps plain row-major tensors in one element type E -- bfloat16 (serving: matrix products on
the bf16 matrix cores, fp32 accumulation) or float32 (everything in true 32-bit) -- runs on the building blocks of
``libpromptcache_blocks.so`` (``_blocks.py``) and steps over FLAT rows: the new tokens of all requests of a step one after another,
each request continuing from what its slot of the ``SlotArena`` holds.  Nothing is padded, and a row reads nothing but its own slot, so
a request's numbers do not depend on the rest of the step.

A forward is a sequence of layer RUNS: layers before the loop, the loop's layers once per pass (the same weights, a cache and states of
the pass's own: the arena has an entry per run), layers after it.  The residual x is fp32; the embedding output x0 joins it again in the
residual step right before each pass but the first.  The turns of a step's rows (cosines and sines of position times frequency) are
tabled once per kind of rotation and serve every layer run.

    h = rms(x) w                                               pcb_post_norm, which also adds the sublayer (and x0) before it
    retention   q | k | v | silu(g) = ONE projection; the recurrence with rotated fp32 queries and keys (pcb_rec_prompt, or pcb_rec_step
                which goes on to the per-head norm and the gate); per-head unit RMS times the gate (pcb_gated_norm); W_o
    attention   q | k = ONE projection; pcb_head_prep: q, k normed and turned, k and the projected k itself (the values) into the slot's
                rows; softmax inside the query's own block with exp(0) more in the denominator (pcb_attn_prompt, or pcb_attn_rows
                for few rows); W_o
    parallel    ONE projection of h gives both halves' inputs: a | g (low ranks) | left q, k, v (biases) | right q, k, v | sigmoid(left g),
                and the step sizes as fp32 rows
                left:  pcb_head_prep, windowed softmax attention times the gate
                right: pcb_causal_conv (SiLU) over q | k | v; the second low-rank projections as ONE block-diagonal product (output gate in
                       E, decay pre-activations in fp32); the delta rule with unit queries and keys (pcb_rec_prompt / pcb_rec_step);
                       per-head norm and gate
                the halves' rows lie side by side, so that ONE projection [W_left | W_right] gives their sum: the right half's norm
                gain carries right_scale / left_scale, the residual step multiplies by left_scale
    ff          W_down relu(W_up h)^2, the square in the first projection's epilogue

and the logits are ``embed . rms(x) w`` for the rows that were asked for.
"""
from __future__ import annotations

import os
from typing import Dict, Optional, Sequence

import numpy as np
import torch

from .. import _blocks as B
from .config import VenitarShape
from .fivesun_hip import rotary_frequencies
from .kv_arena import SlotArena
from .slot_model import SlotKV, SlotModel, StepRows  # noqa: F401

CHUNK = 16      # tokens per chunk of the recurrences (pcb_rec_prompt)


class VenitarHIP(SlotModel):
    GRAPH_MAX_ROWS = 64
    PROMPT_ROWS = int(os.environ.get("PC_VT_PROMPT_ROWS", "16"))   # a request that brings fewer tokens than this attends row by row

    def __init__(self, shape: VenitarShape, weights: Dict[str, torch.Tensor], device="cuda:0", dtype=torch.bfloat16,
                 decode_headroom: int = 256):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Venitar runs in bfloat16 or float32")
        B.load()                                   # fail loudly (or build once) before anything else
        shape.check()
        self.config = shape
        self.device = torch.device(device)
        self.dtype = dtype
        self.decode_headroom = decode_headroom
        self.L = len(shape.layers)
        self.W, self.V = shape.hidden_size, shape.vocab_size
        if self.W > 16384:
            raise ValueError(f"width up to 16384 (got {self.W})")
        dev = self.device

        def e(name):                               # element-type tensor (projections, their biases, convolution taps)
            return weights[name].to(device=dev, dtype=dtype).contiguous()

        def f(name):                               # fp32 tensor (norm gains, decay rates)
            return weights[name].to(device=dev, dtype=torch.float32).contiguous()

        self._rots = []                            # distinct rotations: (base, dims, scaling), frequencies, factor on the turned pairs

        def rot(r):                                # index of a rotation, or -1
            if not r.dims:
                return -1
            if r.dims > 1024:
                raise ValueError(f"up to 1024 rotated columns per head (got {r.dims})")
            key = (r.base, r.dims, r.scaling)
            for i, (k, _, _) in enumerate(self._rots):
                if k == key:
                    return i
            fr, mag = rotary_frequencies(r.base, r.dims, *(r.scaling or ()))
            self._rots.append((key, torch.from_numpy(fr).to(dev), float(mag)))
            return len(self._rots) - 1

        def attention_limits(i, a):
            if a.dim > 256 or a.vdim > 256:
                raise ValueError(f"layer {i}: attention heads take up to 256 key and 256 value columns (got {a.dim} / {a.vdim})")

        self.embed = e("embed")
        self.final_gain = f("final.norm")
        self.layers = []
        for i, l in enumerate(shape.layers):
            p, m = f"l{i}.", f"l{i}.mix."
            ent = dict(cfg=l, norm1=f(p + "norm1"))
            if l.kind == "retention":
                if l.mix.dim > 256:
                    raise ValueError(f"layer {i}: recurrent heads take up to 256 key columns (got {l.mix.dim})")
                ent.update(w_in=torch.cat([e(m + "q"), e(m + "k"), e(m + "v"), e(m + "g")], dim=0).contiguous(), w_out=e(m + "o"), rot=rot(l.mix.rot),
                           decay=torch.tensor(l.mix.decay, dtype=torch.float32, device=dev), step_fits=B.rec_step_fits(l.mix.dim, l.mix.vdim))
            elif l.kind == "attention":
                attention_limits(i, l.mix)
                ent.update(w_in=torch.cat([e(m + "q"), e(m + "k")], dim=0).contiguous(), w_out=e(m + "o"), rot=rot(l.mix.rot), q_gain=f(m + "q.norm"),
                           k_gain=f(m + "k.norm"), sink=torch.zeros(l.mix.heads, dtype=torch.float32, device=dev))
            else:
                attention_limits(i, l.left)
                if l.right.dim > 256 or l.right.conv > 16:
                    raise ValueError(f"layer {i}: recurrent heads take up to 256 key columns and 16 taps (got {l.right.dim}, {l.right.conv})")
                ent.update(self._parallel_weights(l, m, e, f), rot=rot(l.left.rot), step_fits=B.rec_step_fits(l.right.dim, l.right.vdim))
            if l.ff:
                ent.update(norm2=f(p + "norm2"), up=e(p + "mlp.up"), down=e(p + "mlp.down"))
            self.layers.append(ent)
        self.runs = shape.runs()
        self._buf = {}
        self.default_arena: Optional[SlotArena] = None
        self.use_graphs = os.environ.get("PC_VT_GRAPHS", "1") != "0"      # one-token steps replay a captured hipGraph
        self._graphs = {}
        self.max_graphs = 16
        att = [l.mix if l.kind == "attention" else l.left for l in shape.layers if l.kind != "retention"]
        # cache offsets of a row: one table per distinct (key heads, columns of a cached row: key | value)
        self._sigs = sorted({(a.kv_heads, a.dim + a.vdim) for a in att})
        self._max_heads = max([a.heads for a in att], default=1)

    def _parallel_weights(self, l, m, e, f):
        a, b = l.left, l.right
        lp, rp = m + "left.", m + "right."
        ra, rg = e(rp + "a1"), e(rp + "g1")
        if (b.a_rank and ra.shape[0] != b.a_rank) or (b.g_rank and rg.shape[0] != b.g_rank):
            raise ValueError("the low-rank projections' tensors and the configuration disagree")
        # the projection of h: low ranks first, the gate's sigmoid columns last, then the step sizes, which leave it as fp32
        rows = [ra, rg, e(lp + "q"), e(lp + "k"), e(lp + "v"), e(rp + "q"), e(rp + "k"), e(rp + "v"), e(lp + "g"), e(rp + "b")]
        at = np.concatenate([[0], np.cumsum([t.shape[0] for t in rows])]).tolist()
        bias = torch.zeros(at[-1], dtype=self.dtype, device=self.device)
        for j, nm in ((2, "q.b"), (3, "k.b"), (4, "v.b")):
            bias[at[j]:at[j + 1]] = e(lp + nm)
        # the second low-rank projections, block-diagonal over [a | g]: output gate, then decay pre-activations
        HD, HV, na, ng = b.heads * b.dim, b.heads * b.vdim, ra.shape[0], rg.shape[0]
        low = torch.zeros((HV + HD, na + ng), dtype=self.dtype, device=self.device)
        low[:HV, na:] = e(rp + "g2")
        low[HV:, :na] = e(rp + "a2")
        low_b = torch.zeros(HV + HD, dtype=self.dtype, device=self.device)
        low_b[HV:] = e(rp + "dt_bias")
        y_scale = l.left_scale if l.left_scale != 0.0 else 1.0
        w_left = e(lp + "o") if l.left_scale != 0.0 else torch.zeros_like(e(lp + "o"))
        gain = (f(rp + "norm") * (l.right_scale / y_scale)).contiguous()
        return dict(w_in=torch.cat(rows, dim=0).contiguous(), b_in=bias, at=at, w_low=low, b_low=low_b, ranks=na + ng,
                    conv=torch.cat([e(rp + "q.conv"), e(rp + "k.conv"), e(rp + "v.conv")], dim=0).contiguous(),
                    rate=(-torch.exp(f(rp + "A_log"))).contiguous(), gain=gain, gain_rep=gain.repeat(b.heads).contiguous(), y_scale=y_scale,
                    w_out=torch.cat([w_left, e(rp + "o")], dim=1).contiguous())

    # ---- cache and state -------------------------------------------------------------------------------------------------------
    def new_arena(self, slots: int, cap: int) -> SlotArena:
        """Per layer run: rows ``key | value`` of the attention, the recurrences' fp32 matrices, the convolution's last inputs."""
        f32, dims, states = torch.float32, [], []
        for i, _ in self.runs:
            l = self.config.layers[i]
            a = l.mix if l.kind == "attention" else l.left
            dims.append((0, 0) if a is None else (a.kv_heads, a.dim + a.vdim))
            st = []
            if l.kind == "retention":
                st = [((l.mix.heads, l.mix.dim, l.mix.vdim), f32)]
            elif l.kind == "parallel":
                b = l.right
                st = [((b.heads, b.dim, b.vdim), f32)]
                if b.conv > 1:
                    st.append(((b.conv - 1, b.conv_channels), self.dtype))
            states.append(st)
        return SlotArena(dims, slots, cap, self.device, self.dtype, states=states)

    def kv_bytes_per_token(self) -> int:
        es = 2 if self.dtype == torch.bfloat16 else 4
        att = [(l.mix if l.kind == "attention" else l.left) for l in (self.config.layers[i] for i, _ in self.runs)]
        return sum(a.kv_heads * (a.dim + a.vdim) for a in att if a is not None) * es

    # ---- one step ------------------------------------------------------------------------------------------------------------
    @torch.inference_mode()
    def forward_rows(self, arena: SlotArena, slots: Sequence[int], tokens: Sequence[Sequence[int]],
                     want: Optional[Sequence[Sequence[int]]] = None, num_layers: Optional[int] = None,
                     return_streams: bool = False):
        """Append ``tokens[b]`` behind slot ``slots[b]`` for every b, and return fp32 logits ``[n_wanted, vocab]`` for the places
        ``want[b]`` (indices into ``tokens[b]``; default: each request's last token), in request order.  ``num_layers``: only that many
        layer runs.  ``return_streams``: also the residual stream after each layer run, fp32 ``[runs, rows, width]`` (for tests)."""
        dev = self.device
        if not tokens and not slots:
            return torch.empty((0, self.V), dtype=torch.float32, device=dev)
        st = StepRows(arena, slots, tokens, want, self.V)
        T, R, cap, row0 = st.T, st.R, arena.cap, st.row0
        single = all(c == 1 for c in st.counts)
        graphed = self.use_graphs and T <= self.GRAPH_MAX_ROWS and single and num_layers is None and not return_streams
        picked, want_rows = None, st.want_rows
        if graphed:
            if any(len(ws) != 1 for ws in st.want):
                picked = [b for b, ws in enumerate(st.want) for _ in ws]
            want_rows = np.arange(T, dtype=np.int32)
        # attention: tiles of neighbouring queries for requests that bring many tokens, single rows for the others
        big = [b for b, c in enumerate(st.counts) if c >= self.PROMPT_ROWS]
        tile = 64
        if self.dtype == torch.bfloat16 and sum(-(-st.counts[b] // 128) for b in big) * self._max_heads >= 512:
            tile = 128
        p_tiles = [(slots[b], st.starts[b] + q, min(tile, st.counts[b] - q), int(row0[b]) + q) for b in big for q in range(0, st.counts[b], tile)]
        p_tiles.sort(key=lambda t: t[1] + t[2])    # (longer contexts behind the shorter ones: the kernel starts from the last tile)
        small = [b for b, c in enumerate(st.counts) if c < self.PROMPT_ROWS]
        rows = np.concatenate([np.arange(row0[b], row0[b + 1]) for b in small]) if small else np.zeros(0, np.int64)
        s_tiles = np.stack([st.row_slot[rows], st.row_pos[rows], np.ones(rows.size, np.int64), rows], axis=1).astype(np.int32)
        reqs = np.asarray([(s, s0, c, int(row0[b])) for b, (s, s0, c) in enumerate(zip(slots, st.starts, st.counts))], dtype=np.int32)
        idx = np.arange(T, dtype=np.int64) - np.repeat(row0[:-1], st.counts)
        meta = np.stack([st.row_slot, st.row_pos, idx, np.zeros_like(idx)], axis=1).astype(np.int32)
        # the recurrences' chunks, request by request
        n_ch = np.asarray([-(-c // CHUNK) for c in st.counts], dtype=np.int64)
        chunk0 = np.concatenate([[0], np.cumsum(n_ch)])
        at = (np.arange(chunk0[-1]) - np.repeat(chunk0[:-1], n_ch)) * CHUNK
        left = np.repeat(np.asarray(st.counts, dtype=np.int64), n_ch) - at
        chunks = np.stack([np.repeat(row0[:-1], n_ch) + at, np.minimum(left, CHUNK), np.zeros_like(at), np.zeros_like(at)], axis=1).astype(np.int32)
        offs = np.stack([st.row_slot * (g * cap * d) + st.row_pos * d for g, d in self._sigs]) if self._sigs else np.zeros((0, T), np.int64)
        tables = dict(ids=st.ids, pos=st.row_pos.astype(np.int32), want=want_rows, p_tiles=np.asarray(p_tiles, dtype=np.int32).reshape(-1, 4),
                      s_tiles=s_tiles, reqs=reqs, meta=meta, chunks=chunks, chunk0=chunk0[:-1].astype(np.int32))
        sizes = {k: v.size for k, v in tables.items()}
        n32 = sum(sizes.values())
        o64 = (n32 * 4 + 7) // 8 * 8
        blob = np.empty(o64 + offs.size * 8 + 8, dtype=np.uint8)
        blob[:n32 * 4].view(np.int32)[:] = np.concatenate([v.reshape(-1) for v in tables.values()])
        blob[o64:o64 + offs.size * 8].view(np.int64)[:] = offs.reshape(-1)
        dims = dict(T=T, R=R, n_want=int(want_rows.size), n32=n32, o64=o64, sizes=sizes, tile=tile, single=single)
        res = self._decode_graphed(arena, blob, dims) if graphed else None
        if res is None:
            dblob = torch.from_numpy(blob).to(dev)
            logits = torch.empty((dims["n_want"], self.V), dtype=torch.float32, device=dev)
            res = self._run(arena, dblob, dims, logits, num_layers, return_streams)
        for s_, c in zip(slots, st.counts):
            arena.lengths[s_] += c
        if picked is not None:
            res = res[torch.as_tensor(picked, dtype=torch.long, device=dev)] if picked else res[:0]
        return res

    def _tables(self, dblob, d):
        i32 = dblob[:d["n32"] * 4].view(torch.int32)
        at, out = 0, dict(tile=d["tile"], single=d["single"], R=d["R"])
        for name, n in d["sizes"].items():
            out[name] = i32[at:at + n]
            at += n
        no = len(self._sigs)
        out["offs"] = dblob[d["o64"]:d["o64"] + no * d["T"] * 8].view(torch.int64).view(no, d["T"])
        return out

    def _run(self, arena, dblob, d, logits, num_layers=None, return_streams=False):
        """The device side of a step: every launch of the forward, reading the step's tables from ``dblob``."""
        E, f32 = self.dtype, torch.float32
        W, T = self.W, d["T"]
        tb = self._tables(dblob, d)
        runs = self.runs if num_layers is None else self.runs[:num_layers]
        cfg, eps = self.config, self.config.norm_eps
        x, h = self._mat("x", T, W, f32), self._mat("h", T, W, E)
        streams = torch.empty((len(runs), T, W), dtype=f32, device=self.device) if return_streams else None
        B.embed_scaled_rows(self.embed, tb["ids"], cfg.embed_scale, x)
        x0 = None
        if any(joins for _, joins in runs):
            x0 = self._mat("x0", T, W, f32)
            B.embed_scaled_rows(self.embed, tb["ids"], cfg.embed_scale, x0)
        tb["rots"] = []
        for i, (key, freqs, mag) in enumerate(self._rots):
            tb["rots"].append(self._mat(f"rot{i}", T, key[1], f32))
            B.rot_table(tb["pos"], freqs, mag, tb["rots"][-1], T)
        pending = {}                               # the sublayer result (and x0, before a pass) that is still to be added to x
        for r, (i, joins) in enumerate(runs):
            lw = self.layers[i]
            if joins:
                pending["add"] = x0
            B.post_norm(x, gain=lw["norm1"], out=h, eps=eps, n_rows=T, **pending)
            y = self._mat("y1", T, W, f32)
            pending = dict(y=y)
            kind = lw["cfg"].kind
            if kind == "retention":
                self._retention(arena, r, lw, h, y, tb, T)
            elif kind == "attention":
                self._attention(arena, r, lw, h, y, tb, T)
            else:
                self._parallel(arena, r, lw, h, y, tb, T)
                pending["y_scale"] = lw["y_scale"]
            if lw["cfg"].ff:
                B.post_norm(x, gain=lw["norm2"], out=h, eps=eps, n_rows=T, **pending)
                mid, y = self._mat("ff_mid", T, lw["cfg"].ff, E), self._mat("y2", T, W, f32)
                B.linear(h, lw["up"], mid, M=T, act=B.ACT_RELU2)
                B.linear(mid, lw["down"], y, M=T)
                pending = dict(y=y)
            if streams is not None:
                B.post_norm(x, n_rows=T, x_out=streams[r], **pending)
                pending = {}
        if d["n_want"]:
            nw = d["n_want"]
            hn = self._mat("hn", nw, W, E)
            B.post_norm(x, gain=self.final_gain, out=hn, eps=eps, rows=tb["want"], n_rows=nw, **pending)
            B.linear(hn, self.embed, logits, M=nw)
        return (logits, streams) if return_streams else logits

    # ---- recurrences -----------------------------------------------------------------------------------------------------------------
    def _recurrence(self, lw, tb, T, q, k, v, lds_, state, H, Hk, D, Dv, out, ldo, gain, gain_rep, gate, ldg, **kw):
        """The heads' normed and gated outputs in the columns of ``out`` (E, row stride ``ldo``)."""
        eps, R = self.config.norm_eps, tb["R"]
        if tb["single"] and lw["step_fits"]:
            B.rec_step(q, k, v, lds_, tb["reqs"], R, state, H, Hk, D, Dv, out, ldo, eps=eps, gain=gain, gate=gate, ldg=ldg, **kw)
            return
        n_ch = tb["chunks"].numel() // 4
        scratch = self._scratch("rec", B.rec_scratch(n_ch, H, D), torch.float32)
        o = self._mat("rec_o32", T, H * Dv, torch.float32)
        B.rec_prompt(q, k, v, lds_, tb["reqs"], R, tb["chunks"], tb["chunk0"], n_ch, state, H, Hk, D, Dv, scratch, o, **kw)
        B.gated_norm(o, gain_rep, gate, ldg, out, eps, T, group=Dv, ldo=ldo)

    def _rot(self, lw, tb):
        return (tb["rots"][lw["rot"]], self._rots[lw["rot"]][0][1]) if lw["rot"] >= 0 else (None, 0)

    def _retention(self, arena, r, lw, h, y, tb, T):
        m = lw["cfg"].mix
        H, D, Dv = m.heads, m.dim, m.vdim
        HD, HV = H * D, H * Dv
        N = 2 * HD + 2 * HV
        P = self._mat("mix_in", T, N, self.dtype)
        B.linear(h, lw["w_in"], P, M=T, act_split=2 * HD + HV, act2=B.ACT_SILU)
        table, dims = self._rot(lw, tb)
        A = self._mat("mix_out", T, HV, self.dtype)
        self._recurrence(lw, tb, T, P, P[:, HD:], P[:, 2 * HD:], (N, N, N), arena.states[r][0], H, H, D, Dv, A, HV, None, None, P[:, 2 * HD + HV:], N,
                         decay=lw["decay"], k_scale=D ** -0.5, rot=table, rot_dims=dims)
        B.linear(A, lw["w_out"], y, M=T)

    def _delta(self, arena, r, lw, P, N, bt, A, ldo, tb, T):
        """The right half of a parallel mixer: from the projected rows P (row stride N) and the step sizes bt into columns of A."""
        b, at, E = lw["cfg"].right, lw["at"], self.dtype
        H, G, D, Dv = b.heads, b.kv_heads, b.dim, b.vdim
        CC = b.conv_channels
        gate, za = self._mat("out_gate", T, H * Dv, E), self._mat("decay_in", T, H * D, torch.float32)
        B.linear(P, lw["w_low"], gate, M=T, bias=lw["b_low"], act=B.ACT_SIGMOID, ldx=N, split_n=H * Dv, y2=za, y2_f32=True, head_stride2=H * D)
        xc = self._mat("conv", T, CC, E)
        src = P[:, at[5]:]
        state = arena.states[r][1] if b.conv > 1 else self._mat("no_state", 1, CC, E)[:0].view(0, 0, CC)
        if tb["single"]:
            B.conv_step(src, N, lw["conv"], None, True, tb["reqs"], tb["R"], state, xc)
        else:
            B.causal_conv(src, N, lw["conv"], None, True, tb["meta"], state, xc, T)
            if b.conv > 1:
                B.conv_state_update(src, N, tb["reqs"], tb["R"], state)
        self._recurrence(lw, tb, T, xc, xc[:, G * D:], xc[:, 2 * G * D:], (CC, CC, CC), arena.states[r][0], H, G, D, Dv, A, ldo, lw["gain"],
                         lw["gain_rep"], gate, H * Dv, ld=za, ldld=H * D, ld_coef=lw["rate"], ld_softplus=True, beta=bt, ldbeta=H, unit_norm=True,
                         unit_eps=1e-6, q_scale=D ** -0.5)

    # ---- attention --------------------------------------------------------------------------------------------------------------------
    def _attend(self, arena, r, a, q, tb, out, ldo, **kw):
        """Softmax attention of the prepared query rows over the run's cached rows, into columns of ``out``."""
        H, G, D, Dv = a.heads, a.kv_heads, a.dim, a.vdim
        plane = arena.planes[r]
        values = plane.view(-1)[D:]
        ss, hs, rs = arena.slot_stride(r), arena.head_stride(r), D + Dv
        kw.update(window=a.window, block=a.block, ldo=ldo)
        n = tb["p_tiles"].numel() // 4
        if n:
            B.attn_prompt(q, tb["p_tiles"], n, tb["tile"], plane, (rs, hs, ss), values, (rs, hs, ss), H, G, D, Dv, a.scale, out,
                          gate_cols=kw.get("gate") is not None, **kw)
        n = tb["s_tiles"].numel() // 4
        if n:
            # few (row, key head) pairs cannot fill the chip: each is cut into runs of its keys, as many as the visible blocks of 64 allow
            reach = min(v for v in (arena.cap, a.window or arena.cap, a.block or arena.cap))
            splits = max(1, min(64, 512 // (n * G * -(-H // (16 * G))), -(-reach // 64)))
            splits = 1 if -(-reach // 64) <= 3 else splits
            part = self._scratch("attn_part", B.attn_softmax_part(n, H, splits, Dv), torch.float32) if splits > 1 else None
            B.attn_rows(q, tb["s_tiles"], n, plane, (ss, hs, rs), values, (ss, hs, rs), H, G, D, Dv, a.scale, out, n_splits=splits, part=part, **kw)

    def _attention(self, arena, r, lw, h, y, tb, T):
        E, a = self.dtype, lw["cfg"].mix
        H, G, D = a.heads, a.kv_heads, a.dim
        HD, N = H * D, (H + G) * D
        P = self._mat("mix_in", T, N, E)
        B.linear(h, lw["w_in"], P, M=T)
        table, dims = self._rot(lw, tb)
        q, plane = self._mat("q_rows", T, HD, E), arena.planes[r]
        row = dict(row_off=tb["offs"][self._sigs.index((G, 2 * D))], head_stride=arena.head_stride(r))
        segs = [B.head_seg(P, N, H, D, q, norm=True, gain=lw["q_gain"], rot_dims=dims, ld_dst=HD),
                B.head_seg(P[:, HD:], N, G, D, plane, norm=True, gain=lw["k_gain"], rot_dims=dims, **row),
                B.head_seg(P[:, HD:], N, G, D, plane, dst_offset=D, **row)]
        B.head_prep(segs, T, E, table=table, rot_half=True, eps=self.config.norm_eps)
        A = self._mat("mix_out", T, HD, E)
        self._attend(arena, r, a, q, tb, A, HD, sink=lw["sink"])
        B.linear(A, lw["w_out"], y, M=T)

    # ---- both side by side ---------------------------------------------------------------------------------------------------------------
    def _parallel(self, arena, r, lw, h, y, tb, T):
        """Leaves left + (right_scale / left_scale) right in y: the residual step multiplies by what is missing."""
        E, l, at = self.dtype, lw["cfg"], lw["at"]
        a, b = l.left, l.right
        H, G, D, Dv = a.heads, a.kv_heads, a.dim, a.vdim
        N = at[9]
        P, bt = self._mat("mix_in", T, N, E), self._mat("step_sizes", T, b.heads, torch.float32)
        B.linear(h, lw["w_in"], P, M=T, bias=lw["b_in"], act_split=at[8], act2=B.ACT_SIGMOID, split_n=N, y2=bt, y2_f32=True, head_stride2=b.heads)
        K_out = H * Dv + b.heads * b.vdim
        A = self._mat("mix_out", T, K_out, E)
        table, dims = self._rot(lw, tb)
        q, plane = self._mat("q_rows", T, H * D, E), arena.planes[r]
        row = dict(row_off=tb["offs"][self._sigs.index((G, D + Dv))], head_stride=arena.head_stride(r))
        segs = [B.head_seg(P[:, at[2]:], N, H, D, q, rot_dims=dims, ld_dst=H * D), B.head_seg(P[:, at[3]:], N, G, D, plane, rot_dims=dims, **row),
                B.head_seg(P[:, at[4]:], N, G, Dv, plane, dst_offset=D, **row)]
        B.head_prep(segs, T, E, table=table, rot_half=True)
        self._attend(arena, r, a, q, tb, A, K_out, gate=P[:, at[8]:], ldg=N)
        self._delta(arena, r, lw, P, N, bt, A[:, H * Dv:], K_out, tb, T)
        B.linear(A, lw["w_out"], y, M=T)
