"""Pikadra forward pass on MI355X (``config.PikadraShape`` says what the design is).

Like the other flat-row models this one keeps plain row-major tensors in one element type E -- bfloat16 (serving: matrix products on
the bf16 matrix cores, fp32 accumulation) or float32 (everything in true 32-bit) -- runs on the building blocks of
``libpromptcache_blocks.so`` (``_blocks.py``) and steps over FLAT rows: the new tokens of all requests of a step one after another,
each request continuing from what its slot of the ``SlotArena`` holds.  Nothing is padded, and a row reads nothing but its own slot, so
a request's numbers do not depend on the rest of the step.

A forward is a sequence of layer RUNS: layers before the loop, the loop's layers once per pass (the same weights, a cache of the
pass's own: the arena has one plane per run, whose rows are ``latent | rotated key part``), layers after it.  The residual x is fp32;
right before each pass x <- W_in [x; x0] + step_t, x0 being the embedding output (``pcb_post_norm`` leaves x as E beside x0 in one row
matrix, one projection reads it and adds the pass's vector as its bias).

One layer (parallel: one norm feeds both halves, both results join x together):

    h = rms(x) (1 + w)                                         pcb_post_norm, which also adds the layer before
    c_q | latent | key part | gates | shared gate | router     ONE projection of h: sigmoid on the gates, the router's logits to fp32
    c_q, latent normed; key part turned; latent | key part     pcb_head_prep (rotation in halves), the latter into the slot's row
    q = W_uq c_q, its rotated parts turned                     pcb_linear, pcb_head_prep
    attention, per request one of two forms of the same sum
      prompts   keys and values of every head rebuilt from the cached latents (one projection over all of the request's rows),
                pcb_attn_prompt over them, the rotated key part shared by the heads and read from the cache
      few rows  the keys' up-projection folded into the query (q' = W_uk^T q per head), pcb_attn_latent over the cached rows themselves
                with the latent as value, the values' up-projection after it
      exp(sink_h) in the denominator, one sigmoid gate per head on the result
    dense unit / shared expert                                 silu(W_gate h) * (W_up h) (times the token's gate) right beside the heads'
                                                               outputs, so that ONE projection [W_o | W_down] gives their sum
    experts                                                    softmax scores, top-k, buckets, grouped projections; the weighted sum of
                                                               a token's experts joins x in the next layer's pcb_post_norm

and the logits are ``cap tanh(embed . rms(x) (1 + w) scale / cap)`` for the rows that were asked for (the scale rides on the norm's
fp32 gain).
"""
from __future__ import annotations

import os
from typing import Dict, Optional, Sequence

import numpy as np
import torch

from .. import _blocks as B
from .config import PikadraShape
from .fivesun_hip import rotary_frequencies
from .kv_arena import SlotArena
from .slot_model import SlotKV, SlotModel, StepRows  # noqa: F401


class PikadraHIP(SlotModel):
    GRAPH_MAX_ROWS = 64
    PROMPT_ROWS = int(os.environ.get("PC_PK_PROMPT_ROWS", "16"))   # a request that brings fewer tokens than this folds its queries
    REBUILD_RATIO = 64      # ... and so does one that brings less than a 64th of what its slot then holds

    def __init__(self, shape: PikadraShape, weights: Dict[str, torch.Tensor], device="cuda:0", dtype=torch.bfloat16,
                 decode_headroom: int = 256):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Pikadra runs in bfloat16 or float32")
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

        def e(name):                               # element-type tensor (projections, tables)
            return weights[name].to(device=dev, dtype=dtype).contiguous()

        def f(name):                               # fp32 tensor (norm gains, sinks)
            return weights[name].to(device=dev, dtype=torch.float32).contiguous()

        self.embed = e("embed")
        self.final_gain = ((1.0 + f("final.norm")) * shape.logit_scale).contiguous()
        if shape.loop_times:
            self.loop_in, self.loop_step = e("loop.in"), e("loop.step")
        self.layers = []
        for i, l in enumerate(shape.layers):
            p, m, q = f"l{i}.", f"l{i}.mix.", f"l{i}.mlp."
            C, R, H = l.kv_rank, l.rot_dim, l.heads
            if C > 512 or C + R > 768:
                raise ValueError(f"layer {i}: a latent of up to 512 columns and, with its rotated part, 768 (got {C} + {R})")
            if max(l.q_rank, C, R, l.dim) > 16384 or R > 1024:
                raise ValueError(f"layer {i}: query latents of up to 16384 columns, rotated parts of up to 1024")
            if l.ff_kind == "moe" and (l.experts > 2048 or l.top > 64):
                raise ValueError(f"layer {i}: up to 2048 experts, of which a token uses up to 64")
            fr, _ = rotary_frequencies(l.rot_base, l.rot_dims) if l.rot_dims else (np.zeros(0), 1.0)
            rows = [e(m + "dq"), e(m + "dkv"), e(m + "g")]
            if l.shared_ff:
                rows.append(e(q + "shared.sg"))
            ent = dict(cfg=l, gain=(1.0 + f(p + "norm1")).contiguous(), act_from=l.q_rank + C + R, n_in=sum(t.shape[0] for t in rows),
                       q_gain=f(m + "dq.norm"), c_gain=f(m + "dkv.norm"), uq=e(m + "uq"), sink=f(m + "sink"),
                       freqs=torch.from_numpy(fr).to(dev) if l.rot_dims else None,
                       # per head: the key up-projection transposed ([C, dim]: it maps a query to the latent's columns) and the value
                       # up-projection as stored ([vdim, C]); and both as they are, one below the other, for rebuilt rows
                       w_abs=e(m + "uk").view(H, l.dim, C).transpose(1, 2).contiguous(), w_uv=e(m + "uv").view(H, l.vdim, C),
                       w_kv=torch.cat([e(m + "uk"), e(m + "uv")], dim=0).contiguous(),
                       prompts=l.dim + R <= 256 and l.vdim <= 256)
            if l.ff_kind == "moe":
                rows.append(e(q + "router"))
                ent.update(e_gate=torch.stack([e(q + f"e{j}.gate") for j in range(l.experts)]).contiguous(),
                           e_up=torch.stack([e(q + f"e{j}.up") for j in range(l.experts)]).contiguous(),
                           e_down=torch.stack([e(q + f"e{j}.down") for j in range(l.experts)]).contiguous())
            ent["w_in"] = torch.cat(rows, dim=0).contiguous()
            unit = q if l.ff_kind == "dense" else (q + "shared." if l.shared_ff else None)
            out = [e(m + "o")]
            if unit:
                ent.update(gate=e(unit + "gate"), up=e(unit + "up"))
                out.append(e(unit + "down"))
            ent["w_out"] = torch.cat(out, dim=1).contiguous()
            self.layers.append(ent)
        self.runs = shape.runs()
        self._buf = {}
        self.default_arena: Optional[SlotArena] = None
        self.use_graphs = os.environ.get("PC_PK_GRAPHS", "1") != "0"      # one-token steps replay a captured hipGraph
        self._graphs = {}
        self.max_graphs = 16
        # cache offsets of a row: one table per distinct row size of the planes
        self._sigs = sorted({l.kv_rank + l.rot_dim for l in shape.layers})
        self._prompts = any(ent["prompts"] for ent in self.layers)

    # ---- cache -----------------------------------------------------------------------------------------------------------------
    def new_arena(self, slots: int, cap: int) -> SlotArena:
        ls = [self.config.layers[i] for i, _ in self.runs]
        return SlotArena([(1, l.kv_rank + l.rot_dim) for l in ls], slots, cap, self.device, self.dtype)

    def kv_bytes_per_token(self) -> int:
        es = 2 if self.dtype == torch.bfloat16 else 4
        return sum(self.config.layers[i].kv_rank + self.config.layers[i].rot_dim for i, _ in self.runs) * es

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
        T, cap = st.T, arena.cap
        graphed = (self.use_graphs and T <= self.GRAPH_MAX_ROWS and all(c == 1 for c in st.counts) and num_layers is None
                   and not return_streams)
        picked = None
        want_rows = st.want_rows
        if graphed:
            if any(len(ws) != 1 for ws in st.want):
                picked = [b for b, ws in enumerate(st.want) for _ in ws]
            want_rows = np.arange(T, dtype=np.int32)
        # which requests rebuild keys and values (prompts), and which fold their queries into the latent's space
        big = [b for b, (s0, c) in enumerate(zip(st.starts, st.counts))
               if self._prompts and c >= self.PROMPT_ROWS and s0 + c <= self.REBUILD_RATIO * c]
        small = sorted(set(range(st.R)) - set(big))
        row0 = st.row0
        pad = lambda n: -(-n // 32) * 32
        heads = max(l.heads for l in self.config.layers)
        tile = 64
        if self.dtype == torch.bfloat16 and sum(-(-st.counts[b] // 128) for b in big) * heads >= 512:
            tile = 128
        kv_rows, p_tiles, base = [], [], 0
        for b in big:
            n = st.starts[b] + st.counts[b]
            src = slots[b] * cap + np.minimum(np.arange(pad(n), dtype=np.int64), n - 1)     # (the padding repeats the last row)
            kv_rows.append(src.astype(np.int32))
            p_tiles += [(base, st.starts[b] + q, min(tile, st.counts[b] - q), int(row0[b]) + q) for q in range(0, st.counts[b], tile)]
            base += pad(n)
        # (longer contexts behind the shorter ones: the kernel starts from the last tile)
        p_tiles.sort(key=lambda t: t[1] + t[2])
        if big and arena.slots * cap >= 1 << 31:
            raise ValueError("more than 2^31 cached rows in one plane")
        kv_rows = np.concatenate(kv_rows) if kv_rows else np.zeros(0, np.int32)
        p_tiles = np.asarray(p_tiles, dtype=np.int32).reshape(-1, 4)

        def rows_of(reqs):
            return np.concatenate([np.arange(row0[b], row0[b + 1]) for b in reqs]).astype(np.int32) if reqs else np.zeros(0, np.int32)
        s_rows = rows_of(small)
        every = np.arange(T, dtype=np.int32)

        def row_tiles(rows):
            return np.stack([st.row_slot[rows], st.row_pos[rows], np.ones(rows.size, np.int64), rows], axis=1).astype(np.int32)
        # layers whose heads are too wide for the prompt kernel fold all rows
        mixed_sizes = bool(big) and not all(ent["prompts"] for ent in self.layers)
        s_tiles, a_tiles = row_tiles(s_rows), (row_tiles(every) if mixed_sizes else np.zeros((0, 4), np.int32))
        offs = np.stack([st.row_slot * (cap * d) + st.row_pos * d for d in self._sigs])
        tables = dict(ids=st.ids, pos=st.row_pos.astype(np.int32), want=want_rows, kv_rows=kv_rows, p_tiles=p_tiles, s_tiles=s_tiles,
                      s_rows=s_rows if big else np.zeros(0, np.int32), a_tiles=a_tiles)
        sizes = {k: v.size for k, v in tables.items()}
        n32 = sum(sizes.values())
        o64 = (n32 * 4 + 7) // 8 * 8
        blob = np.empty(o64 + offs.size * 8, dtype=np.uint8)
        blob[:n32 * 4].view(np.int32)[:] = np.concatenate([v.reshape(-1) for v in tables.values()])
        blob[o64:].view(np.int64)[:] = offs.reshape(-1)
        dims = dict(T=T, R=st.R, n_want=int(want_rows.size), n32=n32, o64=o64, sizes=sizes, tile=tile)
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
        at, out = 0, {}
        for name, n in d["sizes"].items():
            out[name] = i32[at:at + n]
            at += n
        no = len(self._sigs)
        out["offs"] = dblob[d["o64"]:d["o64"] + no * d["T"] * 8].view(torch.int64).view(no, d["T"])
        return out

    def _run(self, arena, dblob, d, logits, num_layers=None, return_streams=False):
        """The device side of a step: every launch of the forward, reading the step's tables from ``dblob``."""
        dev, E, f32 = self.device, self.dtype, torch.float32
        W, T = self.W, d["T"]
        tb = self._tables(dblob, d)
        tb["tile"] = d["tile"]
        runs = self.runs if num_layers is None else self.runs[:num_layers]
        cfg, eps = self.config, self.config.norm_eps
        x = self._mat("x", T, W, f32)
        h = self._mat("h", T, W, E)
        streams = torch.empty((len(runs), T, W), dtype=f32, device=dev) if return_streams else None
        B.embed_scaled_rows(self.embed, tb["ids"], cfg.embed_scale, x)
        if cfg.loop_times:
            both = self._mat("x_x0", T, 2 * W, E)              # [x; x0] of the passes' entry
            B.post_norm(x, out=both[:, W:], ldo=2 * W, n_rows=T)
        pending = {}                                           # the layer result that is still to be added to x
        for r, (i, starts) in enumerate(runs):
            lw = self.layers[i]
            if starts >= 0:
                B.post_norm(x, out=both, ldo=2 * W, n_rows=T, **pending)
                B.linear(both, self.loop_in, x, M=T, bias=self.loop_step[starts])
                pending = {}
            B.post_norm(x, gain=lw["gain"], out=h, eps=eps, n_rows=T, **pending)
            pending = self._layer(arena, r, lw, h, tb, T)
            if streams is not None:
                B.post_norm(x, n_rows=T, x_out=streams[r], **pending)
                pending = {}
        if d["n_want"]:
            nw = d["n_want"]
            hn = self._mat("hn", nw, W, E)
            B.post_norm(x, gain=self.final_gain, out=hn, eps=eps, rows=tb["want"], n_rows=nw, **pending)
            cap = cfg.logit_softcap
            B.linear(hn, self.embed, logits, M=nw, act=B.ACT_SOFTCAP if cap > 0 else B.ACT_NONE, act_param=cap)
        return (logits, streams) if return_streams else logits

    def _layer(self, arena, r, lw, h, tb, T):
        """One layer run on h = norm(x): what is to be added to x, as ``pcb_post_norm`` takes it."""
        E, f32, l = self.dtype, torch.float32, lw["cfg"]
        H, Dv, N = l.heads, l.vdim, lw["n_in"]
        moe = l.ff_kind == "moe"
        P = self._mat("mix_in", T, N, E)
        logits = self._mat("router", T, l.experts, f32) if moe else None
        B.linear(h, lw["w_in"], P, M=T, act_split=lw["act_from"], act2=B.ACT_SIGMOID, split_n=N if moe else 0, y2=logits, y2_f32=moe,
                 head_stride2=l.experts)
        K_out = lw["w_out"].shape[1]
        A = self._mat("mix_out", T, K_out, E)                  # heads' outputs | gated unit
        if "gate" in lw:
            # (the shared expert's gate, the projection's last column, multiplies its unit here: one number per token)
            B.linear(h, lw["gate"], A[:, H * Dv:], M=T, epilogue=B.EPI_SILU_MUL, w2=lw["up"], act=B.ACT_SILU, ldy=K_out,
                     row_gate=P[:, N - 1:] if moe else None, ld_row_gate=N)
        self._attention(arena, r, lw, P, A, K_out, tb, T)
        y = self._mat("y", T, self.W, f32)
        B.linear(A, lw["w_out"], y, M=T)
        if not moe:
            return dict(y=y)
        return dict(y=y, **self._experts(l, lw, h, logits, T))

    # ---- attention ----------------------------------------------------------------------------------------------------------------
    def _attention(self, arena, r, lw, P, A, ldo, tb, T):
        """Reads the projected rows P, leaves the gated heads' outputs in the first columns of A (row stride ``ldo``)."""
        E, l, eps = self.dtype, lw["cfg"], self.config.norm_eps
        H, D, R, C, Q, N = l.heads, l.dim, l.rot_dim, l.kv_rank, l.q_rank, lw["n_in"]
        DR, CR = D + R, C + R
        plane = arena.planes[r]
        off = tb["offs"][self._sigs.index(CR)]
        turn = dict(rot_dims=l.rot_dims)
        cq = self._mat("q_latent", T, Q, E)
        segs = [B.head_seg(P, N, 1, Q, cq, norm=True, gain=lw["q_gain"], ld_dst=Q),
                B.head_seg(P[:, Q:], N, 1, C, plane, norm=True, gain=lw["c_gain"], row_off=off)]
        if R:
            segs.append(B.head_seg(P[:, Q + C:], N, 1, R, plane, row_off=off, dst_offset=C, **turn))
        rot = dict(pos=tb["pos"], freqs=lw["freqs"], rot_half=True, eps=eps)
        B.head_prep(segs, T, E, **rot)
        q = self._mat("q_rows", T, H * DR, E)
        B.linear(cq, lw["uq"], q, M=T)
        prompts = lw["prompts"] and tb["p_tiles"].numel() > 0
        gate = P[:, Q + CR:]
        if prompts:
            if R:
                B.head_prep([B.head_seg(q[:, D:], H * DR, H, R, q, src_head_stride=DR, ld_dst=H * DR, head_stride=DR, dst_offset=D, **turn)],
                            T, E, **rot)
            self._rebuilt(arena, r, lw, q, A, ldo, gate, N, tb)
        s_tiles = tb["s_tiles"] if lw["prompts"] or not tb["a_tiles"].numel() else tb["a_tiles"]
        n = s_tiles.numel() // 4
        if n:
            rows = tb["s_rows"] if (prompts and n < T) else None
            self._folded(arena, r, lw, q, A, ldo, gate, N, tb, s_tiles, n, rows, T, rot, turned=prompts)

    def _rebuilt(self, arena, r, lw, q, A, ldo, gate, ldg, tb):
        E, l = self.dtype, lw["cfg"]
        H, D, R, Dv, C = l.heads, l.dim, l.rot_dim, l.vdim, l.kv_rank
        CR, plane = C + R, arena.planes[r]
        flat = plane.view(-1, CR)
        M = tb["kv_rows"].numel()
        NK = H * (D + Dv)
        kv = self._mat("kv_rows", M, NK, E)
        B.linear(flat, lw["w_kv"], kv, M=M, row_src=tb["kv_rows"], ldx=CR)
        B.attn_prompt(q, tb["p_tiles"], tb["p_tiles"].numel() // 4, tb["tile"], kv, (NK, D), kv[:, H * D:], (NK, Dv), H, H, D + R, Dv, l.scale, A,
                      ldo=ldo, k_tail=flat[:, C:] if R else None, tail_row_stride=CR, tail_rows=tb["kv_rows"], tail_dim=R, sink=lw["sink"],
                      gate=gate, ldg=ldg)

    def _folded(self, arena, r, lw, q, A, ldo, gate, ldg, tb, tiles, n, rows, T, rot, turned):
        E, l = self.dtype, lw["cfg"]
        H, D, R, Dv, C = l.heads, l.dim, l.rot_dim, l.vdim, l.kv_rank
        DR, CR = D + R, C + R
        qa = self._mat("q_folded", T, H * CR, E)               # per head [W_uk^T q | rotated part]: a query over the cached rows
        if R:
            seg = dict(rot_dims=0 if turned else l.rot_dims)
            B.head_prep([B.head_seg(q[:, D:], H * DR, H, R, qa, src_head_stride=DR, ld_dst=H * CR, head_stride=CR, dst_offset=C, **seg)], T, E,
                        **rot)
        B.linear(q, lw["w_abs"], qa, M=n, row_src=rows, row_dst=rows, n_batch=H, ldx=H * DR, x_batch_stride=DR, ldy=H * CR, y_batch_stride=CR)
        ol = self._mat("o_latent", T, H * C, E)
        splits = self._splits(arena, n, -(-H // 16))
        part = self._scratch("attn_part", B.attn_softmax_part(T, H, splits, C), torch.float32) if splits > 1 else None
        B.attn_latent(qa, tiles, n, arena.planes[r], arena.slot_stride(r), CR, H, CR, C, l.scale, ol, sink=lw["sink"], gate=gate, ldg=ldg,
                      n_splits=splits, part=part)
        B.linear(ol, lw["w_uv"], A, M=n, row_src=rows, row_dst=rows, n_batch=H, ldx=H * C, x_batch_stride=C, ldy=ldo, y_batch_stride=Dv)

    def _splits(self, arena, rows, head_groups):
        # few (row, head group) pairs cannot fill the chip: each is cut into runs of its keys, as many as blocks of 64 keys fit the rows
        return max(1, min(64, 512 // (rows * head_groups), -(-arena.cap // 64)))

    # ---- experts --------------------------------------------------------------------------------------------------------------------
    def _experts(self, l, lw, h, logits, T):
        n_out, P, W = l.experts, T * l.top, self.W
        ex = self._scratch("moe_i", 3 * P + n_out + 1, torch.int32)
        sc = self._scratch("moe_f", 2 * P, torch.float32)
        expert, row_src, row_dst, goff = ex[:P], ex[P:2 * P], ex[2 * P:3 * P], ex[3 * P:3 * P + n_out + 1]
        weight, row_scale = sc[:P], sc[P:2 * P]
        B.router_select(logits, l.top, expert, weight, T, score_fn=B.SCORE_SOFTMAX, renorm=False)
        pair = self._mat("pair", P, W, torch.float32)
        B.moe_plan(expert, weight, P, l.top, n_out, goff, row_src, row_dst, row_scale)
        act = self._mat("moe_act", P, l.expert_ff, self.dtype)
        B.linear(h, lw["e_gate"], act, M=P, epilogue=B.EPI_SILU_MUL, w2=lw["e_up"], act=B.ACT_SILU, row_src=row_src, group_off=goff,
                 n_groups=n_out)
        B.linear(act, lw["e_down"], pair, M=P, row_dst=row_dst, group_off=goff, n_groups=n_out)
        return dict(pair=pair, pair_weight=weight, pair_top=l.top)
