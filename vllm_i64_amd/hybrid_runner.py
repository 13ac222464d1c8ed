"""What the runners over a HybridCache share: step buffers, the grouping of a step's rows, and the sublayers that more than one design is
made of - rotated attention over [values | keys] rows, latent attention, the gated delta rule, gated linear attention, clamped and mixture
feed-forwards - each with its options as parameters.
A design's own file holds its weight layout, its residual and the order in which its sublayers run."""
from __future__ import annotations

import os
from contextlib import contextmanager, nullcontext
from typing import Callable, Dict, Optional

import torch

from . import ops_dense as D

UNIT_EPS = 1e-6     # inside the root of the delta rule's unit vectors: a constant of the mechanism, not of a checkpoint


def pad8(n: int) -> int:
    return (int(n) + 7) // 8 * 8


class HybridRunner:
    MAX_BUFFER_SETS = int(os.environ.get("I64H_MAX_BUFFER_SETS", "8"))
    ATTN_MAX_SEGMENTS = 4
    ATTN_WAVES = {64: 3072, 128: 2048, 256: 1024}     # waves a decode-sized attention launch aims at, by the width of a key head's cached part
    BUFFERS: Optional[Callable] = None                # (runner, rows, logit rows) -> the step's buffers
    SIDE_STREAM = False                               # a second stream for a sublayer that runs beside another one

    def _init_runner(self, cfg, device, dtype: str) -> None:
        if dtype not in ("bfloat16", "float32"):
            raise ValueError(f"dtype {dtype}: bfloat16 or float32")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.exact = dtype == "float32"
        self._bufs: Dict[tuple, object] = {}
        self._pinned: set = set()
        self._arange: Dict[int, torch.Tensor] = {}
        self.side = torch.cuda.Stream(device=self.device) if self.SIDE_STREAM and self.device.type == "cuda" else None

    # ---- two sublayers side by side ----
    @contextmanager
    def _beside(self):
        """The launches of the body run on the side stream (of default priority), behind what the current stream holds so far and beside what
        it gets next, until _meet(); a captured graph keeps the two branches.  Without a side stream they simply run here.  One level only:
        the body forks no further."""
        if self.side is None:
            yield
            return
        self.side.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(self.side):
            yield

    def _meet(self) -> None:
        if self.side is not None:
            torch.cuda.current_stream().wait_stream(self.side)

    # ---- tensors by name and shape, in the two forms the kernels read ----
    def _bf(self, t: torch.Tensor) -> torch.Tensor:
        return t.to(device=self.device, dtype=torch.bfloat16).contiguous()

    def _f(self, t: torch.Tensor) -> torch.Tensor:
        return t.to(device=self.device, dtype=torch.float32).contiguous()

    @staticmethod
    def _reader(weights: Dict[str, torch.Tensor]):
        def need(name, shape):
            if name not in weights:
                raise KeyError(f"tensor '{name}' is missing")
            if tuple(weights[name].shape) != tuple(shape):
                raise ValueError(f"'{name}': shape {tuple(weights[name].shape)}, config says {tuple(shape)}")
            return weights[name]
        return need

    # ---- load-time layout ----
    def _stack(self, parts):
        """Rows of several projections as one weight, every part starting at a multiple of eight rows (rows of zeros between), so that the
        columns of a projection row can be read 16 bytes at a time; returns (weight, first column of each part)."""
        rows, offs, at = [], [], 0
        for t in parts:
            offs.append(at)
            rows.append(t.float())
            at = pad8(at + t.shape[0])
            if at > offs[-1] + t.shape[0]:
                rows.append(torch.zeros(at - offs[-1] - t.shape[0], t.shape[1]))
        return self._bf(torch.cat([r.cpu() for r in rows], 0)), offs

    def _low_rank(self, weights, need, first: str, second: str, out: int):
        """A map of two factors: the rank is the tensors' own; the second factor's columns are padded to where the first one's rows end."""
        if first not in weights or weights[first].dim() != 2:
            raise KeyError(f"tensor '{first}' is missing or is no matrix")
        r = weights[first].shape[0]
        a, b = need(first, (r, self.cfg.width)), need(second, (out, r))
        return a, self._bf(torch.nn.functional.pad(b.float(), (0, pad8(r) - r)))

    # ---- step buffers: the most recent row counts are kept, pinned sets stay for captured graphs ----
    def buffers(self, n: int, m: int):
        key = (n, m)
        B = self._bufs.pop(key, None)
        if B is None:
            B = type(self).BUFFERS(self, n, m)
        self._bufs[key] = B
        loose = [k for k in self._bufs if k not in self._pinned and k != key]
        for k in loose[:max(0, len(loose) + 1 - self.MAX_BUFFER_SETS)]:
            del self._bufs[k]
        return B

    def pin_buffers(self, n: int, m: int) -> None:
        self.buffers(n, m)
        self._pinned.add((n, m))

    def check_sync(self, force: bool = True):
        """No launch of these runners waits on a grid barrier: nothing to read back."""

    def snapshot_state(self):
        """The per-sequence state, for a caller that runs a step which must not count (a warm-up before a graph capture)."""
        return self.kv.snapshot()

    def restore_state(self, held) -> None:
        self.kv.restore(held)

    def _runs(self, n: int, slot_ids: torch.Tensor, tokens_per_seq, rows_are_slots: bool):
        """First rows of the runs of consecutive rows of one sequence, int32 [runs + 1] on the device, and their number."""
        if rows_are_slots:
            t = self._arange.get(n)
            if t is None:
                t = self._arange[n] = torch.arange(n + 1, dtype=torch.int32, device=self.device)
            return t, n
        if tokens_per_seq is None:      # (a caller that does not say how its rows are grouped: read it off the slot ids)
            s = slot_ids.tolist()
            tokens_per_seq, k = [], 0
            for j in range(1, n + 1):
                if j == n or s[j] != s[j - 1]:
                    tokens_per_seq.append(j - k)
                    k = j
        starts = [0]
        for t in tokens_per_seq:
            if int(t) > 0:
                starts.append(starts[-1] + int(t))
        if starts[-1] != n:
            raise ValueError(f"tokens_per_seq adds up to {starts[-1]} rows, the step has {n}")
        return torch.tensor(starts, dtype=torch.int32).to(self.device), len(starts) - 1

    def _splits(self, B, rows: int, heads: int, kv_heads: int, vals: int, width: int, ctx_hint: int, floats):
        """How many waves share a decode row's keys (about ATTN_WAVES waves in the launch, a wave keeping at least two tiles of 32 keys),
        and the workspace their partial results meet in."""
        tasks = rows * kv_heads * ((heads // kv_heads + 15) // 16)
        waves = self.ATTN_WAVES[64 if width <= 64 else (128 if width <= 128 else 256)]
        splits = max(1, min(waves // max(1, tasks), ctx_hint // 64, 64))
        if splits <= 1:
            return 1, None
        key = (rows, heads, kv_heads, vals, splits)
        ws = B.attn_ws.get(key)
        if ws is None:
            ws = B.attn_ws[key] = torch.empty(max(1, floats(splits)), dtype=torch.float32, device=self.device)
        return splits, ws

    # ---- attention over grouped key / value heads, separate keys and values in one cached row ----
    def _kattn(self, B, a, Q, O, rows, kvc, slot_ids, positions, runs, ctx_hint: int, *, bias=None, softcap: float = 0.0, window: int = 0,
               keep_first: int = 0, sink_w=None) -> None:
        """Runs of rows that are one per sequence (a wave takes a token's query heads of one key head, the keys dealt to several waves) and
        runs of prompt portions (a wave takes 16 consecutive rows of one head), each one launch."""
        gs = a.vdim + a.dim
        keys = min(ctx_hint, window + keep_first + 64) if window > 0 else ctx_hint
        for r0, r1, one_per_seq in runs:
            splits, ws = 1, None
            if one_per_seq and not self.exact:
                splits, ws = self._splits(B, r1 - r0, a.heads, a.kv_heads, a.vdim, gs, keys,
                                          lambda s: D.kattn_workspace_floats(r1 - r0, a.heads, a.kv_heads, a.vdim, s))
            D.kattn(Q[r0:r1], rows, None, kvc.block_table, slot_ids[r0:r1], positions[r0:r1], chunk=0, bias=bias, sink=sink_w is not None,
                    heads=a.heads, kv_heads=a.kv_heads, dim=a.dim, vdim=a.vdim, out=O[r0:r1], n=r1 - r0, mode=2 if one_per_seq else 3, splits=splits,
                    workspace=ws, softcap=softcap, window=window, keep_first=keep_first, sink_w=sink_w)

    def _rotary_tables(self, a, d: dict) -> None:
        """Frequency tables of a rotated attention: evaluated in 64 bits on the host, rounded once to fp32."""
        d["inv_freq"], d["rot_mult"], d["v_freq"] = None, 1.0, None
        if a.rot is not None and a.rot.dims:
            fr, d["rot_mult"] = a.rot.frequencies()
            d["inv_freq"] = self._f(torch.tensor(fr, dtype=torch.float64))
        if a.rot is not None and a.rotate_values:
            d["v_freq"] = self._f(torch.tensor([a.rot.base ** (-2.0 * i / a.vdim) for i in range(a.vdim // 2)], dtype=torch.float64))

    def _rotary_attention(self, B, d, a, P, l, n, positions, slot_ids, kvc, runs, ctx_hint, out, scale: float = 1.0) -> None:
        """Rotated attention on the projection rows P (already computed; columns d["q_off"], d["k_off"], d["v_off"]): prep -> paged
        [values | keys] rows and query rows, attention, the turn back and the head gate, out-projection (times `scale`) into `out`."""
        gs = a.vdim + a.dim
        Q = B.a[: n * a.heads * gs].view(n, a.heads * gs)
        rows = kvc.rows[l]
        D.rot_prep(P, q_off=d["q_off"], k_off=d["k_off"], v_off=d["v_off"], heads=a.heads, kv_heads=a.kv_heads, dim=a.dim, vdim=a.vdim, q_norm_w=d.get("q_norm"),
                   k_norm_w=d.get("k_norm"), eps=self.cfg.norm_eps, rot_dims=a.rot.dims if a.rot is not None else 0, interleaved=a.interleaved,
                   inv_freq=d["inv_freq"], rot_mult=d["rot_mult"], head_norm=a.qk_norm == "head", v_freq=d["v_freq"], scale=a.scale, positions=positions,
                   slot_ids=slot_ids, block_table=kvc.block_table, cache=rows, q=Q, n=n, norm_heads=a.qk_norm == "head_weight")
        O = B.b[: n * a.heads * a.vdim].view(n, a.heads * a.vdim)
        self._kattn(B, a, Q, O, rows, kvc, slot_ids, positions, runs, ctx_hint, softcap=a.softcap, window=a.window, keep_first=a.keep_first, sink_w=d.get("sink"))
        if d["v_freq"] is not None or a.head_gate:
            D.rot_post(O, heads=a.heads, vdim=a.vdim, interleaved=a.interleaved, v_freq=d["v_freq"], positions=positions,
                       gate=P if a.head_gate else None, gate_off=d.get("g_off", 0), ldg=P.shape[-1], n=n)
        self._out(O, d["o"], out, scale)

    def _out(self, a, w, out, scale: float = 1.0) -> None:
        D.linear(a, w, out, exact=self.exact, epilogue=D.EPI_STORE if scale == 1.0 else D.EPI_SCALE, scale=scale)

    # ---- latent attention: one cached row per token that all heads share ----
    def _load_latent(self, p: str, m, need, d: dict) -> list:
        """Tensors of a latent attention under the prefix p behind its input projections, which are returned as parts of the layer's input
        weight, in order: queries (or their low-rank row), latent + shared key part, head gates."""
        W, bf, f, H, r = self.cfg.width, self._bf, self._f, m.heads, m.kv_rank
        # a head's score against a cached latent c is q_h . (U_h c) = (U_h^T q_h) . c: the key map transposed per head
        d["uk_t"] = bf(need(p + "uk", (H * m.dim, r)).reshape(H, m.dim, r).transpose(1, 2))      # [H, r, dim]
        d["uv"] = bf(need(p + "uv", (H * m.vdim, r)).reshape(H, m.vdim, r))                      # [H, vdim, r]
        d["c_norm"] = f(need(p + "dkv.norm", (r,)))
        d["sink"] = f(need(p + "sink", (H,))) if m.sink else None
        d["o"] = bf(need(p + "o", (W, H * m.vdim)))
        d["inv_freq"], d["rot_mult"] = None, 1.0
        if m.rot is not None:
            fr, d["rot_mult"] = m.rot.frequencies()
            d["inv_freq"] = f(torch.tensor(fr, dtype=torch.float64))
        if m.q_rank:
            d["q_norm"], d["uq"] = f(need(p + "dq.norm", (m.q_rank,))), bf(need(p + "uq", (m.q_width, m.q_rank)))
        parts = [need(p + "dq", (m.q_rank, W)) if m.q_rank else need(p + "q", (m.q_width, W)), need(p + "dkv", (r + m.rot_dim, W))]
        return parts + ([need(p + "g", (H, W))] if m.head_gate else [])

    def _latent_attention(self, B, d, m, P, l, n, positions, slot_ids, kvc, runs, ctx_hint, out) -> None:
        """Latent attention on the projection rows P (columns d["q_off"]: the queries, or their low-rank row; d["dkv_off"]: latent + shared
        key part; d["g_off"]: head gates): norms and rotation -> paged rows and query rows, queries into latent space per head, attention,
        summed latents into value space per head (times the head's gate), out-projection into `out`."""
        ex, N1 = self.exact, P.shape[-1]
        H, r, rd, qh = m.heads, m.kv_rank, m.rot_dim, m.dim + m.rot_dim
        width = r + rd
        src, q_off = P, d["q_off"]
        if m.q_rank:
            src, q_off = B.q[: n * H * qh].view(n, H * qh), 0
            D.linear(P, d["uq"], src, m=n, a_off=d["q_off"], exact=ex, in_norm_w=d["q_norm"], in_eps=self.cfg.norm_eps)
        cache = kvc.rows[l]
        Q = B.a[: n * H * width]
        D.latent_prep(P, q_off=q_off, dkv_off=d["dkv_off"], heads=H, dim=m.dim, rot_dim=rd, kv_rank=r, rot_dims=m.rot_dims, c_norm_w=d["c_norm"], eps=self.cfg.norm_eps,
                      inv_freq=d["inv_freq"], positions=positions, slot_ids=slot_ids, block_table=kvc.block_table, block_size=kvc.block, cache=cache, q=Q, n=n,
                      q_src=src if m.q_rank else None, rot_mult=d["rot_mult"])
        # queries into latent space, per head: Q[:, h, :r] = q_unrotated[:, h, :] @ U_h
        D.linear(src, d["uk_t"], Q, m=n, n=r, k=m.dim, a_off=q_off, lda=src.shape[-1], ldc=H * width, batch=H, a_batch=qh, w_batch=r * m.dim, c_batch=width, exact=ex)
        olat = B.b[: n * H * r]
        keys = min(ctx_hint, m.window + 64) if m.window > 0 else ctx_hint
        for r0, r1, one_per_seq in runs:
            splits, ws = 1, None
            if one_per_seq and not ex:
                splits, ws = self._splits(B, r1 - r0, H, 1, r, width, keys, lambda s: D.latent_attn_workspace_floats(r1 - r0, H, r, s))
            D.latent_attn(Q[r0 * H * width: r1 * H * width], cache, kvc.block_table, slot_ids[r0:r1], positions[r0:r1], window=m.window, scale=m.scale, heads=H, kv_rank=r,
                          rot_dim=rd, out=olat[r0 * H * r: r1 * H * r], n=r1 - r0, mode=2 if one_per_seq else 3, splits=splits, workspace=ws, sink=d["sink"])
        # summed latents into value space, per head
        og = B.c[: n * H * m.vdim]
        gate = dict(epilogue=D.EPI_ROW_SIGMOID, e=P, e_off=d["g_off"], lde=N1, e_batch=1) if m.head_gate else {}
        D.linear(olat, d["uv"], og, m=n, n=m.vdim, k=r, lda=H * r, ldc=H * m.vdim, batch=H, a_batch=r, w_batch=m.vdim * r, c_batch=m.vdim, exact=ex, **gate)
        D.linear(og, d["o"], out, m=n, k=H * m.vdim, lda=H * m.vdim, exact=ex)

    # ---- gated linear attention ----
    def _gated_linear(self, B, d, r, P, l, n, positions, slot_ids, kvc, seg, nseg, out, scale: float = 1.0) -> None:
        """Gated linear attention on the projection rows P (columns d["rq_off"], d["rk_off"], d["rv_off"], d["rg_off"]: queries, keys, values, output
        gates; d["a1_off"]: the low-rank decay map's first factor).  sigmoid(z)^(1 / tau) = exp(-softplus(-z) / tau): the second factor and
        its bias are held negated, the exponent's rate is d["a_rate"]."""
        rv = r.heads * r.vdim
        F = B.f[: n * r.heads * r.dim].view(n, r.heads * r.dim)
        D.linear(P, d["a2"], F, m=n, a_off=d["a1_off"], exact=self.exact, bias=d["a2_b"], epilogue=D.EPI_DECAY, e=d["a_rate"])
        R, Rn = B.r[: n * rv].view(n, rv), B.rn[: n * rv].view(n, rv)
        D.gla_scan(P, f=F, q_off=d["rq_off"], k_off=d["rk_off"], f_off=0, v_off=d["rv_off"], heads=r.heads, dim=r.dim, vdim=r.vdim, seg_start=seg, nseg=nseg,
                   positions=positions, slot_ids=slot_ids, state=kvc.state[l]["gla"], out=R, n=n, q_scale=r.dim ** -0.5)
        D.gate_norm(R, d["r_norm"], Rn, groups=r.heads, eps=self.cfg.norm_eps, z=P, z_off=d["rg_off"], ldz=P.shape[-1], n=n, gate_after=True, width=rv)
        self._out(Rn, d["o_right"], out, scale)

    # ---- gated delta rule ----
    def _gated_delta(self, B, d, r, P, l, n, positions, slot_ids, kvc, seg, nseg, single: bool, out) -> None:
        """Gated delta rule on the projection rows P: the convolved parts q | k | v from column d["r_off"] on, the write strength's at
        d["rb_off"].  A decay per head comes from the columns d["ra_off"]; a decay per key channel (r.decay 'channel') and its output gate are
        low-rank maps whose first factors' results lie at d["a1_off"] and d["g1_off"]."""
        ex = self.exact
        st = kvc.state[l]
        C, rk, rv = r.conv_channels, r.kv_heads * r.dim, r.heads * r.vdim
        X = B.a[: n * C].view(n, C)
        D.causal_conv(P, off=d["r_off"], channels=C, w=d["conv_w"], bias=None, positions=positions, slot_ids=slot_ids, state=st.get("conv"), out=X, n=n,
                      single_rows=single, seg_start=seg, nseg=nseg)
        G = B.g[: n * 2 * r.heads].view(n, 2 * r.heads)
        cols = dict(q_off=0, k_off=rk, v_off=2 * rk, heads=r.heads, kv_heads=r.kv_heads, dim=r.dim, vdim=r.vdim, n=n)
        channel = r.decay == "channel"
        D.gdn_gates(X, G, P, b_off=d["rb_off"], a_off=-1 if channel else d["ra_off"], a_log=None if channel else d["A_log"],
                    dt_bias=None if channel else d["dt_bias"], unit_eps=UNIT_EPS, q_scale=r.dim ** -0.5, **cols)
        F, Z, z_off, ldz = None, P, d.get("rg_off", 0), P.shape[-1]
        if channel:
            F, Z, z_off, ldz = B.f[: n * r.heads * r.dim].view(n, r.heads * r.dim), B.z[: n * rv].view(n, rv), 0, rv
            D.linear(P, d["a2"], F, m=n, a_off=d["a1_off"], exact=ex, bias=d["dt_bias"], epilogue=D.EPI_DECAY, e=d["a_rate"])
            D.linear(P, d["g2"], Z, m=n, a_off=d["g1_off"], exact=ex)
        R = B.b[: n * rv].view(n, rv)
        D.gdn_scan(X, G, f=F, seg_start=seg, nseg=nseg, positions=positions, slot_ids=slot_ids, state=st["gdn"], out=R, **cols)
        Rn = B.c[: n * rv].view(n, rv)
        D.gate_norm(R, d["r_norm"], Rn, groups=r.heads, eps=self.cfg.norm_eps, z=Z, z_off=z_off, ldz=ldz, n=n, gate_after=True, width=rv, sigmoid=r.gate == "sigmoid")
        D.linear(Rn, d["o_right"], out, exact=ex)

    # ---- mixture of experts ----
    def _load_moe(self, p: str, f, need, d: dict) -> None:
        """Router, stacked experts and shared expert of a mixture under the tensor prefix p."""
        W, bf = self.cfg.width, self._bf
        router = need(p + "router", (f.entries, W))
        if f.shared_ff and f.shared_gate:       # one more row behind the router's: the shared expert's gate
            router = torch.cat([router, need(p + "shared.sg", (1, W))], 0)
        d["router"] = bf(router)
        d["router_b"] = self._f(need(p + "router.b", (f.entries,))) if f.router_bias else None
        # per expert [gate rows; up rows], all experts stacked: one grouped launch for the pair, one for the way down
        d["gate_up"] = bf(torch.stack([torch.cat([need(f"{p}e{e}.gate", (f.ff, W)), need(f"{p}e{e}.up", (f.ff, W))], 0) for e in range(f.experts)]))
        d["e_down"] = bf(torch.stack([need(f"{p}e{e}.down", (W, f.ff)) for e in range(f.experts)]))
        if f.shared_ff:
            s = f.shared_ff
            d["s_gate_up"] = bf(torch.cat([need(p + "shared.gate", (s, W)), need(p + "shared.up", (s, W))], 0))
            d["s_down"] = bf(need(p + "shared.down", (W, s)))

    @staticmethod
    def moe_buffers(B, model, n: int) -> None:
        """The step buffers of _moe_ff on B (model.max_top == 0: no mixtures)."""
        i32, f32 = dict(dtype=torch.int32, device=model.device), dict(dtype=torch.float32, device=model.device)
        t = model.max_top
        B.ey = torch.empty(n * t, model.cfg.width, **f32) if t else None   # the chosen experts' outputs, grouped by expert
        B.idx = torch.empty(n * max(t, 1), **i32)
        B.wgt = torch.empty(n * max(t, 1), **f32)
        B.pair_token = torch.empty(n * max(t, 1), **i32)
        B.pair_row = torch.empty(n * max(t, 1), **i32)
        B.pair_wgt = torch.empty(n * max(t, 1), **f32)
        B.group_off = torch.empty(model.max_experts + 1, **i32)
        B.sgate = torch.empty(n, **f32)
        B.sact = torch.empty(n * max(model.max_shared, 1), **f32)

    def _moe_sizes(self, mlps) -> None:
        moes = [m for m in mlps if m is not None and m.kind == "moe"]
        self.max_top = max([m.top for m in moes] or [0])
        self.max_experts = max([m.experts for m in moes] or [0])
        self.max_shared = max([m.shared_ff for m in moes] or [0])
        self.max_act = max([m.ff for m in mlps if m is not None and m.kind == "dense"] + [m.ff * m.top for m in moes] + [0])

    @staticmethod
    def _glu(limit: float, alpha: float) -> dict:
        """The gate / up epilogue of a feed-forward: clamped by `limit`, or silu."""
        return dict(epilogue=D.EPI_CLAMP_GLU, act_a=alpha, act_b=limit) if limit > 0 else dict(epilogue=D.EPI_SILU_MUL)

    def _load_dense(self, p: str, f, need, d: dict) -> None:
        W = self.cfg.width
        d["ff_gate_up"] = self._bf(torch.cat([need(p + "gate", (f.ff, W)), need(p + "up", (f.ff, W))], 0))
        d["ff_down"] = self._bf(need(p + "down", (W, f.ff)))

    def _dense_glu(self, B, d, n, h, out) -> None:
        f = d["mlp"]
        act = B.act[: n * f.ff].view(n, f.ff)
        D.linear(h, d["ff_gate_up"], act, exact=self.exact, **self._glu(f.limit, f.glu_alpha))
        D.linear(act, d["ff_down"], out, exact=self.exact)

    def _moe_ff(self, B, d, n, h, out, shared_out, record: Optional[dict] = None, tag: str = "", beside: bool = False) -> None:
        """out <- the mixture of d["mlp"] on h fp32 [n, width]; shared_out [n, width] receives the shared expert's rows on the way (beside: on
        the side stream, while the routed experts run)."""
        f, ex, W = d["mlp"], self.exact, self.cfg.width
        E, top = f.experts, f.top
        gate = B.sgate if f.shared_ff and f.shared_gate else None
        shared = None
        if f.shared_ff:
            with self._beside() if beside else nullcontext():
                sact = B.sact[: n * f.shared_ff].view(n, f.shared_ff)
                D.linear(h, d["s_gate_up"], sact, exact=ex, **self._glu(f.shared_limit, f.glu_alpha))
                shared = D.linear(sact, d["s_down"], shared_out, exact=ex)
        # the router's products in 32 bits in both modes (a choice between experts is not rounding's to make), inside the choice's launch
        D.route_topk(None, h=h, w=d["router"], entries=f.entries, correction=d.get("correction"), groups=f.groups, keep=f.keep, top=top, scale=f.scale,
                     idx=B.idx, wgt=B.wgt, n=n, bias=d["router_b"], chosen_softmax=f.chosen_softmax, gate_out=gate, sigmoid_scores=f.sigmoid_scores, raw_weights=f.raw_weights)
        if record is not None:
            record[f"{tag}.route"] = B.idx[: n * top].view(n, top).clone()
        pair_wgt = B.pair_wgt if f.weigh_input else None      # the weight multiplies what the expert reads, not what it returns
        D.moe_plan(B.idx, n=n, top=top, experts=E, group_off=B.group_off, pair_token=B.pair_token, pair_row=B.pair_row, wgt=B.wgt, pair_wgt=pair_wgt)
        # the (token, expert) pairs lie grouped by expert: one launch runs every expert over its own rows, the counts stay on the device
        act = B.act[: n * top * f.ff].view(n * top, f.ff)
        D.linear(h, d["gate_up"], act, m=n, a_rows=B.pair_token, batch=E, w_batch=2 * f.ff * W, exact=ex, group_off=B.group_off, row_scale=pair_wgt, **self._glu(f.limit, f.glu_alpha))
        D.linear(act, d["e_down"], B.ey, m=n, batch=E, w_batch=W * f.ff, exact=ex, group_off=B.group_off)
        if shared is not None and beside:
            self._meet()
        D.moe_combine(B.ey, B.pair_row, None if f.weigh_input else B.wgt, h, shared, out, n=n, top=top, width=W, shared_gate=gate)
