"""Runner of the Pukatar design on one MI355X: a decoder whose layers run mixer and feed-forward side by side on one normed input, with a
stretch of layers that repeats under the same weights:

  x0 = ln(embed[token]);   x = x0
  layer:  h = ln1(x);  x <- x + (mixer(h) + ff(h))                       ln: centred norm with weight and offset
  loop:   layers start .. stop - 1 run `times` times, every pass with a cache and state of its own; in front of pass t:
          x <- W_in [x; x0] + step[t]
  attention      grouped key / value heads, rotation in halves of the first rot.dims values of a head, a window in which the first
                 keep_first positions stay visible, a learned sink per head in the softmax's denominator
  channel_delta  gated delta rule with a decay per head and KEY CHANNEL (a low-rank map): S <- diag(g) S, u = beta (v - S^T k),
                 S <- S + k u^T, o = S^T q on unit q, k behind short causal convolutions + silu; RMS norm per head, times the
                 sigmoid of a low-rank gate; out-projection
  dense          W_down (silu(W_gate h) * W_up h)
  moe            the top experts by router logit, weighted by the softmax over the chosen logits; an expert bounds its gate from above
                 and its other factor from both sides, g sigmoid(1.702 g) (u + 1); a shared expert times a sigmoid per token
  logits = head . ln(x)

The residual, norms, angles, decays, the recurrence and its state, router, scores and softmax are fp32 in both modes; "bfloat16" rounds
the inputs of the matrix products to bf16 (fp32 sums on the matrix cores) and keeps cached rows in bf16, "float32" keeps everything in
32 bits.  torch holds memory and streams; every arithmetic step is a libi64hip_dense.so kernel.  The step interface is I64MoEModel's, so
the same engine, scheduler and decoders drive it."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from . import ops_dense as D
from .config import PukatarConfig
from .hybrid_runner import HybridRunner
from .model import attention_segments
from .paged_cache import HybridCache


class _StepBuffers:
    def __init__(self, model: "PukatarModel", n: int, m: int):
        f32 = dict(dtype=torch.float32, device=model.device)
        W = model.cfg.width
        self.x = [torch.empty(1, n, W, **f32) for _ in range(2 if model.cfg.loop is not None else 1)]   # the residual; a pass moves it to the other
        self.e = torch.empty(1, n, W, **f32)                    # embedding rows
        self.x0 = torch.empty(n, W, **f32) if model.cfg.loop is not None else None    # the embedding output's part of what a pass starts from
        self.h = torch.empty(n, W, **f32)                       # the normed input of the current layer
        self.y = torch.empty(n, W, **f32)                       # the mixer's result
        self.y2 = torch.empty(n, W, **f32)                      # the feed-forward's
        self.y3 = torch.empty(n if model.max_shared else 0, W, **f32)
        self.p = torch.empty(n * model.max_proj, **f32)         # everything projected from the layer's input
        self.a = torch.empty(n * model.max_a, **f32)            # query rows / convolution output
        self.b = torch.empty(n * model.max_b, **f32)            # attention output / recurrence output
        self.c = torch.empty(n * model.max_rv, **f32)           # normed recurrence output
        self.f = torch.empty(n * model.max_rk, **f32)           # decays per key channel
        self.z = torch.empty(n * model.max_rv, **f32)           # raw output gates
        self.g = torch.empty(n * 2 * model.max_delta_heads, **f32)      # write strengths
        self.act = torch.empty(n * max(model.max_act, 1), **f32)
        HybridRunner.moe_buffers(self, model, n)
        self.xf = torch.empty(m, W, **f32)
        self.logits = torch.empty(m, model.cfg.vocab, **f32)
        self.attn_ws: Dict[tuple, torch.Tensor] = {}


class PukatarModel(HybridRunner):
    BUFFERS = _StepBuffers
    SIDE_STREAM = True

    def __init__(self, cfg: PukatarConfig, weights: Dict[str, torch.Tensor], device="cuda:0", dtype: str = "bfloat16", max_seqs: int = 4,
                 num_kv_blocks: int = 256, kv_block: int = 16, cache_dtype: Optional[torch.dtype] = None):
        self._init_runner(cfg, device, dtype)
        dev, bf, f, need, W = self.device, self._bf, self._f, self._reader(weights), cfg.width
        self._norm = lambda name: (f(need(name, (W,))), f(need(name + ".b", (W,))))
        self.embed, self.head = bf(need("embed", (cfg.vocab, W))), bf(need("head", (cfg.vocab, W)))
        self.embed_norm, self.final_norm = self._norm("embed.norm"), self._norm("final.norm")
        self.ones1 = torch.ones(1, dtype=torch.float32, device=dev)
        if cfg.loop is not None:
            # W_in [x; x0] = A x + B x0: the second part is the same for every pass and is computed once
            w = need("loop.in", (W, 2 * W))
            self.loop_x, self.loop_x0 = bf(w[:, :W]), bf(w[:, W:])
            self.loop_step = f(need("loop.step", (cfg.loop.times, W)))
        self.layers: List[dict] = [self._load_layer(i, L, weights, need) for i, L in enumerate(cfg.layers)]
        self.layer_runs = cfg.layer_runs()
        specs = []
        for i, _ in self.layer_runs:      # one cache and state per run of a layer
            L = cfg.layers[i]
            m = L.mixer
            if L.type == "attention":
                specs.append({"rows": m.kv_heads * (m.vdim + m.dim), "kscale": False})
            else:
                state = {"gdn": (m.heads, m.vdim, m.dim)}
                if m.conv > 1:
                    state["conv"] = (m.conv - 1, m.conv_channels)
                specs.append({"state": state})
        deltas = [L.mixer for L in cfg.layers if L.type == "channel_delta"]
        self.max_proj = max(d["ld"] for d in self.layers)
        self.max_a = max(d["n_a"] for d in self.layers)
        self.max_b = max(d["n_b"] for d in self.layers)
        self.max_rk = max([m.heads * m.dim for m in deltas] or [0])
        self.max_rv = max([m.heads * m.vdim for m in deltas] or [0])
        self.max_delta_heads = max([m.heads for m in deltas] or [0])
        self._moe_sizes([l.mlp for l in cfg.layers])
        if cache_dtype is None:
            cache_dtype = torch.float32 if self.exact else torch.bfloat16
        self.kv = HybridCache(specs, num_kv_blocks, max_seqs, dev, dtype=cache_dtype, block=kv_block)

    # ---- load-time layout work: one weight for everything that reads the layer's input; small vectors and tables in fp32 ----
    def _load_layer(self, i: int, L, weights, need) -> dict:
        W, p, bf, f = self.cfg.width, f"l{i}.", self._bf, self._f
        d = dict(type=L.type, m=L.mixer, mlp=L.mlp)
        d["norm1"] = self._norm(p + "norm1")
        m, mp = L.mixer, p + "mix."
        if L.type == "attention":
            nq, nk, nv = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
            d["w_in"], (d["q_off"], d["k_off"], d["v_off"]) = self._stack([need(mp + "q", (nq, W)), need(mp + "k", (nk, W)), need(mp + "v", (nv, W))])
            d["sink"] = f(need(mp + "sink", (m.heads,)))
            self._rotary_tables(m, d)
            d["o"] = bf(need(mp + "o", (W, m.heads * m.vdim)))
            d["n_a"], d["n_b"] = m.heads * (m.vdim + m.dim), m.heads * m.vdim
        else:
            rk, rv, nd = m.kv_heads * m.dim, m.heads * m.vdim, m.heads * m.dim
            a1, d["a2"] = self._low_rank(weights, need, mp + "a1", mp + "a2", nd)
            g1, d["g2"] = self._low_rank(weights, need, mp + "g1", mp + "g2", rv)
            conv = torch.cat([need(mp + "q", (rk, W)), need(mp + "k", (rk, W)), need(mp + "v", (rv, W))], 0)      # the three convolved parts side by side
            d["w_in"], (d["r_off"], d["a1_off"], d["g1_off"], d["rb_off"]) = self._stack([conv, a1, g1, need(mp + "b", (m.heads, W))])
            d["conv_w"] = f(torch.cat([need(mp + "q.conv", (rk, m.conv)), need(mp + "k.conv", (rk, m.conv)), need(mp + "v.conv", (rv, m.conv))], 0))
            d["a_rate"] = f(need(mp + "A_log", (m.heads,))).exp().repeat_interleave(m.dim).contiguous()      # exp(A_log), per key channel of every head
            d["dt_bias"] = f(need(mp + "dt_bias", (nd,)))
            d["r_norm"] = f(need(mp + "norm", (m.vdim,)))
            d["o_right"] = bf(need(mp + "o", (W, rv)))
            d["n_a"], d["n_b"] = m.conv_channels, rv
        d["ld"] = d["w_in"].shape[0]
        ff = L.mlp
        if ff is not None and ff.kind == "dense":
            self._load_dense(p + "mlp.", ff, need, d)
        elif ff is not None:
            self._load_moe(p + "mlp.", ff, need, d)
        return d

    def _feed_forward(self, B, d, n, record, r) -> None:
        if d["mlp"].kind == "dense":
            self._dense_glu(B, d, n, B.h, B.y2)
        else:
            self._moe_ff(B, d, n, B.h, B.y2, B.y3, record, f"r{r}")

    @torch.no_grad()
    def forward(self, token_ids: torch.Tensor, positions: torch.Tensor, slot_ids: torch.Tensor, ctx_len: Optional[torch.Tensor] = None,
                logit_rows: Optional[torch.Tensor] = None, max_ctx_hint: int = 0, record: Optional[dict] = None, kv=None,
                rows_are_slots: bool = False, tokens_per_seq: Optional[List[int]] = None) -> torch.Tensor:
        """token_ids int64 [N]; positions / slot_ids int32 [N], rows in sequence order (the rows of a sequence consecutive, positions
        consecutive, continuing what the sequence's slot and pages hold; position 0 starts a sequence afresh); logit_rows int32 [M]
        selects the rows whose logits are wanted (None = all).  Returns fp32 logits [M, V].  record: dict filled with the residual after
        every layer run ("r<k>.x") and every mixture run's chosen experts ("r<k>.route", int32 [N, top]).  kv: a HybridCache other than the
        runner's own.  tokens_per_seq (rows per sequence, in order) or rows_are_slots (every row a sequence of its own) say how the rows are
        grouped; without them the slot ids are read back.  ctx_len and max_ctx_hint belong to the shared step interface."""
        cfg = self.cfg
        kvc = kv if kv is not None else self.kv
        n = token_ids.numel()
        M = logit_rows.numel() if logit_rows is not None else n
        B = self.buffers(n, M)
        if n == 0:
            return B.logits
        eps, ex, hint = cfg.norm_eps, self.exact, int(max_ctx_hint)
        seg, nseg = self._runs(n, slot_ids, tokens_per_seq, rows_are_slots)
        if tokens_per_seq is not None:
            runs = attention_segments(tokens_per_seq, n, self.ATTN_MAX_SEGMENTS)
        else:
            runs = [(0, n, bool(rows_are_slots))]
        # every row the only row of its sequence (a decode step): the convolutions then store their carried inputs in the launch that reads them
        single = bool(rows_are_slots) or (tokens_per_seq is not None and all(int(t) <= 1 for t in tokens_per_seq))
        read = lambda norm, h, **kw: dict(norm_w=norm[0], norm_b=norm[1], eps=eps, h=h, h_center=True, **kw)
        D.embed_scaled(token_ids, self.embed, 1.0, B.e)
        cur = 0
        D.streams_step(B.e, **read(self.embed_norm, B.x[0]))
        if cfg.loop is not None:
            D.linear(B.x[0][0], self.loop_x0, B.x0, exact=ex)
        for r, (l, t) in enumerate(self.layer_runs):
            d = self.layers[l]
            if t is not None:
                D.linear(B.x[cur][0], self.loop_x, B.x[1 - cur][0], exact=ex, bias=self.loop_step[t], epilogue=D.EPI_ADD, e=B.x0, lde=cfg.width)
                cur = 1 - cur
            if r == 0 or t is not None:      # (elsewhere the launch that wrote the residual has normed it)
                D.streams_step(B.x[cur], **read(d["norm1"], B.h))
            # mixer and feed-forward read the same input and meet at the residual: they run side by side
            if d["mlp"] is not None:
                with self._beside():
                    self._feed_forward(B, d, n, record, r)
            P = B.p[: n * d["ld"]].view(n, d["ld"])
            D.linear(B.h, d["w_in"], P, exact=ex)
            if d["type"] == "attention":
                self._rotary_attention(B, d, d["m"], P, r, n, positions, slot_ids, kvc, runs, hint, B.y)
            else:
                self._gated_delta(B, d, d["m"], P, r, n, positions, slot_ids, kvc, seg, nseg, single, B.y)
            write = dict(y=B.y, out_w=self.ones1)
            if d["mlp"] is not None:
                write["y2"] = B.y2
                self._meet()
            if r + 1 < len(self.layer_runs) and self.layer_runs[r + 1][1] is None:
                write.update(read(self.layers[self.layer_runs[r + 1][0]]["norm1"], B.h))
            D.streams_step(B.x[cur], **write)
            if record is not None:
                record[f"r{r}.x"] = B.x[cur][0].clone()
        D.streams_step(B.x[cur], **read(self.final_norm, B.xf, rows=logit_rows))
        D.linear(B.xf, self.head, B.logits, exact=ex)
        return B.logits
