"""Runner of the Vepelix design on one MI355X: a pre-norm decoder with a learned factor per column on every sublayer's result and a stretch
of layers that repeats under the same weights:

  x0 = embed[token];   x = x0
  layer:  x <- x + ls1 * mixer(rms(x) (1 + norm1));   x <- x + ls2 * ff(rms(x) (1 + norm2))
  loop:   layers start .. stop - 1 run `times` times, every pass with a cache and state of its own; in front of every pass but the first:
          x <- x + x0
  latent_attention  queries through a normed low-rank row; one cached row per token - a normed latent, from which every head's unrotated keys
                    and its values are maps, and a rotated key part that all heads share (interleaved pairs, frequencies optionally scaled); a
                    learned sink per head in the softmax's denominator; a sigmoid gate per head
  parallel          left_scale * left + right_scale * right on the same input.  left: windowed attention, queries and keys RMS-normed per head
                    (weights the heads share) and rotated in interleaved pairs.  right: gated linear attention with a decay per key channel
                    (a low-rank map), S <- diag(alpha) S + k v^T, o = S^T q; RMS norm per head times silu(gate)
  dense             the gate bounded from above, the other factor from both sides, W_down (g sigmoid(1.702 g) (u + 1))
  moe               the top experts by sigmoid score, the score (as it is) on the expert's input; a shared expert
  logits = head . (rms(x) (1 + final.norm))

The residual, norms, angles, decays, the recurrence and its state, router, scores and softmax are fp32 in both modes; "bfloat16" rounds
the inputs of the matrix products to bf16 (fp32 sums on the matrix cores) and keeps cached rows in bf16, "float32" keeps everything in
32 bits.  torch holds memory and streams; every arithmetic step is a libi64hip_dense.so kernel.  The step interface is I64MoEModel's, so
the same engine, scheduler and decoders drive it."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from . import ops_dense as D
from .config import VepelixConfig
from .hybrid_runner import HybridRunner
from .model import attention_segments
from .paged_cache import HybridCache


class _StepBuffers:
    def __init__(self, model: "VepelixModel", n: int, m: int):
        f32 = dict(dtype=torch.float32, device=model.device)
        W = model.cfg.width
        self.xe = torch.empty(2 if model.repeats else 1, n, W, **f32)      # the residual; the embedding output, where a further pass adds it
        self.h = torch.empty(n, W, **f32)                       # the normed input of the current sublayer
        self.y = torch.empty(n, W, **f32)                       # a sublayer's result
        self.y2 = torch.empty(n, W, **f32)                      # that of the right one of two side-by-side mixers / the shared expert's
        self.p = torch.empty(n * model.max_proj, **f32)         # everything projected from the mixer's input
        self.q = torch.empty(n * model.max_q, **f32)            # the queries of the latent heads
        self.a = torch.empty(n * model.max_a, **f32)            # query rows of the attention
        self.b = torch.empty(n * model.max_b, **f32)            # attention output
        self.c = torch.empty(n * model.max_c, **f32)            # values of the latent heads
        self.f = torch.empty(n * model.max_rk, **f32)           # decays per key channel
        self.r = torch.empty(n * model.max_rv, **f32)           # recurrence output
        self.rn = torch.empty(n * model.max_rv, **f32)          # ... normed and gated
        self.act = torch.empty(n * max(model.max_act, 1), **f32)
        HybridRunner.moe_buffers(self, model, n)
        self.xf = torch.empty(m, W, **f32)
        self.logits = torch.empty(m, model.cfg.vocab, **f32)
        self.attn_ws: Dict[tuple, torch.Tensor] = {}


class VepelixModel(HybridRunner):
    BUFFERS = _StepBuffers
    SIDE_STREAM = True

    def __init__(self, cfg: VepelixConfig, weights: Dict[str, torch.Tensor], device="cuda:0", dtype: str = "bfloat16", max_seqs: int = 4,
                 num_kv_blocks: int = 256, kv_block: int = 16, cache_dtype: Optional[torch.dtype] = None):
        self._init_runner(cfg, device, dtype)
        dev, bf, f, need, W = self.device, self._bf, self._f, self._reader(weights), cfg.width
        self._norm = lambda name: f(1.0 + need(name, (W,)).float())      # (stored as the distance from one)
        self.embed, self.head = bf(need("embed", (cfg.vocab, W))), bf(need("head", (cfg.vocab, W)))
        self.final_norm = self._norm("final.norm")
        self.ones1 = torch.ones(1, dtype=torch.float32, device=dev)
        self.layers: List[dict] = [self._load_layer(i, L, weights, need) for i, L in enumerate(cfg.layers)]
        self.layer_runs = cfg.layer_runs()
        self.repeats = any(t for _, t in self.layer_runs)
        specs = []
        for i, _ in self.layer_runs:      # one cache and state per run of a layer
            m = cfg.layers[i].mixer
            if cfg.layers[i].type == "latent_attention":
                specs.append({"rows": m.cache_width, "kscale": False})
            else:
                a, r = m.left, m.right
                specs.append({"rows": a.kv_heads * (a.vdim + a.dim), "kscale": False, "state": {"gla": (r.heads, r.vdim, r.dim)}})
        latents = [L.mixer for L in cfg.layers if L.type == "latent_attention"]
        rights = [L.mixer.right for L in cfg.layers if L.type == "parallel"]
        self.max_proj = max(d["ld"] for d in self.layers)
        self.max_a = max(d["n_a"] for d in self.layers)
        self.max_b = max(d["n_b"] for d in self.layers)
        self.max_c = max([m.heads * m.vdim for m in latents] or [0])
        self.max_q = max([m.q_width for m in latents] or [0])
        self.max_rk = max([r.heads * r.dim for r in rights] or [0])
        self.max_rv = max([r.heads * r.vdim for r in rights] or [0])
        self._moe_sizes([l.mlp for l in cfg.layers])
        if cache_dtype is None:
            cache_dtype = torch.float32 if self.exact else torch.bfloat16
        self.kv = HybridCache(specs, num_kv_blocks, max_seqs, dev, dtype=cache_dtype, block=kv_block)

    # ---- load-time layout work: one weight for everything that reads the mixer's input; small vectors and tables in fp32 ----
    def _load_layer(self, i: int, L, weights, need) -> dict:
        W, p, bf, f = self.cfg.width, f"l{i}.", self._bf, self._f
        d = dict(type=L.type, m=L.mixer, mlp=L.mlp)
        d["norm1"], d["ls1"] = self._norm(p + "norm1"), f(need(p + "ls1", (W,)))
        m = L.mixer
        if L.type == "latent_attention":
            d["w_in"], (d["q_off"], d["dkv_off"], d["g_off"]) = self._stack(self._load_latent(p + "mix.", m, need, d))
            d["n_a"], d["n_b"] = m.heads * m.cache_width, m.heads * m.kv_rank
        else:
            a, r, lp, rp = m.left, m.right, p + "mix.left.", p + "mix.right."
            rk, rv = r.heads * r.dim, r.heads * r.vdim
            a1, a2 = self._low_rank(weights, need, rp + "a1", rp + "a2", rk)
            d["w_in"], (d["q_off"], d["k_off"], d["v_off"], d["rq_off"], d["rk_off"], d["rv_off"], d["rg_off"], d["a1_off"]) = self._stack(
                [need(lp + "q", (a.heads * a.dim, W)), need(lp + "k", (a.kv_heads * a.dim, W)), need(lp + "v", (a.kv_heads * a.vdim, W)),
                 need(rp + "q", (rk, W)), need(rp + "k", (rk, W)), need(rp + "v", (rv, W)), need(rp + "g", (rv, W)), a1])
            d["q_norm"], d["k_norm"] = f(need(lp + "q.norm", (a.dim,))), f(need(lp + "k.norm", (a.dim,)))
            self._rotary_tables(a, d)
            d["o"] = bf(need(lp + "o", (W, a.heads * a.vdim)))
            d["a2"], d["a2_b"] = -a2, f(-need(rp + "a2.b", (rk,)).float())
            d["a_rate"] = torch.full((rk,), 1.0 / r.tau, dtype=torch.float32, device=self.device)
            d["r_norm"] = f(need(rp + "norm", (r.vdim,)))
            d["o_right"] = bf(need(rp + "o", (W, rv)))
            d["n_a"], d["n_b"] = a.heads * (a.vdim + a.dim), a.heads * a.vdim
        d["ld"] = d["w_in"].shape[0]
        if L.mlp is not None:
            d["norm2"], d["ls2"] = self._norm(p + "norm2"), f(need(p + "ls2", (W,)))
            if L.mlp.kind == "dense":
                self._load_dense(p + "mlp.", L.mlp, need, d)
            else:
                self._load_moe(p + "mlp.", L.mlp, need, d)
        return d

    # ---- sublayers: the input is B.h, the result lands in B.y (and B.y2, to be added) ----
    def _mixer(self, B, d, r, n, positions, slot_ids, kvc, seg, nseg, runs, hint) -> dict:
        """Returns the operands of the residual's write."""
        m = d["m"]
        P = B.p[: n * d["ld"]].view(n, d["ld"])
        D.linear(B.h, d["w_in"], P, exact=self.exact)
        if d["type"] == "latent_attention":
            self._latent_attention(B, d, m, P, r, n, positions, slot_ids, kvc, runs, hint, B.y)
            return dict(y=B.y)
        with self._beside():      # attention and recurrence share nothing but the projection rows
            self._rotary_attention(B, d, m.left, P, r, n, positions, slot_ids, kvc, runs, hint, B.y, m.left_scale)
        self._gated_linear(B, d, m.right, P, r, n, positions, slot_ids, kvc, seg, nseg, B.y2, m.right_scale)
        self._meet()
        return dict(y=B.y, y2=B.y2)

    def _feed_forward(self, B, d, n, record, r) -> None:
        if d["mlp"].kind == "dense":
            self._dense_glu(B, d, n, B.h, B.y)
        else:
            self._moe_ff(B, d, n, B.h, B.y, B.y2, record, f"r{r}", beside=True)

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
        seg, nseg = self._runs(n, slot_ids, tokens_per_seq, rows_are_slots)
        if tokens_per_seq is not None:
            runs = attention_segments(tokens_per_seq, n, self.ATTN_MAX_SEGMENTS)
        else:
            runs = [(0, n, bool(rows_are_slots))]
        read = lambda w, h, **kw: dict(norm_w=w, eps=cfg.norm_eps, h=h, **kw)
        D.embed_bigram(token_ids, positions, slot_ids, self.embed, B.xe)      # (a plane each for the residual and the embedding output)
        x = B.xe[0:1]
        for r, (l, t) in enumerate(self.layer_runs):
            d = self.layers[l]
            if r == 0:
                D.streams_step(x, **read(d["norm1"], B.h))
            elif t:
                D.streams_step(x, y=B.xe[1], out_w=self.ones1, **read(d["norm1"], B.h))
            # (elsewhere the launch that wrote the residual has normed it)
            write = self._mixer(B, d, r, n, positions, slot_ids, kvc, seg, nseg, runs, int(max_ctx_hint))
            write.update(out_w=self.ones1, y_scale=d["ls1"])
            if d["mlp"] is not None:
                D.streams_step(x, **write, **read(d["norm2"], B.h))
                self._feed_forward(B, d, n, record, r)
                write = dict(y=B.y, out_w=self.ones1, y_scale=d["ls2"])
            if r + 1 < len(self.layer_runs) and not self.layer_runs[r + 1][1]:
                write.update(read(self.layers[self.layer_runs[r + 1][0]]["norm1"], B.h))
            D.streams_step(x, **write)
            if record is not None:
                record[f"r{r}.x"] = B.xe[0].clone()
        D.streams_step(x, **read(self.final_norm, B.xf, rows=logit_rows))
        D.linear(B.xf, self.head, B.logits, exact=self.exact)
        return B.logits
