"""CPU oracle (TEST INFRASTRUCTURE ONLY) of the Vepelix design: a plain, slow restatement of its equations in 64-bit torch, one
function per mechanism, one whole sequence at a time, token-by-token loops for everything recurrent or causal, no cache, no state
object and no code shared with vllm_i64_amd/.  However the product path cuts, batches, pages and slots a sequence, its logits at a
position must agree with this file's.

Notation: T tokens, width w; weights `W[name]` as stored ([out, in] matrices); `m` a mixer's entry of the config, `f` a layer's 'mlp'
entry, `p` the prefix of the tensors.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def one_plus_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """The stored weight is the distance from one."""
    return rms(x, eps) * (1.0 + w)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


# ---- rotation ------------------------------------------------------------------------------------------------------------------------
def frequencies(rot: dict):
    """([dims / 2] frequencies, the factor on sine and cosine).  With scaling: pairs that turn often within `original` positions keep their
    frequency, slow ones are divided by `factor`, between the two a linear ramp over the pair's index."""
    base, dims = float(rot["base"]), int(rot["dims"])
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return plain, 1.0

    def index_of(turns: float) -> float:      # the (real) pair index, times two over two, whose period fits `turns` times into `original`
        return dims * math.log(float(sc["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(float(sc["fast"]))), 0)
    hi = min(math.ceil(index_of(float(sc["slow"]))), dims - 1)
    span = max(hi - lo, 0.001)
    out = []
    for i, f in enumerate(plain):
        r = (i - lo) / span
        r = 0.0 if r < 0.0 else (1.0 if r > 1.0 else r)
        out.append(r * f / float(sc["factor"]) + (1.0 - r) * f)
    return out, 1.0 + 0.1 * math.log(float(sc["factor"]))


def rotate_pairs(x: torch.Tensor, pos: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [T, heads, d]: values 2i and 2i + 1 of every head turn against each other, i < dims / 2; the rest pass."""
    if not rot:
        return x
    fs, mult = frequencies(rot)
    out = x.clone()
    for i, f in enumerate(fs):
        a = pos.to(F64) * f
        c, s = (torch.cos(a) * mult).unsqueeze(-1), (torch.sin(a) * mult).unsqueeze(-1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


# ---- attention over a window, queries and keys normed per head -------------------------------------------------------------------------
def sees(i: int, j: int, mask: Optional[dict]) -> bool:
    size = int((mask or {}).get("size") or 0)
    return j <= i and (size <= 0 or i - j < size)


def window_attention(W: Dict[str, torch.Tensor], p: str, m: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    T = h.shape[0]
    H, G = int(m["heads"]), int(m.get("kv_heads", m["heads"]))
    d, dv = int(m["dim"]), int(m.get("vdim", m["dim"]))
    q, k, v = (h @ W[p + "q"].T).reshape(T, H, d), (h @ W[p + "k"].T).reshape(T, G, d), (h @ W[p + "v"].T).reshape(T, G, dv)
    pos = torch.arange(T)
    q = rotate_pairs(rms(q, eps) * W[p + "q.norm"], pos, m.get("rot"))
    k = rotate_pairs(rms(k, eps) * W[p + "k.norm"], pos, m.get("rot"))
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        js = [j for j in range(i + 1) if sees(i, j, m.get("mask"))]
        for a in range(H):
            g = a // (H // G)
            out[i, a] = torch.softmax((k[js, g] @ q[i, a]) * float(m["scale"]), 0) @ v[js, g]
    return out.reshape(T, H * dv) @ W[p + "o"].T


# ---- gated linear attention ------------------------------------------------------------------------------------------------------------
def channel_decay(z: torch.Tensor, tau: float) -> torch.Tensor:
    return torch.sigmoid(z) ** (1.0 / tau)


def gated_linear_recurrence(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, alpha: torch.Tensor) -> torch.Tensor:
    """q, k, alpha [T, H, d], v [T, H, dv]: the rows of a head's state decay by their channel's factor, the token writes, then reads."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=F64)
    o = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for t in range(T):
        S = alpha[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        o[t] = (q[t].unsqueeze(-1) * S).sum(-2)
    return o


def linear_attention(W: Dict[str, torch.Tensor], p: str, m: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m.get("vdim", m["dim"]))
    q = (h @ W[p + "q"].T).reshape(T, H, d) * d ** -0.5
    k, v = (h @ W[p + "k"].T).reshape(T, H, d), (h @ W[p + "v"].T).reshape(T, H, dv)
    alpha = channel_decay((h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"], float(m["tau"])).reshape(T, H, d)
    o = rms(gated_linear_recurrence(q, k, v, alpha), eps) * W[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel_mixer(W: Dict[str, torch.Tensor], p: str, m: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    return float(m["left_scale"]) * window_attention(W, p + "left.", m["left"], eps, h) + \
        float(m["right_scale"]) * linear_attention(W, p + "right.", m["right"], eps, h)


# ---- latent attention --------------------------------------------------------------------------------------------------------------------
def sink_softmax(s: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """Weights of the scores s when one more term exp(sink), which has no value, counts in the denominator."""
    top = torch.maximum(s.max(), sink)
    e = torch.exp(s - top)
    return e / (e.sum() + torch.exp(sink - top))


def latent_attention(W: Dict[str, torch.Tensor], p: str, m: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    T = h.shape[0]
    H, d, dr, dv, r = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    pos = torch.arange(T)
    q = ((rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]) @ W[p + "uq"].T).reshape(T, H, d + dr)
    qn, qr = q[..., :d], rotate_pairs(q[..., d:], pos, m.get("rot"))
    down = h @ W[p + "dkv"].T
    c = rms(down[:, :r], eps) * W[p + "dkv.norm"]
    kr = rotate_pairs(down[:, r:].reshape(T, 1, dr), pos, m.get("rot"))[:, 0]
    kn, v = (c @ W[p + "uk"].T).reshape(T, H, d), (c @ W[p + "uv"].T).reshape(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        for a in range(H):
            s = (kn[:i + 1, a] @ qn[i, a] + kr[:i + 1] @ qr[i, a]) * float(m["scale"])
            out[i, a] = sink_softmax(s, W[p + "sink"][a]) @ v[:i + 1, a]
    out = out * torch.sigmoid(h @ W[p + "g"].T).unsqueeze(-1)
    return out.reshape(T, H * dv) @ W[p + "o"].T


# ---- feed-forwards -------------------------------------------------------------------------------------------------------------
def clamped_ff(W: Dict[str, torch.Tensor], p: str, limit: float, h: torch.Tensor) -> torch.Tensor:
    """The gate bounded from above, the other factor from both sides and shifted by one."""
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def expert(W: Dict[str, torch.Tensor], p: str, h: torch.Tensor) -> torch.Tensor:
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(z: torch.Tensor, top: int):
    """z [T, experts] -> the `top` entries of the largest sigmoid scores and those scores as they are."""
    s = torch.sigmoid(z)
    idx = z.topk(top, -1).indices       # (the sigmoid keeps the order)
    return idx, s.gather(1, idx)


def mixture_ff(W: Dict[str, torch.Tensor], p: str, f: dict, h: torch.Tensor, forced: Optional[torch.Tensor] = None, chosen: Optional[list] = None) -> torch.Tensor:
    """A chosen expert sees its score times the row.  forced [T, top]: experts to use instead of the router's own choice (their weights still
    come from the router's logits) - for comparisons with an implementation in lower precision, where a close call may fall the other
    way; chosen receives the choice."""
    z = h @ W[p + "router"].T
    idx, wgt = route(z, int(f["router"]["top"]))
    if forced is not None:
        idx = forced.to(torch.int64)
        wgt = torch.sigmoid(z.gather(1, idx))
    if chosen is not None:
        chosen.append(idx)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(idx[t].tolist(), wgt[t]):
            out[t] += expert(W, f"{p}e{e}.", g * h[t:t + 1])[0]
    if f.get("shared"):
        out = out + expert(W, p + "shared.", h)
    return out


def feed_forward(W: Dict[str, torch.Tensor], p: str, f: dict, h: torch.Tensor, **route_options) -> torch.Tensor:
    return clamped_ff(W, p, float(f["limit"]), h) if f.get("kind", "dense") == "dense" else mixture_ff(W, p, f, h, **route_options)


# ---- the model -----------------------------------------------------------------------------------------------------------------
def layer_runs(config: dict):
    """[(layer, pass that starts in front of it or None)] in the order they run."""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    runs = [(i, None) for i in range(a)]
    for t in range(int(loop["times"])):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], layers_out: Optional[list] = None, routes: Optional[dict] = None,
            chosen: Optional[dict] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence (64-bit).  layers_out receives the residual after every layer run; routes: layer run -> experts
    [T, top] to use instead of the router's choice; chosen (a dict) receives every mixture layer run's choice."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    x0 = W["embed"][tokens]
    x = x0
    for r, (i, t) in enumerate(layer_runs(config)):
        if t:                                   # every pass but the first starts from the residual plus the embedding
            x = x + x0
        L, p = config["layers"][i], f"l{i}."
        h = one_plus_norm(x, W[p + "norm1"], eps)
        if L["type"] == "parallel":
            y = parallel_mixer(W, p + "mix.", L["mixer"], eps, h)
        elif L["type"] == "latent_attention":
            y = latent_attention(W, p + "mix.", L["mixer"], eps, h)
        else:
            raise ValueError(L["type"])
        x = x + W[p + "ls1"] * y
        if L.get("mlp"):
            got: list = []
            opts = dict(forced=(routes or {}).get(r), chosen=got) if L["mlp"].get("kind") == "moe" else {}
            x = x + W[p + "ls2"] * feed_forward(W, p + "mlp.", L["mlp"], one_plus_norm(x, W[p + "norm2"], eps), **opts)
            if got and chosen is not None:
                chosen[r] = got[0]
        if layers_out is not None:
            layers_out.append(x.clone())
    return one_plus_norm(x, W["final.norm"], eps) @ W["head"].T
