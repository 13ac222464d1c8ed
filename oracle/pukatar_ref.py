"""CPU oracle (TEST INFRASTRUCTURE ONLY) of the Pukatar design: a plain, slow restatement of its equations in 64-bit torch, one
function per mechanism, one whole sequence at a time, token-by-token loops for everything recurrent or causal, no cache, no state
object and no code shared with vllm_i64_amd/.  However the product path cuts, batches, pages and slots a sequence, its logits at a
position must agree with this file's.

Notation: T tokens, width w; weights `W[name]` as stored ([out, in] matrices); `m` a layer's 'mixer' entry of the config, `f` its
'mlp' entry, `p` the prefix of its tensors.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

F64 = torch.float64


def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt(c.pow(2).mean(-1, keepdim=True) + eps) * w + b


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.logaddexp(z, torch.zeros_like(z))


# ---- rotation, visibility, softmax with a sink -------------------------------------------------------------------------------------
def rotate_halves(x: torch.Tensor, pos: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """x [T, heads, d]: value i < dims / 2 of every head turns against value i + dims / 2 by pos * base^(-2i / dims)."""
    half = dims // 2
    out = x.clone()
    for i in range(half):
        a = pos.to(F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a).unsqueeze(-1), torch.sin(a).unsqueeze(-1)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def sees(i: int, j: int, mask: Optional[dict]) -> bool:
    """A window of mask.size positions that ends at the query, and the first mask.keep_first positions of the sequence for everyone."""
    if j > i:
        return False
    if not mask or not mask.get("size"):
        return True
    return i - j < int(mask["size"]) or j < int(mask.get("keep_first") or 0)


def sink_softmax(s: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """Weights of the scores s when one more term exp(sink), which has no value, counts in the denominator."""
    top = torch.maximum(s.max(), sink)
    e = torch.exp(s - top)
    return e / (e.sum() + torch.exp(sink - top))


def windowed_attention(W: Dict[str, torch.Tensor], p: str, m: dict, h: torch.Tensor) -> torch.Tensor:
    T = h.shape[0]
    H, G = int(m["heads"]), int(m.get("kv_heads", m["heads"]))
    d, dv = int(m["dim"]), int(m.get("vdim", m["dim"]))
    q, k, v = (h @ W[p + "q"].T).reshape(T, H, d), (h @ W[p + "k"].T).reshape(T, G, d), (h @ W[p + "v"].T).reshape(T, G, dv)
    rot = m.get("rot")
    if rot:
        pos = torch.arange(T)
        q, k = rotate_halves(q, pos, float(rot["base"]), int(rot["dims"])), rotate_halves(k, pos, float(rot["base"]), int(rot["dims"]))
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        js = [j for j in range(i + 1) if sees(i, j, m.get("mask"))]
        for a in range(H):
            g = a // (H // G)
            out[i, a] = sink_softmax((k[js, g] @ q[i, a]) * float(m["scale"]), W[p + "sink"][a]) @ v[js, g]
    return out.reshape(T, H * dv) @ W[p + "o"].T


# ---- delta rule with a decay per key channel ---------------------------------------------------------------------------------------
def short_convolution(w: torch.Tensor, x: torch.Tensor) -> torch.Tensor:
    """Per channel over time, the last column of w [channels, taps] on the current token, nothing before the first token; then silu."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1 - j)
            if s >= 0:
                out[t] = out[t] + w[:, j] * x[s]
    return silu(out)


def channel_decay(z: torch.Tensor, a_log: torch.Tensor, dt_bias: torch.Tensor, d: int) -> torch.Tensor:
    """z [T, H * d] -> factors in (0, 1), [T, H, d]: exp(-exp(a_log_h) softplus(z + dt_bias))."""
    T, H = z.shape[0], a_log.numel()
    step = softplus(z + dt_bias).reshape(T, H, d)
    return torch.exp(-torch.exp(a_log).reshape(1, H, 1) * step)


def channel_delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, beta: torch.Tensor, g: torch.Tensor) -> torch.Tensor:
    """q, k, g [T, H, d], v [T, H, dv], beta [T, H]: every row of the state decays by its own channel's factor, the state is corrected
    towards v along k with strength beta, and is read by q after the write."""
    T, H, d = q.shape
    dv = v.shape[-1]
    S = torch.zeros(H, d, dv, dtype=F64)
    o = torch.zeros(T, H, dv, dtype=F64)
    for t in range(T):
        S = S * g[t].unsqueeze(-1)
        u = beta[t].reshape(H, 1) * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(-2)
        o[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return o


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def channel_delta(W: Dict[str, torch.Tensor], p: str, m: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    T = h.shape[0]
    H, G = int(m["heads"]), int(m.get("kv_heads", m["heads"]))
    d, dv = int(m["dim"]), int(m.get("vdim", m["dim"]))
    q = short_convolution(W[p + "q.conv"], h @ W[p + "q"].T).reshape(T, G, d)
    k = short_convolution(W[p + "k.conv"], h @ W[p + "k"].T).reshape(T, G, d)
    v = short_convolution(W[p + "v.conv"], h @ W[p + "v"].T).reshape(T, H, dv)
    own = torch.arange(H) // (H // G)
    q, k = (unit(q) * d ** -0.5)[:, own], unit(k)[:, own]
    beta = torch.sigmoid(h @ W[p + "b"].T)
    g = channel_decay((h @ W[p + "a1"].T) @ W[p + "a2"].T, W[p + "A_log"], W[p + "dt_bias"], d)
    o = channel_delta_rule(q, k, v, beta, g)
    o = o / torch.sqrt(o.pow(2).mean(-1, keepdim=True) + eps) * W[p + "norm"]
    o = o * torch.sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T).reshape(T, H, dv)
    return o.reshape(T, H * dv) @ W[p + "o"].T


# ---- feed-forwards -------------------------------------------------------------------------------------------------------------
def dense_ff(W: Dict[str, torch.Tensor], p: str, h: torch.Tensor) -> torch.Tensor:
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def clamped_expert(W: Dict[str, torch.Tensor], p: str, limit: float, h: torch.Tensor) -> torch.Tensor:
    """The gate bounded from above, the other factor from both sides and shifted by one."""
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def route(z: torch.Tensor, top: int):
    """z [T, experts] -> the `top` largest logits' indices and the softmax over those alone."""
    v, idx = z.topk(top, -1)
    return idx, torch.softmax(v, -1)


def mixture_ff(W: Dict[str, torch.Tensor], p: str, f: dict, h: torch.Tensor, forced: Optional[torch.Tensor] = None, chosen: Optional[list] = None) -> torch.Tensor:
    """forced [T, top]: experts to use instead of the router's own choice (their weights still come from the router's logits) - for
    comparisons with an implementation in lower precision, where a close call may fall the other way; chosen receives the choice."""
    z = h @ W[p + "router"].T + W[p + "router.b"]
    idx, wgt = route(z, int(f["router"]["top"]))
    if forced is not None:
        idx = forced.to(torch.int64)
        wgt = torch.softmax(z.gather(1, idx), -1)
    if chosen is not None:
        chosen.append(idx)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(idx[t].tolist(), wgt[t]):
            out[t] += g * clamped_expert(W, f"{p}e{e}.", float(f["expert"]["limit"]), h[t:t + 1])[0]
    if f.get("shared"):
        out = out + torch.sigmoid(h @ W[p + "shared.sg"].T) * clamped_expert(W, p + "shared.", float(f["shared"]["limit"]), h)
    return out


def feed_forward(W: Dict[str, torch.Tensor], p: str, f: Optional[dict], h: torch.Tensor, **route_options) -> torch.Tensor:
    if not f:
        return torch.zeros_like(h)
    return dense_ff(W, p, h) if f.get("kind", "dense") == "dense" else mixture_ff(W, p, f, h, **route_options)


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


def enter_pass(W: Dict[str, torch.Tensor], t: int, x: torch.Tensor, x0: torch.Tensor) -> torch.Tensor:
    """What a pass over the repeated layers starts from: a map of the residual and the embedding output side by side, plus the pass's vector."""
    return torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], layers_out: Optional[list] = None, routes: Optional[dict] = None,
            chosen: Optional[dict] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence (64-bit).  layers_out receives the residual after every layer run; routes: layer run -> experts
    [T, top] to use instead of the router's choice; chosen (a dict) receives every mixture layer run's choice."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    x0 = layer_norm(W["embed"][tokens], W["embed.norm"], W["embed.norm.b"], eps)
    x = x0
    for r, (i, t) in enumerate(layer_runs(config)):
        if t is not None:
            x = enter_pass(W, t, x, x0)
        L, p = config["layers"][i], f"l{i}."
        h = layer_norm(x, W[p + "norm1"], W[p + "norm1.b"], eps)
        if L["type"] == "attention":
            y = windowed_attention(W, p + "mix.", L["mixer"], h)
        elif L["type"] == "channel_delta":
            y = channel_delta(W, p + "mix.", L["mixer"], eps, h)
        else:
            raise ValueError(L["type"])
        got: list = []
        opts = dict(forced=(routes or {}).get(r), chosen=got) if (L.get("mlp") or {}).get("kind") == "moe" else {}
        x = x + (y + feed_forward(W, p + "mlp.", L.get("mlp"), h, **opts))
        if got and chosen is not None:
            chosen[r] = got[0]
        if layers_out is not None:
            layers_out.append(x.clone())
    return layer_norm(x, W["final.norm"], W["final.norm.b"], eps) @ W["head"].T
