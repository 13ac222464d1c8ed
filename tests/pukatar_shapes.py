"""Small Pukatar configurations and random weights for the tests (no GPU needed to import)."""
import json

import torch


def attn(heads, kv_heads, dim, vdim, rot=None, mask=None, scale=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5}
    if kv_heads is not None:
        m["kv_heads"] = kv_heads
    if rot is not None:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    if mask is not None:
        m["mask"] = {"size": mask[0], "keep_first": mask[1]} if isinstance(mask, tuple) else {"size": mask}
    return {"type": "attention", "mixer": m}


def delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def layer(mix, mlp):
    return dict(mix, mlp=mlp)


# nothing equal and no size a multiple of four, a loop in the middle / the branches a config may leave out (no loop, no mask, no rotation,
# no kept tokens, one tap, all heads their own key head, a layer without feed-forward, a mixture without shared expert) / sizes the
# matrix-core kernels take, every layer inside the loop / other orders: a loop at the end, a window of one token, more kept tokens than the
# window has, a loop that runs once, a single chosen expert
SHAPES = {
    "odd": {"architecture": "Pukatar", "vocab": 83, "width": 42, "norm": {"eps": 1e-5}, "loop": {"start": 1, "stop": 3, "times": 3},
            "layers": [layer(attn(6, 2, 10, 14, (500.0, 6), (13, 3)), dense(50)),
                       layer(delta(4, 2, 10, 6, 3), moe(5, 2, 22, 0.7, (18, 1.1))),
                       layer(attn(3, 3, 18, 6, (90.0, 18), (21, 2), scale=0.4), moe(6, 3, 14, 1.3, (26, 0.5))),
                       layer(delta(3, 1, 14, 9, 5), dense(30)),
                       layer(delta(2, 2, 5, 22, 2), None)],
            "ranks": {1: (3, 7), 3: (10, 4), 4: (1, 9)}},
    "plain": {"architecture": "Pukatar", "vocab": 64, "width": 32, "norm": {"eps": 1e-6},
              "layers": [layer(delta(1, 1, 8, 16, 1), dense(40)),
                         layer(attn(2, None, 16, 8), None),
                         layer(attn(4, 1, 8, 8, (100.0, 4), 9), moe(3, 3, 16, 2.0)),
                         layer(delta(2, 1, 16, 8, 4), moe(4, 1, 24, 1.0, (8, 3.0)))],
              "ranks": {0: (8, 8), 3: (16, 4)}},
    "wide": {"architecture": "Pukatar", "vocab": 200, "width": 128, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 4, "times": 2},
             "layers": [layer(attn(8, 2, 64, 48, (10000.0, 32), (50, 5)), dense(192)),
                        layer(delta(4, 4, 64, 32, 4), moe(8, 3, 48, 1.2, (64, 1.7))),
                        layer(delta(2, 1, 32, 80, 3), dense(160)),
                        layer(attn(4, 4, 32, 64, (5000.0, 32), (33, 40)), moe(4, 2, 32, 0.9, (40, 0.8)))],
             "ranks": {1: (24, 16), 2: (8, 32)}},
    "tail": {"architecture": "Pukatar", "vocab": 51, "width": 36, "norm": {"eps": 1e-6}, "loop": {"start": 2, "stop": 4, "times": 1},
             "layers": [layer(delta(6, 3, 17, 3, 4), moe(7, 1, 12, 0.6, (20, 0.9))),
                        layer(attn(4, 2, 12, 20, (777.0, 8), (1, 4)), dense(28)),
                        layer(attn(5, 1, 6, 4, (64.0, 2), (6, 11)), dense(44)),
                        layer(delta(1, 1, 24, 12, 2), None)],
             "ranks": {0: (5, 11), 3: (2, 2)}},
}


def config_of(name):
    c = json.loads(json.dumps(SHAPES[name]))
    c.pop("ranks")
    return c


def expert_weights(w, p, W, ff, lin):
    w.update({p + "gate": lin(ff, W), p + "up": lin(ff, W), p + "down": lin(W, ff)})


def make_weights(name, seed=0):
    shape = SHAPES[name]
    g = torch.Generator().manual_seed(seed)
    W = shape["width"]
    rn = lambda *s, std=1.0: (torch.randn(*s, generator=g) * std).to(torch.bfloat16)
    un = lambda lo, hi, *s: (torch.rand(tuple(s), generator=g) * (hi - lo) + lo).to(torch.bfloat16)
    lin = lambda o, i: rn(o, i, std=i ** -0.5)
    w = {"embed": rn(shape["vocab"], W, std=0.3), "head": lin(shape["vocab"], W)}

    def norm(p):
        w.update({p: un(0.5, 1.5, W), p + ".b": rn(W, std=0.3)})

    norm("embed.norm"), norm("final.norm")
    if "loop" in shape:
        w.update({"loop.in": lin(W, 2 * W), "loop.step": rn(shape["loop"]["times"], W, std=0.5)})
    for i, L in enumerate(shape["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        mp = p + "mix."
        norm(p + "norm1")
        H, G, d, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
        if L["type"] == "attention":
            w.update({mp + "q": rn(H * d, W, std=2.0 * W ** -0.5), mp + "k": lin(G * d, W), mp + "v": lin(G * dv, W), mp + "sink": rn(H, std=2.0), mp + "o": lin(W, H * dv)})
        else:
            ra, rg = shape["ranks"][i]
            w.update({mp + "q": lin(G * d, W), mp + "k": lin(G * d, W), mp + "v": lin(H * dv, W), mp + "q.conv": rn(G * d, m["conv"], std=0.6),
                      mp + "k.conv": rn(G * d, m["conv"], std=0.6), mp + "v.conv": rn(H * dv, m["conv"], std=0.6), mp + "b": lin(H, W), mp + "a1": lin(ra, W),
                      mp + "a2": lin(H * d, ra), mp + "A_log": un(-3.0, 0.5, H), mp + "dt_bias": rn(H * d), mp + "norm": un(0.5, 1.5, dv), mp + "g1": lin(rg, W),
                      mp + "g2": lin(H * dv, rg), mp + "o": lin(W, H * dv)})
        if f and f["kind"] == "dense":
            expert_weights(w, p + "mlp.", W, f["ff"], lin)
        elif f:
            E = f["router"]["experts"]
            w.update({p + "mlp.router": rn(E, W, std=2.0 * W ** -0.5), p + "mlp.router.b": rn(E)})
            for e in range(E):
                expert_weights(w, f"{p}mlp.e{e}.", W, f["expert"]["ff"], lin)
            if f.get("shared"):
                expert_weights(w, p + "mlp.shared.", W, f["shared"]["ff"], lin)
                w[p + "mlp.shared.sg"] = rn(1, W, std=2.0 * W ** -0.5)
    return w


def tokens(name, n, seed):
    return torch.randint(0, SHAPES[name]["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
