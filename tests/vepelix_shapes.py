"""Small Vepelix configurations and random weights for the tests (no GPU needed to import)."""
import json

import torch


def rotation(base, dims, scaling=None):
    r = {"base": base, "dims": dims}
    if scaling is not None:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, base=5000.0, scaling=(4.0, 60, 6.0, 0.5), scale=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                                                  "scale": scale if scale is not None else (dim + rot_dim) ** -0.5, "rot": rotation(base, rot_dim, scaling)}}


def parallel(heads, kv_heads, dim, vdim, rot, size, rec_heads, rec_dim, rec_vdim, tau, scales, scale=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": rot, "scale": scale if scale is not None else dim ** -0.5}
    if size:
        left["mask"] = {"size": size}
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": rec_heads, "dim": rec_dim, "vdim": rec_vdim, "tau": tau}, "left_scale": scales[0], "right_scale": scales[1]}}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(mix, mlp):
    return dict(mix, mlp=mlp)


# nothing equal and no size a multiple of four, a loop in the middle that runs three times / the branches a config may leave out (no loop,
# no scaling of frequencies, no mask, all heads their own key head, a layer without feed-forward, a mixture without shared expert, a rank of one)
# / sizes the matrix-core kernels take, every layer inside the loop / other orders: a loop of one layer at the end, a loop that runs once, a
# window of one token, factors of one, a time constant of one, negative and equal constants
SHAPES = {
    "odd": {"architecture": "Vepelix", "vocab": 83, "width": 42, "norm": {"eps": 1e-5}, "loop": {"start": 1, "stop": 3, "times": 3},
            "layers": [layer(latent(3, 10, 6, 14, 18, 22), dense(50, 0.8)),
                       layer(parallel(6, 2, 10, 14, rotation(500.0, 6, (8.0, 40, 4.0, 1.0)), 13, 5, 18, 7, 5.0, (1.3, 0.7)), moe(5, 2, 22, 18)),
                       layer(latent(5, 6, 2, 9, 27, 13, scaling=None, scale=0.3), moe(6, 3, 14, 26)),
                       layer(parallel(3, 3, 18, 6, rotation(90.0, 18), 21, 2, 9, 22, 12.0, (0.6, 1.9), scale=0.4), None),
                       layer(latent(1, 33, 10, 5, 7, 3), moe(4, 1, 11))],
            "ranks": {1: 3, 3: 10}},
    "plain": {"architecture": "Vepelix", "vocab": 64, "width": 32, "norm": {"eps": 1e-6},
              "layers": [layer(parallel(2, 2, 8, 8, rotation(10000.0, 8), 0, 1, 8, 16, 16.0, (1.0, 1.0)), dense(40, 2.0)),
                         layer(latent(4, 8, 8, 8, 16, 1, scaling=None), None),
                         layer(parallel(4, 1, 16, 24, rotation(100.0, 4), 9, 2, 16, 8, 4.0, (2.0, 0.5)), moe(3, 3, 16)),
                         layer(latent(2, 16, 4, 32, 8, 24), moe(4, 1, 24, 8))],
              "ranks": {0: 8, 2: 1}},
    "wide": {"architecture": "Vepelix", "vocab": 200, "width": 128, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 4, "times": 2},
             "layers": [layer(latent(4, 32, 16, 48, 48, 64), dense(192, 1.5)),
                        layer(parallel(8, 2, 64, 48, rotation(10000.0, 32, (4.0, 100, 16.0, 2.0)), 50, 4, 64, 32, 10.0, (0.9, 1.4)), moe(8, 3, 48, 64)),
                        layer(latent(18, 16, 8, 16, 128, 40), moe(4, 2, 32, 40)),
                        layer(parallel(4, 4, 32, 64, rotation(5000.0, 32, (2.0, 50, 3.0, 1.0)), 33, 2, 32, 80, 3.0, (1.1, 0.8)), dense(160, 0.7))],
             "ranks": {1: 24, 3: 8}},
    "tail": {"architecture": "Vepelix", "vocab": 51, "width": 36, "norm": {"eps": 1e-6}, "loop": {"start": 3, "stop": 4, "times": 4},
             "layers": [layer(parallel(5, 1, 6, 4, rotation(64.0, 2), 1, 6, 17, 3, 1.0, (-0.8, 1.0)), moe(7, 1, 12, 20)),
                        layer(latent(2, 12, 4, 20, 24, 16), dense(28, 1.0)),
                        layer(latent(2, 12, 4, 20, 24, 16), None),
                        layer(parallel(4, 2, 12, 20, rotation(777.0, 12, (16.0, 30, 8.0, 8.0)), 6, 3, 24, 12, 2.0, (1.2, 1.2)), dense(44, 3.0))],
             "ranks": {0: 5, 3: 2}},
    "once": {"architecture": "Vepelix", "vocab": 40, "width": 24, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 1, "times": 1},
             "layers": [layer(latent(2, 8, 4, 8, 16, 8), moe(1, 1, 8, 8))],
             "ranks": {}},
}


def config_of(name):
    c = json.loads(json.dumps(SHAPES[name]))
    c.pop("ranks")
    return c


def make_weights(name, seed=0):
    shape = SHAPES[name]
    g = torch.Generator().manual_seed(seed)
    W = shape["width"]
    rn = lambda *s, std=1.0: (torch.randn(*s, generator=g) * std).to(torch.bfloat16)
    un = lambda lo, hi, *s: (torch.rand(tuple(s), generator=g) * (hi - lo) + lo).to(torch.bfloat16)
    lin = lambda o, i, gain=1.0: rn(o, i, std=gain * i ** -0.5)
    w = {"embed": rn(shape["vocab"], W, std=0.7), "head": lin(shape["vocab"], W), "final.norm": un(-0.5, 0.5, W)}

    def glu(p, ff, gain=1.0):
        w.update({p + "gate": lin(ff, W, gain), p + "up": lin(ff, W, gain), p + "down": lin(W, ff)})

    for i, L in enumerate(shape["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        mp = p + "mix."
        w.update({p + "norm1": un(-0.5, 0.5, W), p + "ls1": un(-1.5, 1.5, W)})
        if L["type"] == "latent_attention":
            H, d, rd, dv, r, rq = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            w.update({mp + "dq": lin(rq, W), mp + "dq.norm": un(0.5, 1.5, rq), mp + "uq": lin(H * (d + rd), rq, 2.0), mp + "dkv": lin(r + rd, W), mp + "dkv.norm": un(0.5, 1.5, r),
                      mp + "uk": lin(H * d, r), mp + "uv": lin(H * dv, r), mp + "sink": rn(H, std=2.0), mp + "g": lin(H, W, 2.0), mp + "o": lin(W, H * dv)})
        else:
            a, r, lp, rp = m["left"], m["right"], mp + "left.", mp + "right."
            rk, rv, rank = r["heads"] * r["dim"], r["heads"] * r["vdim"], shape["ranks"][i]
            w.update({lp + "q": lin(a["heads"] * a["dim"], W), lp + "k": lin(a["kv_heads"] * a["dim"], W), lp + "v": lin(a["kv_heads"] * a["vdim"], W), lp + "q.norm": un(0.5, 2.0, a["dim"]),
                      lp + "k.norm": un(0.5, 1.5, a["dim"]), lp + "o": lin(W, a["heads"] * a["vdim"]), rp + "q": lin(rk, W), rp + "k": lin(rk, W), rp + "v": lin(rv, W), rp + "g": lin(rv, W),
                      rp + "o": lin(W, rv), rp + "norm": un(0.5, 1.5, r["vdim"]), rp + "a1": lin(rank, W), rp + "a2": lin(rk, rank), rp + "a2.b": rn(rk, std=2.0)})
        if f:
            w.update({p + "norm2": un(-0.5, 0.5, W), p + "ls2": un(-1.5, 1.5, W)})
        if f and f["kind"] == "dense":
            glu(p + "mlp.", f["ff"], 1.5)
        elif f:
            w[p + "mlp.router"] = lin(f["router"]["experts"], W, 2.0)
            for e in range(f["router"]["experts"]):
                glu(f"{p}mlp.e{e}.", f["expert"]["ff"], 1.5)
            if f.get("shared"):
                glu(p + "mlp.shared.", f["shared"]["ff"])
    return w


def tokens(name, n, seed):
    return torch.randint(0, SHAPES[name]["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
