"""The Pukatar design on the GPU against the CPU oracle (oracle/pukatar_ref.py): every mechanism alone, then whole models of several
small shapes under every way of cutting, batching, paging and slotting their sequences, through the engine and the command line.
Weights are random and bf16-representable; where random weights would hide a fault (a far key among many, a window's edge, a sink, a
state that has to last) the inputs are made so that it shows.  Mechanism tests feed the kernels projection rows directly: the oracle gets
the same rows as its input and selector matrices as its projections."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import pukatar_ref as R
from tests.pukatar_shapes import SHAPES, config_of, make_weights, tokens
from tests.test_gpu_fukatar import Rows, agrees, close, cuts_of, pages, replay, same_to_rounding, selectors, steps_of

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64


@pytest.fixture(scope="module")
def dev():
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    return torch.device("cuda:0")


def make_model(name, dtype, dev, max_tokens=512, max_seqs=4, seed=0, block=16):
    from vllm_i64_amd.config import PukatarConfig
    from vllm_i64_amd.pukatar import PukatarModel
    return PukatarModel(PukatarConfig.from_dict(config_of(name)), make_weights(name, seed), device=dev, dtype=dtype, max_seqs=max_seqs,
                        num_kv_blocks=(max_tokens + block - 1) // block, kv_block=block)


def oracle_logits(name, toks, seed=0):
    return R.forward(config_of(name), make_weights(name, seed), toks)


def whole_prompt(model, name, toks, dtype, slot=0, layers_too=False):
    """The model's logits for the whole prompt in one step, checked against the oracle under the model's own expert choices - which must be
    the oracle's for (nearly) every token: a close call may fall the other way in lower precision, and stays in state and cache then."""
    dev, n = model.device, len(toks)
    model.kv.reserve(slot, n)
    rec = {}
    got = model.forward(torch.tensor(toks, dtype=torch.int64, device=dev), torch.arange(n, dtype=torch.int32, device=dev),
                        torch.full((n,), slot, dtype=torch.int32, device=dev), record=rec, tokens_per_seq=[n]).cpu().clone()
    model.kv.free(slot)
    routes = {int(k[1:].split(".")[0]): v.cpu() for k, v in rec.items() if k.endswith(".route")}
    layers, free = [], {}
    W = make_weights(name)
    R.forward(config_of(name), W, toks, chosen=free)
    want = R.forward(config_of(name), W, toks, layers, routes=routes)
    assert set(routes) == set(free)
    for r, idx in routes.items():
        other = int((idx.long().sort(-1).values != free[r].sort(-1).values).any(-1).sum())
        assert other <= (max(1, 0.3 * n) if dtype == "bfloat16" else 0.02 * n), f"layer run {r}: the experts chosen differ from the oracle's for {other} of {n} tokens"
    if layers_too:
        for r, x in enumerate(layers):
            assert agrees(rec[f"r{r}.x"], x, dtype), f"residual after layer run {r}"
    assert agrees(got, want, dtype)
    return got


# =================================================== mechanisms alone =============================================================
@pytest.mark.parametrize("M", [1, 5, 40, 150])
@pytest.mark.parametrize("exact", [False, True])
@pytest.mark.parametrize("K,N", [(72, 52), (45, 30)])
def test_linear_epilogues(dev, M, exact, K, N):
    """Clamped gate / up pair, an added matrix (with a bias), and decays exp(-rate softplus(z + bias)) with one rate per column."""
    from vllm_i64_amd import ops_dense as D
    g = torch.Generator().manual_seed(M + K)
    rnd = lambda t: t if exact else t.to(torch.bfloat16).float()
    a = rnd(torch.randn(M, K, generator=g))
    w = (torch.randn(2 * N, K, generator=g) * 2.0 * K ** -0.5).to(torch.bfloat16)
    bias, e, rate = torch.randn(N, generator=g), torch.randn(M, N + 3, generator=g), torch.rand(N, generator=g) * 3.0
    z = a.double() @ w.double().T
    out = torch.empty(M, N, device=dev)
    D.linear(a.to(dev), w.to(dev), out, exact=exact, epilogue=D.EPI_CLAMP_GLU, act_a=1.702, act_b=0.8)
    u, v = z[:, :N].clamp(max=0.8), z[:, N:].clamp(-0.8, 0.8)
    assert float((u == 0.8).double().mean()) > 0.1 and float((v == -0.8).double().mean()) > 0.1      # (the premise)
    assert close(out, u * torch.sigmoid(1.702 * u) * (v + 1.0), 1e-5)
    wn = w[:N].contiguous().to(dev)
    D.linear(a.to(dev), wn, out, exact=exact, epilogue=D.EPI_ADD, bias=bias.to(dev), e=e.to(dev), e_off=2, lde=N + 3)
    assert close(out, z[:, :N] + bias.double() + e[:, 2:N + 2].double(), 1e-5)
    D.linear(a.to(dev), wn, out, exact=exact, epilogue=D.EPI_DECAY, bias=bias.to(dev), e=rate.to(dev))
    assert close(out, torch.exp(-rate.double() * R.softplus(z[:, :N] + bias.double())), 1e-5)


@pytest.mark.parametrize("W", [24, 300])
def test_residual_takes_the_sum_of_two_results_and_a_centred_norm_with_offset(dev, W):
    from vllm_i64_amd import ops_dense as D
    g = torch.Generator().manual_seed(W)
    n, eps = 7, 1e-5
    x, y, y2 = torch.randn(1, n, W, generator=g) + 3.0, torch.randn(n, W, generator=g) * 3 + 2.0, torch.randn(n, W, generator=g) - 1.0      # (means that matter)
    w, b, wf, bf_ = (torch.rand(W, generator=g) + 0.5 for _ in range(4))
    ones, xs, h = torch.ones(1, device=dev), x.to(dev).clone(), torch.empty(n, W, device=dev)
    D.streams_step(xs, y=y.to(dev), y2=y2.to(dev), out_w=ones, norm_w=w.to(dev), norm_b=b.to(dev), eps=eps, h=h, h_center=True)
    want = x[0].double() + y.double() + y2.double()
    assert close(xs[0], want, 1e-6) and close(h, R.layer_norm(want, w.double(), b.double(), eps), 1e-5)
    D.streams_step(xs, y=y.to(dev), out_w=ones)
    want = want + y.double()
    rows = torch.tensor([5, 0, 5, 2], dtype=torch.int32, device=dev)
    hr = torch.empty(4, W, device=dev)
    D.streams_step(xs, norm_w=wf.to(dev), norm_b=bf_.to(dev), eps=eps, h=hr, rows=rows, h_center=True)
    assert close(xs[0], want, 1e-6) and close(hr, R.layer_norm(want[rows.cpu().long()], wf.double(), bf_.double(), eps), 1e-5)


# ---- attention ---------------------------------------------------------------------------------------------------------------------
def attention_entry(H, G, d, dv, dims, window, keep, scale=0.37):
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": scale}
    if dims:
        m["rot"] = {"base": 300.0, "dims": dims}
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    return m


def run_attention(dev, m, sink, rows_of, lens, cut_sizes, cache_dtype, block, splits=1):
    """rows_of: slot -> [T, q | k | v] projection rows.  The kernels under cuts over scattered pages; returns slot -> [T, H * dv]."""
    from vllm_i64_amd import ops_dense as D
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    dims = (m.get("rot") or {}).get("dims", 0)
    inv = torch.tensor([m["rot"]["base"] ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64).float().to(dev) if dims else None
    mask = m.get("mask") or {"size": 0, "keep_first": 0}
    gs, nq, nk = dv + d, H * d, G * d
    per_seq = (max(lens.values()) + block - 1) // block
    bt = pages(dev, 3, per_seq, block, 5)
    cache = torch.full((3 * per_seq, block, G * gs), 7.0, dtype=cache_dtype, device=dev)
    got = {s: [] for s in lens}
    for runs in steps_of(lens, cut_sizes):
        r = Rows(dev, runs)
        P = torch.cat([rows_of[s][p:p + c] for s, p, c in runs]).float().to(dev).contiguous()
        Q = torch.empty(r.n, H * gs, device=dev)
        D.rot_prep(P, q_off=0, k_off=nq, v_off=nq + nk, heads=H, kv_heads=G, dim=d, vdim=dv, q_norm_w=None, k_norm_w=None, eps=1e-6, rot_dims=dims, interleaved=False,
                   inv_freq=inv, rot_mult=1.0, head_norm=False, v_freq=None, scale=m["scale"], positions=r.pos, slot_ids=r.slots, block_table=bt, cache=cache, q=Q, n=r.n)
        O = torch.empty(r.n, H * dv, device=dev)
        one = all(c == 1 for _, _, c in runs)
        D.kattn(Q, cache, None, bt, r.slots, r.pos, chunk=0, bias=None, sink=sink is not None, sink_w=sink.float().to(dev) if sink is not None else None, heads=H,
                kv_heads=G, dim=d, vdim=dv, out=O, n=r.n, mode=2 if one else 3, splits=splits if one else 1, window=mask["size"], keep_first=mask["keep_first"])
        row = 0
        for s, p, c in runs:
            got[s].append(O[row:row + c].cpu())
            row += c
    return {s: torch.cat(v) for s, v in got.items()}


def attention_oracle(m, sink, rows):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    sel, _ = selectors({"q": H * d, "k": G * d, "v": G * dv})
    W = {"x." + k: v for k, v in sel.items()}
    W.update({"x.sink": sink.double(), "x.o": torch.eye(H * dv, dtype=F64)})
    return R.windowed_attention(W, "x.", m, rows.double())


@pytest.mark.parametrize("H,G,d,dv,dims,window,keep", [(3, 3, 16, 16, 16, 20, 4), (6, 2, 10, 14, 6, 7, 3), (4, 1, 24, 40, 0, 0, 0), (2, 2, 130, 6, 64, 33, 0), (5, 1, 6, 4, 2, 1, 40)])
@pytest.mark.parametrize("block,cut_sizes", [(16, [300]), (4, [1]), (8, [2, 11, 1, 64])])
def test_windowed_attention_in_32_bits(dev, H, G, d, dv, dims, window, keep, block, cut_sizes):
    g = torch.Generator().manual_seed(H * d + block)
    m = attention_entry(H, G, d, dv, dims, window, keep)
    sink = torch.linspace(-5.0, 5.0, H)
    lens = {2: 70, 0: 33, 1: 5}
    rows = {s: torch.randn(T, H * d + G * d + G * dv, generator=g) for s, T in lens.items()}
    got = run_attention(dev, m, sink, rows, lens, cut_sizes, torch.float32, block)
    for s in lens:
        assert close(got[s], attention_oracle(m, sink, rows[s]), 2e-5), s


@pytest.mark.parametrize("H,G,d,dv,dims,window,keep", [(3, 3, 16, 16, 8, 37, 4), (8, 2, 48, 32, 48, 64, 40), (34, 2, 32, 16, 30, 5, 1), (2, 1, 64, 256, 64, 0, 0), (4, 2, 40, 64, 12, 1, 0),
                                                       (4, 2, 16, 16, 16, 90, 70)])
@pytest.mark.parametrize("block,cut_sizes,splits", [(16, [200], 1), (4, [1], 1), (4, [1], 3), (16, [2, 11, 1, 40], 2)])
def test_windowed_attention_matrix_core_form(dev, H, G, d, dv, dims, window, keep, block, cut_sizes, splits):
    """The bf16 cache rounds keys and values after the rotation; scores, sinks and softmax stay in 32 bits."""
    g = torch.Generator().manual_seed(H * d + block)
    m = attention_entry(H, G, d, dv, dims, window, keep)
    sink = torch.linspace(-5.0, 5.0, H)
    lens = {2: 170, 0: 33, 1: 5}
    rows = {s: torch.randn(T, H * d + G * d + G * dv, generator=g) for s, T in lens.items()}
    got = run_attention(dev, m, sink, rows, lens, cut_sizes, torch.bfloat16, block, splits)
    for s in lens:
        assert close(got[s], attention_oracle(m, sink, rows[s]), 2.5e-2), s


@pytest.mark.parametrize("mode", ["prompt", "decode"])
@pytest.mark.parametrize("cache_dtype,block,T,window,keep,splits", [(torch.float32, 16, 200, 50, 5, 1), (torch.bfloat16, 8, 330, 100, 4, 1), (torch.bfloat16, 16, 330, 96, 36, 3),
                                                                    (torch.bfloat16, 16, 150, 64, 0, 2)])
def test_one_key_stands_out_at_every_edge(dev, mode, cache_dtype, block, T, window, keep, splits):
    """One key alone lines up with the last query (along a dimension that is not rotated; all others are orthogonal to it): if it is inside the
    window or among the kept first positions the head returns its value, one step further it must have no part in the result at all."""
    H, G, d, dv = 2, 1, 16, 16
    m = attention_entry(H, G, d, dv, 8, window, keep, scale=1.5)
    sink = torch.full((H,), -3.0)
    g = torch.Generator().manual_seed(T)
    last = T - 1
    places = {0, keep - 1, keep, keep + 1, block - 1, block, 31, 32, last - window - 1, last - window, last - window + 1, last - window + 2, last - block, last}
    for target in sorted(p for p in places if 0 <= p <= last):
        rows = torch.zeros(T, H * d + G * d + G * dv)
        v = torch.randn(T, dv, generator=g).to(torch.bfloat16).float()
        rows[:, H * d + G * d:] = v
        rows[:, H * d + 14] = 1.0
        rows[target, H * d + 14], rows[target, H * d + 15] = 0.0, 3.0
        rows[:, 15], rows[:, d + 15] = 4.0, 4.0
        want = attention_oracle(m, sink, rows)
        seen = R.sees(last, target, m["mask"])
        assert close(want[-1].reshape(H, dv), v[target].double().expand(H, dv), 1e-4) == seen      # (the premise)
        got = run_attention(dev, m, sink, {1: rows}, {1: T}, [T] if mode == "prompt" else [T - 1, 1], cache_dtype, block, splits)
        assert close(got[1][-1], want[-1], 2e-5 if cache_dtype == torch.float32 else 1e-2), target


def test_window_slides_over_decoded_tokens_and_first_tokens_stay(dev):
    """Every position of a long decoding: the window's far edge walks over page borders and over the kept first positions."""
    H, G, d, dv = 4, 2, 16, 16
    m = attention_entry(H, G, d, dv, 16, 24, 6)
    sink = torch.linspace(-4.0, 2.0, H)
    rows = torch.randn(150, H * d + G * d + G * dv, generator=torch.Generator().manual_seed(0)) * 1.5
    for cache_dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2.5e-2)):
        got = run_attention(dev, m, sink, {0: rows}, {0: 150}, [3] + [1] * 147, cache_dtype, 8, 2)
        assert close(got[0], attention_oracle(m, sink, rows), tol)


# ---- gated delta rule with a decay per key channel ----------------------------------------------------------------------------------
def delta_weights(m, g, a_log=None):
    H, G, d, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    return {"q.conv": torch.randn(G * d, taps, generator=g) * 0.6, "k.conv": torch.randn(G * d, taps, generator=g) * 0.6, "v.conv": torch.randn(H * dv, taps, generator=g) * 0.6,
            "A_log": torch.rand(H, generator=g) * 3.0 - 2.5 if a_log is None else torch.full((H,), a_log), "dt_bias": torch.randn(H * d, generator=g),
            "norm": torch.rand(dv, generator=g) + 0.5}


def delta_run(dev, m, w, h, lens, cut_sizes, eps):
    """h: slot -> [T, q | k | v | b | a | g] raw projections (a: per head and key channel, g: per head and value channel)."""
    from vllm_i64_amd import ops_dense as D
    H, G, d, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    rk, rv, nd = G * d, H * dv, H * d
    C = 2 * rk + rv
    N1 = C + H + nd + rv
    conv_w = torch.cat([w["q.conv"], w["k.conv"], w["v.conv"]], 0).float().contiguous().to(dev)
    conv_state = torch.full((3, taps - 1, C), 9.0, device=dev) if taps > 1 else None
    state = torch.full((3, H, dv, d), 9.0, device=dev)
    eye = torch.eye(nd).to(torch.bfloat16).to(dev)
    rate = w["A_log"].float().exp().repeat_interleave(d).to(dev)
    got = {s: [] for s in lens}
    for runs in steps_of(lens, cut_sizes):
        r = Rows(dev, runs)
        P = torch.cat([h[s][p:p + c] for s, p, c in runs]).float().to(dev).contiguous()
        X, Gt, F, O, On = (torch.empty(r.n, k, device=dev) for k in (C, 2 * H, nd, rv, rv))
        D.causal_conv(P, off=0, channels=C, w=conv_w, bias=None, positions=r.pos, slot_ids=r.slots, state=conv_state, out=X, n=r.n,
                      single_rows=all(c == 1 for _, _, c in runs), seg_start=r.seg, nseg=r.nseg)
        cols = dict(q_off=0, k_off=rk, v_off=2 * rk, heads=H, kv_heads=G, dim=d, vdim=dv, n=r.n)
        D.gdn_gates(X, Gt, P, b_off=C, a_off=-1, a_log=None, dt_bias=None, unit_eps=1e-6, q_scale=d ** -0.5, **cols)
        D.linear(P, eye, F, m=r.n, a_off=C + H, exact=True, bias=w["dt_bias"].float().to(dev), epilogue=D.EPI_DECAY, e=rate)
        D.gdn_scan(X, Gt, f=F, seg_start=r.seg, nseg=r.nseg, positions=r.pos, slot_ids=r.slots, state=state, out=O, **cols)
        D.gate_norm(O, w["norm"].float().to(dev), On, groups=H, eps=eps, z=P, z_off=C + H + nd, ldz=N1, n=r.n, gate_after=True, width=rv, sigmoid=True)
        row = 0
        for s, p, c in runs:
            got[s].append(On[row:row + c].cpu())
            row += c
    return {s: torch.cat(v) for s, v in got.items()}


def delta_oracle(m, w, rows, eps):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    sel, _ = selectors({"q": G * d, "k": G * d, "v": H * dv, "b": H, "a1": H * d, "g1": H * dv})
    W = {"x." + k: v for k, v in sel.items()}
    W.update({"x." + k: w[k].double() for k in ("q.conv", "k.conv", "v.conv", "A_log", "dt_bias", "norm")})
    W.update({"x.a2": torch.eye(H * d, dtype=F64), "x.g2": torch.eye(H * dv, dtype=F64), "x.o": torch.eye(H * dv, dtype=F64)})
    return R.channel_delta(W, "x.", m, eps, rows.double())


@pytest.mark.parametrize("H,G,d,dv,taps", [(3, 3, 40, 24, 4), (4, 2, 16, 64, 3), (1, 1, 130, 8, 1), (6, 2, 8, 33, 5), (2, 1, 64, 20, 2), (2, 2, 200, 40, 4)])
@pytest.mark.parametrize("cut_sizes", [[200], [1], [2, 5, 1, 3, 90], [7, 2]])
def test_channel_delta_rule_under_cuts(dev, H, G, d, dv, taps, cut_sizes):
    g = torch.Generator().manual_seed(H * d + taps)
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "conv": taps}
    w = delta_weights(m, g)
    lens = {2: 120, 0: 31, 1: 4}
    h = {s: torch.randn(T, 2 * G * d + 2 * H * dv + H + H * d, generator=g) for s, T in lens.items()}
    got = delta_run(dev, m, w, h, lens, cut_sizes, 1e-5)
    for s in lens:
        assert close(got[s], delta_oracle(m, w, h[s], 1e-5), 5e-5), s


@pytest.mark.parametrize("cut_sizes", [[300], [1]])
def test_channel_delta_rule_in_a_launch_of_many_runs(dev, cut_sizes):
    """Enough workgroups for the form with two value columns per lane."""
    g = torch.Generator().manual_seed(1)
    m = {"heads": 48, "kv_heads": 48, "dim": 32, "vdim": 64, "conv": 2}
    w = delta_weights(m, g)
    lens = {2: 40, 0: 33, 1: 2}
    h = {s: torch.randn(T, 2 * 48 * 32 + 2 * 48 * 64 + 48 + 48 * 32, generator=g) for s, T in lens.items()}
    got = delta_run(dev, m, w, h, lens, cut_sizes, 1e-6)
    for s in lens:
        assert close(got[s], delta_oracle(m, w, h[s], 1e-6), 5e-5), s


@pytest.mark.parametrize("channel", [True, False])
@pytest.mark.parametrize("H,G,d,dv", [(4, 2, 64, 32), (3, 3, 40, 24), (2, 1, 128, 128), (2, 2, 200, 40), (1, 1, 12, 5), (8, 8, 256, 256)])
def test_delta_scan_forms_agree_bit_for_bit(dev, channel, H, G, d, dv):
    """Loads straight into registers, or tokens staged through LDS with one, two or four value columns per lane: runs of unequal length (also
    one row, a tile of rows, one more), continued from slots' states or fresh, in scattered slots."""
    from vllm_i64_amd import _lib, ops_dense as D
    g = torch.Generator().manual_seed(d + dv)
    r = Rows(dev, [(4, 0, 33), (1, 7, 1), (0, 3, 16), (3, 0, 17), (2, 50, 70)])
    C = 2 * G * d + H * dv
    X, Gt, F = torch.randn(r.n, C, generator=g) * 0.2, torch.rand(r.n, 2 * H, generator=g), torch.rand(r.n, H * d, generator=g)
    S0 = torch.randn(5, H, dv, d, generator=g)
    X, Gt, F = X.to(dev), Gt.to(dev), F.to(dev)
    got = []
    try:
        for form in (1, 2, 3, 4, 0):
            _lib.call_dense("i64h_set_gdn_scan_form", form)
            S, O = S0.to(dev).clone(), torch.full((r.n, H * dv), 7.0, device=dev)
            D.gdn_scan(X, Gt, f=F if channel else None, q_off=0, k_off=G * d, v_off=2 * G * d, heads=H, kv_heads=G, dim=d, vdim=dv, seg_start=r.seg, nseg=r.nseg,
                       positions=r.pos, slot_ids=r.slots, state=S, out=O, n=r.n)
            got.append((O.cpu(), S.cpu()))
    finally:
        _lib.call_dense("i64h_set_gdn_scan_form", 0)
    for O, S in got[1:]:
        assert torch.equal(O, got[0][0]) and torch.equal(S, got[0][1])
    own = torch.arange(H) // (H // G)
    at = 0
    for slot, p, c in [(4, 0, 33), (1, 7, 1), (0, 3, 16), (3, 0, 17), (2, 50, 70)]:      # (the fresh runs against the oracle's recurrence)
        x, gt, f = (t[at:at + c].cpu().double() for t in (X, Gt, F))
        if p == 0:
            q, k, v = x[:, :G * d].reshape(c, G, d)[:, own], x[:, G * d:2 * G * d].reshape(c, G, d)[:, own], x[:, 2 * G * d:].reshape(c, H, dv)
            dec = f.reshape(c, H, d) if channel else gt[:, H:].unsqueeze(-1).expand(c, H, d)
            assert close(got[0][0][at:at + c], R.channel_delta_rule(q, k, v, gt[:, :H], dec).reshape(c, H * dv), 2e-5)
        at += c


@pytest.mark.parametrize("cut_sizes", [[500], [1], [64, 3]])
def test_channel_delta_rule_keeps_one_channel_and_forgets_another(dev, cut_sizes):
    """What the first token wrote along a channel whose decay is next to one is still there 500 tokens later; along a channel that decays
    fast it is gone (a decay taken per head, a state lost at a cut or a slot's stale state taken over would show)."""
    g = torch.Generator().manual_seed(7)
    m = {"heads": 2, "kv_heads": 1, "dim": 12, "vdim": 10, "conv": 1}
    w = delta_weights(m, g, a_log=0.0)
    w["q.conv"], w["k.conv"], w["v.conv"] = torch.ones(12, 1), torch.ones(12, 1), torch.ones(20, 1)
    T, a0 = 500, 44 + 2
    N1 = 44 + 2 + 24 + 20
    h = torch.randn(T, N1, generator=g)
    w["dt_bias"] = torch.full((24,), -12.0)              # (softplus next to zero: nothing decays ...)
    h[:, a0:a0 + 24] = 0.0
    h[:, a0 + 1] = h[:, a0 + 13] = 11.0                  # (... but the second channel of either head)
    h[:, 12:14] = 0.0                                    # (silu(0) = 0: no later key has a part along the first two channels)
    h[0, 12:24] = 0.0
    h[:, 44:46] = 3.0                                    # strong writes
    for channel, lasts in ((0, True), (1, False)):
        hc = h.clone()
        hc[0, 12 + channel] = 5.0
        hc[T - 1, :12] = 0.0
        hc[T - 1, channel] = 9.0                         # the last query asks along that channel
        want = delta_oracle(m, w, hc, 1e-6)
        o_last = want[-1].abs().max()
        assert (float(o_last) > 0.05) == lasts           # (the premise)
        got = delta_run(dev, m, w, {1: hc}, {1: T}, cut_sizes, 1e-6)[1]
        assert close(got, want, 1e-4) and abs(float(got[-1].abs().max()) - float(o_last)) < 1e-3


# ---- router and experts --------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("E,top", [(6, 2), (12, 12), (16, 4), (5, 1), (70, 9), (1, 1)])
def test_router_bias_choice_and_softmax_over_the_chosen(dev, E, top):
    from vllm_i64_amd import ops_dense as D
    g = torch.Generator().manual_seed(E + top)
    n = 301
    gi, gw, gate = torch.empty(n, top, dtype=torch.int32, device=dev), torch.empty(n, top, device=dev), torch.empty(n, device=dev)
    b = torch.randn(E, generator=g) * 2.0
    for spread in (2.0, 60.0):      # (wide: a softmax over all entries would underflow for most of them)
        z = torch.randn(n, E, generator=g) * spread
        idx, wgt = R.route(z.double() + b.double(), top)
        D.route_topk(z.to(dev), entries=E, correction=None, groups=1, keep=1, top=top, scale=1.0, idx=gi, wgt=gw, n=n, bias=b.to(dev), chosen_softmax=True)
        assert torch.equal(gi.cpu().long(), idx) and close(gw, wgt, 1e-5)
    for K in (72, 45):
        h = torch.randn(n, K, generator=g)
        w = (torch.randn(E + 1, K, generator=g) * 2 * K ** -0.5).to(torch.bfloat16)
        z = h.double() @ w.double().T
        idx, wgt = R.route(z[:, :E] + b.double(), top)
        D.route_topk(None, h=h.to(dev), w=w.to(dev), entries=E, correction=None, groups=1, keep=1, top=top, scale=1.0, idx=gi, wgt=gw, n=n, bias=b.to(dev),
                     chosen_softmax=True, gate_out=gate)
        same = (gi.cpu().long() == idx).all(-1)
        assert float(same.double().mean()) > 0.99 and close(gw.cpu()[same], wgt[same], 1e-4)      # (a close call in 32 bits may fall the other way)
        assert close(gate, torch.sigmoid(z[:, E]), 1e-5)


@pytest.mark.parametrize("name,l", [("odd", 1), ("odd", 2), ("plain", 2), ("plain", 3), ("wide", 1), ("wide", 3), ("tail", 0)])
@pytest.mark.parametrize("n", [1, 7, 200])
def test_mixture_of_experts_alone(dev, name, l, n):
    model = make_model(name, "float32", dev)
    cfg, w = config_of(name), {k: v.double() for k, v in make_weights(name).items()}
    h = torch.randn(n, cfg["width"], generator=torch.Generator().manual_seed(n + l))
    B = model.buffers(n, 1)
    B.h.copy_(h)
    model._moe_ff(B, model.layers[l], n, B.h, B.y2, B.y3)
    idx = B.idx[: n * model.layers[l]["mlp"].top].view(n, -1).cpu()
    want = R.mixture_ff(w, f"l{l}.mlp.", cfg["layers"][l]["mlp"], h.double(), forced=idx)
    assert close(B.y2, want, 2e-5)


@pytest.mark.parametrize("n", [3, 100])
def test_dense_feed_forward_alone(dev, n):
    model = make_model("odd", "float32", dev)
    w = {k: v.double() for k, v in make_weights("odd").items()}
    h = torch.randn(n, 42, generator=torch.Generator().manual_seed(n))
    B = model.buffers(n, 1)
    B.h.copy_(h)
    model._dense_glu(B, model.layers[0], n, B.h, B.y2)
    assert close(B.y2, R.dense_ff(w, "l0.mlp.", h.double()), 2e-5)


# =================================================== whole models =================================================================
@pytest.mark.parametrize("name", list(SHAPES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompt_and_residual_after_every_layer_run(dev, name, dtype):
    whole_prompt(make_model(name, dtype, dev), name, tokens(name, 140, 1), dtype, slot=2, layers_too=True)


@pytest.mark.parametrize("name", list(SHAPES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_cuts_batches_and_reuse(dev, name, dtype):
    """Token by token from the first token; portions of changing size down to two tokens; four live requests of unequal length in a
    pool that only fits with page reuse, more requests than slots over the run; a request left out of steps.  Every request's whole
    prompt is checked against the oracle first; the schedules must then give the same logits."""
    from vllm_i64_amd.engine import Engine
    model = make_model(name, dtype, dev, max_tokens=4 * 64, max_seqs=4)
    reqs = {"a": tokens(name, 61, 2), "b": tokens(name, 38, 3), "c": tokens(name, 1, 4), "d": tokens(name, 50, 5), "e": tokens(name, 33, 6), "f": tokens(name, 64, 7)}
    want = {i: whole_prompt(model, name, t, dtype, slot=3) for i, t in reqs.items()}
    eng = Engine(model)
    got = replay(eng, {"b": reqs["b"]}, [[("b", 1)] for _ in range(38)])
    assert same_to_rounding(got["b"], want["b"], dtype)
    got = replay(eng, {"a": reqs["a"]}, [[("a", c)] for _, c in cuts_of(61, [2, 17, 1, 3, 16, 2, 5])])
    assert same_to_rounding(got["a"], want["a"], dtype)
    sched = [[("a", 30), ("b", 2)], [("a", 1), ("b", 20), ("c", 1), ("d", 7)], [("b", 1), ("d", 2), ("e", 16)], [("a", 28), ("b", 1), ("d", 1), ("e", 1)],
             [("a", 2), ("b", 14), ("d", 40), ("e", 2)], [("e", 14), ("f", 33)], [("f", 1)], [("f", 30)]]
    got = replay(eng, reqs, sched)
    for i in reqs:
        assert same_to_rounding(got[i], want[i], dtype), i
    assert model.kv.free_blocks == model.kv.num_blocks and not eng.seqs


@pytest.mark.parametrize("name", ["odd", "wide"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_past_many_pages(dev, name, dtype):
    from vllm_i64_amd.engine import Engine
    toks = tokens(name, 300, 8)
    model = make_model(name, dtype, dev, max_tokens=304, max_seqs=1)
    want = whole_prompt(model, name, toks, dtype)
    got = replay(Engine(model), {"x": toks}, [[("x", 9)]] + [[("x", 1)] for _ in range(291)])
    assert same_to_rounding(got["x"], want, dtype)


def test_every_pass_has_its_own_cache_and_state(dev):
    """Decoding continues a prompt: were a cache or state shared between the passes of the loop, the second pass would overwrite what the
    first one needs for the next token; and the passes do differ (the premise)."""
    from vllm_i64_amd.engine import Engine
    name = "odd"
    toks = tokens(name, 40, 30)
    model = make_model(name, "float32", dev, max_tokens=64, max_seqs=1)
    eng = Engine(model)
    got = replay(eng, {"x": toks}, [[("x", 25)]] + [[("x", 1)] for _ in range(15)])["x"]
    want = oracle_logits(name, toks)
    assert agrees(got, want, "float32")
    runs = model.cfg.layer_runs()
    first, second = [r for r, (l, _) in enumerate(runs) if l == 1][:2]
    assert not close(model.kv.state[first]["gdn"], model.kv.state[second]["gdn"], 1e-2)
    once = config_of(name)
    once["loop"]["times"] = 1
    w = make_weights(name)
    w["loop.step"] = w["loop.step"][:1]
    assert not agrees(R.forward(once, w, toks), want, "bfloat16")


@pytest.mark.parametrize("name", ["odd", "plain", "tail"])
def test_greedy_generation_through_the_engine(dev, name):
    """More prompts than slots; the engine's own scheduler, batching and sampling; against the oracle's greedy continuation."""
    from vllm_i64_amd.engine import Engine, SamplingParams
    model = make_model(name, "float32", dev, max_tokens=3 * 64, max_seqs=2)
    prompts = [tokens(name, n, 20 + n) for n in (5, 19, 1, 12)]
    new = 6
    want = []
    for p in prompts:
        t = list(p)
        for _ in range(new):
            t.append(int(oracle_logits(name, t)[-1].argmax()))
        want.append(t[len(p):])
    eng = Engine(model, max_batch_tokens=16)
    assert eng.generate(prompts, SamplingParams(max_new_tokens=new)) == want


def test_graph_decoder_steps_match_the_oracle(dev):
    """The batch decoder (a captured HIP graph replayed per step) from the first token on: convolution inputs, the delta rule's state and the
    pages of every pass advance inside the graph."""
    from vllm_i64_amd import _lib
    if not os.path.exists(_lib.LIB_PATH):
        pytest.skip("the batch decoder takes its argmax from the first library, which is not built")
    from vllm_i64_amd.model import GreedyDecoder
    name = "odd"
    model = make_model(name, "float32", dev, max_tokens=256, max_seqs=3)
    prompts = [tokens(name, n, 40 + n) for n in (4, 11, 17)]
    dec = GreedyDecoder(model, 3, use_graph=True)
    dec.prefill([torch.tensor(p) for p in prompts], reserve_extra=12)
    seqs = [list(p) + [int(t)] for p, t in zip(prompts, dec.tokens.tolist())]
    for _ in range(9):
        dec.step()
        torch.cuda.synchronize()
        for s, t in zip(seqs, dec.tokens.tolist()):
            s.append(int(t))
    for p, s in zip(prompts, seqs):
        t = list(p)
        for _ in range(10):
            t.append(int(oracle_logits(name, t)[-1].argmax()))
        assert s == t


def test_trace_command_on_a_checkpoint_folder(dev, tmp_path):
    from safetensors.torch import save_file
    name = "tail"
    ck = tmp_path / "ck"
    ck.mkdir()
    (ck / "config.json").write_text(json.dumps(config_of(name)))
    save_file(make_weights(name), str(ck / "model.safetensors"))
    toks = tokens(name, 21, 9)
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": toks[:10], "want": [0, 9]}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[10:12], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "q", "tokens": toks[12:], "want": [8]}, {"id": "r", "tokens": toks[:3], "want": [2]}], "end": ["q", "r"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(ck), "--dtype", "float32", "--out", str(out), "--max-tokens", "128"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    import numpy as np
    want = oracle_logits(name, toks)
    V = SHAPES[name]["vocab"]
    a = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(-1, V))
    c = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(-1, V))
    assert not (out / "1.f32").exists()
    assert agrees(a, want[[0, 9]], "float32") and agrees(c, torch.stack([want[20], want[2]]), "float32")
