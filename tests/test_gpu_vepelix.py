"""The Vepelix design on the GPU against the CPU oracle (oracle/vepelix_ref.py): every mechanism alone, then whole models of several
small shapes under every way of cutting, batching, paging and slotting their sequences, through the engine and the command line.
Weights are random and bf16-representable; where random weights would hide a fault (a far key among many, a window's edge, a sink, a
state that has to last) weights and inputs are made so that it shows."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import vepelix_ref as R
from tests.test_gpu_fukatar import Rows, agrees, close, cuts_of, pages, replay, same_to_rounding, steps_of
from tests.vepelix_shapes import SHAPES, config_of, latent, make_weights, parallel, rotation, tokens

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64


@pytest.fixture(scope="module")
def dev():
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    return torch.device("cuda:0")


def make_model(name, dtype, dev, max_tokens=512, max_seqs=4, seed=0, block=16, config=None, weights=None, cache_dtype=None):
    from vllm_i64_amd.config import VepelixConfig
    from vllm_i64_amd.vepelix import VepelixModel
    return VepelixModel(VepelixConfig.from_dict(config if config is not None else config_of(name)), weights if weights is not None else make_weights(name, seed), device=dev,
                        dtype=dtype, max_seqs=max_seqs, num_kv_blocks=(max_tokens + block - 1) // block, kv_block=block, cache_dtype=cache_dtype)


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
def test_linear_row_gates_and_row_factors(dev, M, exact, K, N):
    """One sigmoid gate for all columns of a row and batch, on column blocks of wider matrices; a factor on the input row of a gate / up pair
    (which is not a factor on the result: the premise)."""
    from vllm_i64_amd import ops_dense as D
    g = torch.Generator().manual_seed(M + K)
    rnd = lambda t: t if exact else t.to(torch.bfloat16).float()
    H = 3
    a = rnd(torch.randn(M, H * K, generator=g))
    w = (torch.randn(H, N, K, generator=g) * K ** -0.5).to(torch.bfloat16)
    e = torch.randn(M, H + 4, generator=g) * 2
    out = torch.empty(M, H * N, device=dev)
    D.linear(a.to(dev), w.to(dev), out, m=M, n=N, k=K, lda=H * K, ldc=H * N, batch=H, a_batch=K, w_batch=N * K, c_batch=N, exact=exact, epilogue=D.EPI_ROW_SIGMOID, e=e.to(dev),
             e_off=2, lde=H + 4, e_batch=1)
    want = torch.cat([a[:, h * K:(h + 1) * K].double() @ w[h].double().T * torch.sigmoid(e[:, 2 + h:3 + h].double()) for h in range(H)], 1)
    assert close(out, want, 1e-5)
    w2 = (torch.randn(2 * N, K, generator=g) * 2 * K ** -0.5).to(torch.bfloat16)
    s = torch.rand(M, generator=g)
    x, z = a[:, :K].contiguous(), a[:, :K].double() @ w2.double().T
    zs = z * s.double().unsqueeze(-1)
    o2 = torch.empty(M, N, device=dev)
    D.linear(x.to(dev), w2.to(dev), o2, exact=exact, epilogue=D.EPI_SILU_MUL, row_scale=s.to(dev))
    want = R.silu(zs[:, :N]) * zs[:, N:]
    assert close(o2, want, 1e-5) and not close(want, R.silu(z[:, :N]) * z[:, N:] * s.double().unsqueeze(-1), 1e-2)
    D.linear(x.to(dev), w2.to(dev), o2, exact=exact, epilogue=D.EPI_CLAMP_GLU, act_a=1.702, act_b=0.8, row_scale=s.to(dev))
    u, v = zs[:, :N].clamp(max=0.8), zs[:, N:].clamp(-0.8, 0.8)
    assert close(o2, u * torch.sigmoid(1.702 * u) * (v + 1.0), 1e-5)


@pytest.mark.parametrize("M", [1, 8, 9, 40, 64, 150])
@pytest.mark.parametrize("exact", [False, True])
@pytest.mark.parametrize("K,N,off,ld", [(72, 52, 8, 88), (45, 30, 3, 50), (512, 200, 0, 512), (1, 9, 2, 6)])
def test_linear_norms_its_input(dev, M, exact, K, N, off, ld):
    """Columns of a wider matrix, RMS-normed with weights on the way into the product; rows of very different size, and one of zeros."""
    from vllm_i64_amd import ops_dense as D
    g = torch.Generator().manual_seed(M + K)
    a = torch.randn(M, ld, generator=g) * torch.logspace(-3, 3, M).unsqueeze(-1)
    a[M // 2] = 0.0
    w, nw, eps = (torch.randn(N, K, generator=g) * K ** -0.5).to(torch.bfloat16), torch.rand(K, generator=g) + 0.5, 1e-5
    out = torch.empty(M, N, device=dev)
    D.linear(a.to(dev), w.to(dev), out, a_off=off, m=M, exact=exact, in_norm_w=nw.to(dev), in_eps=eps)
    want = (R.rms(a[:, off:off + K].double(), eps) * nw.double()) @ w.double().T
    assert not out[M // 2].any()
    scale = want.abs().max(-1).values.clamp_min(1e-9)
    err = ((out.cpu().double() - want).abs().max(-1).values / scale).max()
    assert float(err) < (1e-5 if exact else 2e-2)
    if not exact:      # what is rounded to bf16 is the row times the weights
        x = (a[:, off:off + K] * nw).to(torch.bfloat16).double() @ w.double().T / torch.sqrt(a[:, off:off + K].double().pow(2).mean(-1, keepdim=True) + eps)
        assert float(((out.cpu().double() - x).abs().max(-1).values / scale).max()) < 2e-5


@pytest.mark.parametrize("W", [24, 300, 1024, 2056, 5000, 30])
@pytest.mark.parametrize("n", [1, 7])
@pytest.mark.parametrize("form", [0, 1])
def test_residual_takes_results_times_a_factor_per_column(dev, W, n, form):
    from vllm_i64_amd import _lib
    try:
        _lib.call_dense("i64h_set_residual_form", form)
        check_residual(dev, W, n)
    finally:
        _lib.call_dense("i64h_set_residual_form", 1)


def check_residual(dev, W, n):
    from vllm_i64_amd import ops_dense as D
    g = torch.Generator().manual_seed(W)
    eps = 1e-5
    x, y, y2 = torch.randn(1, n, W, generator=g), torch.randn(n, W, generator=g) * 3, torch.randn(n, W, generator=g)
    ls, w = torch.randn(W, generator=g), torch.rand(W, generator=g) - 0.5
    ones, xs, h = torch.ones(1, device=dev), x.to(dev).clone(), torch.empty(n, W, device=dev)
    nw = (1.0 + w).to(dev)
    D.streams_step(xs, y=y.to(dev), y2=y2.to(dev), y_scale=ls.to(dev), out_w=ones, norm_w=nw, eps=eps, h=h)
    want = x[0].double() + ls.double() * (y.double() + y2.double())
    assert close(xs[0], want, 1e-6) and close(h, R.one_plus_norm(want, w.double(), eps), 1e-5)
    D.streams_step(xs, y=y.to(dev), y_scale=ls.to(dev), out_w=ones)
    want = want + ls.double() * y.double()
    D.streams_step(xs, y=y2.to(dev), out_w=ones, norm_w=nw, eps=eps, h=h)      # (another pass: something added as it is, the norm with it)
    want = want + y2.double()
    rows = torch.tensor([n - 1, 0, n // 2], dtype=torch.int32, device=dev)
    hr = torch.empty(3, W, device=dev)
    D.streams_step(xs, norm_w=nw, eps=eps, h=hr, rows=rows)
    assert close(xs[0], want, 1e-6) and close(h, R.one_plus_norm(want, w.double(), eps), 1e-5) and close(hr, R.one_plus_norm(want[rows.cpu().long()], w.double(), eps), 1e-5)
    b = torch.randn(W, generator=g)
    half = torch.full((1,), 0.5, device=dev)
    D.streams_step(xs, y=y.to(dev), out_w=half, norm_w=nw, norm_b=b.to(dev), eps=eps, h=h, h_center=True)      # (a centred norm with offset; half the result)
    want = want + 0.5 * y.double()
    c = want - want.mean(-1, keepdim=True)
    assert close(xs[0], want, 1e-6) and close(h, R.rms(c, eps) * (1.0 + w.double()) + b.double(), 1e-5)


# ---- mixers of a model, their input rows given -----------------------------------------------------------------------------------------
def run_mixer(model, r, rows_of, lens, cut_sizes, seed=5):
    """The mixer of layer run r on given input rows (slot -> [T, width]) under cuts, over scattered pages that hold other things before; returns
    slot -> [T, width]."""
    from vllm_i64_amd.model import attention_segments
    dev, kv = model.device, model.kv
    d = model.layers[model.layer_runs[r][0]]
    per_seq = max(kv.blocks_for(T) for T in lens.values())
    kv.block_table[:3, :per_seq] = pages(dev, 3, per_seq, kv.block, seed)
    kv.rows[r].fill_(7.0)
    for t in kv.state[r].values():
        t.fill_(9.0)
    got = {s: [] for s in lens}
    for runs in steps_of(lens, cut_sizes):
        s = Rows(dev, runs)
        B = model.buffers(s.n, 1)
        B.h.copy_(torch.cat([rows_of[q][p:p + c] for q, p, c in runs]))
        per = [c for _, _, c in runs]
        w = model._mixer(B, d, r, s.n, s.pos, s.slots, kv, s.seg, s.nseg, attention_segments(per, s.n, model.ATTN_MAX_SEGMENTS), max(p + c for _, p, c in runs))
        y = (w["y"] + w["y2"] if "y2" in w else w["y"]).cpu()
        row = 0
        for q, p, c in runs:
            got[q].append(y[row:row + c].clone())
            row += c
    return {q: torch.cat(v) for q, v in got.items()}


def mixer_oracle(config, weights, l, rows):
    W = {k: v.double() for k, v in weights.items()}
    L = config["layers"][l]
    fn = R.latent_attention if L["type"] == "latent_attention" else R.parallel_mixer
    return fn(W, f"l{l}.mix.", L["mixer"], float(config["norm"]["eps"]), rows.double())


MIXERS = [("odd", 0, 0), ("odd", 1, 1), ("odd", 2, 2), ("odd", 7, 3), ("odd", 8, 4), ("plain", 0, 0), ("plain", 1, 1), ("plain", 2, 2), ("plain", 3, 3), ("wide", 0, 0), ("wide", 1, 1),
          ("wide", 2, 2), ("wide", 3, 3), ("tail", 0, 0), ("tail", 3, 3)]


@pytest.mark.parametrize("name,r,l", MIXERS)
@pytest.mark.parametrize("dtype,block,cut_sizes", [("float32", 16, [200]), ("float32", 4, [1]), ("float32", 8, [2, 11, 1, 40]), ("bfloat16", 16, [200]), ("bfloat16", 4, [1]),
                                                   ("bfloat16", 8, [2, 11, 1, 40])])
def test_mixers_alone_under_cuts(dev, name, r, l, dtype, block, cut_sizes):
    """Unequal sequences side by side, whole, token by token, and in portions down to two tokens and one."""
    model = make_model(name, dtype, dev, max_tokens=3 * 128, block=block)
    lens = {2: 101, 0: 33, 1: 5}
    g = torch.Generator().manual_seed(r + block)
    rows = {s: torch.randn(T, model.cfg.width, generator=g) for s, T in lens.items()}
    if dtype == "bfloat16":
        rows = {s: t.to(torch.bfloat16).float() for s, t in rows.items()}
    got = run_mixer(model, r, rows, lens, cut_sizes)
    for s in lens:
        want = mixer_oracle(config_of(name), make_weights(name), l, rows[s])
        assert close(got[s], want, 3e-5) if dtype == "float32" else agrees(got[s], want, dtype), s


def one_layer(width, mix):
    return {"architecture": "Vepelix", "vocab": 8, "width": width, "norm": {"eps": 1e-6}, "layers": [dict(mix, mlp=None)]}


def zero_weights(config, **given):
    """Zeros of the shapes that the tests' weights have, but for the given tensors of layer 0's mixer."""
    SHAPES["_made"] = dict(config, ranks={0: 2})
    try:
        w = {k: torch.zeros_like(v) for k, v in make_weights("_made").items()}
    finally:
        del SHAPES["_made"]
    for k, v in given.items():
        k = "l0.mix." + k.replace("__", ".")
        assert w[k].shape == v.shape, k
        w[k] = v.to(torch.bfloat16)
    return w


def pick(out, width, at):
    """[out, width] that hands the input's values from column `at` on through."""
    t = torch.zeros(out, width)
    t[torch.arange(out), at + torch.arange(out)] = 1.0
    return t


@pytest.mark.parametrize("mode", ["prompt", "decode"])
@pytest.mark.parametrize("dtype,block,T,window", [("float32", 16, 200, 50), ("bfloat16", 8, 330, 100), ("bfloat16", 16, 330, 96), ("bfloat16", 16, 150, 64), ("float32", 4, 40, 1)])
def test_window_attention_one_key_stands_out_at_every_edge(dev, mode, dtype, block, T, window):
    """One key alone lines up with the last query (along a dimension that is not rotated; all others are orthogonal to it): inside the window the
    head returns its value, one step further it must have no part in the result at all."""
    d = dv = 16
    config = one_layer(64, parallel(2, 1, d, dv, rotation(300.0, 8, (4.0, 60, 6.0, 0.5)), window, 1, 8, 8, 2.0, (1.0, 1.0), scale=1.5))
    w = zero_weights(config, left__q=torch.cat([pick(d, 64, 0), pick(d, 64, 0)]), left__k=pick(d, 64, 16), left__v=pick(dv, 64, 32), left__q__norm=torch.ones(d),
                     left__k__norm=torch.ones(d), left__o=torch.cat([torch.eye(2 * dv), torch.zeros(32, 2 * dv)]))
    model = make_model("", dtype, dev, max_tokens=3 * T + 3 * block, block=block, config=config, weights=w)
    g = torch.Generator().manual_seed(T)
    last = T - 1
    places = {0, block - 1, block, 31, 32, last - window - 1, last - window, last - window + 1, last - window + 2, last - block, last}
    for target in sorted(p for p in places if 0 <= p <= last):
        h = torch.zeros(T, 64)
        h[:, 15] = 2.0                                        # queries
        h[:, 16 + 14] = 1.0                                   # keys
        h[target, 16 + 14], h[target, 16 + 15] = 0.0, 3.0
        h[:, 32:48] = torch.randn(T, dv, generator=g).to(torch.bfloat16).float()
        want = mixer_oracle(config, w, 0, h)
        seen = R.sees(last, target, {"size": window})
        assert close(want[-1, :2 * dv].reshape(2, dv), h[target, 32:48].double().expand(2, dv), 1e-4) == seen      # (the premise)
        got = run_mixer(model, 0, {1: h}, {1: T}, [T] if mode == "prompt" else [T - 1, 1])
        assert close(got[1][-1], want[-1], 2e-5 if dtype == "float32" else 1e-2), target


def test_window_slides_over_decoded_tokens(dev):
    """Every position of a long decoding: the window's far edge walks over page borders."""
    config = one_layer(40, parallel(4, 2, 16, 16, rotation(300.0, 16, (4.0, 60, 6.0, 0.5)), 24, 2, 8, 12, 6.0, (1.0, 0.3)))
    SHAPES["_made"] = dict(config, ranks={0: 4})
    try:
        w = make_weights("_made")
    finally:
        del SHAPES["_made"]
    h = torch.randn(150, 40, generator=torch.Generator().manual_seed(0)).to(torch.bfloat16).float()
    want = mixer_oracle(config, w, 0, h)
    for dtype in ("float32", "bfloat16"):
        model = make_model("", dtype, dev, max_tokens=3 * 152, block=8, config=config, weights=w)
        got = run_mixer(model, 0, {0: h}, {0: 150}, [3] + [1] * 147)[0]
        assert close(got, want, 3e-5) if dtype == "float32" else agrees(got, want, dtype)


@pytest.mark.parametrize("mode", ["prompt", "decode"])
@pytest.mark.parametrize("dtype,block,T", [("float32", 16, 200), ("bfloat16", 8, 530), ("bfloat16", 16, 300)])
def test_latent_attention_one_cached_row_stands_out(dev, mode, dtype, block, T):
    """One latent alone lines up with the last query: at the first position, far back, at page borders and at the query itself the heads return
    what their value maps make of it, times their gates."""
    r, rd, H, dv = 16, 8, 2, 16
    config = one_layer(64, latent(H, r, rd, dv, r, 16, base=300.0, scale=1.5))
    eye = torch.eye(r)
    uq = torch.zeros(H * (r + rd), 16)
    uq[:r], uq[r + rd:2 * r + rd] = eye, eye                   # (no rotated part in the queries)
    gate = torch.zeros(H, 64)
    gate[0, 48], gate[1, 48] = 0.5, -1.0
    w = zero_weights(config, dq=pick(16, 64, 0), dq__norm=torch.ones(16), uq=uq, dkv=torch.cat([pick(r, 64, 16), pick(rd, 64, 32)]), dkv__norm=torch.ones(r), uk=torch.cat([eye, eye]),
                     uv=torch.cat([eye, 2.0 * eye]), sink=torch.tensor([-3.0, 2.0]), g=gate, o=torch.cat([torch.eye(H * dv), torch.zeros(32, H * dv)]))
    model = make_model("", dtype, dev, max_tokens=3 * T + 3 * block, block=block, config=config, weights=w)
    g = torch.Generator().manual_seed(T)
    last = T - 1
    for target in sorted({0, 1, block - 1, block, 31, 32, T // 2, last - block, last - 1, last}):
        h = torch.zeros(T, 64)
        h[:, 15], h[:, 48] = 2.0, 1.0
        h[:, 16:30] = torch.randn(T, 14, generator=g).to(torch.bfloat16).float()
        h[target, 16:30], h[target, 16 + 15] = 0.0, 3.0
        h[:, 32:40] = torch.randn(T, rd, generator=g).to(torch.bfloat16).float()
        want = mixer_oracle(config, w, 0, h)
        c = torch.zeros(r, dtype=F64)
        c[15] = 4.0
        gates = torch.sigmoid(torch.tensor([0.5, -1.0], dtype=F64))
        assert close(want[-1, :H * dv], torch.cat([gates[0] * c, gates[1] * 2.0 * c]), 1e-3)      # (the premise)
        got = run_mixer(model, 0, {1: h}, {1: T}, [T] if mode == "prompt" else [T - 1, 1])
        assert close(got[1][-1], want[-1], 2e-5 if dtype == "float32" else 1e-2), target


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cut_sizes", [[90], [1], [2, 31, 1]])
def test_latent_attention_the_rotated_shared_key_decides(dev, dtype, cut_sizes):
    """No unrotated scores at all: what a head attends to follows from the rotation of the shared key part (its layout, its scaled frequencies and
    the factor on sine and cosine, which is squared in the score)."""
    r, rd, H, dv = 16, 8, 3, 16
    config = one_layer(64, latent(H, 8, rd, dv, r, 24, base=50.0, scaling=(8.0, 30, 4.0, 1.0), scale=2.0))
    g = torch.Generator().manual_seed(3)
    uq = torch.zeros(H * (8 + rd), 24)
    for a in range(H):
        uq[a * (8 + rd) + 8:(a + 1) * (8 + rd), 8 * a:8 * a + 8] = torch.eye(rd)
    w = zero_weights(config, dq=pick(24, 64, 0), dq__norm=torch.ones(24), uq=uq, dkv=torch.cat([pick(r, 64, 24), pick(rd, 64, 40)]), dkv__norm=torch.ones(r), uv=torch.randn(H * dv, r, generator=g),
                     sink=torch.tensor([-20.0, 0.0, 3.0]), o=torch.cat([torch.eye(H * dv), torch.zeros(64 - H * dv, H * dv)]))
    h = torch.randn(90, 64, generator=g).to(torch.bfloat16).float()
    want = mixer_oracle(config, w, 0, h)
    plain = json.loads(json.dumps(config))
    del plain["layers"][0]["mixer"]["rot"]["scaling"]
    assert not close(mixer_oracle(plain, w, 0, h), want, 0.2)      # (the premise)
    model = make_model("", dtype, dev, max_tokens=3 * 96, block=4, config=config, weights=w)
    got = run_mixer(model, 0, {2: h}, {2: 90}, cut_sizes)[2]
    assert close(got, want, 3e-5) if dtype == "float32" else agrees(got, want, dtype)


# ---- gated linear attention -------------------------------------------------------------------------------------------------------------
def linear_attention_run(dev, H, d, dv, tau, rows, lens, cut_sizes):
    """rows: slot -> [T, q | k | v | z] (z [H * d] the decay's raw values, bias included)."""
    from vllm_i64_amd import ops_dense as D
    nd, rv = H * d, H * dv
    state = torch.full((3, H, dv, d), 9.0, device=dev)
    eye, rate, zero = (-torch.eye(nd)).to(torch.bfloat16).to(dev), torch.full((nd,), 1.0 / tau, device=dev), torch.zeros(nd, device=dev)
    got = {s: [] for s in lens}
    for runs in steps_of(lens, cut_sizes):
        r = Rows(dev, runs)
        P = torch.cat([rows[s][p:p + c] for s, p, c in runs]).float().to(dev).contiguous()
        F, O = torch.empty(r.n, nd, device=dev), torch.empty(r.n, rv, device=dev)
        D.linear(P, eye, F, m=r.n, a_off=2 * nd + rv, exact=True, bias=zero, epilogue=D.EPI_DECAY, e=rate)
        D.gla_scan(P, f=F, q_off=0, k_off=nd, f_off=0, v_off=2 * nd, heads=H, dim=d, vdim=dv, seg_start=r.seg, nseg=r.nseg, positions=r.pos, slot_ids=r.slots, state=state, out=O,
                   n=r.n, q_scale=d ** -0.5)
        row = 0
        for s, p, c in runs:
            got[s].append(O[row:row + c].cpu())
            row += c
    return {s: torch.cat(v) for s, v in got.items()}


def linear_attention_oracle(H, d, dv, tau, rows):
    T, nd = rows.shape[0], H * d
    x = rows.double()
    q, k, v, z = x[:, :nd].reshape(T, H, d), x[:, nd:2 * nd].reshape(T, H, d), x[:, 2 * nd:2 * nd + H * dv].reshape(T, H, dv), x[:, 2 * nd + H * dv:].reshape(T, H, d)
    return R.gated_linear_recurrence(q * d ** -0.5, k, v, R.channel_decay(z, tau)).reshape(T, H * dv)


@pytest.mark.parametrize("H,d,dv,tau", [(3, 40, 24, 16.0), (4, 16, 64, 1.0), (1, 130, 8, 3.0), (6, 8, 33, 7.0), (2, 64, 20, 2.0), (2, 200, 40, 9.0), (48, 32, 64, 5.0)])
@pytest.mark.parametrize("cut_sizes", [[200], [1], [2, 5, 1, 3, 90], [7, 2]])
def test_gated_linear_attention_under_cuts(dev, H, d, dv, tau, cut_sizes):
    g = torch.Generator().manual_seed(H * d)
    lens = {2: 60 if H > 8 else 120, 0: 31, 1: 4}
    rows = {s: torch.randn(T, 3 * H * d + H * dv, generator=g) for s, T in lens.items()}
    got = linear_attention_run(dev, H, d, dv, tau, rows, lens, cut_sizes)
    for s in lens:
        assert close(got[s], linear_attention_oracle(H, d, dv, tau, rows[s]), 2e-5), s


@pytest.mark.parametrize("H,d,dv", [(4, 64, 32), (3, 40, 24), (2, 128, 128), (2, 200, 40), (1, 12, 5)])
@pytest.mark.parametrize("own_matrix", [True, False])
@pytest.mark.parametrize("own_keys", [True, False])
def test_gated_linear_scan_forms_agree_bit_for_bit(dev, H, d, dv, own_matrix, own_keys):
    """Loads straight into registers, or tokens staged through LDS with one, two or four value columns per lane; decays in a matrix of their own or
    as columns of the projections; keys of their own or one minus the decay: runs of unequal length, continued from slots' states or fresh, in scattered slots."""
    from vllm_i64_amd import _lib, ops_dense as D
    g = torch.Generator().manual_seed(d + dv)
    runs = [(4, 0, 33), (1, 7, 1), (0, 3, 16), (3, 0, 17), (2, 50, 70)]
    r = Rows(dev, runs)
    nd = H * d
    P, F = torch.randn(r.n, 3 * nd + H * dv, generator=g), torch.rand(r.n, nd, generator=g)
    P[:, 2 * nd + H * dv:] = F
    S0 = torch.randn(5, H, dv, d, generator=g)
    Pd, Fd = P.to(dev), F.to(dev)
    got = []
    try:
        for form in (1, 2, 3, 4, 0):
            _lib.call_dense("i64h_set_gdn_scan_form", form)
            S, O = S0.to(dev).clone(), torch.full((r.n, H * dv), 7.0, device=dev)
            D.gla_scan(Pd, f=Fd if own_matrix else None, q_off=0, k_off=nd if own_keys else -1, f_off=0 if own_matrix else 2 * nd + H * dv, v_off=2 * nd, heads=H, dim=d, vdim=dv, seg_start=r.seg,
                       nseg=r.nseg, positions=r.pos, slot_ids=r.slots, state=S, out=O, n=r.n, q_scale=0.3)
            got.append((O.cpu(), S.cpu()))
    finally:
        _lib.call_dense("i64h_set_gdn_scan_form", 0)
    for O, S in got[1:]:
        assert torch.equal(O, got[0][0]) and torch.equal(S, got[0][1])
    at = 0
    for slot, p, c in runs:      # (the fresh runs against the oracle's recurrence)
        x, f = P[at:at + c].double(), F[at:at + c].double()
        if p == 0:
            k = x[:, nd:2 * nd] if own_keys else 1.0 - f
            o = R.gated_linear_recurrence(0.3 * x[:, :nd].reshape(c, H, d), k.reshape(c, H, d), x[:, 2 * nd:2 * nd + H * dv].reshape(c, H, dv), f.reshape(c, H, d))
            assert close(got[0][0][at:at + c], o.reshape(c, H * dv), 2e-5)
        at += c


@pytest.mark.parametrize("cut_sizes", [[500], [1], [64, 3]])
def test_gated_linear_attention_keeps_one_channel_and_forgets_another(dev, cut_sizes):
    """What the first token wrote along a channel whose decay is next to one is still there 500 tokens later; along a channel that decays
    fast it is gone (a decay taken per head, a state lost at a cut or a slot's stale state taken over would show)."""
    H, d, dv, tau, T = 2, 12, 10, 4.0, 500
    nd = H * d
    g = torch.Generator().manual_seed(7)
    rows = torch.randn(T, 3 * nd + H * dv, generator=g)
    z0 = 2 * nd + H * dv
    rows[:, z0:] = 16.0                                       # (sigmoid next to one: nothing decays ...)
    rows[:, z0 + 1] = rows[:, z0 + d + 1] = -3.0              # (... but the second channel of either head)
    for a in range(H):
        rows[:, nd + a * d:nd + a * d + 2] = 0.0              # no later key has a part along the first two channels
        rows[0, nd + a * d:nd + (a + 1) * d] = 0.0
    for channel, lasts in ((0, True), (1, False)):
        x = rows.clone()
        x[T - 1, :nd] = 0.0
        for a in range(H):
            x[0, nd + a * d + channel] = 2.0
            x[T - 1, a * d + channel] = 9.0                   # the last query asks along that channel
        want = linear_attention_oracle(H, d, dv, tau, x)
        o_last = float(want[-1].abs().max())
        assert (o_last > 0.5) == lasts                        # (the premise)
        got = linear_attention_run(dev, H, d, dv, tau, {1: x}, {1: T}, cut_sizes)[1]
        assert close(got, want, 5e-5) and abs(float(got[-1].abs().max()) - o_last) < 1e-3


# ---- router and experts --------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("E,top", [(6, 2), (12, 12), (16, 4), (5, 1), (70, 9), (1, 1), (300, 3)])
@pytest.mark.parametrize("n", [2, 301, 700])
def test_router_takes_sigmoid_scores_as_they_are(dev, E, top, n):
    """Few rows take a workgroup each, many a wave each."""
    from vllm_i64_amd import ops_dense as D
    g = torch.Generator().manual_seed(E + top)
    gi, gw = torch.empty(n, top, dtype=torch.int32, device=dev), torch.empty(n, top, device=dev)
    kw = dict(entries=E, groups=1, keep=1, top=top, idx=gi, wgt=gw, n=n, sigmoid_scores=True)
    for spread in (2.0, 60.0):      # (wide: most scores round to one or are next to zero, the choice is the logits' all the same)
        z = torch.randn(n, E, generator=g) * spread
        idx, wgt = R.route(z.double(), top)
        D.route_topk(z.to(dev), correction=None, scale=1.0, raw_weights=True, **kw)
        assert torch.equal(gi.cpu().long(), idx) and close(gw, wgt, 1e-5)
    z = torch.randn(n, E, generator=g) * 2.0
    idx, wgt = R.route(z.double(), top)
    D.route_topk(z.to(dev), correction=None, scale=2.5, **kw)                                # renormalised, times a scale
    assert torch.equal(gi.cpu().long(), idx) and close(gw, 2.5 * wgt / wgt.sum(-1, keepdim=True), 1e-5)
    z, c = torch.randn(n, E, generator=g), torch.randn(E, generator=g)
    D.route_topk(z.to(dev), correction=c.to(dev), scale=1.0, raw_weights=True, **kw)      # a corrected choice, uncorrected weights
    pickd = (torch.sigmoid(z.double()) + c.double()).topk(top, -1).indices
    same = (gi.cpu().long() == pickd).all(-1)
    assert int((~same).sum()) <= max(1, n // 100) and close(gw.cpu()[same], torch.sigmoid(z.double()).gather(1, pickd)[same], 1e-5)
    for K in (72, 45, 1300):
        h = torch.randn(n, K, generator=g)
        w = (torch.randn(E, K, generator=g) * 2 * K ** -0.5).to(torch.bfloat16)
        idx, wgt = R.route(h.double() @ w.double().T, top)
        D.route_topk(None, h=h.to(dev), w=w.to(dev), correction=None, scale=1.0, raw_weights=True, **kw)
        same = (gi.cpu().long() == idx).all(-1)
        assert int((~same).sum()) <= max(1, n // 100) and close(gw.cpu()[same], wgt[same], 1e-5)      # (a close call in 32 bits may fall the other way)
        b, gate, w1 = torch.randn(E, generator=g), torch.empty(n, device=dev), (torch.randn(E + 1, K, generator=g) * 2 * K ** -0.5).to(torch.bfloat16)
        z = h.double() @ w1.double().T
        D.route_topk(None, h=h.to(dev), w=w1.to(dev), bias=b.to(dev), gate_out=gate, correction=None, scale=1.0, raw_weights=True, **kw)
        idx, wgt = R.route(z[:, :E] + b.double(), top)
        same = (gi.cpu().long() == idx).all(-1)
        assert int((~same).sum()) <= max(1, n // 100) and close(gw.cpu()[same], wgt[same], 1e-5) and close(gate, torch.sigmoid(z[:, E]), 1e-5)


@pytest.mark.parametrize("name,l", [("odd", 1), ("odd", 2), ("odd", 4), ("plain", 2), ("plain", 3), ("wide", 1), ("wide", 2), ("tail", 0), ("once", 0)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n", [1, 7, 64, 200])
def test_mixture_of_experts_alone(dev, name, l, dtype, n):
    """The score multiplies what an expert reads: on the result it would be another function (the premise)."""
    model = make_model(name, dtype, dev)
    cfg, w = config_of(name), {k: v.double() for k, v in make_weights(name).items()}
    h = torch.randn(n, cfg["width"], generator=torch.Generator().manual_seed(n + l)).to(torch.bfloat16).float()
    B = model.buffers(n, 1)
    for beside in (False, True):
        B.h.copy_(h)
        B.y.fill_(5.0)
        model._moe_ff(B, model.layers[l], n, B.h, B.y, B.y2, beside=beside)
        torch.cuda.synchronize()
        idx = B.idx[: n * model.layers[l]["mlp"].top].view(n, -1).cpu()
        p, f = f"l{l}.mlp.", cfg["layers"][l]["mlp"]
        want = R.mixture_ff(w, p, f, h.double(), forced=idx)
        assert close(B.y, want, 2e-5) if dtype == "float32" else agrees(B.y, want, dtype)
    s = torch.sigmoid((h.double() @ w[p + "router"].T).gather(1, idx.long()))
    outside = sum(s[:, k:k + 1] * torch.cat([R.expert(w, f"{p}e{e}.", h[t:t + 1].double()) for t, e in enumerate(idx[:, k].tolist())]) for k in range(idx.shape[1]))
    if f.get("shared"):
        outside = outside + R.expert(w, p + "shared.", h.double())
    assert not close(outside, want, 1e-2)


@pytest.mark.parametrize("name,l", [("odd", 0), ("plain", 0), ("wide", 3)])
@pytest.mark.parametrize("n", [3, 100])
def test_dense_feed_forward_alone(dev, name, l, n):
    model = make_model(name, "float32", dev)
    w, f = {k: v.double() for k, v in make_weights(name).items()}, config_of(name)["layers"][l]["mlp"]
    h = torch.randn(n, model.cfg.width, generator=torch.Generator().manual_seed(n)) * 1.5
    B = model.buffers(n, 1)
    B.h.copy_(h)
    model._dense_glu(B, model.layers[l], n, B.h, B.y)
    assert float((h.double() @ w[f"l{l}.mlp.gate"].T > f["limit"]).double().mean()) > 0.03      # (the bound matters)
    assert close(B.y, R.clamped_ff(w, f"l{l}.mlp.", f["limit"], h.double()), 2e-5)


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


def test_every_pass_has_its_own_cache_and_state_and_adds_the_embedding(dev):
    """Decoding continues a prompt: were a cache or state shared between the passes of the loop, the second pass would overwrite what the
    first one needs for the next token; the passes do differ, and the added embedding matters (the premises)."""
    from vllm_i64_amd.engine import Engine
    name = "odd"
    toks = tokens(name, 40, 30)
    model = make_model(name, "float32", dev, max_tokens=64, max_seqs=1)
    got = replay(Engine(model), {"x": toks}, [[("x", 25)]] + [[("x", 1)] for _ in range(15)])["x"]
    want = oracle_logits(name, toks)
    assert agrees(got, want, "float32")
    first, second = [r for r, (l, _) in enumerate(model.cfg.layer_runs()) if l == 1][:2]
    assert not close(model.kv.state[first]["gla"], model.kv.state[second]["gla"], 1e-2)
    once = config_of(name)
    once["loop"]["times"] = 1
    assert not agrees(R.forward(once, make_weights(name), toks), want, "bfloat16")
    flat = config_of(name)                                     # the same layers in the same order without a loop: nothing is added
    loop = flat.pop("loop")
    order = list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], len(flat["layers"])))
    w = make_weights(name)
    fw = {k: v for k, v in w.items() if not k.startswith("l")}
    for j, i in enumerate(order):
        fw.update({f"l{j}." + k[len(f"l{i}."):]: v for k, v in w.items() if k.startswith(f"l{i}.")})
    flat["layers"] = [flat["layers"][i] for i in order]
    assert not agrees(R.forward(flat, fw, toks), want, "bfloat16")


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


@pytest.mark.parametrize("name", ["odd", "tail"])
def test_graph_decoder_steps_match_the_oracle(dev, name):
    """The batch decoder (a captured HIP graph replayed per step) from the first token on: the recurrence's state and the pages of every pass
    advance inside the graph, the two branches of a step included."""
    from vllm_i64_amd import _lib
    if not os.path.exists(_lib.LIB_PATH):
        pytest.skip("the batch decoder takes its argmax from the first library, which is not built")
    from vllm_i64_amd.model import GreedyDecoder
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
