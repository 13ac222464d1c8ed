"""The Vepelix design without a GPU: configuration, order of layer runs, registry, weight layout, and the oracle's own mechanisms against
written-out forms."""
import math

import pytest
import torch

from oracle import vepelix_ref as R
from tests.test_gpu_fukatar import close
from tests.vepelix_shapes import SHAPES, config_of, make_weights, rotation, tokens

F64 = torch.float64


def test_configuration_round_trip_and_design_flags():
    from vllm_i64_amd.config import VepelixConfig
    for name in SHAPES:
        c = VepelixConfig.from_dict(config_of(name))
        assert VepelixConfig.from_dict(c.to_dict()) == c
        for l in c.layers:
            if l.type == "latent_attention":
                assert l.mixer.sink and l.mixer.head_gate and l.mixer.q_rank > 0 and l.mixer.rot is not None and l.mixer.window == 0
            else:
                assert l.mixer.left.interleaved and l.mixer.left.qk_norm == "head_weight" and not l.mixer.left.sink and not l.mixer.left.rotate_values
            if l.mlp is not None and l.mlp.kind == "moe":
                assert l.mlp.sigmoid_scores and l.mlp.raw_weights and l.mlp.weigh_input and not l.mlp.shared_gate and not l.mlp.router_bias and l.mlp.limit == 0
    odd, plain = VepelixConfig.from_dict(config_of("odd")), VepelixConfig.from_dict(config_of("plain"))
    a, r = odd.layers[1].mixer.left, odd.layers[1].mixer.right
    assert (a.window, a.rot.dims, a.rot.factor, r.tau, odd.layers[1].mixer.left_scale, odd.layers[1].mixer.right_scale) == (13, 6, 8.0, 5.0, 1.3, 0.7)
    assert (odd.layers[0].mlp.limit, odd.layers[1].mlp.shared_ff, odd.layers[4].mlp.shared_ff) == (0.8, 18, 0)
    assert plain.loop is None and plain.layers[0].mixer.left.window == 0 and plain.layers[1].mlp is None and plain.layers[1].mixer.rot.factor == 0


def test_configuration_refuses_what_the_design_has_not():
    from vllm_i64_amd.config import VepelixConfig
    for change in (lambda c: c["layers"][0].update(type="mamba2"), lambda c: c.update(loop={"start": 2, "stop": 2, "times": 2}),
                   lambda c: c.update(loop={"start": 0, "stop": 9, "times": 2}), lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4),
                   lambda c: c["layers"][0]["mlp"].pop("limit"), lambda c: c["layers"][1]["mlp"]["router"].update(top=9),
                   lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=12), lambda c: c["layers"][1]["mixer"]["right"].update(tau=0.0),
                   lambda c: c["layers"][0]["mixer"].pop("q_rank"), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5)):
        bad = config_of("odd")
        change(bad)
        with pytest.raises(ValueError):
            VepelixConfig.from_dict(bad)


def test_layer_runs_and_where_passes_begin():
    from vllm_i64_amd.config import VepelixConfig
    want = {"odd": [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None), (4, None)], "plain": [(i, None) for i in range(4)],
            "wide": [(0, 0), (1, None), (2, None), (3, None), (0, 1), (1, None), (2, None), (3, None)],
            "tail": [(0, None), (1, None), (2, None), (3, 0), (3, 1), (3, 2), (3, 3)], "once": [(0, 0)]}
    for name, runs in want.items():
        assert VepelixConfig.from_dict(config_of(name)).layer_runs() == runs == R.layer_runs(config_of(name))


def test_registry_names_the_design_and_loader_takes_sizes_from_the_tensors(monkeypatch):
    from vllm_i64_amd import registry, vepelix
    assert "vepelix" in registry.architectures() and registry.architecture_of(config_of("odd")) == "Vepelix"
    seen = {}
    monkeypatch.setattr(vepelix, "VepelixModel", lambda cfg, tensors, **kw: seen.update(cfg=cfg, kw=kw))
    cfg = config_of("odd")
    del cfg["vocab"], cfg["width"], cfg["layers"][2]["mixer"]["q_rank"]
    registry._load_vepelix(cfg, make_weights("odd"), device="cpu", dtype="float32", max_seqs=2, max_tokens=100)
    c = seen["cfg"]
    assert (c.vocab, c.width, c.layers[2].mixer.q_rank, c.layers[0].mixer.q_rank) == (83, 42, 13, 22) and seen["kw"]["num_kv_blocks"] == 7


def test_weights_on_the_host_cover_every_run_and_keep_the_layout():
    """Layout work alone (no launch): every layer run has its own cache and state, projections start at multiples of eight columns, the decay
    map's second factor is held negated with zeros in its padding, norms are one plus what is stored."""
    from vllm_i64_amd.config import VepelixConfig
    from vllm_i64_amd.vepelix import VepelixModel
    for name in SHAPES:
        w = make_weights(name)
        cfg = VepelixConfig.from_dict(config_of(name))
        m = VepelixModel(cfg, w, device="cpu", dtype="float32", max_seqs=2, num_kv_blocks=3)
        assert len(m.kv.rows) == len(m.kv.state) == len(cfg.layer_runs())
        held = [t.data_ptr() for t in m.kv.rows if t is not None] + [t.data_ptr() for d in m.kv.state for t in d.values()]
        assert len(set(held)) == len(held)
        assert m.repeats == (name not in ("plain", "once"))
        for i, d in enumerate(m.layers):
            assert torch.equal(d["norm1"], 1.0 + w[f"l{i}.norm1"].float())
            if d["type"] == "latent_attention":
                assert d["q_off"] % 8 == d["dkv_off"] % 8 == d["g_off"] % 8 == 0
                assert torch.equal(d["w_in"][d["dkv_off"]: d["dkv_off"] + d["m"].cache_width], w[f"l{i}.mix.dkv"])
                continue
            ra = SHAPES[name]["ranks"][i]
            assert d["a1_off"] % 8 == d["rk_off"] % 8 == d["rg_off"] % 8 == 0
            assert torch.equal(d["w_in"][d["a1_off"]: d["a1_off"] + ra], w[f"l{i}.mix.right.a1"]) and not d["w_in"][d["a1_off"] + ra:].any()
            assert torch.equal(d["a2"][:, :ra], -w[f"l{i}.mix.right.a2"]) and not d["a2"][:, ra:].any()
    bad = make_weights("odd")
    bad["l1.mix.right.a2"] = bad["l1.mix.right.a2"][:-1]
    with pytest.raises(ValueError):
        VepelixModel(VepelixConfig.from_dict(config_of("odd")), bad, device="cpu")
    del bad["l1.mix.right.a2"]
    with pytest.raises(KeyError):
        VepelixModel(VepelixConfig.from_dict(config_of("odd")), bad, device="cpu")


def test_oracle_visibility():
    assert [j for j in range(10) if R.sees(7, j, {"size": 4})] == [4, 5, 6, 7]
    assert [j for j in range(10) if R.sees(2, j, {"size": 4})] == [0, 1, 2]
    assert [j for j in range(10) if R.sees(5, j, {"size": 1})] == [5]
    assert [j for j in range(10) if R.sees(3, j, None)] == [0, 1, 2, 3]


def test_oracle_sink_counts_once_and_unscaled():
    s = R.sink_softmax(torch.tensor([1.0, 2.0], dtype=F64), torch.tensor(0.5, dtype=F64))
    den = math.exp(1.0) + math.exp(2.0) + math.exp(0.5)
    assert close(s, torch.tensor([math.exp(1.0) / den, math.exp(2.0) / den], dtype=F64), 1e-12)


def test_frequencies_of_oracle_and_product_agree_and_follow_the_ramp():
    from vllm_i64_amd.config import RotaryConfig
    for base, dims, scaling in ((10000.0, 16, None), (10000.0, 16, (4.0, 4096, 32.0, 1.0)), (500.0, 6, (8.0, 40, 4.0, 1.0)), (777.0, 12, (16.0, 30, 8.0, 8.0)), (5000.0, 2, (4.0, 60, 6.0, 0.5))):
        r = rotation(base, dims, scaling)
        f, mult = R.frequencies(r)
        g, m2 = RotaryConfig.from_dict(r).frequencies()
        assert max(abs(a - b) / b for a, b in zip(f, g)) < 1e-12 and abs(mult - m2) < 1e-12
    # 4096 positions make 32 turns at pair index 16 ln(4096 / 64 pi) / (2 ln 10000) = 2.6 and one turn at 5.6: pairs up to 2 stay, from 6 on divided
    f, mult = R.frequencies(rotation(10000.0, 16, (4.0, 4096, 32.0, 1.0)))
    plain = [10000.0 ** (-2.0 * i / 16) for i in range(8)]
    want = [p / 4.0 * r + p * (1.0 - r) for p, r in zip(plain, (0, 0, 0, 0.25, 0.5, 0.75, 1, 1))]
    assert close(torch.tensor(f, dtype=F64), torch.tensor(want, dtype=F64), 1e-12) and abs(mult - (1.0 + 0.1 * math.log(4.0))) < 1e-12


def test_oracle_rotation_turns_neighbours():
    x = torch.arange(6, dtype=F64).reshape(1, 1, 6) + 1.0
    r = R.rotate_pairs(x, torch.tensor([3]), rotation(16.0, 4))[0, 0]
    a, b = 3.0, 3.0 * 16.0 ** -0.5
    want = [1 * math.cos(a) - 2 * math.sin(a), 2 * math.cos(a) + 1 * math.sin(a), 3 * math.cos(b) - 4 * math.sin(b), 4 * math.cos(b) + 3 * math.sin(b), 5.0, 6.0]
    assert close(r, torch.tensor(want, dtype=F64), 1e-12)


def test_oracle_linear_recurrence_decays_each_channel_and_reads_after_the_write():
    q = torch.tensor([[[1.0, 0.0]], [[1.0, 10.0]]], dtype=F64)
    k = torch.tensor([[[0.6, 0.8]], [[0.0, 2.0]]], dtype=F64)
    v = torch.tensor([[[1.0, 2.0, 3.0]], [[5.0, 0.0, 1.0]]], dtype=F64)
    alpha = torch.tensor([[[0.3, 0.3]], [[0.5, 0.25]]], dtype=F64)
    o = R.gated_linear_recurrence(q, k, v, alpha)
    assert close(o[0, 0], 0.6 * v[0, 0], 1e-12)
    assert close(o[1, 0], (0.5 * 0.6 + 10.0 * 0.25 * 0.8) * v[0, 0] + 20.0 * v[1, 0], 1e-12)
    a = R.channel_decay(torch.tensor([0.0, 3.0], dtype=F64), 4.0)
    assert close(a, torch.tensor([0.5 ** 0.25, (1.0 / (1.0 + math.exp(-3.0))) ** 0.25], dtype=F64), 1e-12)


def test_oracle_bounds_of_the_dense_feed_forward():
    one = torch.ones(1, 1, dtype=F64)
    W = {"e.gate": one, "e.up": one, "e.down": one}
    for z, g, u in ((0.5, 0.5, 0.5), (3.0, 1.5, 1.5), (-4.0, -4.0, -1.5)):
        want = g / (1.0 + math.exp(-1.702 * g)) * (u + 1.0)
        assert abs(float(R.clamped_ff(W, "e.", 1.5, torch.full((1, 1), z, dtype=F64))) - want) < 1e-12


def test_oracle_router_keeps_the_scores_and_the_weight_is_on_the_input():
    idx, w = R.route(torch.tensor([[0.0, 3.0, 1.0, 2.0]], dtype=F64), 2)
    assert idx.tolist() == [[1, 3]] and close(w[0], torch.tensor([1.0 / (1.0 + math.exp(-3.0)), 1.0 / (1.0 + math.exp(-2.0))], dtype=F64), 1e-12)
    one = torch.ones(1, 1, dtype=F64)
    W = {"router": 0.0 * one, "e0.gate": one, "e0.up": one, "e0.down": one}
    got = float(R.mixture_ff(W, "", {"router": {"experts": 1, "top": 1}}, 4.0 * one))       # score one half: the expert sees 2
    assert abs(got - 4.0 / (1.0 + math.exp(-2.0))) < 1e-12


def test_oracle_runs_every_shape():
    for name in SHAPES:
        layers = []
        z = R.forward(config_of(name), make_weights(name), tokens(name, 12, 1), layers)
        assert z.shape == (12, SHAPES[name]["vocab"]) and bool(torch.isfinite(z).all()) and len(layers) == len(R.layer_runs(config_of(name)))
