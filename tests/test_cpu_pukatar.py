"""The Pukatar design without a GPU: configuration, order of layer runs, registry, weight layout, and the oracle's own mechanisms against
written-out forms."""
import math

import pytest
import torch

from oracle import pukatar_ref as R
from tests.pukatar_shapes import SHAPES, config_of, make_weights, tokens
from tests.test_gpu_fukatar import close

F64 = torch.float64


def test_configuration_round_trip_and_design_flags():
    from vllm_i64_amd.config import PukatarConfig
    for name in SHAPES:
        c = PukatarConfig.from_dict(config_of(name))
        assert PukatarConfig.from_dict(c.to_dict()) == c
        for l in c.layers:
            if l.type == "attention":
                assert l.mixer.sink and not l.mixer.interleaved and l.mixer.qk_norm is None and not l.mixer.rotate_values and not l.mixer.head_gate
            else:
                assert (l.mixer.decay, l.mixer.gate) == ("channel", "sigmoid")
            if l.mlp is not None and l.mlp.kind == "moe":
                assert l.mlp.router_bias and l.mlp.chosen_softmax and l.mlp.shared_gate and l.mlp.limit > 0
    odd, plain = PukatarConfig.from_dict(config_of("odd")), PukatarConfig.from_dict(config_of("plain"))
    assert (odd.layers[0].mixer.window, odd.layers[0].mixer.keep_first, odd.layers[1].mlp.limit, odd.layers[1].mlp.shared_limit) == (13, 3, 0.7, 1.1)
    assert plain.loop is None and plain.layers[1].mixer.kv_heads == 2 and plain.layers[1].mixer.window == 0 and plain.layers[1].mixer.rot is None
    assert plain.layers[1].mlp is None and plain.layers[2].mixer.keep_first == 0 and plain.layers[2].mlp.shared_ff == 0


def test_configuration_refuses_what_the_design_has_not():
    from vllm_i64_amd.config import PukatarConfig
    for change in (lambda c: c["layers"][0].update(type="mamba2"), lambda c: c.update(loop={"start": 2, "stop": 2, "times": 2}),
                   lambda c: c.update(loop={"start": 0, "stop": 9, "times": 2}), lambda c: c["layers"][3]["mixer"].update(kv_heads=2),
                   lambda c: c["layers"][1]["mlp"]["expert"].pop("limit"), lambda c: c["layers"][1]["mlp"]["router"].update(top=9),
                   lambda c: c["layers"][0]["mixer"]["rot"].update(dims=12), lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1)):
        bad = config_of("odd")
        change(bad)
        with pytest.raises(ValueError):
            PukatarConfig.from_dict(bad)


def test_layer_runs_and_where_passes_begin():
    from vllm_i64_amd.config import PukatarConfig
    want = {"odd": [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None), (4, None)], "plain": [(i, None) for i in range(4)],
            "wide": [(0, 0), (1, None), (2, None), (3, None), (0, 1), (1, None), (2, None), (3, None)], "tail": [(0, None), (1, None), (2, 0), (3, None)]}
    for name, runs in want.items():
        assert PukatarConfig.from_dict(config_of(name)).layer_runs() == runs == R.layer_runs(config_of(name))


def test_registry_names_the_design_and_loader_takes_sizes_from_the_tensors(monkeypatch):
    from vllm_i64_amd import pukatar, registry
    assert "pukatar" in registry.architectures() and registry.architecture_of(config_of("odd")) == "Pukatar"
    seen = {}
    monkeypatch.setattr(pukatar, "PukatarModel", lambda cfg, tensors, **kw: seen.update(cfg=cfg, kw=kw))
    cfg = config_of("odd")
    del cfg["vocab"], cfg["width"], cfg["layers"][3]["mixer"]["conv"]
    registry._load_pukatar(cfg, make_weights("odd"), device="cpu", dtype="float32", max_seqs=2, max_tokens=100)
    c = seen["cfg"]
    assert (c.vocab, c.width, c.layers[3].mixer.conv, c.layers[1].mixer.conv) == (83, 42, 5, 3) and seen["kw"]["num_kv_blocks"] == 7


def test_weights_on_the_host_cover_every_run_and_keep_the_layout():
    """Layout work alone (no launch): every layer run has its own cache or state, projections start at multiples of eight columns, the low-rank
    factors' padding is zero."""
    from vllm_i64_amd.config import PukatarConfig
    from vllm_i64_amd.pukatar import PukatarModel
    for name in SHAPES:
        w = make_weights(name)
        cfg = PukatarConfig.from_dict(config_of(name))
        m = PukatarModel(cfg, w, device="cpu", dtype="float32", max_seqs=2, num_kv_blocks=3)
        assert len(m.kv.rows) == len(m.kv.state) == len(cfg.layer_runs())
        held = [t.data_ptr() for t in m.kv.rows if t is not None] + [t.data_ptr() for d in m.kv.state for t in d.values()]
        assert len(set(held)) == len(held)
        for i, d in enumerate(m.layers):
            if d["type"] != "channel_delta":
                continue
            ra, rg = SHAPES[name]["ranks"][i]
            assert d["a1_off"] % 8 == d["g1_off"] % 8 == d["rb_off"] % 8 == 0
            assert torch.equal(d["w_in"][d["a1_off"]: d["a1_off"] + ra], w[f"l{i}.mix.a1"]) and not d["w_in"][d["a1_off"] + ra: d["g1_off"]].any()
            assert torch.equal(d["a2"][:, :ra], w[f"l{i}.mix.a2"]) and not d["a2"][:, ra:].any() and not d["g2"][:, rg:].any()
    bad = make_weights("odd")
    bad["l1.mix.a2"] = bad["l1.mix.a2"][:-1]
    with pytest.raises(ValueError):
        PukatarModel(PukatarConfig.from_dict(config_of("odd")), bad, device="cpu")
    del bad["l1.mix.a2"]
    with pytest.raises(KeyError):
        PukatarModel(PukatarConfig.from_dict(config_of("odd")), bad, device="cpu")


def test_oracle_visibility():
    m = {"size": 4, "keep_first": 2}
    assert [j for j in range(10) if R.sees(7, j, m)] == [0, 1, 4, 5, 6, 7]
    assert [j for j in range(10) if R.sees(2, j, m)] == [0, 1, 2]
    assert [j for j in range(10) if R.sees(5, j, {"size": 1, "keep_first": 0})] == [5]
    assert [j for j in range(10) if R.sees(3, j, None)] == [0, 1, 2, 3]
    assert [j for j in range(10) if R.sees(4, j, {"size": 2, "keep_first": 9})] == [0, 1, 2, 3, 4]


def test_oracle_sink_counts_once_and_unscaled():
    s = R.sink_softmax(torch.tensor([1.0, 2.0], dtype=F64), torch.tensor(0.5, dtype=F64))
    den = math.exp(1.0) + math.exp(2.0) + math.exp(0.5)
    assert close(s, torch.tensor([math.exp(1.0) / den, math.exp(2.0) / den], dtype=F64), 1e-12)


def test_oracle_rotation_turns_halves():
    x = torch.arange(6, dtype=F64).reshape(1, 1, 6) + 1.0
    r = R.rotate_halves(x, torch.tensor([3]), 16.0, 4)[0, 0]
    a, b = 3.0, 3.0 * 16.0 ** -0.5
    want = [1 * math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b), 3 * math.cos(a) + 1 * math.sin(a), 4 * math.cos(b) + 2 * math.sin(b), 5.0, 6.0]
    assert close(r, torch.tensor(want, dtype=F64), 1e-12)


def test_oracle_delta_rule_decays_each_channel_by_its_own_factor():
    d, dv = 3, 2
    v = torch.tensor([[[1.0, 2.0]], [[0.0, 0.0]]], dtype=F64)
    k = torch.tensor([[[0.6, 0.8, 0.0]], [[0.0, 0.0, 1.0]]], dtype=F64)
    q = torch.tensor([[[1.0, 0.0, 0.0]], [[1.0, 10.0, 0.0]]], dtype=F64)
    g = torch.tensor([[[0.3, 0.3, 0.3]], [[0.5, 0.25, 0.125]]], dtype=F64)
    o = R.channel_delta_rule(q, k, v, torch.ones(2, 1, dtype=F64), g)
    assert close(o[0, 0], 0.6 * v[0, 0], 1e-12)                                  # read after the write, the first write not decayed
    assert close(o[1, 0], (0.5 * 0.6 + 10.0 * 0.25 * 0.8) * v[0, 0], 1e-12)
    # a repeated key replaces what it stored (decayed), up to the write strength
    o = R.channel_delta_rule(k[[0, 0]], k[[0, 0]], torch.stack([v[0], 3.0 * v[0]]), torch.tensor([[1.0], [0.5]], dtype=F64), torch.ones(2, 1, d, dtype=F64))
    assert close(o[1, 0], 2.0 * v[0, 0], 1e-12)
    a = R.channel_decay(torch.zeros(1, 4, dtype=F64), torch.tensor([0.0, 1.0], dtype=F64), torch.zeros(4, dtype=F64), 2)
    assert close(a[0], torch.tensor([[0.5, 0.5], [0.5 ** math.e] * 2], dtype=F64), 1e-12)


def test_oracle_expert_bounds():
    one = torch.ones(1, 1, dtype=F64)
    W = {"e.gate": one, "e.up": one, "e.down": one}
    for z, g, u in ((0.5, 0.5, 0.5), (3.0, 1.5, 1.5), (-4.0, -4.0, -1.5)):
        want = g / (1.0 + math.exp(-1.702 * g)) * (u + 1.0)
        assert abs(float(R.clamped_expert(W, "e.", 1.5, torch.full((1, 1), z, dtype=F64))) - want) < 1e-12


def test_oracle_router_softmax_over_the_chosen():
    idx, w = R.route(torch.tensor([[0.0, 3.0, 1.0, 2.0]], dtype=F64), 2)
    assert idx.tolist() == [[1, 3]] and close(w[0], torch.tensor([1.0 / (1.0 + math.exp(-1.0)), 1.0 / (1.0 + math.exp(1.0))], dtype=F64), 1e-12)


def test_oracle_runs_every_shape():
    for name in SHAPES:
        layers = []
        z = R.forward(config_of(name), make_weights(name), tokens(name, 12, 1), layers)
        assert z.shape == (12, SHAPES[name]["vocab"]) and bool(torch.isfinite(z).all()) and len(layers) == len(R.layer_runs(config_of(name)))
