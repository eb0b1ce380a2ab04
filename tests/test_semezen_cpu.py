"""Semezen on the CPU: configuration, tensor list, cache plan, random-weights folder, and the plain implementation held to closed
forms of its own."""
import copy
import math

import pytest
import torch

import plain_semezen as P
import tiny_semezen as TS
from photon_infer_amd.config import SemezenConfig
from photon_infer_amd.errors import ConfigError, UnsupportedModelError
from photon_infer_amd.parts import StateSpec
from photon_infer_amd.parts.model import plan_cache
from photon_infer_amd.registry import build_model_spec, config_from_dict, load_config

F64 = torch.float64


@pytest.mark.parametrize("name", list(TS.ALL))
def test_configuration_round_trip_and_registry(name):
    raw = TS.ALL[name][0]
    cfg = config_from_dict(raw)
    assert isinstance(cfg, SemezenConfig) and cfg.architecture == "Semezen"
    assert SemezenConfig.from_dict(cfg.to_dict()) == cfg
    assert cfg.vocab_size == raw["vocab"] and cfg.hidden_size == raw["width"] and len(cfg.layers) == len(raw["layers"])


def test_errors_name_their_key():
    def broken(edit):
        raw = copy.deepcopy(TS.TINY_A)
        edit(raw)
        return raw
    cases = [(lambda r: r["layers"][1]["mixer"].pop("scale"), "scale"), (lambda r: r["layers"][0]["mixer"].pop("width"), "width"),
             (lambda r: r["layers"][1]["mixer"].update(heads=3), "kv_heads"), (lambda r: r["layers"][1]["mixer"].update(vdim=24), "vdim"),
             (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=7), "rot.dims"), (lambda r: r["layers"][1]["mixer"]["rot"]["scaling"].update(high=1.0), "high"),
             (lambda r: r["layers"][1]["mixer"]["mask"].update(size=0), "size"), (lambda r: r["layers"][1]["mlp"]["router"].update(top=6), "router.top"),
             (lambda r: r["layers"][1]["mlp"]["expert"].pop("limit"), "limit"), (lambda r: r.pop("streams"), "streams"), (lambda r: r.pop("norm"), "norm")]
    for edit, word in cases:
        with pytest.raises(ConfigError, match=word):
            SemezenConfig.from_dict(broken(edit))
    with pytest.raises(UnsupportedModelError, match="layer type"):
        SemezenConfig.from_dict(broken(lambda r: r["layers"][0].update(type="gla")))
    with pytest.raises(UnsupportedModelError, match="feed-forward kind"):
        SemezenConfig.from_dict(broken(lambda r: r["layers"][0]["mlp"].update(kind="glu")))
    with pytest.raises(UnsupportedModelError, match="residual streams"):
        build_model_spec(SemezenConfig.from_dict(broken(lambda r: r.update(streams=17))))


def test_tensor_list():
    spec = build_model_spec(SemezenConfig.from_dict(TS.TINY_C))
    shapes = {s.name: s.shape for s in spec.tensor_specs()}
    assert len(shapes) == len(spec.tensor_specs())
    assert shapes["l0.hc1.in"] == (5,) and shapes["l0.hc1.mix"] == (5, 5) and shapes["l0.shift"] == (90,)
    assert shapes["l0.mix.q"] == (72, 90) and shapes["l0.mix.k.b"] == (36,) and shapes["l0.mix.g"] == (72, 90) and shapes["l0.mix.o"] == (90, 72)
    assert shapes["l1.mix.z.b"] == (37,) and shapes["l1.mix.o"] == (90, 37) and shapes["l1.mlp.e8.down"] == (90, 36) and shapes["l1.mlp.router"] == (9, 90)
    assert shapes["l2.mlp.up"] == (52, 90) and shapes["final.norm"] == (90,) and shapes["head"] == (257, 90)
    assert "l0.mix.v" not in shapes and "l0.mix.g.b" not in shapes and "l2.mlp.gate" not in shapes
    assert "l0.norm2" not in shapes and "l0.hc2.in" not in shapes                        # no feed-forward, nothing in front of it


def test_cache_plan_has_pages_per_window_and_a_token_before_for_every_layer():
    plan = plan_cache(build_model_spec(SemezenConfig.from_dict(TS.TINY_A)))
    assert [g.window for g in plan.groups] == [7, 20]
    assert [g.owners for g in plan.groups] == [((1, 0),), ((3, 0),)]
    assert [k for k, _ in plan.states] == [(0, 0), (0, 1), (1, 1), (2, 0), (2, 1), (3, 1)]
    assert [s.shape for _, s in plan.states] == [(48,), (64,), (64,), (80,), (64,), (64,)]
    assert all(isinstance(s, StateSpec) and s.dtype == torch.float32 for _, s in plan.states)
    plan = plan_cache(build_model_spec(SemezenConfig.from_dict(TS.TINY_C)))
    assert [g.window for g in plan.groups] == [None, 5]
    assert not plan_cache(build_model_spec(SemezenConfig.from_dict(TS.TINY_E))).groups


def test_folder_with_random_weights(tmp_path):
    d = TS.make_model_dir(tmp_path, "A", seed=3)
    cfg = load_config(d)
    raw, W = P.read_model_folder(d)
    assert set(W) == {s.name for s in build_model_spec(cfg).tensor_specs()}
    logits = P.forward(raw, W, [5, 6, 7, 8])
    assert logits.shape == (4, 300) and bool(torch.isfinite(logits).all())
    assert float(W["l0.mix.z.b"].float().mean()) < -2.0 and 0.2 < float(W["l0.shift"].float().mean()) < 0.8


# ----------------------------------------------------------------------------- the plain implementation's own closed forms
def test_streams_are_mixed_from_the_streams_as_they_were():
    X = [torch.tensor([1.0, 2.0], dtype=F64), torch.tensor([10.0, 20.0], dtype=F64)]
    y = torch.tensor([100.0, 200.0], dtype=F64)
    swap = torch.tensor([[0.0, 1.0], [1.0, 0.0]], dtype=F64)
    got = P.mix_streams(X, y, swap, torch.tensor([0.0, 0.5], dtype=F64))
    assert torch.equal(got[0], X[1]) and torch.equal(got[1], X[0] + 0.5 * y)
    one_way = torch.tensor([[1.0, 3.0], [0.0, 1.0]], dtype=F64)                          # from the first to the second only
    got = P.mix_streams(X, y, one_way, torch.zeros(2, dtype=F64))
    assert torch.equal(got[0], X[0]) and torch.equal(got[1], X[1] + 3.0 * X[0])


def test_shift_takes_the_token_before_as_it_was():
    h = torch.arange(1.0, 5.0, dtype=F64)[:, None].expand(4, 3)
    share = torch.tensor([0.0, 0.5, 1.0], dtype=F64)
    want = torch.tensor([[1.0, 0.5, 0.0], [2.0, 1.5, 1.0], [3.0, 2.5, 2.0], [4.0, 3.5, 3.0]], dtype=F64)
    assert torch.equal(P.shift_in(h, share), want)


def test_frequencies_in_three_bands():
    sc = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}
    freq = [P.rope_frequency(i, 16, 1000.0, sc) for i in range(8)]
    plain = [1000.0 ** (-2.0 * i / 16) for i in range(8)]
    kinds = set()
    for f, p in zip(freq, plain):
        wave = 2 * math.pi / p
        if wave < 16:
            assert f == p
            kinds.add("kept")
        elif wave > 64:
            assert f == p / 8
            kinds.add("slowed")
        else:
            assert p / 8 < f < p
            kinds.add("blended")
    assert kinds == {"kept", "slowed", "blended"}
    from photon_infer_amd.config.llama import RopeScaling
    from photon_infer_amd.parts import rope_frequencies
    made = rope_frequencies(16, 1000.0, RopeScaling("llama3", 8.0, 1.0, 4.0, 64))
    assert torch.allclose(made, torch.tensor(freq, dtype=F64), rtol=1e-12)


def test_rotation_of_paired_halves_keeps_a_head_s_length():
    x = torch.randn(2, 10, dtype=F64)
    y = P.rotate_halves(x, 7, 6, 30.0)
    assert torch.equal(y[:, 6:], x[:, 6:]) and torch.allclose((y * y).sum(-1), (x * x).sum(-1))
    for i in range(3):
        a = 7 * 30.0 ** (-2.0 * i / 6)
        assert torch.allclose(y[:, i], x[:, i] * math.cos(a) - x[:, i + 3] * math.sin(a))
        assert torch.allclose(y[:, i + 3], x[:, i + 3] * math.cos(a) + x[:, i] * math.sin(a))


def test_window_holds_exactly_its_size():
    T, W = 12, 4
    q, k = torch.zeros(T, 1, dtype=F64), torch.zeros(T, 1, dtype=F64)
    v = torch.arange(T, dtype=F64)[:, None]
    out = P.window_attention(q, k, v, 1.0, W)
    for i in range(T):
        lo = max(0, i - W + 1)
        assert math.isclose(float(out[i]), (lo + i) / 2.0)
    assert torch.equal(P.window_attention(q, k, v, 1.0, 1), v)


def test_gate_that_is_shut_keeps_and_one_that_is_open_takes():
    T = 6
    u = torch.tensor([2.0, -1.0, 0.0, -3.0, 1.0, 5.0], dtype=F64)[:, None]
    cand = [2.5, 1 / (1 + math.e), 0.5, 1 / (1 + math.e ** 3), 1.5, 5.5]
    out = P.gru_walk(torch.ones(T, 1, dtype=F64), u)
    assert torch.allclose(out[:, 0], torch.tensor(cand, dtype=F64))
    z = torch.zeros(T, 1, dtype=F64)
    z[1] = 1.0
    assert torch.allclose(P.gru_walk(z, u)[1:, 0], torch.full((5,), cand[1], dtype=F64)) and float(P.gru_walk(z, u)[0]) == 0.0
    half = P.gru_walk(torch.full((T, 1), 0.5, dtype=F64), u)
    assert math.isclose(float(half[5]), sum(c * 0.5 ** (6 - i) for i, c in enumerate(cand)))


def test_routing_by_sigmoids_that_are_not_renormalised():
    z = torch.tensor([0.0, 2.0, -1.0, 1.0], dtype=F64)
    order, w = P.route(z, 2)
    assert order == [1, 3] and torch.allclose(w, torch.sigmoid(z[[1, 3]]))
    assert P.route(torch.zeros(4, dtype=F64), 2)[0] == [0, 1]                            # equal scores: the lower index


def test_weight_multiplies_the_expert_s_input():
    """A unit that is clamped at once does not grow with its weight beyond the clamp: weighing the input is not weighing the output."""
    D, F = 4, 3
    W = {"router": torch.zeros(1, D, dtype=F64), "e0.gate": torch.randn(F, D, dtype=F64) * 50, "e0.up": torch.randn(F, D, dtype=F64) * 50,
         "e0.down": torch.randn(D, F, dtype=F64)}
    h = torch.randn(5, D, dtype=F64)
    mlp = {"router": {"experts": 1, "top": 1}, "expert": {"ff": F, "limit": 0.5}}
    got = P.routed_experts(h, mlp, W, "")
    assert torch.allclose(got, P.clamped_unit(0.5 * h, W, "e0.", 0.5))
    assert not torch.allclose(got, 0.5 * P.clamped_unit(h, W, "e0.", 0.5))


def test_gelu_is_the_exact_one():
    x = torch.linspace(-6, 6, 101, dtype=F64)
    assert torch.allclose(P.gelu(x), torch.nn.functional.gelu(x), atol=1e-14)
    assert not torch.allclose(P.gelu(x), torch.nn.functional.gelu(x, approximate="tanh"), atol=1e-5)
