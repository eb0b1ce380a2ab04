"""Roserax on the CPU: configuration, tensor list, cache plan and kept pages, work lists, random-weights folder, and the plain
implementation held to closed forms of its own."""
import copy
import math

import pytest
import torch

import plain_roserax as P
import tiny_roserax as TR
from photon_infer_amd.cache import CacheManager
from photon_infer_amd.config import RoseraxConfig
from photon_infer_amd.errors import ConfigError, UnsupportedModelError
from photon_infer_amd.ops.fast import AttentionPlanner
from photon_infer_amd.parts.model import plan_cache
from photon_infer_amd.registry import build_model_spec, config_from_dict, load_config

F64 = torch.float64


@pytest.mark.parametrize("name", list(TR.ALL))
def test_configuration_round_trip_and_registry(name):
    raw = TR.ALL[name][0]
    cfg = config_from_dict(raw)
    assert isinstance(cfg, RoseraxConfig) and cfg.architecture == "Roserax"
    assert RoseraxConfig.from_dict(cfg.to_dict()) == cfg and cfg.to_dict() == raw
    assert cfg.vocab_size == raw["vocab"] and cfg.hidden_size == raw["width"] and len(cfg.layers) == len(raw["layers"])


def test_errors_name_their_key():
    def broken(edit):
        raw = copy.deepcopy(TR.TINY_A)
        edit(raw)
        return raw
    cases = [(lambda r: r["layers"][0]["mixer"].pop("scale"), "scale"), (lambda r: r["layers"][0]["mixer"].update(heads=3), "kv_heads"),
             (lambda r: r["layers"][0]["mixer"]["mask"].update(size=0), "size"), (lambda r: r["layers"][0]["mixer"]["mask"].update(keep_first=-1), "keep_first"),
             (lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(count=4), "groups"), (lambda r: r["layers"][0]["mlp"]["router"].update(top=5), "choices"),
             (lambda r: r["layers"][0]["mlp"].pop("expert"), "expert"), (lambda r: r["layers"][1]["mixer"].update(decay=[0.5]), "decay"),
             (lambda r: r["layers"][1]["mixer"].update(decay=[0.5, 0.5, 1.5]), "decay"), (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=18), "dims"),
             (lambda r: r["layers"][2]["mixer"]["rot"].update(dims=6), "rot_dim"), (lambda r: r["layers"][2]["mixer"].pop("q_rank"), "q_rank"),
             (lambda r: r.pop("logit_scale"), "logit_scale"), (lambda r: r.pop("embedding"), "embedding"), (lambda r: r.pop("layers"), "layers")]
    for edit, word in cases:
        with pytest.raises(ConfigError, match=word):
            RoseraxConfig.from_dict(broken(edit))
    with pytest.raises(UnsupportedModelError, match="layer type"):
        RoseraxConfig.from_dict(broken(lambda r: r["layers"][0].update(type="gla")))
    with pytest.raises(UnsupportedModelError, match="feed-forward kind"):
        RoseraxConfig.from_dict(broken(lambda r: r["layers"][1]["mlp"].update(kind="glu")))


def test_tensor_list():
    spec = build_model_spec(RoseraxConfig.from_dict(TR.TINY_C))
    shapes = {s.name: s.shape for s in spec.tensor_specs()}
    assert len(shapes) == len(spec.tensor_specs())
    assert shapes["embed"] == (257, 90) and shapes["final.norm"] == (90,) and "head" not in shapes
    assert shapes["l0.mix.q"] == (30, 90) and shapes["l0.mix.v"] == (21, 90) and shapes["l0.mix.g"] == (21, 90) and shapes["l0.mix.o"] == (90, 21)
    assert shapes["l1.mix.q.norm"] == (12,) and shapes["l1.mix.k.norm"] == (12,) and shapes["l1.mix.v"] == (30, 90) and shapes["l1.mix.o"] == (90, 60)
    assert shapes["l2.mix.dq"] == (11, 90) and shapes["l2.mix.uq"] == (48, 11) and shapes["l2.mix.dkv"] == (36, 90) and shapes["l2.mix.g"] == (42, 90)
    assert shapes["l1.mlp.up"] == (52, 90) and shapes["l3.mlp.router"] == (7, 90) and shapes["l3.mlp.e6.gate"] == (36, 90)
    assert shapes["l1.norm1b"] == (90,) and shapes["l1.norm2b"] == (90,)
    assert "l0.norm2" not in shapes and "l0.norm2b" not in shapes and "l1.mlp.gate" not in shapes and "l1.mix.sink" not in shapes
    assert "l1.mix.g" not in shapes


def test_cache_plan_has_a_group_per_window_and_kept_tokens():
    plan = plan_cache(build_model_spec(RoseraxConfig.from_dict(TR.TINY_A)))
    assert [(g.window, g.keep_first) for g in plan.groups] == [(None, 0), (21, 5), (40, 19)]
    assert [g.owners for g in plan.groups] == [((2, 0),), ((0, 0),), ((3, 0),)]
    assert [(k, s.shape) for k, s in plan.states] == [((1, 0), (3 * 16 * 24,)), ((4, 0), (2 * 8 * 16,))]
    twice = copy.deepcopy(TR.TINY_A)
    twice["layers"][3]["mixer"]["mask"] = {"size": 21, "keep_first": 6}           # the same window, other kept tokens
    assert [(g.window, g.keep_first) for g in plan_cache(build_model_spec(RoseraxConfig.from_dict(twice))).groups] == [(None, 0), (21, 5), (21, 6)]
    assert not plan_cache(build_model_spec(RoseraxConfig.from_dict(TR.TINY_E))).groups


@pytest.mark.parametrize("W,keep,page", [(6, 3, 4), (6, 4, 4), (9, 5, 4), (1, 1, 4), (5, 30, 4), (3, 0, 2)])
def test_pages_of_kept_tokens_stay_and_pages_between_go(W, keep, page):
    m = CacheManager([None, W], page, [40, 40], 2, 128, keep_first=[0, keep])
    s, length = m.admit("a"), 0
    for n in [2, 1, 3, 1, 7, 1, 1, 19, 1, 2, 9, 1, 1, 30, 1]:
        m.reserve("a", n)
        row = m.table_rows(1, [s])[0]
        for pos in range(length, length + n):           # every key a query of this step may read is there
            assert all(row[key // page] >= 0 for key in range(pos + 1) if pos - key < W or key < keep)
        m.commit("a", n)
        length += n
        row, blocks = m.table_rows(1, [s])[0], -(-length // page)
        needed = [b < -(-keep // page) or b >= max(0, length - W + 1) // page for b in range(blocks)]
        assert [row[b] >= 0 for b in range(blocks)] == needed and (row[blocks:] == -1).all()
        assert 40 - m.free_pages(1) == sum(needed)
        m.check_invariants()
    m.release("a")
    assert m.free_pages(0) == 40 and m.free_pages(1) == 40
    s2 = m.admit("b")
    m.reserve("b", 3)
    assert m.table_rows(1, [s2])[0][0] >= 0
    m.check_invariants()


def test_work_lists_count_the_kept_rounds():
    """A late portion's tile walks its window's rounds of 128 keys and the rounds of the kept keys in front of them."""
    from photon_infer_amd.errors import CacheError
    near = AttentionPlanner(tile_rows=16, window=100, num_kv_heads=2, singles_apart=True, units=256)
    kept = AttentionPlanner(tile_rows=16, window=100, num_kv_heads=2, singles_apart=True, units=256, keep=130)
    assert near != kept and hash(near) != hash(kept)
    for planner in (near, kept):
        arrays, _ = planner.plan([16, 40], [5000, 40])
        assert arrays["req"].tolist() == [0, 1, 1, 1] and sorted(t for t in arrays["order"].tolist() if t >= 0) == [0, 1, 2, 3]
    assert kept.plan([16], [5000])[0]["order"].tolist()[0] == 0
    with pytest.raises(CacheError, match="kept first tokens"):
        CacheManager([None, 8], 4, 8, 2, 64, keep_first=[0])


def test_folder_with_random_weights(tmp_path):
    d = TR.make_model_dir(tmp_path, "A", seed=3)
    cfg = load_config(d)
    raw, W = P.read_model_folder(d)
    assert set(W) == {s.name for s in build_model_spec(cfg).tensor_specs()}
    logits = P.forward(raw, W, [5, 6, 7, 8])
    assert logits.shape == (4, 300) and bool(torch.isfinite(logits).all())


# ----------------------------------------------------------------------------- the plain implementation's own closed forms
def test_mask_holds_the_window_and_the_first_tokens():
    seen = P.kept_window_mask(12, 3, 2)
    for i in range(12):
        assert set(torch.nonzero(seen[i]).view(-1).tolist()) == {j for j in range(i + 1) if j > i - 3 or j < 2}
    assert torch.equal(P.kept_window_mask(5, 1, 0), torch.eye(5, dtype=torch.bool))
    assert int(P.causal_mask(6).sum()) == 21


def test_one_in_the_denominator():
    s = torch.tensor([[0.3, -0.2], [-800.0, -900.0], [700.0, 1.0]], dtype=F64)
    seen = torch.tensor([[True, True], [True, True], [True, False]])
    p = P.softmax_over(s, seen, one=True)
    assert torch.allclose(p[0], torch.exp(s[0]) / (1.0 + torch.exp(s[0]).sum()))
    assert float(p[1].sum()) < 1e-300 and torch.allclose(p[2], torch.tensor([1.0, 0.0], dtype=F64))
    assert math.isclose(float(P.softmax_over(s[:1], seen[:1], one=False).sum()), 1.0)


def test_rotation_of_paired_halves():
    x = torch.randn(3, 2, 10, dtype=F64)
    pos = torch.tensor([0, 7, 100])
    y = P.rotate_halves(x, pos, 6, 30.0)
    assert torch.equal(y[..., 6:], x[..., 6:]) and torch.equal(y[0], x[0]) and torch.allclose((y * y).sum(-1), (x * x).sum(-1))
    a = 7 * 30.0 ** (-2.0 / 6)
    assert torch.allclose(y[1, :, 1], x[1, :, 1] * math.cos(a) - x[1, :, 4] * math.sin(a))
    assert torch.allclose(y[1, :, 4], x[1, :, 4] * math.cos(a) + x[1, :, 1] * math.sin(a))


def test_retention_is_a_decayed_sum():
    T, H, d, dv = 9, 2, 3, 4
    q, k, v = (torch.randn(T, H, n, dtype=F64) for n in (d, d, dv))
    decay = [0.5, 1.0]
    o, S = P.retention_heads(q, k, v, decay)
    for h in range(H):
        for t in range(T):
            want = sum(decay[h] ** (t - j) * float(q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert torch.allclose(o[t, h], want)
    o1, S1 = P.retention_heads(q[:4], k[:4], v[:4], decay)
    o2, S2 = P.retention_heads(q[4:], k[4:], v[4:], decay, S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)


def test_groups_bound_the_choice():
    s = torch.tensor([0.30, 0.01, 0.20, 0.19, 0.02, 0.28], dtype=F64)
    assert P.choose_experts(s, 2, 1, 1) == [0, 5]
    assert P.choose_experts(s, 2, 3, 1) == [0, 1]                 # the group of the best one, even of a poor second
    assert P.choose_experts(s, 2, 3, 2) == [0, 5] and P.choose_experts(s, 3, 3, 2) == [0, 5, 4]
    assert math.isclose(P.choice_margin(s, 2, 3, 1), math.log(0.30 / 0.28))
    assert math.isclose(P.choice_margin(s, 3, 3, 2), min(math.log(0.28 / 0.20), math.log(0.02 / 0.01)))


def test_weights_are_the_scores_themselves():
    D, F, E = 4, 3, 4
    W = {"router": torch.zeros(E, D, dtype=F64)}
    for e in range(E):
        W[f"e{e}.gate"], W[f"e{e}.up"], W[f"e{e}.down"] = (torch.randn(*s, dtype=F64) for s in ((F, D), (F, D), (D, F)))
    h = torch.randn(2, D, dtype=F64)
    got = P.routed_ff(h, {"router": {"experts": E, "top": 1}}, W)
    assert torch.allclose(got, 0.25 * (P.silu(h @ W["e0.gate"].T) * (h @ W["e0.up"].T)) @ W["e0.down"].T)
