"""Gekopel on the CPU: limiting cases of the plain implementation's mechanisms (each checked against
a form that is obviously right), the product's distance buckets, config.json in and out, what the
architecture refuses, the cache layout (chunks of pages for the attention layers, a state and the
convolutions' last inputs for the others), the release of a passed chunk's pages, and the loader's
tensor names."""

import copy
import math

import numpy as np
import pytest
import torch

import gekopel_cases as cases
import plain_gekopel as P
from mini_gpt_inference_amd.cache.manager import CacheManager, GroupGeometry
from mini_gpt_inference_amd.config.model_config import ConfigError, read_config_json
from mini_gpt_inference_amd.config.registry import architecture_of
from mini_gpt_inference_amd.models import gekopel
from mini_gpt_inference_amd.parts.base import KVNeed, PartSpec, StateNeed
from mini_gpt_inference_amd.parts.mixers import GatedAttention, distance_buckets
from mini_gpt_inference_amd.parts.feedforward import RoutedExperts
from mini_gpt_inference_amd.parts.model import DecoderModel, KVRun, LayerRun, LayerSpec, ModelSpec


def _rnd(g, *shape):
    return torch.randn(*shape, generator=g, dtype=P.DTYPE)


# ---------------------------------------------------------------- the plain mechanisms
def test_short_convolution_is_a_sum_over_the_last_taps_with_zeros_before_the_start():
    g = torch.Generator().manual_seed(0)
    T, C, J = 7, 3, 4
    u, w = _rnd(g, T, C), _rnd(g, C, J)
    got = P.short_conv(u, w)
    for t in range(T):
        for c in range(C):
            want = sum(float(w[c, j]) * float(u[t - J + 1 + j, c]) for j in range(J) if t - J + 1 + j >= 0)
            assert math.isclose(float(got[t, c]), want, abs_tol=1e-12)
    assert torch.allclose(P.short_conv(u, w[:, -1:]), u * w[:, -1])


def test_delta_rule_against_its_product_form():
    """S_t = g_t (I - beta_t k_t k_t^T) S_(t-1) + beta_t k_t v_t^T, and the read-out sees the token's own write."""
    g = torch.Generator().manual_seed(1)
    T, H, G, D, E = 9, 4, 2, 5, 3
    q, k = P.unit_length(_rnd(g, T, G, D)), P.unit_length(_rnd(g, T, G, D))
    v, beta = _rnd(g, T, H, E), torch.rand(T, H, generator=g, dtype=P.DTYPE)
    decay = torch.rand(T, H, generator=g, dtype=P.DTYPE)
    got = P.delta_recurrence(q, k, v, beta, decay)
    for a in range(H):
        S = torch.zeros(D, E, dtype=P.DTYPE)
        for t in range(T):
            kt = k[t, a // 2]
            S = decay[t, a] * (S - beta[t, a] * torch.outer(kt, kt @ S)) + beta[t, a] * torch.outer(kt, v[t, a])
            assert torch.allclose(got[t, a], q[t, a // 2] @ S, atol=1e-12)


def test_delta_rule_limits():
    """beta 1 and no decay: a key read right after its write gives its value back, whatever was there before;
    beta 0: nothing is ever written; a decay of 0: only the token's own write is left."""
    g = torch.Generator().manual_seed(2)
    T, D, E = 6, 8, 4
    k = P.unit_length(_rnd(g, T, 1, D)) * math.sqrt(1.0 + 1e-6)
    k = k / k.norm(dim=-1, keepdim=True)
    v, one = _rnd(g, T, 1, E), torch.ones(T, 1, dtype=P.DTYPE)
    assert torch.allclose(P.delta_recurrence(k, k, v, one, one), v, atol=1e-12)
    assert float(P.delta_recurrence(k, k, v, 0 * one, one).abs().max()) == 0.0
    q = P.unit_length(_rnd(g, T, 1, D))
    got = P.delta_recurrence(q, k, v, 0.3 * one, 0 * one)
    assert torch.allclose(got, 0.3 * (q * k).sum(-1, keepdim=True) * v, atol=1e-12)


def test_chunks_bias_and_sink():
    g = torch.Generator().manual_seed(3)
    T, H, G, D, E, C = 11, 2, 1, 4, 3, 4
    q, k, v = _rnd(g, T, H, D), _rnd(g, T, G, D), _rnd(g, T, G, E)
    rel, sink = _rnd(g, 6, H), _rnd(g, H)
    bias = P.distance_bias(rel, 9, T)
    got = P.chunk_attention(q, k, v, 0.7, bias, sink, C)
    for i in range(T):
        for a in range(H):
            keys = [j for j in range(i + 1) if j // C == i // C]
            s = [0.7 * float(q[i, a] @ k[j, 0]) + float(rel[P.distance_bucket(i - j, 6, 9), a]) for j in keys]
            den = sum(math.exp(x) for x in s) + math.exp(float(sink[a]))
            want = sum(math.exp(x) / den * v[j, 0] for x, j in zip(s, keys))
            assert torch.allclose(got[i, a], want, atol=1e-12)
    # the first token of a chunk sees itself only; chunk 0: every earlier key
    assert torch.allclose(got[8], torch.stack([v[8, 0] * float(torch.sigmoid(0.7 * (q[8, a] @ k[8, 0]) + rel[0, a] - sink[a]))
                                               for a in range(H)]), atol=1e-12)
    assert torch.allclose(P.chunk_attention(q, k, v, 0.7, bias, sink, 0), P.chunk_attention(q, k, v, 0.7, bias, sink, 50))
    # a sink far below the scores does nothing
    far = P.chunk_attention(q, k, v, 0.7, bias, sink - 1000.0, C)
    assert torch.allclose(far[0], v[0].expand(H, E))


def test_distance_buckets():
    """One distance a bucket below half of them, never falling, the last one from bias_max on at the latest; the
    product's list ends with the first distance of the last bucket."""
    for buckets, bias_max in ((32, 90), (16, 24), (4, 9), (2, 2), (40, 500), (6, 4)):
        rows = [P.distance_bucket(n, buckets, bias_max) for n in range(bias_max + 40)]
        assert rows[:buckets // 2] == list(range(buckets // 2))
        assert all(b >= a for a, b in zip(rows, rows[1:])) and rows[bias_max] == buckets - 1
        mine = distance_buckets(buckets, bias_max)
        assert mine == rows[:len(mine)] and mine[-1] == buckets - 1 and set(rows[len(mine) - 1:]) == {buckets - 1}
        if len(mine) > 1:
            assert mine[-2] < buckets - 1
    # ln(24 / 8) / ln(72 / 8) is one half exactly: on a bucket's edge
    assert distance_buckets(16, 72)[24] == 12 and distance_buckets(16, 72)[23] == 11
    for bad in ((5, 20), (8, 4), (0, 10)):
        with pytest.raises(ValueError):
            distance_buckets(*bad)


def test_grouped_choice():
    """The correction counts for the choice and not for the weight; only the best groups' experts can be chosen,
    also where all their choice scores are negative (what is left out counts as minus infinity)."""
    scores = torch.tensor([[0.9, 0.1, 0.5, 0.45, 0.6, 0.05]], dtype=P.DTYPE)
    zero = torch.zeros(6, dtype=P.DTYPE)
    assert sorted(P.grouped_choice(scores, zero, 2, 1, 1)[0].tolist()) == [0, 4]
    # groups (0.9 + 0.1), (0.5 + 0.45), (0.6 + 0.05): the second beats the third though 4 is the second best expert
    assert sorted(P.grouped_choice(scores, zero, 2, 3, 2)[0].tolist()) == [0, 2]
    assert sorted(P.grouped_choice(scores, zero, 3, 3, 1)[0].tolist()[:2]) == [0, 1]
    down = zero - 2.0
    down[2:4] += 0.5
    assert sorted(P.grouped_choice(scores, down, 2, 3, 1)[0].tolist()) == [2, 3]
    g = torch.Generator().manual_seed(4)
    W, F = 6, 5
    h = _rnd(g, 7, W)
    tensors = {"m.router": _rnd(g, 6, W), "m.correction": _rnd(g, 6) * 0.2, "m.shared.up": _rnd(g, 3, W),
               "m.shared.down": _rnd(g, W, 3), "m.shared.sg": _rnd(g, 1, W)}
    for e in range(6):
        tensors.update({f"m.e{e}.up": _rnd(g, F, W), f"m.e{e}.down": _rnd(g, W, F)})
    mlp = {"router": {"experts": 6, "top": 2, "scale": 1.7, "groups": {"count": 3, "keep": 2}}, "shared": {"ff": 3}}
    got = P.routed_experts(h, tensors, "m.", mlp)
    s = P.sigmoid(h @ tensors["m.router"].T)
    for t in range(7):
        c = s[t] + tensors["m.correction"]
        groups = sorted(range(3), key=lambda i: -float(c[2 * i] + c[2 * i + 1]))[:2]
        chosen = sorted([e for i in groups for e in (2 * i, 2 * i + 1)], key=lambda e: -float(c[e]))[:2]
        total = sum(float(s[t, e]) for e in chosen)
        want = sum(1.7 * float(s[t, e]) / total * (tensors[f"m.e{e}.down"] @ P.relu_squared(tensors[f"m.e{e}.up"] @ h[t]))
                   for e in chosen)
        want = want + P.sigmoid(tensors["m.shared.sg"] @ h[t]) * (tensors["m.shared.down"] @ P.relu_squared(tensors["m.shared.up"] @ h[t]))
        assert torch.allclose(got[t], want, atol=1e-12)


def test_what_the_test_models_are_sensitive_to(tmp_path):
    """Changing a chunk by one, a bias row, a sink, a tap, a decay constant, the step sizes' projection, the head
    norm, the correction, the groups, the router's scale, the shared expert's gate, a norm behind a sublayer, the
    embedding's scale or the positions moves the logits by far more than the tolerances."""
    folder = cases.write_model(str(tmp_path / "A"), "A")
    cfg, w = P.read_model_folder(folder)
    ids = list(np.random.default_rng(0).integers(0, cfg["vocab"], 60))
    base = P.forward(cfg, w, ids)

    def moved(cfg2=None, w2=None):
        return float((P.forward(cfg2 or cfg, w2 or w, ids) - base).abs().max())

    def with_layer(i, change):
        layers = copy.deepcopy(cfg["layers"])
        change(layers[i])
        return {**cfg, "layers": layers}

    assert moved(with_layer(0, lambda l: l["mixer"]["mask"].update(size=8))) > 0.05
    assert moved(with_layer(2, lambda l: l["mixer"]["mask"].update(size=38))) > 0.05
    assert moved(with_layer(2, lambda l: l["mixer"].update(bias_max=20))) > 0.005
    assert moved(w2={**w, "l2.mix.rel": w["l2.mix.rel"].flip(0)}) > 0.05
    assert moved(w2={**w, "l0.mix.sink": w["l0.mix.sink"] - 50.0}) > 0.05
    assert moved(w2={**w, "l1.mix.k.conv": w["l1.mix.k.conv"].flip(1)}) > 0.05
    assert moved(w2={**w, "l1.mix.A_log": w["l1.mix.A_log"] + 1.0}) > 0.005
    assert moved(w2={**w, "l1.mix.dt_bias": w["l1.mix.dt_bias"] + 1.0}) > 0.005
    assert moved(w2={**w, "l1.mix.b": -w["l1.mix.b"]}) > 0.05
    assert moved(w2={**w, "l1.mix.norm": w["l1.mix.norm"] + torch.linspace(0.0, 2.0, 24, dtype=P.DTYPE)}) > 0.05
    assert moved(w2={**w, "l1.mlp.correction": w["l1.mlp.correction"].flip(0)}) > 0.05
    assert moved(with_layer(1, lambda l: l["mlp"]["router"]["groups"].update(keep=1))) > 0.05
    assert moved(with_layer(1, lambda l: l["mlp"]["router"].update(scale=1.0))) > 0.05
    assert moved(w2={**w, "l1.mlp.shared.sg": -w["l1.mlp.shared.sg"]}) > 0.05
    assert moved(w2={**w, "l1.norm2b": w["l1.norm2b"] + 0.5}) > 0.05
    assert moved({**cfg, "embedding": {"scale": 4.0}}) > 0.05
    assert moved(w2={**w, "pos": w["pos"].flip(0)}) > 0.05


def test_residuals_are_reported_layer_by_layer(tmp_path):
    folder = cases.write_model(str(tmp_path / "D"), "D")
    cfg, w = P.read_model_folder(folder)
    res = []
    logits = P.forward(cfg, w, [1, 2, 3, 4, 5], residuals=res)
    assert len(res) == len(cfg["layers"]) and res[0].shape == (5, cfg["width"]) and logits.shape == (5, cfg["vocab"])
    # causal: a later token does not change an earlier position
    assert torch.allclose(P.forward(cfg, w, [1, 2, 3]), logits[:3], atol=1e-9)


# ---------------------------------------------------------------- configuration
@pytest.mark.parametrize("name", sorted(cases.RAW))
def test_config_round_trip(name, tmp_path):
    cfg = gekopel.config_from_json(cases.RAW[name])
    assert gekopel.config_from_json(gekopel.config_to_json(cfg)) == cfg
    folder = cases.write_model(str(tmp_path / name), name)
    raw = read_config_json(folder)
    assert architecture_of(raw).name == "Gekopel" and gekopel.config_from_json(raw) == cfg


def test_random_configurations_are_accepted_and_round_trip():
    rng = np.random.default_rng(4)
    for _ in range(30):
        raw, _ = cases.random_raw(rng)
        cfg = gekopel.config_from_json(raw)
        assert gekopel.config_from_json(gekopel.config_to_json(cfg)) == cfg
        DecoderModel(gekopel.model_spec(cfg))


@pytest.mark.parametrize("edit", [
    lambda r: r["layers"][0].update(type="gla"),
    lambda r: r["layers"][0]["mixer"].update(kv_heads=3),
    lambda r: r["layers"][0]["mixer"].update(bias_max=0),
    lambda r: r["layers"][0]["mixer"]["mask"].update(size=-1),
    lambda r: r["layers"][1]["mixer"].update(conv=0),
    lambda r: r["layers"][1]["mixer"].update(kv_heads=4),
    lambda r: r["layers"][1].pop("mixer"),
    lambda r: r["layers"][0]["mlp"].update(kind="gated"),
    lambda r: r["layers"][0]["mlp"].update(ff=0),
    lambda r: r["layers"][1]["mlp"]["router"].update(top=7),
    lambda r: r["layers"][1]["mlp"]["router"].update(top=5),
    lambda r: r["layers"][1]["mlp"]["router"]["groups"].update(count=4),
    lambda r: r["layers"][1]["mlp"]["router"]["groups"].update(keep=4),
    lambda r: r["layers"][1]["mlp"]["shared"].update(ff=-1),
    lambda r: r.update(layers=[]),
    lambda r: r.update(max_positions=0),
])
def test_refusals(edit):
    raw = copy.deepcopy(cases.RAW["A"])
    edit(raw)
    with pytest.raises(ConfigError):
        gekopel.config_from_json(raw)


def test_parts_refuse_what_their_kernels_do_not_combine():
    with pytest.raises(ValueError):
        GatedAttention(32, 2, 1, 16, 16, 0.25, sinks=True, score_bias=True)
    with pytest.raises(ValueError):
        GatedAttention(32, 2, 1, 16, 16, 0.25, bias_max=20, softcap=5.0)
    with pytest.raises(ValueError):
        RoutedExperts(32, 16, 6, 3, groups=(3, 1))
    with pytest.raises(ValueError):
        RoutedExperts(32, 16, 6, 2, activation="gelu")


# ---------------------------------------------------------------- model as data
def test_cache_layout_and_tensor_names():
    cfg = cases.config("A")
    model = DecoderModel(gekopel.model_spec(cfg))
    layout = model.cache_layout
    assert [b.kind for run in layout.run_bindings for b in run.values()] == ["kv", "state", "kv", "state"]
    # an attention layer keeps pages of max(dim, vdim) rounded up to 32 channels a head, a chunk of them
    assert [(g.n_kv_head, g.head_dim, g.n_pools, g.window, g.chunked) for g in layout.groups] == [(2, 32, 1, 7, True),
                                                                                                 (1, 32, 1, 37, True)]
    # delta: heads * dim * vdim, and the last taps - 1 rows of q, k and v
    assert layout.state_numels == [6 * 16 * 24 + 2 * (2 * 2 * 16 + 6 * 24), 3 * 8 * 40 + 1 * (2 * 3 * 8 + 3 * 40)]
    wanted = model.weight_requests()
    plan_names = {name: tuple(shape) for name, shape, _, _ in gekopel.init_plan(cfg)}
    assert set(wanted) == set(plan_names)
    for name, req in wanted.items():
        assert req.fits(plan_names[name]), name
    assert "l3.norm2" not in wanted and "l1.mix.v.conv" in wanted and "l0.mlp.up" in wanted
    assert "l1.mlp.e5.down" in wanted and "l1.mlp.e6.down" not in wanted and "l1.mlp.e0.gate" not in wanted
    assert "l1.mlp.shared.sg" in wanted and "l2.mlp.shared.sg" not in wanted and "l2.mlp.correction" in wanted
    # the number of distance buckets comes from the stored table
    assert wanted["l0.mix.rel"].shape == (-1, 4)
    assert model.graph_safe and model.plan_safe and model.spec.max_positions == 500


def test_a_chunk_as_large_as_another_layers_window_keeps_a_group_of_its_own():
    """Pages of a chunk go at once when the chunk is passed, those of a sliding window one by one: layers of both
    kinds do not share a page table.  A run that reads a chunked cache through a sliding window of the same size
    needs the window's pages."""
    w = 32

    def spec(chunked, window):
        names = {n: f"{chunked}.{n}" for n in ("q_weight", "k_weight", "v_weight", "out_weight")}
        mixer = PartSpec("gated_attention", {"width": w, "n_head": 2, "n_kv_head": 1, "head_dim": 16, "value_dim": 16, "scale": 0.25,
                                             "window": window, "chunked": chunked}, names)
        return LayerSpec(PartSpec("pre_norm_mixer", {"width": w}), norm1=PartSpec("rms_norm", {"width": w, "eps": 1e-5},
                                                                                 {"weight": "n"}), mixer=mixer)

    def layout(layers, order):
        return DecoderModel(ModelSpec(w, 9, PartSpec("token_embedding", {"vocab_size": 9, "width": w}, {"weight": "e"}),
                                      PartSpec("none"), tuple(layers), tuple(order),
                                      PartSpec("rms_norm", {"width": w, "eps": 1e-5}, {"weight": "f"}),
                                      PartSpec("linear_head", {"vocab_size": 9, "width": w, "tied": False}, {"weight": "h"}))).cache_layout

    got = layout([spec(True, 24), spec(False, 24)], [LayerRun(0), LayerRun(1), LayerRun(0)])
    assert [(g.window, g.chunked, g.n_pools) for g in got.groups] == [(24, True, 2), (24, False, 1)]
    got = layout([spec(True, 24), spec(False, 24)], [LayerRun(0), LayerRun(1, reads_cache_of=0)])
    assert [(g.window, g.chunked) for g in got.groups] == [(24, False)]
    got = layout([spec(True, 24), spec(True, 24)], [LayerRun(0), LayerRun(1, reads_cache_of=0)])
    assert [(g.window, g.chunked) for g in got.groups] == [(24, True)]
    # no chunk size: every earlier key is seen
    assert GatedAttention(w, 2, 1, 16, 16, 0.25, chunked=True).cache_need() == KVNeed(1, 32, 0)


def test_a_passed_chunks_pages_come_back_at_once():
    cm = CacheManager([GroupGeometry(4, 32, 10, 0, True), GroupGeometry(4, 32, 10, 0, False)], 2)
    slot = cm.acquire_slot()
    assert cm.reserve(slot, 40)
    for computed, chunk_pages, window_pages in ((3, 0, 0), (9, 0, 0), (10, 2, 0), (13, 2, 1), (19, 2, 2), (20, 5, 2), (29, 5, 5),
                                                (30, 7, 5)):
        cm.release_passed(slot, computed)
        # chunk: everything below floor(computed / 10) * 10 in whole pages; window: below computed - 9
        assert 10 - cm.held_pages(slot, 0) == chunk_pages, computed
        assert 10 - cm.held_pages(slot, 1) == window_pages, computed
        assert cm.check() == 0
    assert cm.free_slot(slot) and cm.num_free_pages(0) == 32


def test_keys_seen_by_distance_kinds():
    chunk, window, both = KVRun(1, 1, 8, 10, chunked=True), KVRun(1, 1, 8, 10), KVRun(1, 1, 8, 10, keep_first=3, chunked=True)
    assert [chunk.keys_seen(n) for n in (1, 10, 11, 25)] == [1, 10, 1, 5]
    assert [window.keys_seen(n) for n in (1, 10, 11, 25)] == [1, 10, 10, 10]
    assert [both.keys_seen(n) for n in (1, 10, 11, 25)] == [1, 10, 4, 8]
    assert KVRun(1, 1, 8, 0).keys_seen(25) == 25


def test_a_model_of_delta_layers_only_still_has_a_group_of_pages():
    layout = DecoderModel(gekopel.model_spec(cases.config("E"))).cache_layout
    assert [(g.n_pools, g.window) for g in layout.groups] == [(0, 0)]
    assert [b.kind for run in layout.run_bindings for b in run.values()] == ["state", "state"]
    needs = [p.cache_need() for layer in DecoderModel(gekopel.model_spec(cases.config("E"))).layers
             for r, p in layer.parts.items() if r == "mixer"]
    assert needs == [StateNeed(n) for n in layout.state_numels]
