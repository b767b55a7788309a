"""Telapel on the CPU: limiting cases of the plain implementation's mechanisms (each checked against a form that is
obviously right), config.json in and out, what the architecture and its parts refuse, the cache layout (a state and the
convolution's last inputs for a recurrence, padded latent rows, a window's pages; layers that use another's tensors keep a
cache of their own), the packed order of the gates' matrices, and the loader's tensor names."""

import copy
import json
import math

import numpy as np
import pytest
import torch

import plain_telapel as P
import telapel_cases as cases
from mini_gpt_inference_amd.config.model_config import ConfigError, read_config_json
from mini_gpt_inference_amd.config.registry import architecture_of
from mini_gpt_inference_amd.models import telapel
from mini_gpt_inference_amd.ops import kernels
from mini_gpt_inference_amd.parts.base import StateNeed
from mini_gpt_inference_amd.parts.feedforward import GatedMLP, RoutedExperts
from mini_gpt_inference_amd.parts.mixers import GatedAttention, GatedDiagonalState, LatentAttention, geometric_slopes
from mini_gpt_inference_amd.parts.model import DecoderModel
from mini_gpt_inference_amd.parts.positions import RotaryHalf, RotaryInterleaved


def _rnd(g, *shape):
    return torch.randn(*shape, generator=g, dtype=P.DTYPE)


# ---------------------------------------------------------------- the plain mechanisms
def test_short_convolution_with_a_bias():
    g = torch.Generator().manual_seed(0)
    T, C, J = 7, 3, 4
    u, w, b = _rnd(g, T, C), _rnd(g, C, J), _rnd(g, C)
    got = P.short_conv(u, w, b)
    for t in range(T):
        for c in range(C):
            want = float(b[c]) + sum(float(w[c, j]) * float(u[t - J + 1 + j, c]) for j in range(J) if t - J + 1 + j >= 0)
            assert math.isclose(float(got[t, c]), want, abs_tol=1e-12)
    assert torch.allclose(P.short_conv(u, w[:, -1:]), u * w[:, -1])


def test_recurrence_is_a_weighted_sum_of_the_inputs():
    """S_t = sum_s (a_(s+1) .. a_t) sqrt(1 - a_s^2) i_s u_s, also for the first token; with r = 0 nothing decays and
    nothing enters; with a large decay only the token's own input is left."""
    g = torch.Generator().manual_seed(1)
    T, C = 8, 3
    u, r, i = _rnd(g, T, C), torch.rand(T, C, generator=g, dtype=P.DTYPE), torch.rand(T, C, generator=g, dtype=P.DTYPE)
    lam = _rnd(g, C) - 2.0
    got = P.gated_recurrence(u, r, i, lam)
    a = torch.exp(-8.0 * r * torch.log(1.0 + torch.exp(lam)))
    for t in range(T):
        want = torch.zeros(C, dtype=P.DTYPE)
        for s in range(t + 1):
            want = want + a[s + 1:t + 1].prod(dim=0) * torch.sqrt(1.0 - a[s] ** 2) * i[s] * u[s]
        assert torch.allclose(got[t], want, atol=1e-12)
    assert torch.allclose(got[0], torch.sqrt(1.0 - a[0] ** 2) * i[0] * u[0])
    assert float(P.gated_recurrence(u, 0 * r, i, lam).abs().max()) == 0.0
    assert torch.allclose(P.gated_recurrence(u, 0 * r + 1, i, lam + 50.0), i * u, atol=1e-12)


def test_block_product_is_a_block_diagonal_matrix():
    g = torch.Generator().manual_seed(2)
    u, w, b = _rnd(g, 5, 12), _rnd(g, 3, 4, 4), _rnd(g, 3, 4)
    assert torch.allclose(P.block_product(u, w, b), u @ torch.block_diag(*w).T + b.reshape(-1), atol=1e-12)


def test_interleaved_rotation_turns_neighbours_and_keeps_distances():
    g = torch.Generator().manual_seed(3)
    x = _rnd(g, 1, 6).expand(9, 6)
    y = P.rotate_pairs(x, 100.0)
    assert torch.allclose(y[0], x[0])
    z = torch.view_as_complex(x[0].view(3, 2).contiguous())
    f = torch.tensor([1.0, 100.0 ** (-2 / 6), 100.0 ** (-4 / 6)], dtype=P.DTYPE)
    want = torch.view_as_real(z * torch.exp(1j * 5 * f)).reshape(6)
    assert torch.allclose(y[5], want, atol=1e-12)
    k = P.rotate_pairs(_rnd(g, 1, 6).expand(9, 6), 100.0)
    assert math.isclose(float(y[7] @ k[4]), float(y[3] @ k[0]), abs_tol=1e-12)
    half, inter = RotaryHalf(6, 100.0), RotaryInterleaved(6, 100.0)
    assert inter.interleaved and not half.interleaved and torch.allclose(torch.tensor(inter.frequency_values(), dtype=P.DTYPE), f)


def test_latent_attention_as_explicit_sums():
    g = torch.Generator().manual_seed(4)
    T, W, H, D, R2, E, Q, R, eps = 6, 10, 2, 4, 4, 3, 7, 5, 1e-5
    m = {"heads": H, "dim": D, "rot_dim": R2, "vdim": E, "q_rank": Q, "kv_rank": R, "scale": 0.4, "rot": {"base": 30.0, "dims": R2}}
    w = {"dq": _rnd(g, Q, W), "dq.norm": _rnd(g, Q), "uq": _rnd(g, H * (D + R2), Q), "dkv": _rnd(g, R + R2, W), "dkv.norm": _rnd(g, R),
         "uk": _rnd(g, H * D, R), "uv": _rnd(g, H * E, R), "o": _rnd(g, W, H * E)}
    h = _rnd(g, T, W)
    got = P.latent_mixer(h, w, "", m, eps)
    norm = lambda v, gain: v / math.sqrt(float((v * v).mean()) + eps) * gain
    turned = lambda v, p: P.rotate_pairs(v.expand(p + 1, R2), 30.0)[p]
    for i in range(T):
        heads = []
        q = (w["uq"] @ norm(w["dq"] @ h[i], w["dq.norm"])).view(H, D + R2)
        for a in range(H):
            s, v = [], []
            for j in range(i + 1):
                row = w["dkv"] @ h[j]
                c = norm(row[:R], w["dkv.norm"])
                s.append(0.4 * float(q[a, :D] @ (w["uk"][a * D:(a + 1) * D] @ c) + turned(q[a, D:], i) @ turned(row[R:], j)))
                v.append(w["uv"][a * E:(a + 1) * E] @ c)
            den = sum(math.exp(x) for x in s)
            heads.append(sum(math.exp(x) / den * y for x, y in zip(s, v)))
        assert torch.allclose(got[i], w["o"] @ torch.cat(heads), atol=1e-10)


def test_window_cap_slope_and_sink():
    g = torch.Generator().manual_seed(5)
    T, H, G, D, E, N = 11, 4, 2, 4, 3, 4
    q, k, v = _rnd(g, T, H, D), _rnd(g, T, G, D), _rnd(g, T, G, E)
    slope = P.slopes(H)
    assert slope.tolist() == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8] == geometric_slopes(H)
    got = P.window_attention(q, k, v, 0.7, 1.5, slope, N)
    for i in range(T):
        for a in range(H):
            keys = [j for j in range(T) if 0 <= i - j < N]
            s = [1.5 * math.tanh(0.7 * float(q[i, a] @ k[j, a // 2]) / 1.5) - float(slope[a]) * (i - j) for j in keys]
            den = 1.0 + sum(math.exp(x) for x in s)
            want = sum(math.exp(x) / den * v[j, a // 2] for x, j in zip(s, keys))
            assert torch.allclose(got[i, a], want, atol=1e-12)
    assert torch.allclose(P.window_attention(q, k, v, 0.7, 1.5, slope, 0), P.window_attention(q, k, v, 0.7, 1.5, slope, 50))
    assert torch.allclose(P.window_attention(q, k, v, 0.7, 0.0, slope, N), P.window_attention(q, k, v, 0.7, 1e6, slope, N), atol=1e-9)
    # without the sink the slope may be counted from the key's end as well; with it that is another result
    shifted = lambda sink: (P.window_attention(q, k, v, 0.7, 0.0, slope, 0, sink), slope)
    plain, _ = shifted(None)
    assert float((P.window_attention(q, k, v, 0.7, 0.0, slope, 0) - plain).abs().max()) > 1e-2


def test_query_temperature_steps():
    t = P.query_temperature(10, 0.5, 4)
    # floor((p + 1) / 4) is 0 for p = 0 .. 2, 1 for 3 .. 6, 2 from 7 on
    assert torch.allclose(t, torch.tensor([1.0] * 3 + [1 + 0.5 * math.log(2)] * 4 + [1 + 0.5 * math.log(3)] * 3, dtype=P.DTYPE))


def test_clamped_unit():
    z = torch.tensor([-9.0, -1.0, 0.5, 3.0], dtype=P.DTYPE)
    u = torch.tensor([-5.0, 0.25, 1.0, 7.0], dtype=P.DTYPE)
    got = P.clamped_swish_unit(z, u, 2.0)
    want = [g / (1 + math.exp(-1.702 * g)) * (h + 1) for g, h in ((-9.0, -2.0), (-1.0, 0.25), (0.5, 1.0), (2.0, 2.0))]
    assert torch.allclose(got, torch.tensor(want, dtype=P.DTYPE))      # the gate is held from above only


def test_grouped_choice_and_experts():
    scores = torch.softmax(torch.tensor([[3.0, 0.1, 2.0, 1.9, 2.5, 0.0]], dtype=P.DTYPE), dim=-1)
    assert sorted(P.grouped_choice(scores, 2, 1, 1)[0].tolist()) == [0, 4]
    # groups rank by their best: (3.0), (2.0), (2.5): the second group is out, whatever its second best
    assert sorted(P.grouped_choice(scores, 3, 3, 2)[0].tolist()) == [0, 1, 4]
    g = torch.Generator().manual_seed(6)
    W, F, S = 6, 5, 3
    h = _rnd(g, 7, W)
    tensors = {"m.router": _rnd(g, 6, W), "m.shared.gate": _rnd(g, S, W), "m.shared.up": _rnd(g, S, W), "m.shared.down": _rnd(g, W, S)}
    for e in range(6):
        tensors.update({f"m.e{e}.gate": _rnd(g, F, W), f"m.e{e}.up": _rnd(g, F, W), f"m.e{e}.down": _rnd(g, W, F)})
    mlp = {"router": {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 2}}, "expert": {"ff": F, "limit": 0.8},
           "shared": {"ff": S, "limit": 0.3}}
    got = P.routed_experts(h, tensors, "m.", mlp)

    def unit(name, x, limit):
        gate, up = torch.clamp(tensors[name + ".gate"] @ x, max=limit), torch.clamp(tensors[name + ".up"] @ x, -limit, limit)
        return tensors[name + ".down"] @ (gate * torch.sigmoid(1.702 * gate) * (up + 1))

    for t in range(7):
        s = torch.softmax(tensors["m.router"] @ h[t], dim=-1)
        groups = sorted(range(3), key=lambda i: -max(float(s[2 * i]), float(s[2 * i + 1])))[:2]
        chosen = sorted([e for i in groups for e in (2 * i, 2 * i + 1)], key=lambda e: -float(s[e]))[:2]
        total = sum(float(s[e]) for e in chosen)
        want = sum(float(s[e]) / total * unit(f"m.e{e}", h[t], 0.8) for e in chosen) + unit("m.shared", h[t], 0.3)
        assert torch.allclose(got[t], want, atol=1e-12)


def test_what_the_test_models_are_sensitive_to(tmp_path):
    """Changing any constant or small tensor moves the logits by far more than the tolerances."""
    folder = cases.write_model(str(tmp_path / "A"), "A")
    cfg, w = P.read_model_folder(folder)
    ids = list(np.random.default_rng(0).integers(0, cfg["vocab"], 40))
    base = P.forward(cfg, w, ids)

    def moved(cfg2=None, **w2):
        return float((P.forward(cfg2 or cfg, {**w, **w2}, ids) - base).abs().max())

    def with_layers(change, *which):
        layers = copy.deepcopy(cfg["layers"])
        for i in which:
            change(layers[i])
        return {**cfg, "layers": layers}

    assert moved(with_layers(lambda l: l["mixer"]["mask"].update(size=8), 1, 4)) > 0.02
    assert moved(with_layers(lambda l: l["mixer"].update(softcap=1.0), 1, 4)) > 0.02
    assert moved(with_layers(lambda l: l["mixer"]["q_temp"].update(every=4), 1, 4)) > 0.02
    assert moved(with_layers(lambda l: l["mixer"]["rot"].update(base=50.0), 2, 5)) > 0.02
    assert moved(with_layers(lambda l: l["mixer"].update(scale=0.5), 2, 5)) > 0.02
    assert moved(with_layers(lambda l: l["mlp"]["router"]["groups"].update(keep=1), 0, 3, 6)) > 0.02
    assert moved(with_layers(lambda l: l["mlp"]["expert"].update(limit=0.5), 0, 3, 6)) > 0.02
    assert moved(with_layers(lambda l: l["mlp"]["shared"].update(limit=1.0), 0, 3, 6)) > 0.02
    for name in ("l0.mix.conv", "l1.mix.q.conv", "l1.mix.k.conv"):
        assert moved(**{name: w[name].flip(1)}) > 0.02, name
    for name in ("l0.mix.conv.b", "l0.mix.x.b", "l0.mix.y.b", "l0.mix.ra.b", "l0.mix.ri.b", "l0.mix.lam", "l1.mix.q.b", "l1.mix.k.b",
                 "l1.mix.k.norm", "l1.mix.q.norm", "l2.mix.dq.norm", "l2.mix.dkv.norm", "l0.norm1", "l0.norm2", "final.norm"):
        assert moved(**{name: w[name] + torch.linspace(-1.0, 1.0, w[name].numel(), dtype=P.DTYPE).view_as(w[name])}) > 0.02, name
    for name in ("l0.mix.ra", "l0.mix.ri"):
        assert moved(**{name: w[name].transpose(1, 2)}) > 0.02, name
    # a layer that uses another's tensors uses them
    own = with_layers(lambda l: l.pop("weights_of"), 3)
    other = {n.replace("l0.", "l3."): t for n, t in w.items() if n.startswith("l0.")}
    assert moved(own, **other) < 1e-9
    other["l3.mix.lam"] = other["l3.mix.lam"] + 1.0
    assert moved(own, **other) > 0.01


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
    cfg = telapel.config_from_json(cases.RAW[name])
    assert telapel.config_from_json(telapel.config_to_json(cfg)) == cfg
    folder = cases.write_model(str(tmp_path / name), name)
    raw = read_config_json(folder)
    assert architecture_of(raw).name == "Telapel" and telapel.config_from_json(raw) == cfg


def test_random_configurations_are_accepted_and_round_trip():
    rng = np.random.default_rng(4)
    for _ in range(30):
        raw = cases.random_raw(rng)
        cfg = telapel.config_from_json(raw)
        assert telapel.config_from_json(telapel.config_to_json(cfg)) == cfg
        DecoderModel(telapel.model_spec(cfg))


@pytest.mark.parametrize("edit", [
    lambda r: r["layers"][0].update(type="gla"),
    lambda r: r["layers"][0]["mixer"].update(blocks=5),
    lambda r: r["layers"][0]["mixer"].update(conv=0),
    lambda r: r["layers"][0].pop("mixer"),
    lambda r: r["layers"][1]["mixer"].update(kv_heads=4),
    lambda r: r["layers"][1]["mixer"].update(vdim=16),
    lambda r: r["layers"][1]["mixer"]["mask"].update(size=-1),
    lambda r: r["layers"][1]["mixer"]["q_temp"].update(every=0),
    lambda r: r["layers"][1]["mixer"].update(softcap=-1.0),
    lambda r: r["layers"][2]["mixer"].update(q_rank=0),
    lambda r: r["layers"][2]["mixer"]["rot"].update(dims=6),
    lambda r: r["layers"][2]["mixer"].pop("rot"),
    lambda r: r["layers"][0]["mlp"].update(kind="dense"),
    lambda r: r["layers"][0]["mlp"]["router"].update(top=5),
    lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(count=4),
    lambda r: r["layers"][0]["mlp"]["expert"].update(limit=0.0),
    lambda r: r["layers"][0]["mlp"]["shared"].update(ff=-1),
    lambda r: r["layers"][3].update(weights_of=3),
    lambda r: r["layers"][3].update(weights_of=1),
    lambda r: r["layers"][3]["mixer"].update(conv=4),
    lambda r: r.update(layers=[]),
])
def test_refusals(edit):
    raw = json.loads(json.dumps(cases.RAW["A"]))      # (layers of the case share their entries)
    edit(raw)
    with pytest.raises(ConfigError):
        telapel.config_from_json(raw)


def test_parts_refuse_what_their_kernels_do_not_combine():
    for bad in (dict(slopes=[0.5]), dict(slopes=[0.5, 0.25], bias_max=20), dict(slopes=[0.5, 0.25], score_bias=True),
                dict(sink_score=0.0, sinks=True), dict(query_temperature=(0.5, 0)), dict(values_from_keys=True, value_mix="keep")):
        with pytest.raises(ValueError):
            GatedAttention(32, 2, 1, 16, 16, 0.25, **bad)
    with pytest.raises(ValueError):
        LatentAttention(32, 2, 16, 16, 24, 0.25, gate="row")
    with pytest.raises(ValueError):
        LatentAttention(32, 2, 16, 16, 24, 0.25, q_rank=16)
    with pytest.raises(ValueError):
        GatedDiagonalState(32, 30, 4, 2)
    with pytest.raises(ValueError):
        GatedDiagonalState(32, 32, 4, 10)
    with pytest.raises(ValueError):
        RoutedExperts(32, 16, 6, 2, activation="clamped_swish")
    with pytest.raises(ValueError):
        RoutedExperts(32, 16, 6, 2, groups=(3, 2), group_best=3)
    with pytest.raises(ValueError):
        GatedMLP(32, 16, activation="clamped_swish", limit=0.0)


# ---------------------------------------------------------------- model as data
def test_cache_layout_and_tensor_names():
    cfg = cases.config("A")
    model = DecoderModel(telapel.model_spec(cfg))
    layout = model.cache_layout
    assert [b.kind for run in layout.run_bindings for b in run.values()] == ["state", "kv", "kv", "state", "kv", "kv", "state"]
    # attention: pages of 24 rounded up to 32 channels a head behind a window of 7; latents: rows of 24 + 8 values, joint.
    # Each layer that uses another's tensors has a pool, or a state, of its own
    assert [(g.n_kv_head, g.head_dim, g.n_pools, g.window, g.joint) for g in layout.groups] == [(2, 32, 2, 7, False), (1, 32, 2, 0, True)]
    recurrence, attention = 48 + 2 * 48, 1 * (6 + 2) * 32
    assert layout.state_numels == [recurrence, attention, recurrence, attention, recurrence]
    assert len(model.layers) == 3 and [run.layer for run in model.spec.order] == [0, 1, 2, 0, 1, 2, 0]
    wanted = model.weight_requests()
    plan_names = {name: tuple(shape) for name, shape, _, _ in telapel.init_plan(cfg)}
    assert set(wanted) == set(plan_names)
    for name, req in wanted.items():
        assert req.fits(plan_names[name]), name
    assert "l3.norm1" not in wanted and "l1.mix.v" not in wanted and "l1.mix.k.conv" in wanted and "head" not in wanted
    assert "l2.mlp.e3.down" in wanted and "l2.mlp.e4.down" not in wanted and "l2.mlp.shared.up" not in wanted
    assert "l1.norm1" in wanted and "l1.norm2" not in wanted
    assert model.graph_safe and model.plan_safe and model.spec.max_positions is None
    other = DecoderModel(telapel.model_spec(cases.config("B"))).weight_requests()
    assert "l2.norm1" in other and "l2.norm2" not in other


def test_one_tap_keeps_no_inputs():
    layout = DecoderModel(telapel.model_spec(cases.config("C"))).cache_layout
    # (the first attention layer's and the recurrence's convolution have one tap; the last layer's has six)
    assert layout.state_numels == [36, 5 * (4 + 4) * 32]


def test_cached_latent_rows_take_the_next_size_of_the_kernels():
    row = lambda rank, rot: LatentAttention(32, 2, 8, 8, rank, 0.3, rot_dim=rot, rotary={"kind": "rotary_interleaved", "dims": rot, "base": 10.0},
                                            gate=None, sinks=False, q_rank=16).row
    assert [row(16, 8), row(24, 8), row(40, 8), row(56, 8), row(58, 8), row(120, 8), row(122, 8), row(512, 64)] == \
        [32, 32, 64, 64, 128, 128, 136, 576]


def test_a_model_of_recurrences_only_still_has_a_group_of_pages():
    model = DecoderModel(telapel.model_spec(cases.config("E")))
    assert [(g.n_pools, g.window) for g in model.cache_layout.groups] == [(0, 0)]
    assert model.cache_layout.state_numels == [80 * 4, 32 * 2, 32 * 2]
    assert [layer.mixer.cache_need() for layer in model.layers] == [StateNeed(80 * 4), StateNeed(32 * 2)]


@pytest.mark.parametrize("blocks,block", [(2, 16), (1, 48), (3, 64), (2, 144)])
def test_packed_gates_hold_every_matrix_element_once(blocks, block):
    g = torch.Generator().manual_seed(block)
    r, i = (torch.randn(blocks, block, block, generator=g).to(torch.bfloat16) for _ in range(2))
    packed = kernels.pack_diagonal_gates(r, i)
    assert tuple(packed.shape) == (blocks * block // 16, 2, -(-block // 32), 64, 8)
    for tile in range(blocks * block // 16):
        b, c0 = tile * 16 // block, tile * 16 % block
        for gate, w in enumerate((r, i)):
            for step in range(packed.shape[2]):
                for lane in (0, 5, 17, 40, 63):
                    k = step * 32 + lane // 16 * 8
                    want = w[b, c0 + lane % 16, k:k + 8] if k < block else torch.zeros(8, dtype=torch.bfloat16)
                    assert torch.equal(packed[tile, gate, step, lane], want)
    assert kernels.pack_diagonal_gates(r.float(), i.float()) is None
    assert kernels.pack_diagonal_gates(r[:, :12, :12].contiguous(), i[:, :12, :12].contiguous()) is None


def test_costs_count_a_layers_second_run():
    once = DecoderModel(telapel.model_spec(cases.config("D")))
    tensors = {n: torch.zeros(r.shape, dtype=torch.bfloat16 if r.role != "vector" else torch.float32)
               for n, r in once.weight_requests().items()}
    once.bind(tensors)
    cost = once.cost()
    assert [(k.n_head, k.n_kv_head, k.head_dim, k.window, k.tensors) for k in cost.kv_runs] == [(2, 1, 32, 0, 1), (2, 1, 32, 33, 2)]
    assert cost.state_floats == 16 * 4 + 3 * (2 + 1) * 32
