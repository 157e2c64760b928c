"""Pozozen without a GPU: the configuration reader and its errors, the order of looped layers, the tensors it expects, the cache
units of side-by-side mixers and of every pass, the random-weights folder, and pins of the plain implementation (each mechanism
against a second, independent formulation)."""

from __future__ import annotations

import copy
import math

import pytest
import torch

from plain import pozozen_plain as plain
from pozozen_cases import CASES, SINGLE, make_tensors

F64 = torch.float64


# -- configuration and weights ---------------------------------------------------------

def test_config_is_found_by_its_architecture_key_and_states_the_layers_as_parts():
    from lockstep_amd.config import PozozenConfig, config_from_dict

    cfg = config_from_dict(CASES["A"]["raw"])
    assert isinstance(cfg, PozozenConfig) and cfg.order() == [0, 1, 2, 1, 2, 3]
    spec = cfg.model_spec()
    assert [layer.mixer.kind for layer in spec.layers] == ["matrix_memory", "side_by_side", "matrix_memory", "side_by_side"]
    assert all(layer.arrangement.kind == "hyper_connections" and layer.arrangement["copies"] == 3 and layer.arrangement["learned"]
               and layer.arrangement["residual_mult"] == 0.6 for layer in spec.layers)
    first, second = spec.layers[0].mixer, spec.layers[1].mixer
    assert (first["num_heads"], first["head_dim"], first["value_dim"], first["gate_cap"], first["eps"], first["denom_eps"]) == (
        3, 20, 24, 8.0, 1e-5, 1e-6)
    left, right = second["branches"]["left"], second["branches"]["right"]
    assert left.kind == "sink_attention" and right.kind == "state_space"
    assert (left["num_heads"], left["num_kv_heads"], left["window"], left["sink"], left["bias"], left["scale"], left["out_scale"]) == (
        4, 2, 21, None, True, 0.5, 0.7)
    assert left["position"].kind == "no_position" and spec.layers[3].mixer["branches"]["left"]["window"] is None
    assert (right["num_heads"], right["value_dim"], right["state_size"], right["groups"], right["taps"], right["norm_parts"],
            right["out_scale"]) == (4, 16, 24, 2, 3, 2, 0.8)
    ff = spec.layers[0].feed_forward
    assert (ff["experts"], ff["identity"], ff["top"], ff["groups"], ff["score"], ff["shared"]["intermediate_size"]) == (
        6, 2, 2, {"count": 4, "keep": 2}, "softmax_all", 40)
    assert spec.layers[2].feed_forward is None and spec.layers[1].feed_forward["shared"] is None
    assert spec.layers[3].feed_forward["groups"] is None and spec.layers[3].feed_forward["identity"] == 0
    assert [(e.layer, e.cache, e.further) for e in spec.schedule] == [
        (0, 0, ()), (1, 1, (2,)), (2, 3, ()), (1, 4, (5,)), (2, 6, ()), (3, 7, (8,))]
    assert spec.cache_units() == 9 and spec.residual_copies == 3 and spec.final_norm["copies"] == 3
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    plain_stream = config_from_dict(CASES["C"]["raw"])
    assert plain_stream.order() == [0, 1, 2] * 3
    assert not plain_stream.model_spec().layers[0].arrangement["learned"] and plain_stream.model_spec().residual_copies == 1


def test_the_expected_tensors():
    from lockstep_amd.config import config_from_dict
    from lockstep_amd.engine.model import collect_weight_specs

    names = {w.name: w for w in collect_weight_specs(config_from_dict(CASES["A"]["raw"]).model_spec())}
    assert names["embed"].shape == (128, 64) and names["head"].shape == (128, 64) and names["final.norm.b"].shape == (64,)
    assert names["l0.mix.q"].shape == (60, 64) and names["l0.mix.v"].shape == (72, 64) and names["l0.mix.norm"].shape == (72,)
    assert names["l0.mix.i"].shape == (3, 64) and names["l0.mix.f.b"].shape == (3,) and names["l0.mix.o"].shape == (64, 72)
    assert names["l0.mlp.router"].shape == (8, 64) and names["l0.mlp.correction"].shape == (8,) and "l0.mlp.router.b" not in names
    assert "l0.mlp.e5.up" in names and "l0.mlp.e6.up" not in names and names["l0.mlp.shared.down"].shape == (64, 40)
    assert names["l1.mix.left.v.b"].shape == (32,) and names["l1.mix.right.in"].shape == (64 + 64 + 96 + 4, 64)
    assert names["l1.mix.right.conv"].shape == (160, 3) and names["l1.mix.right.conv"].kind == "vector"
    assert names["l1.mix.right.A_log"].shape == (4,) and names["l1.mix.right.norm"].shape == (64,)
    assert names["l2.norm2"].optional and names["l2.norm2.b"].optional and names["l2.hc2.mix"].optional and "l2.mlp.router" not in names
    assert names["l1.hc1.mix"].shape == (3, 3) and not names["l1.hc1.mix"].optional and "l1.mlp.shared.up" not in names
    plain_stream = {w.name for w in collect_weight_specs(config_from_dict(CASES["C"]["raw"]).model_spec())}
    assert not any(".hc" in name for name in plain_stream) and "l2.mix.right.D" in plain_stream


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda c: c["layers"][0]["mixer"].update(gate_cap=0), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(groups=3), "groups"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(norm_groups=5), "norm_groups"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("state"), "state"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "moe"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "top"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=1), "groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=5), "groups"),
    (lambda c: c["layers"][0]["mlp"]["shared"].pop("ff"), "shared"),
    (lambda c: c["loop"].update(stop=9), "loop"),
    (lambda c: c["loop"].update(times=0), "times"),
    (lambda c: c.update(streams=0), "streams"),
    (lambda c: c["norm"].update(eps=0.0), "eps"),
    (lambda c: c.pop("width"), "width"),
])
def test_a_wrong_or_missing_key_is_named_when_the_configuration_is_read(change, message):
    from lockstep_amd.config import ConfigError, config_from_dict

    raw = copy.deepcopy(CASES["A"]["raw"])
    change(raw)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(raw)


def cache_units(raw):
    from lockstep_amd.config import config_from_dict
    from lockstep_amd.parts import part_class

    spec = config_from_dict(raw).model_spec()
    units = [None] * spec.cache_units()
    for run in spec.schedule:
        mixer = part_class(spec.layers[run.layer].arrangement.kind)(spec.layers[run.layer]).mixer
        units[run.cache] = mixer.cache_spec()
        for unit, further in zip(run.further, mixer.further_specs()):
            units[unit] = further
    return units


def test_cache_units_of_every_pass_and_of_both_halves_of_a_parallel_mixer():
    from lockstep_amd.cache import CacheManager
    from lockstep_amd.parts import PagedKVSpec, StateSpec

    units = cache_units(CASES["A"]["raw"])
    assert units[0] == StateSpec((3 * 20 * 25 + 12,), "float32")      # S, n and the maxima
    assert units[1] == units[4] == PagedKVSpec(2, 24, 21, value_dim=16)
    assert units[2] == units[5] == StateSpec((4 * 24 * 16 + 3 * 160,), "float32")    # S and the ring of the convolution's inputs
    assert units[7] == PagedKVSpec(3, 16, None, value_dim=24)
    cache = CacheManager(units, page_size=8, num_pages=32, max_requests=2, max_tokens_per_request=256)
    assert sorted(len(g.units) for g in cache.groups) == [1, 2]
    cache.open("r")
    cache.reserve("r", 100)
    cache.commit("r", 100)
    held = {g.spec.window: sum(p >= 0 for p in cache.request_pages("r", g.index)) for g in cache.groups}
    assert held == {21: 3, None: 13}                    # (positions 80 .. 100 of the window, all of the other)
    cache.audit()


def test_a_mixer_that_is_not_one_product_in_and_one_out_cannot_be_a_branch():
    from lockstep_amd.config.base import PartSpec
    from lockstep_amd.parts import build_part

    with pytest.raises(ValueError, match="branch"):
        build_part(PartSpec("side_by_side", {"branches": {"a": PartSpec("min_gru", {"hidden_size": 8, "state_size": 8})}}), "m")


def test_random_weights_folder_round_trip(tmp_path):
    from lockstep_amd.config import config_from_dict, config_from_dir
    from lockstep_amd.engine.model import collect_weight_specs
    from lockstep_amd.weights import load_weights, write_random_model

    cfg = config_from_dict(SINGLE["loop"]["raw"])
    folder = write_random_model(cfg, tmp_path / "m", seed=3)
    assert config_from_dir(folder).to_dict() == cfg.to_dict()
    weights = load_weights(folder, collect_weight_specs(cfg.model_spec()), {})
    assert weights.get("l1.mix.right.in").shape == (32 + 64 + 2, 64) and weights.get("l0.mix.i.b").shape == (2,)


# -- pins of the plain implementation -----------------------------------------------------

def test_layer_norm_against_the_librarys():
    x = torch.randn((5, 24), dtype=F64) * 3 + 2
    w, b = torch.rand(24, dtype=F64), torch.randn(24, dtype=F64)
    assert torch.allclose(plain.layer_norm(x, w, b, 1e-3), torch.nn.functional.layer_norm(x, (24,), w, b, 1e-3))
    assert torch.allclose(plain.unit_rms(x, 1e-3), x * torch.rsqrt((x ** 2).mean(-1, keepdim=True) + 1e-3))


def test_gates_by_the_librarys_functions():
    z = torch.linspace(-40, 40, 81, dtype=F64)
    assert torch.allclose(plain.softplus(z), torch.nn.functional.softplus(z, threshold=100))
    assert torch.allclose(plain.log_sigmoid(z), torch.nn.functional.logsigmoid(z))
    assert torch.allclose(plain.silu(z), torch.nn.functional.silu(z))


def test_window_attention_against_the_librarys():
    q, k, v = torch.randn((17, 8), dtype=F64), torch.randn((17, 8), dtype=F64), torch.randn((17, 5), dtype=F64)
    at = torch.arange(17)
    for window in (None, 1, 4, 100):
        far = at[:, None] - at[None, :]
        seen = (far >= 0) & (far < (window or 1000))
        want = torch.nn.functional.scaled_dot_product_attention(q[None], k[None], v[None], attn_mask=seen[None], scale=0.3)[0]
        assert torch.allclose(plain.window_attention(q, k, v, 0.3, window), want)


def test_the_convolution_against_the_librarys():
    x, taps, bias = torch.randn((9, 6), dtype=F64), torch.randn((6, 4), dtype=F64), torch.randn(6, dtype=F64)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (3, 0)), taps[:, None], bias, groups=6)[0].T
    assert torch.allclose(plain.causal_conv(x, taps, bias), want)
    assert torch.allclose(plain.causal_conv(x, taps[:, :1], bias), x * taps[:, 0] + bias)


def test_the_state_space_recurrence_is_attention_with_decaying_weights():
    n, e, N = 12, 5, 7
    x, b, c = torch.randn((n, e), dtype=F64), torch.randn((n, N), dtype=F64), torch.randn((n, N), dtype=F64)
    dt, rate, skip = torch.rand(n, dtype=F64), torch.tensor(1.3, dtype=F64), torch.tensor(0.4, dtype=F64)
    total = torch.cumsum(-rate * dt, dim=0)
    w = torch.exp(total[:, None] - total[None, :]) * dt[None, :] * (c @ b.T)
    want = torch.tril(w) @ x + skip * x
    assert torch.allclose(plain.state_space(x, b, c, dt, rate, skip), want)
    once = plain.state_space(x, b, c, dt, torch.tensor(1e9, dtype=F64), skip)      # a head that forgets at once
    assert torch.allclose(once, (dt * (c * b).sum(-1))[:, None] * x + skip * x)


def test_the_matrix_memory_does_not_depend_on_its_stabiliser_but_for_the_floor():
    """Without a maximum: sums of exp(i_s + f_(s+1) + ... + f_t), a denominator of at least one in these units, and the small
    addend in units of the maximum."""
    n, d, e = 10, 6, 4
    q, k, v = torch.randn((n, d), dtype=F64), torch.randn((n, d), dtype=F64), torch.randn((n, e), dtype=F64)
    i, f = torch.randn(n, dtype=F64) * 2, -torch.rand(n, dtype=F64)
    got = plain.matrix_memory(q, k, v, i, f)
    m = 0.0
    for t in range(n):
        m = max(float(f[t]) + m, float(i[t]))
        w = torch.stack([torch.exp(i[s] + f[s + 1:t + 1].sum()) for s in range(t + 1)]) * (k[:t + 1] @ q[t])
        want = (w @ v[:t + 1]) / (max(abs(float(w.sum())), 1.0) + 1e-6 * math.exp(m))
        assert torch.allclose(got[t], want), t


def test_the_choice_of_experts_by_hand():
    scores = torch.tensor([[0.30, 0.05, 0.25, 0.10, 0.20, 0.10]], dtype=F64)
    none = torch.zeros(6, dtype=F64)
    chosen, w = plain.choose(scores, none, 2, 1, 1)
    assert chosen.tolist() == [[0, 2]] and torch.allclose(w, torch.tensor([[0.30, 0.25]], dtype=F64) / 0.55)
    chosen, w = plain.choose(scores, none, 2, 3, 1)                     # (the first group alone, though its second is the smallest)
    assert chosen.tolist() == [[0, 1]] and torch.allclose(w, torch.tensor([[0.30, 0.05]], dtype=F64) / 0.35)
    correction = torch.tensor([-1.0, -1.0, -1.0, -1.0, -0.9, -2.0], dtype=F64)
    chosen, w = plain.choose(scores, correction, 3, 3, 2)               # choice scores are negative and still beat closed groups
    assert chosen.tolist() == [[0, 4, 1]] or chosen.tolist() == [[4, 0, 1]]
    assert torch.allclose(w.sum(), torch.tensor(1.0, dtype=F64))
    chosen, _ = plain.choose(scores, torch.tensor([0, 1.0, 0, 0, 0, 0], dtype=F64), 1, 1, 1)
    assert chosen.tolist() == [[1]]


def test_one_copy_with_plain_weights_is_the_residual_sum_and_a_loop_is_the_layers_again():
    raw = SINGLE["loop"]["raw"]
    tensors = make_tensors(raw, seed=4)
    unrolled = dict(copy.deepcopy(raw), layers=raw["layers"] * 2)
    unrolled.pop("loop")
    repeated = dict(tensors)
    for name, t in tensors.items():
        if name.startswith("l") and name[1].isdigit():
            repeated[f"l{int(name[1]) + 2}{name[2:]}"] = t
    tokens = list(range(9))
    want = plain.PlainPozozen(raw, tensors).forward(tokens)
    assert torch.allclose(plain.PlainPozozen(unrolled, repeated).forward(tokens), want)
    bare_stream = {k: v for k, v in raw.items() if k != "streams"}
    one = dict(tensors)
    for i in range(2):
        for name in ("in", "out", "mix"):
            one[f"l{i}.hc1.{name}"] = torch.ones((1, 1) if name == "mix" else 1)
    assert torch.allclose(plain.PlainPozozen(bare_stream, tensors).forward(tokens),
                          plain.PlainPozozen(dict(raw, streams=1), one).forward(tokens))
    assert not torch.allclose(plain.PlainPozozen(bare_stream, tensors).forward(tokens), want, atol=1e-2)


def test_identity_experts_and_the_shared_expert_in_the_feed_forward():
    raw = SINGLE["experts"]["raw"]
    tensors = make_tensors(raw, seed=5)
    model = plain.PlainPozozen(raw, tensors)
    mlp, h = raw["layers"][0]["mlp"], torch.randn((40, 64), dtype=F64)
    scores = torch.softmax(h @ model.w["l0.mlp.router"].T, dim=-1)
    chosen, weight = plain.choose(scores, model.w["l0.mlp.correction"], 4, 4, 2)
    dense = torch.stack([model.gated(f"l0.mlp.e{e}", h) if e < 9 else h for e in range(12)], dim=1)         # [T, R, W]
    w = torch.zeros((40, 12), dtype=F64).scatter_(1, chosen, weight)
    want = (w[:, :, None] * dense).sum(1) + model.gated("l0.mlp.shared", h)
    assert torch.allclose(model.experts("l0.mlp", mlp, h), want)
    assert bool((chosen >= 9).any()) and bool((chosen < 9).any())
