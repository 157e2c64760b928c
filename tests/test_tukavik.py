"""Tukavik without a GPU: the configuration reader and its errors, the tensors it expects, the cache units and the
layers that share a latent, the random-weights folder, and pins of the plain implementation (each mechanism against a
second, independent formulation)."""

from __future__ import annotations

import copy
import math

import pytest
import torch

from plain import tukavik_plain as plain
from tukavik_cases import CASES, SINGLE, make_tensors

F64 = torch.float64


# -- configuration and weights ---------------------------------------------------------

def test_config_is_found_by_its_architecture_key_and_states_the_layers_as_parts():
    from lockstep_amd.config import TukavikConfig, config_from_dict

    cfg = config_from_dict(CASES["A"]["raw"])
    assert isinstance(cfg, TukavikConfig)
    spec = cfg.model_spec()
    assert [layer.mixer.kind for layer in spec.layers] == ["latent_attention", "min_gru", "latent_attention", "latent_attention", "min_gru"]
    assert all(layer.arrangement.kind == "sandwich_residual" for layer in spec.layers)
    assert [layer.arrangement["depth_average"]["index"] for layer in spec.layers] == [0, 1, 2, 3, 4]
    first, second, third, fourth, _ = (layer.mixer for layer in spec.layers)
    assert (first["num_heads"], first["head_dim"], first["value_dim"], first["kv_rank"], first["q_rank"]) == (4, 16, 24, 32, None)
    assert (first["rot_dim"], first["sink"], first["window"], first["scale"], first["eps"]) == (0, None, None, 0.3, 1e-5)
    assert first["position"].kind == "no_position" and not first["reads_other"]
    assert second["state_size"] == 80
    assert (third["q_rank"], third["reads_other"], fourth["q_rank"], fourth["reads_other"]) == (24, False, 56, True)
    assert spec.layers[1].feed_forward is None and spec.layers[0].feed_forward["activation"] == "xielu"
    assert spec.layers[0].feed_forward["intermediate_size"] == 96
    assert spec.embedding["positions"] == {"base": 10000.0} and spec.head["name"] == "embed"
    assert [(e.layer, e.cache, e.writes_cache) for e in spec.schedule] == [
        (0, 0, True), (1, 1, True), (2, 2, True), (3, 2, False), (4, 4, True)]
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()


def test_the_expected_tensors():
    from lockstep_amd.config import config_from_dict
    from lockstep_amd.engine.model import collect_weight_specs

    names = {w.name: w for w in collect_weight_specs(config_from_dict(CASES["B"]["raw"]).model_spec())}
    assert names["embed"].shape == (200, 96) and names["final.norm"].shape == (96,) and "head" not in names
    assert names["l0.mix.z"].shape == (96, 96) and names["l0.mix.x.b"].shape == (96,) and names["l0.dwa"].shape == (2,)
    assert names["l1.mix.dq"].shape == (12, 96) and names["l1.mix.uq"].shape == (40, 12) and names["l1.mix.o"].shape == (96, 8)
    assert names["l1.norm2"].optional and names["l1.norm2b"].optional and "l1.mlp.up" not in names
    assert names["l2.mix.q"].shape == (60, 96) and names["l2.mix.dkv"].shape == (20, 96) and "l2.mix.dq" not in names
    assert names["l2.mix.uk"].shape == (60, 20) and names["l2.mix.uv"].shape == (100, 20) and names["l2.mlp.act"].shape == (2,)
    assert not names["l2.norm2"].optional and names["l2.norm1b"].kind == "vector"
    assert "l4.mix.dkv" not in names and names["l4.mix.uk"].shape == (40, 20) and names["l4.dwa"].shape == (6,)


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][2]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][1]["mixer"].update(width=0), "width"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=1), "no latent of its own"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=0), "kv_rank"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=3), "no latent of its own"),
    (lambda c: c["layers"][0]["mixer"].update(kv_from=2, kv_rank=40), "runs after"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=9), "not another layer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "dense"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"),
    (lambda c: c["norm"].update(eps=0.0), "eps"),
    (lambda c: c.pop("width"), "width"),
])
def test_a_wrong_or_missing_key_is_named_when_the_configuration_is_read(change, message):
    from lockstep_amd.config import ConfigError, config_from_dict

    raw = copy.deepcopy(CASES["A"]["raw"])
    change(raw)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(raw)


def test_cache_units_of_the_mixers_and_of_a_shared_latent():
    from lockstep_amd.cache import CacheManager
    from lockstep_amd.config import config_from_dict
    from lockstep_amd.parts import PagedKVSpec, StateSpec, part_class

    spec = config_from_dict(CASES["B"]["raw"]).model_spec()
    units = [None] * spec.cache_units()
    for run in spec.schedule:
        layer = part_class(spec.layers[run.layer].arrangement.kind)(spec.layers[run.layer])
        if run.writes_cache:
            units[run.cache] = layer.mixer.cache_spec()
    assert units[0] == StateSpec((96,), "float32") and units[3] == StateSpec((24,), "float32")
    assert units[1] == PagedKVSpec(1, 24, None, value_dim=24)
    assert units[2] == PagedKVSpec(1, 24, None, value_dim=20)          # (keys padded to a multiple of eight)
    assert len(units) == 4 and spec.schedule[4].cache == 2             # the last layer has no unit of its own
    cache = CacheManager(units, page_size=8, num_pages=32, max_requests=2, max_tokens_per_request=256)
    cache.open("r")
    cache.reserve("r", 100)
    cache.commit("r", 100)
    assert all(sum(p >= 0 for p in cache.request_pages("r", g.index)) == 13 for g in cache.groups)
    cache.audit()


def test_random_weights_folder_round_trip(tmp_path):
    from lockstep_amd.config import config_from_dict, config_from_dir
    from lockstep_amd.engine.model import collect_weight_specs
    from lockstep_amd.weights import load_weights, write_random_model

    cfg = config_from_dict(SINGLE["shared"]["raw"])
    folder = write_random_model(cfg, tmp_path / "m", seed=3)
    assert config_from_dir(folder).to_dict() == cfg.to_dict()
    weights = load_weights(folder, collect_weight_specs(cfg.model_spec()), {})
    assert weights.get("l0.mix.dkv").shape == (40, 64) and weights.get("l1.dwa").shape == (3,)


# -- pins of the plain implementation -----------------------------------------------------

def test_position_vectors_are_unit_circles_that_turn():
    v = plain.position_vectors(50, 10)
    assert torch.equal(v[0], torch.tensor([0.0, 1.0] * 5, dtype=F64))
    z = torch.complex(v[:, 1::2], v[:, 0::2])                 # cos + i sin
    f = torch.tensor([10000.0 ** (-i / 5) for i in range(5)], dtype=F64)
    assert torch.allclose(z[1:] / z[:-1], torch.polar(torch.ones(5, dtype=F64), f).expand(49, 5))
    assert torch.allclose(plain.position_vectors(9, 7)[:, 6], torch.sin(torch.arange(9, dtype=F64) * 10000.0 ** (-6 / 7)))


def test_norms_against_the_librarys():
    x = torch.randn((5, 24), dtype=F64) * 3 + 2
    w = torch.rand(24, dtype=F64)
    assert torch.allclose(plain.layer_norm(x, w, 1e-3), torch.nn.functional.layer_norm(x, (24,), w, None, 1e-3))
    assert torch.allclose(plain.rms_norm(x, w, 1e-3), x * torch.rsqrt((x ** 2).mean(-1, keepdim=True) + 1e-3) * w)


def test_xielu_by_its_pieces_and_its_slope():
    p, q = torch.tensor(0.3, dtype=F64), torch.tensor(-0.7, dtype=F64)
    up, down = math.log1p(math.exp(0.3)), 0.5 + math.log1p(math.exp(-0.7))
    assert float(plain.xielu(torch.tensor(2.0, dtype=F64), p, q)) == pytest.approx(4 * up + 1.0)
    assert float(plain.xielu(torch.tensor(-1.5, dtype=F64), p, q)) == pytest.approx(down * (math.exp(-1.5) + 0.5) - 0.75)
    assert float(plain.xielu(torch.tensor(0.0, dtype=F64), p, q)) == 0.0
    z = torch.linspace(-3, 3, 121, dtype=F64, requires_grad=True)
    plain.xielu(z, p, q).sum().backward()
    want = torch.where(z > 0, 2 * up * z, down * (torch.exp(z) - 1)) + 0.5
    assert torch.allclose(z.grad, want.detach())


def test_the_recurrence_is_a_weighted_mean_of_the_candidates():
    z = torch.rand((6, 3), dtype=F64)
    u = torch.randn((6, 3), dtype=F64)
    c = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    S = plain.gated_average(z, u)
    for t in range(6):
        want = sum(z[s] * c[s] * torch.prod(1 - z[s + 1:t + 1], dim=0) for s in range(t + 1))
        assert torch.allclose(S[t], want)
    assert torch.allclose(plain.gated_average(torch.ones_like(z), u), c)         # an open gate keeps nothing
    assert float(plain.gated_average(torch.zeros_like(z), u).abs().max()) == 0.0


def test_attention_against_the_librarys_and_in_the_latents_space():
    """What the engine computes (queries multiplied into the latent's space, one shared key/value head, the heads'
    outputs multiplied out of it) equals keys and values a head."""
    raw = SINGLE["latent_2"]["raw"]
    model = plain.PlainTukavik(raw, make_tensors(raw, seed=2))
    m, w = raw["layers"][0]["mixer"], model.w
    h = torch.randn((9, raw["width"]), dtype=F64)
    c = model.latent(0, h)
    want = model.attention(0, m, h, c)
    q = plain.rms_norm(h @ w["l0.mix.dq"].T, w["l0.mix.dq.norm"], 1e-5) @ w["l0.mix.uq"].T
    q = q.view(9, m["heads"], m["dim"])
    moved = torch.einsum("thd,hdr->htr", q, w["l0.mix.uk"].view(m["heads"], m["dim"], -1))
    mixed = torch.nn.functional.scaled_dot_product_attention(moved, c.expand(m["heads"], -1, -1), c.expand(m["heads"], -1, -1),
                                                             is_causal=True, scale=m["scale"])
    out = torch.einsum("htr,hvr->thv", mixed, w["l0.mix.uv"].view(m["heads"], m["vdim"], -1)).reshape(9, -1)
    assert torch.allclose(out @ w["l0.mix.o"].T, want)


def test_the_average_over_depth():
    xs = [torch.randn((4, 6), dtype=F64) for _ in range(3)]
    shares = torch.tensor([0.5, -1.0, 2.0], dtype=F64)
    assert torch.allclose(plain.depth_average(xs, shares), 0.5 * xs[0] - xs[1] + 2.0 * xs[2])
    # shares that are zero but for the last leave a plain residual stream; other shares do not
    raw = CASES["A"]["raw"]
    tensors = make_tensors(raw, seed=5)
    last_only = {n: torch.cat([torch.zeros_like(t[:-1]), torch.ones_like(t[-1:])]) if n.endswith(".dwa") else t
                 for n, t in tensors.items()}
    tokens = list(range(7))
    model = plain.PlainTukavik(raw, last_only)
    w, x = model.w, model.w["embed"][tokens] + plain.position_vectors(7, raw["width"])
    latents = {}
    for i, layer in enumerate(raw["layers"]):
        h = plain.layer_norm(x, w[f"l{i}.norm1"], 1e-5)
        if layer["type"] == "mingru":
            y = model.recurrence(i, h)
        else:
            if "kv_from" not in layer["mixer"]:
                latents[i] = model.latent(i, h)
            y = model.attention(i, layer["mixer"], h, latents[layer["mixer"].get("kv_from", i)])
        x = x + plain.layer_norm(y, w[f"l{i}.norm1b"], 1e-5)
        if layer["mlp"]:
            y = model.feed_forward(i, plain.layer_norm(x, w[f"l{i}.norm2"], 1e-5))
            x = x + plain.layer_norm(y, w[f"l{i}.norm2b"], 1e-5)
    want = plain.layer_norm(x, w["final.norm"], 1e-5) @ w["embed"].T
    assert torch.allclose(model.forward(tokens), want)
    assert not torch.allclose(plain.PlainTukavik(raw, tensors).forward(tokens), want, atol=1e-2)


def test_a_shared_latent_is_the_first_layers_own():
    raw = SINGLE["shared"]["raw"]
    tensors = make_tensors(raw, seed=6)
    tokens = list(range(12))
    want = plain.PlainTukavik(raw, tensors).forward(tokens)
    changed = dict(tensors)
    changed["l0.mix.dkv.norm"] = tensors["l0.mix.dkv.norm"] * 2
    changed["l0.mix.uk"], changed["l0.mix.uv"] = tensors["l0.mix.uk"] / 2, tensors["l0.mix.uv"] / 2
    got = plain.PlainTukavik(raw, changed).forward(tokens)           # layer 0 sees what it saw, layer 1 a latent twice as large
    assert not torch.allclose(got, want, atol=1e-3)
    changed["l1.mix.uk"], changed["l1.mix.uv"] = tensors["l1.mix.uk"] / 2, tensors["l1.mix.uv"] / 2
    assert torch.allclose(plain.PlainTukavik(raw, changed).forward(tokens), want)
