"""Small Pozozen configurations and weights for the tests.  The configurations differ from each other in every size and
option: residual copies (three, one, none at all), loops (a part of the layers twice, all of them three times, none), the order of
the layers, heads of both halves of a parallel mixer (grouped, as many key/value heads as query heads, a single one, sixteen on
one), key, value and state sizes (equal and unequal, no multiples of 4 or of 16, one row), windows (shorter than a page, no multiple
of a page or of a key tile, longer than any sequence, none), convolutions of one to five taps, groups of B and C, parts of the gated
norm, experts with and without groups, identity experts, a shared expert (all experts for every token, one a token, groups of
one), layers without a feed-forward, factors of both signs, widths that are no multiple of 4."""

from __future__ import annotations

import json

import torch


def attention(heads, kv_heads, dim, vdim, window, scale):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        out["mask"] = {"size": window}
    return out


def space(heads, vdim, state, groups=1, taps=4, parts=1):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": taps, "norm_groups": parts}


def parallel(left, right, left_scale=0.7, right_scale=0.8):
    return {"type": "parallel", "mixer": {"left": left, "left_scale": left_scale, "right": right, "right_scale": right_scale}}


def memory(heads, dim, vdim, cap=8.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def moe(layer, ff, experts, top, identity=0, groups=None, shared=None):
    router = {"experts": experts, "top": top}
    if identity:
        router["identity"] = identity
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared:
        mlp["shared"] = {"ff": shared}
    return dict(layer, mlp=mlp)


def bare(layer):
    return dict(layer, mlp=None)


def config(width, vocab, layers, streams=None, loop=None, mult=0.6, eps=1e-5):
    out = {"architecture": "Pozozen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "layers": layers}
    if streams is not None:
        out["streams"] = streams
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CASES = {
    # three copies, the middle two layers twice; a window of 21 on pages of 8; groups of B and C, a gated norm in two parts
    "A": dict(page_size=8, raw=config(64, 128, [
        moe(memory(3, 20, 24), 32, experts=6, top=2, identity=2, groups=(4, 2), shared=40),
        moe(parallel(attention(4, 2, 24, 16, 21, 0.5), space(4, 16, 24, groups=2, taps=3, parts=2)), 24, experts=5, top=3, identity=1,
            groups=(3, 2)),
        bare(memory(2, 32, 16, cap=5.0)),
        moe(parallel(attention(3, 3, 16, 24, None, 0.3), space(2, 40, 16), left_scale=1.0, right_scale=-0.5), 32, experts=7, top=2,
            shared=16),
    ], streams=3, loop=(1, 3, 2))),
    # one copy behind hyper-connections; sizes that are no multiples of 8; a window longer than any sequence; two taps and five;
    # a factor of one everywhere; the best group alone
    "B": dict(page_size=16, raw=config(96, 200, [
        moe(parallel(attention(6, 1, 12, 40, 1000, 0.4), space(3, 20, 40, taps=2, parts=3), left_scale=1.0, right_scale=1.0), 24, experts=8,
            top=1, identity=4, groups=(6, 1)),
        moe(memory(1, 40, 50), 16, experts=3, top=3, shared=8),
        moe(parallel(attention(2, 2, 40, 6, 37, 0.3), space(6, 10, 6, groups=3, taps=5)), 40, experts=9, top=4),
    ], streams=1, mult=1.0, eps=1e-3)),
    # a plain residual stream of an odd width; sixteen heads on one with a window shorter than a page; a state of one row, a
    # convolution of one tap, one head; a state of 70 rows and 9 columns; all of it three times; more identity experts than others
    "C": dict(page_size=16, raw=config(45, 64, [
        moe(parallel(attention(16, 1, 8, 4, 5, 0.6), space(1, 9, 1, taps=1)), 12, experts=2, top=2, identity=3, groups=(5, 3)),
        moe(memory(2, 70, 9, cap=20.0), 10, experts=1, top=1, identity=1, shared=20),
        bare(parallel(attention(1, 1, 40, 8, 11, 0.2), space(5, 6, 70, taps=4, parts=5))),
    ], loop=(0, 3, 3), eps=1e-6)),
}

SINGLE = {
    "parallel": dict(page_size=8, raw=config(64, 96, [bare(parallel(attention(4, 2, 32, 16, 20, 0.4), space(4, 24, 32)))], streams=2)),
    "attention": dict(page_size=8, raw=config(64, 96, [bare(parallel(attention(4, 2, 32, 16, 20, 0.4), space(2, 8, 8), right_scale=0.0))])),
    "space": dict(page_size=8, raw=config(64, 96, [bare(parallel(attention(1, 1, 8, 8, 20, 0.4), space(4, 24, 32, groups=2, parts=2),
                                                                left_scale=0.0))])),
    "memory": dict(page_size=8, raw=config(64, 96, [bare(memory(4, 32, 24))], streams=2)),
    "loop": dict(page_size=8, raw=config(64, 96, [bare(memory(2, 16, 16)), bare(parallel(attention(2, 1, 16, 16, 20, 0.4), space(2, 16, 16)))],
                                         streams=2, loop=(0, 2, 2))),
    "experts": dict(page_size=8, raw=config(64, 96, [moe(memory(1, 8, 8), 40, experts=9, top=4, identity=3, groups=(4, 2), shared=24)],
                                            streams=4)),
    # a stream of eight copies of a width that is no multiple of 4
    "copies": dict(page_size=8, raw=config(90, 96, [moe(memory(2, 16, 12), 20, experts=3, top=2)], streams=8)),
}


def make_tensors(raw: dict, seed: int, spread: float = 1.0) -> dict:
    """Random bfloat16 weights for ``raw`` through the package's seeded random-weights mode, then: biases, taps, gates, decays and
    the streams' weights are drawn wide enough to matter, the heads' decays from one that forgets at once to one that
    hardly does, routers so that they decide clearly, with corrections that change the choice."""
    from lockstep_amd.config import config_from_dict
    from lockstep_amd.weights import random_tensors

    tensors = random_tensors(config_from_dict(raw), seed, std=0.1 * spread, norm_std=0.2, dtype=torch.bfloat16)
    g = torch.Generator().manual_seed(seed + 1000)

    def draw(name, width, centre=0.0):
        if name in tensors:
            tensors[name] = (centre + torch.randn(tensors[name].shape, generator=g) * width).to(torch.bfloat16)

    draw("embed", 1.0)
    draw("final.norm.b", 0.2)
    for i in range(len(raw["layers"])):
        p = f"l{i}.mix"
        for name in ("q.b", "k.b", "v.b"):
            draw(f"{p}.left.{name}", 0.4)
        draw(f"{p}.right.conv", 0.5)
        draw(f"{p}.right.conv.b", 0.2)
        draw(f"{p}.right.A_log", 1.8, centre=0.5)
        draw(f"{p}.right.dt_bias", 0.7, centre=-2.0)
        draw(f"{p}.right.D", 0.4, centre=0.6)
        draw(f"{p}.i.b", 1.0)
        draw(f"{p}.f.b", 1.5, centre=3.5)
        for name in ("i", "f"):
            if f"{p}.{name}" in tensors:
                tensors[f"{p}.{name}"] = (tensors[f"{p}.{name}"].float() * 2.5).to(torch.bfloat16)
        for half in ("norm1", "norm2"):
            draw(f"l{i}.{half}.b", 0.2)
        draw(f"l{i}.mlp.router", 0.6)
        draw(f"l{i}.mlp.correction", 0.4)
        for half in ("hc1", "hc2"):
            draw(f"l{i}.{half}.in", 0.3, centre=0.5)
            draw(f"l{i}.{half}.out", 0.3, centre=1.0)
            if f"l{i}.{half}.mix" in tensors:
                n = tensors[f"l{i}.{half}.mix"].shape[0]
                tensors[f"l{i}.{half}.mix"] = (0.8 * torch.eye(n) + torch.randn((n, n), generator=g) * 0.2).to(torch.bfloat16)
    return tensors


def write_model(folder, raw: dict, tensors: dict):
    from lockstep_amd.weights import save_file

    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(raw))
    save_file(tensors, folder / "model.safetensors")
    return folder
