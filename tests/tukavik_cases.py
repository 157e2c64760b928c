"""Small Tukavik configurations and weights for the tests.  The configurations differ from each other in every size
and option: the order of the layers, one to sixteen heads, key and value sizes (equal and unequal, no multiples of 16
or of 8), latents of sizes that are no multiple of 8, queries with and without a latent of their own, layers that read
the latent of an earlier one (of either kind, once or twice, with other heads and sizes), recurrences narrower and
wider than the model and of a single channel, layers without a feed-forward, widths that are no multiple of 4."""

from __future__ import annotations

import json

import torch


def latent(heads, dim, vdim, kv_rank, scale, q_rank=None, kv_from=None):
    """``latent_attention``, or ``latent_attention_2`` where the queries have a latent (``q_rank``)."""
    mixer = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale}
    if q_rank is not None:
        mixer["q_rank"] = q_rank
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention" if q_rank is None else "latent_attention_2", "mixer": mixer}


def recurrence(width):
    return {"type": "mingru", "mixer": {"width": width}}


def dense(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff})


def bare(layer):
    return dict(layer, mlp=None)


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Tukavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


CASES = {
    # every mixer; a latent read by the layer behind it with other heads and sizes
    "A": dict(page_size=8, raw=config(64, 128, [
        dense(latent(4, 16, 24, kv_rank=32, scale=0.3), 96),
        bare(recurrence(80)),
        dense(latent(3, 24, 16, kv_rank=40, scale=0.25, q_rank=24), 48),
        bare(latent(6, 8, 40, kv_rank=40, scale=0.4, q_rank=56, kv_from=2)),
        dense(recurrence(40), 32),
    ])),
    # a recurrence first, as wide as the model; a latent of 20 elements (padded keys) that belongs to a layer without
    # a query latent and is read by one with; two independent latents of other sizes; another eps
    "B": dict(page_size=16, raw=config(96, 200, [
        dense(recurrence(96), 40),
        bare(latent(1, 40, 8, kv_rank=24, scale=0.2, q_rank=12)),
        dense(latent(5, 12, 20, kv_rank=20, scale=0.5), 64),
        dense(recurrence(24), 24),
        dense(latent(2, 20, 28, kv_rank=20, scale=0.4, q_rank=16, kv_from=2), 80),
    ], eps=1e-3)),
    # an odd width; a single head, then sixteen and two heads on its latent; a recurrence of one channel; one unit in
    # a feed-forward
    "C": dict(page_size=16, raw=config(45, 64, [
        dense(latent(1, 8, 8, kv_rank=16, scale=0.6, q_rank=8), 16),
        bare(latent(16, 12, 4, kv_rank=16, scale=0.3, q_rank=20, kv_from=0)),
        dense(recurrence(1), 1),
        bare(latent(2, 16, 24, kv_rank=16, scale=0.4, q_rank=33, kv_from=0)),
    ], eps=1e-6)),
}

SINGLE = {
    "latent": dict(page_size=8, raw=config(64, 96, [bare(latent(4, 16, 24, kv_rank=32, scale=0.5))])),
    "latent_2": dict(page_size=8, raw=config(64, 96, [bare(latent(4, 16, 24, kv_rank=24, scale=0.5, q_rank=40))])),
    "shared": dict(page_size=8, raw=config(64, 96, [bare(latent(3, 16, 24, kv_rank=40, scale=0.5)),
                                                    bare(latent(2, 24, 16, kv_rank=40, scale=0.5, q_rank=24, kv_from=0))])),
    "recurrence": dict(page_size=8, raw=config(64, 96, [bare(recurrence(100))])),
    "dense": dict(page_size=8, raw=config(64, 96, [dense(recurrence(16), 200)])),
}


def make_tensors(raw: dict, seed: int, spread: float = 1.0) -> dict:
    """Random bfloat16 weights for ``raw`` through the package's seeded random-weights mode, then: token vectors as
    large as the position vectors, gates of the recurrence that differ from token to token and mostly remember, biases,
    the activation's two numbers and the shares of earlier layers (of both signs) wide enough to matter."""
    from lockstep_amd.config import config_from_dict
    from lockstep_amd.weights import random_tensors

    tensors = random_tensors(config_from_dict(raw), seed, std=0.12 * spread, norm_std=0.2, dtype=torch.bfloat16)
    g = torch.Generator().manual_seed(seed + 1000)

    def draw(name, width, centre=0.0):
        if name in tensors:
            tensors[name] = (centre + torch.randn(tensors[name].shape, generator=g) * width).to(torch.bfloat16)

    draw("embed", 0.7)
    for i in range(len(raw["layers"])):
        draw(f"l{i}.mix.z", 0.15)
        draw(f"l{i}.mix.z.b", 0.7, centre=-1.5)
        draw(f"l{i}.mix.x.b", 0.5)
        draw(f"l{i}.mlp.act", 0.8)
        draw(f"l{i}.dwa", 0.4)
        tensors[f"l{i}.dwa"][-1] = 1.0
    return tensors


def write_model(folder, raw: dict, tensors: dict):
    from lockstep_amd.weights import save_file

    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(raw))
    save_file(tensors, folder / "model.safetensors")
    return folder
