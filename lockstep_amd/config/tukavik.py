"""Tukavik: a decoder with layer norms on both sides of every sublayer, whose layers hand on a learned average
of all results so far, and each of which names one of three mixers.

* embedding: ``embed[token]`` plus a vector of sines and cosines of the position; the head is the same table.
* a layer: ``x += norm1b(mixer(norm1(x)))``, then ``x += norm2b(ff(norm2(x)))`` (or the first half alone); what
  goes on is ``sum_j dwa[j] X_j`` over the embedding's output ``X_0`` and the layers' results ``X_1, ...`` so far.
* ``mingru``: a recurrence of one number a channel whose gates read the current token only, a SiLU gate behind.
* ``latent_attention``: causal attention without positions whose keys and values are projections of one cached,
  normalised latent a token.
* ``latent_attention_2``: the same with queries that pass a normalised latent of their own; a layer with
  ``kv_from`` reads the latent that an earlier layer caches.
* feed-forward ``dense``: two matrices with xIELU (two learned numbers a layer) between them.

``config.json`` is nested: ``architecture`` (the name), ``vocab``, ``width``, ``norm.eps`` and ``layers``, a list
whose entries give ``type``, the mixer's sizes and constants under ``mixer`` and the feed-forward under ``mlp``
(null for a layer without one).  Layer ``i``'s tensors start with ``l<i>.``: ``norm1``, ``norm1b``, ``norm2``,
``norm2b``, ``dwa``, ``mix.*``, ``mlp.{up,down,act}``; beside them ``embed`` and ``final.norm``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any

from .base import ConfigError, LayerSpec, ModelConfig, ModelSpec, PartSpec, ScheduleEntry
from .registry import register_architecture

#: base of the position vectors' frequencies; fixed by the design
POSITION_BASE = 10000.0
MIXERS = ("mingru", "latent_attention", "latent_attention_2")


def _need(mapping, key: str, where: str):
    if not isinstance(mapping, dict) or key not in mapping:
        raise ConfigError(f"config.json: {where} lacks the key {key!r}")
    return mapping[key]


def _positive_int(value, what: str) -> int:
    if not isinstance(value, int) or isinstance(value, bool) or value <= 0:
        raise ConfigError(f"{what} must be a positive integer, got {value!r}")
    return value


@register_architecture
@dataclass(frozen=True)
class TukavikConfig(ModelConfig):
    architecture: str
    vocab: int
    width: int
    norm: Any
    layers: Any

    architecture_names = ("Tukavik", "tukavik")

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def to_dict(self) -> dict:
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": dict(self.norm),
                "layers": [dict(layer) for layer in self.layers]}

    def init_scheme(self):
        return {"std": 0.05, "norm_std": 0.1}

    def validate(self) -> None:
        _positive_int(self.vocab, "vocab")
        _positive_int(self.width, "width")
        if not float(_need(self.norm, "eps", "norm")) > 0:
            raise ConfigError("norm.eps must be positive")
        if not isinstance(self.layers, (list, tuple)) or not self.layers:
            raise ConfigError("layers must be a non-empty list")
        for i, layer in enumerate(self.layers):
            kind = _need(layer, "type", f"layers[{i}]")
            if kind not in MIXERS:
                raise ConfigError(f"layers[{i}].type {kind!r} is not one of {', '.join(MIXERS)}")
            if not isinstance(_need(layer, "mixer", f"layers[{i}]"), dict):
                raise ConfigError(f"layers[{i}].mixer must be a mapping")
            mlp = layer.get("mlp")
            if mlp is not None and _need(mlp, "kind", f"layers[{i}].mlp") != "dense":
                raise ConfigError(f"layers[{i}].mlp.kind {mlp['kind']!r} is not dense")
        self.model_spec()        # every key the layers need, now rather than at the first step

    # -- the mixers as parts ------------------------------------------------------------
    def _source(self, i: int) -> int:
        """The layer whose cache unit layer ``i`` uses: itself, or the one whose latent it reads (``kv_from``)."""
        m = self.layers[i]["mixer"]
        source = m.get("kv_from")
        if source is None:
            return i
        where = f"layers[{i}].mixer.kv_from"
        if not isinstance(source, int) or isinstance(source, bool) or not 0 <= source < len(self.layers) or source == i:
            raise ConfigError(f"{where} {source!r} is not another layer")
        other = self.layers[source]
        if other.get("type") not in ("latent_attention", "latent_attention_2") or other["mixer"].get("kv_from") is not None:
            raise ConfigError(f"{where}: layer {source} has no latent of its own")
        if source > i:
            raise ConfigError(f"{where}: layer {source} runs after layer {i}")
        if other["mixer"].get("kv_rank") != m.get("kv_rank"):
            raise ConfigError(f"{where}: layer {source} has another kv_rank")
        return source

    def _mixer(self, i: int, layer) -> PartSpec:
        kind, m, where = layer["type"], layer["mixer"], f"layers[{i}].mixer"
        need = lambda key: _positive_int(_need(m, key, where), f"{where}.{key}")  # noqa: E731
        if kind == "mingru":
            return PartSpec("min_gru", {"hidden_size": self.width, "state_size": need("width")})
        return PartSpec("latent_attention", {
            "hidden_size": self.width, "num_heads": need("heads"), "head_dim": need("dim"), "rot_dim": 0,
            "value_dim": need("vdim"), "q_rank": need("q_rank") if kind == "latent_attention_2" else None,
            "kv_rank": need("kv_rank"), "eps": float(self.norm["eps"]), "position": PartSpec("no_position", {}),
            "scale": float(_need(m, "scale", where)), "window": None, "sink": None, "reads_other": self._source(i) != i})

    def model_spec(self) -> ModelSpec:
        width, eps, n = self.width, float(self.norm["eps"]), len(self.layers)
        norm = lambda name, **more: PartSpec("layernorm", dict(size=width, eps=eps, name=name, **more))  # noqa: E731
        layers, schedule = [], []
        for i, layer in enumerate(self.layers):
            mlp = layer.get("mlp")
            arrangement = PartSpec("sandwich_residual", {
                "mixer_prefix": "mix", "feed_forward_prefix": "mlp", "mixer_norm_name": "norm1",
                "mixer_post_norm_name": "norm1b", "feed_forward_norm_name": "norm2", "feed_forward_post_norm_name": "norm2b",
                "depth_average": {"name": "dwa", "index": i, "layers": n}})
            feed_forward = None if mlp is None else PartSpec("mlp", {
                "hidden_size": width, "activation": "xielu",
                "intermediate_size": _positive_int(_need(mlp, "ff", f"layers[{i}].mlp"), f"layers[{i}].mlp.ff")})
            layers.append(LayerSpec(
                prefix=f"l{i}", arrangement=arrangement, mixer=self._mixer(i, layer), feed_forward=feed_forward,
                mixer_norm=norm(f"l{i}.norm1"), feed_forward_norm=norm(f"l{i}.norm2", optional=mlp is None),
                parts={"mixer_post_norm": norm(f"l{i}.norm1b"),
                       "feed_forward_post_norm": norm(f"l{i}.norm2b", optional=mlp is None)}))
            source = i if layer["type"] == "mingru" else self._source(i)
            schedule.append(ScheduleEntry(layer=i, cache=source, writes_cache=source == i))
        return ModelSpec(
            hidden_size=width, vocab_size=self.vocab,
            embedding=PartSpec("token_embedding", {"name": "embed", "vocab_size": self.vocab, "hidden_size": width,
                                                   "positions": {"base": POSITION_BASE}}),
            layers=tuple(layers), schedule=tuple(schedule), final_norm=norm("final.norm"),
            head=PartSpec("linear_head", {"name": "embed", "tied_to": None, "vocab_size": self.vocab, "hidden_size": width}),
            max_positions=None)
