"""Pozozen: a decoder over a residual stream of several copies (hyper-connections) whose layers each name one of two
mixers, some of them run several times in a row, with a feed-forward of routed experts.

* ``parallel``: two mixers side by side on the same input: grouped-query attention with biased projections and a sliding
  window, without positions, and Mamba-2's state-space recurrence behind a short convolution; each enters the sum with a
  factor of its own.
* ``mlstm``: xLSTM's matrix memory with capped exponential gates, a running maximum and a normaliser.
* feed-forward: a softmax router with a correction that counts for the choice only, groups of experts of which the best are
  kept, experts that return their input, and a shared expert; or none.

Norms are layer norms with weight and bias; what a sublayer returns enters the stream times ``residual_mult``.

``config.json`` is nested: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``residual_mult``, ``streams`` (the copies of the
residual stream; absent: one plain residual stream), ``loop`` (``start``, ``stop``, ``times``: the layers ``start .. stop - 1`` run ``times``
times in a row with the same weights, each pass with its own cache units; absent: once) and ``layers``, a list whose entries give
``type``, the mixer's sizes and constants under ``mixer`` and the feed-forward under ``mlp`` (null for a layer without one).  Layer
``i``'s tensors start with ``l<i>.``: ``norm1``, ``norm2`` (each with ``.b``), ``mix.*`` (``mix.left.*`` and ``mix.right.*`` of a parallel mixer),
``mlp.*``, ``hc1.*``, ``hc2.*``; beside them ``embed``, ``final.norm``, ``final.norm.b`` and ``head``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any

from .base import ConfigError, LayerSpec, ModelConfig, ModelSpec, PartSpec, ScheduleEntry
from .registry import register_architecture

#: added to the denominator of the matrix memory's read-out; fixed by the design
DENOM_EPS = 1e-6


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
class PozozenConfig(ModelConfig):
    architecture: str
    vocab: int
    width: int
    norm: Any
    residual_mult: float
    layers: Any
    streams: Any = None
    loop: Any = None

    architecture_names = ("Pozozen", "pozozen")

    @classmethod
    def from_dict(cls, raw):
        return super().from_dict({"streams": None, "loop": None, "residual_mult": 1.0, **raw})

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": dict(self.norm),
               "residual_mult": self.residual_mult, "layers": [dict(layer) for layer in self.layers]}
        if self.streams is not None:
            out["streams"] = self.streams
        if self.loop is not None:
            out["loop"] = dict(self.loop)
        return out

    def init_scheme(self):
        return {"std": 0.05, "norm_std": 0.1}

    def validate(self) -> None:
        _positive_int(self.vocab, "vocab")
        _positive_int(self.width, "width")
        if not float(_need(self.norm, "eps", "norm")) > 0:
            raise ConfigError("norm.eps must be positive")
        float(self.residual_mult)
        if self.streams is not None:
            _positive_int(self.streams, "streams")
        if not isinstance(self.layers, (list, tuple)) or not self.layers:
            raise ConfigError("layers must be a non-empty list")
        for i, layer in enumerate(self.layers):
            kind = _need(layer, "type", f"layers[{i}]")
            if kind not in ("parallel", "mlstm"):
                raise ConfigError(f"layers[{i}].type {kind!r} is not one of parallel, mlstm")
            if not isinstance(_need(layer, "mixer", f"layers[{i}]"), dict):
                raise ConfigError(f"layers[{i}].mixer must be a mapping")
            mlp = layer.get("mlp")
            if mlp is not None and _need(mlp, "kind", f"layers[{i}].mlp") != "moe":
                raise ConfigError(f"layers[{i}].mlp.kind {mlp['kind']!r} is not moe")
        self.model_spec()        # every key the layers need, now rather than at the first step

    # -- the order of the layers ----------------------------------------------------------
    def order(self) -> list[int]:
        """The layers in the order of their runs."""
        n = len(self.layers)
        if self.loop is None:
            return list(range(n))
        start, stop = _need(self.loop, "start", "loop"), _need(self.loop, "stop", "loop")
        times = _positive_int(_need(self.loop, "times", "loop"), "loop.times")
        if not all(isinstance(v, int) and not isinstance(v, bool) for v in (start, stop)) or not 0 <= start <= stop <= n:
            raise ConfigError(f"loop.start {start!r} and loop.stop {stop!r} do not bound a run of the {n} layers")
        return list(range(start)) + list(range(start, stop)) * times + list(range(stop, n))

    # -- the mixers as parts ------------------------------------------------------------
    def _attention(self, m, where: str, factor: float) -> PartSpec:
        need = lambda key: _positive_int(_need(m, key, where), f"{where}.{key}")  # noqa: E731
        heads, kv_heads = need("heads"), need("kv_heads")
        if heads % kv_heads:
            raise ConfigError(f"{where}: {heads} heads are not a multiple of {kv_heads} kv_heads")
        mask = m.get("mask")
        window = _positive_int(_need(mask, "size", where + ".mask"), where + ".mask.size") if mask else None
        return PartSpec("sink_attention", {
            "hidden_size": self.width, "num_heads": heads, "num_kv_heads": kv_heads, "head_dim": need("dim"),
            "value_dim": need("vdim"), "scale": float(_need(m, "scale", where)), "position": PartSpec("no_position", {}),
            "window": window, "sink": None, "bias": True, "out_scale": factor})

    def _state_space(self, m, where: str, factor: float) -> PartSpec:
        need = lambda key: _positive_int(_need(m, key, where), f"{where}.{key}")  # noqa: E731
        heads, groups, vdim, parts = need("heads"), need("groups"), need("vdim"), need("norm_groups")
        if heads % groups:
            raise ConfigError(f"{where}: {heads} heads are not a multiple of {groups} groups")
        if heads * vdim % parts:
            raise ConfigError(f"{where}: {heads * vdim} elements do not fall into {parts} norm_groups")
        return PartSpec("state_space", {
            "hidden_size": self.width, "num_heads": heads, "value_dim": vdim, "state_size": need("state"), "groups": groups,
            "taps": need("conv"), "norm_parts": parts, "eps": float(self.norm["eps"]), "out_scale": factor})

    def _mixer(self, i: int, layer) -> PartSpec:
        m, where = layer["mixer"], f"layers[{i}].mixer"
        if layer["type"] == "parallel":
            left, right = _need(m, "left", where), _need(m, "right", where)
            return PartSpec("side_by_side", {"branches": {
                "left": self._attention(left, where + ".left", float(_need(m, "left_scale", where))),
                "right": self._state_space(right, where + ".right", float(_need(m, "right_scale", where)))}})
        need = lambda key: _positive_int(_need(m, key, where), f"{where}.{key}")  # noqa: E731
        cap = float(_need(m, "gate_cap", where))
        if not cap > 0:
            raise ConfigError(f"{where}.gate_cap must be positive, got {cap}")
        return PartSpec("matrix_memory", {
            "hidden_size": self.width, "num_heads": need("heads"), "head_dim": need("dim"), "value_dim": need("vdim"),
            "gate_cap": cap, "eps": float(self.norm["eps"]), "denom_eps": DENOM_EPS})

    def _feed_forward(self, i: int, mlp) -> PartSpec:
        where = f"layers[{i}].mlp"
        router, expert = _need(mlp, "router", where), _need(mlp, "expert", where)
        experts = _positive_int(_need(router, "experts", where + ".router"), where + ".router.experts")
        top = _positive_int(_need(router, "top", where + ".router"), where + ".router.top")
        identity = router.get("identity") or 0
        if not isinstance(identity, int) or isinstance(identity, bool) or identity < 0:
            raise ConfigError(f"{where}.router.identity must be a number of experts, got {identity!r}")
        routed = experts + identity
        groups = router.get("groups")
        if groups is not None:
            count = _positive_int(_need(groups, "count", where + ".router.groups"), where + ".router.groups.count")
            keep = _positive_int(_need(groups, "keep", where + ".router.groups"), where + ".router.groups.keep")
            if routed % count or keep > count:
                raise ConfigError(f"{where}.router.groups: {routed} experts do not fall into {count} groups of which {keep} are kept")
            groups = {"count": count, "keep": keep}
        most = routed if groups is None else groups["keep"] * (routed // groups["count"])
        if top > most:
            raise ConfigError(f"{where}.router.top {top} exceeds the {most} experts that can be chosen")
        shared = mlp.get("shared")
        shared_spec = None
        if shared is not None:
            shared_spec = PartSpec("gated_mlp", {
                "hidden_size": self.width, "activation": "silu",
                "intermediate_size": _positive_int(_need(shared, "ff", where + ".shared"), where + ".shared.ff"),
                "gate_name": "gate", "up_name": "up", "down_name": "down"})
        return PartSpec("routed_experts", {
            "hidden_size": self.width,
            "intermediate_size": _positive_int(_need(expert, "ff", where + ".expert"), where + ".expert.ff"),
            "experts": experts, "top": top, "limit": None, "alpha": 1.0, "shared": shared_spec, "score": "softmax_all",
            "router_bias": False, "groups": groups, "identity": identity})

    def model_spec(self) -> ModelSpec:
        width, eps = self.width, float(self.norm["eps"])
        copies = 1 if self.streams is None else int(self.streams)
        arrangement = PartSpec("hyper_connections", {
            "mixer_prefix": "mix", "feed_forward_prefix": "mlp", "mixer_norm_name": "norm1", "feed_forward_norm_name": "norm2",
            "copies": copies, "learned": self.streams is not None, "residual_mult": float(self.residual_mult),
            "mixer_streams_prefix": "hc1", "feed_forward_streams_prefix": "hc2"})
        norm = lambda name, **more: PartSpec("layernorm", dict(size=width, eps=eps, name=name, bias=True, **more))  # noqa: E731
        layers = []
        for i, layer in enumerate(self.layers):
            mlp = layer.get("mlp")
            layers.append(LayerSpec(
                prefix=f"l{i}", arrangement=arrangement, mixer=self._mixer(i, layer),
                feed_forward=None if mlp is None else self._feed_forward(i, mlp),
                mixer_norm=norm(f"l{i}.norm1"), feed_forward_norm=norm(f"l{i}.norm2", optional=mlp is None)))
        schedule, unit = [], 0
        for i in self.order():            # every run of a layer has cache units of its own
            two = self.layers[i]["type"] == "parallel"
            schedule.append(ScheduleEntry(layer=i, cache=unit, further=(unit + 1,) if two else ()))
            unit += 2 if two else 1
        return ModelSpec(
            hidden_size=width, vocab_size=self.vocab,
            embedding=PartSpec("token_embedding", {"name": "embed", "vocab_size": self.vocab, "hidden_size": width, "copies": copies}),
            layers=tuple(layers), schedule=tuple(schedule), final_norm=norm("final.norm", copies=copies),
            head=PartSpec("linear_head", {"name": "head", "tied_to": None, "vocab_size": self.vocab, "hidden_size": width}),
            max_positions=None, residual_copies=copies)
