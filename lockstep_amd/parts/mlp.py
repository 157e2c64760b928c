"""Gated feed-forward: ``down(act(gate(x)) * up(x))``, with biases if asked for; with the
SiLU activation and without biases this is the reference's SwiGLU MLP
(engine/model/qwen3.py:368-370, engine/kernels/swiglu.py:25-29).  Gate and up
are one matrix product over their rows interleaved in tiles of 16, whose
epilogue applies the activation, so the two projections never leave the
kernel."""

from __future__ import annotations

import math

import torch

from ..config.base import PartSpec
from ..ops import ADD_F32, STORE_F32, SWIGLU, interleave_gate_up
from .base import FeedForward, PendingAdd, WeightSpec, deferred_rows, register_part


@register_part("gated_mlp")
class GatedMLP(FeedForward):
    """Parameters: ``hidden_size``, ``intermediate_size``, ``activation`` (``silu``, ``gelu``,
    ``gelu_tanh``, ``relu``), ``bias`` (optional, default False: ``gate_proj.bias``, ``up_proj.bias``
    and ``down_proj.bias``), and optionally the tensor names below the prefix, ``gate_name``,
    ``up_name``, ``down_name`` (default ``gate_proj.weight`` and so on; biases then ``<name>.b``).

    SiLU without biases is the fast path (the activation is the product's epilogue).  Anything else
    stores the gate/up product in float32 and applies biases and activation in a pass of its own,
    and adds the down projection to the residual stream at once rather than leaving it to the next
    norm, so that the order of the additions (stream + product, then + bias) is the same at every
    batch size."""

    graph_safe = True
    repeatable = True

    def __init__(self, spec: PartSpec, prefix: str = ""):
        super().__init__(spec, prefix)
        self.hidden = int(spec["hidden_size"])
        self.inter = int(spec["intermediate_size"])
        self.activation = str(spec["activation"])
        self.bias = bool(spec.params.get("bias", False))
        if self.activation not in ("silu", "gelu", "gelu_tanh", "relu"):
            raise ValueError(f"activation {self.activation!r} is not built; known: silu, gelu, gelu_tanh, relu")
        self.fused = self.activation == "silu" and not self.bias
        self.w_gate_up = self.w_down = self.b_gate_up = self.b_down = None

    @classmethod
    def names(cls, spec: PartSpec, prefix: str):
        """(weight, bias) tensor names of gate, up and down."""
        out = []
        for key, default in (("gate_name", "gate_proj"), ("up_name", "up_proj"), ("down_name", "down_proj")):
            given = spec.params.get(key)
            out.append((f"{prefix}.{given}", f"{prefix}.{given}.b") if given else
                       (f"{prefix}.{default}.weight", f"{prefix}.{default}.bias"))
        return out

    @classmethod
    def weight_specs(cls, spec: PartSpec, prefix: str) -> list[WeightSpec]:
        h, i = int(spec["hidden_size"]), int(spec["intermediate_size"])
        (gate, gate_b), (up, up_b), (down, down_b) = cls.names(spec, prefix)
        out = [WeightSpec(gate, (i, h)), WeightSpec(up, (i, h)), WeightSpec(down, (h, i))]
        if spec.params.get("bias", False):
            out += [WeightSpec(gate_b, (i,), kind="vector"), WeightSpec(up_b, (i,), kind="vector"),
                    WeightSpec(down_b, (h,), kind="vector")]
        return out

    def load(self, weights, rt) -> None:
        (gate_name, gate_b), (up_name, up_b), (down_name, down_b) = self.names(self.spec, self.prefix)
        gate = weights.get(gate_name)
        up = weights.get(up_name)
        if gate.dtype != up.dtype:
            gate, up = gate.to(torch.float32), up.to(torch.float32)
        self.w_gate_up = rt.matrix(interleave_gate_up(gate, up) if self.fused else torch.cat([gate, up], dim=0))
        self.w_down = rt.matrix(weights.get(down_name))
        if self.bias:
            self.b_gate_up = rt.vector(torch.cat([weights.get(gate_b).to(torch.float32), weights.get(up_b).to(torch.float32)]))
            self.b_down = rt.vector(weights.get(down_b))

    def forward(self, ctx, x, out, accumulate: bool, norm=None, defer: bool = False):
        """``norm``: when given, ``x`` is the float32 residual stream and ``norm``
        (an RMSNorm part) is applied inside the first matrix product.  ``defer``: the
        addition to ``out`` may be left to the caller (a ``PendingAdd`` is returned)."""
        rt = ctx.rt
        k = rt.kernels
        act = ctx.buf("mlp.act", (ctx.n_tokens, self.inter), rt.dtype)
        fused_norm = {} if norm is None else {"norm_weight": norm.weight, "eps": norm.eps}
        if not self.fused:
            wide = ctx.buf("mlp.gate_up", (ctx.n_tokens, 2 * self.inter), torch.float32)
            k.gemm(x, self.w_gate_up, wide, STORE_F32, **fused_norm)
            k.bias_act(wide, self.b_gate_up, act, self.activation, gated=True)
            k.gemm(act, self.w_down, out, ADD_F32 if accumulate else STORE_F32)
            if self.b_down is not None:
                k.bias_act(out, self.b_down, out)
            return None
        k.gemm(x, self.w_gate_up, act, SWIGLU, **fused_norm)
        if defer and accumulate and 0 < ctx.n_tokens <= deferred_rows(ctx, self.inter, out.shape[1]):
            slices = k.gemm_slices_count(self.inter)
            partials = ctx.buf("mlp.down_slices", (slices * ctx.n_tokens, out.shape[1]), torch.float32)
            partials = partials.view(slices, ctx.n_tokens, out.shape[1])
            k.gemm_slices(act, self.w_down, partials)
            return PendingAdd(partials)
        k.gemm(act, self.w_down, out, ADD_F32 if accumulate else STORE_F32)
        return None


@register_part("mlp")
class MLP(FeedForward):
    """``down(act(up(x)))``: a feed-forward of two matrices.  Parameters: ``hidden_size``, ``intermediate_size``,
    ``activation`` (``xielu``, or ``silu``, ``gelu``, ``gelu_tanh``, ``relu``), and optionally the tensor names below the
    prefix ``up_name``, ``down_name`` (default ``up``, ``down``) and, for ``xielu``, ``act_name`` (default ``act``).

    ``xielu`` has two learned numbers (p, q): ``softplus(p) z^2 + z/2`` above zero, ``(1/2 + softplus(q)) (e^z - 1 - z) +
    z/2`` elsewhere.  It is the up product's epilogue; the softplus of both numbers is taken once, at load.  The other
    activations store the up product in float32 and run as a pass of their own."""

    graph_safe = True
    repeatable = True

    def __init__(self, spec: PartSpec, prefix: str = ""):
        super().__init__(spec, prefix)
        self.hidden = int(spec["hidden_size"])
        self.inter = int(spec["intermediate_size"])
        self.activation = str(spec["activation"])
        if self.activation not in ("xielu", "silu", "gelu", "gelu_tanh", "relu"):
            raise ValueError(f"activation {self.activation!r} is not built; known: xielu, silu, gelu, gelu_tanh, relu")
        self.w_up = self.w_down = self.factors = None

    @classmethod
    def names(cls, spec: PartSpec, prefix: str):
        return tuple(f"{prefix}.{spec.params.get(key, default)}" for key, default in
                     (("up_name", "up"), ("down_name", "down"), ("act_name", "act")))

    @classmethod
    def weight_specs(cls, spec: PartSpec, prefix: str) -> list[WeightSpec]:
        h, i = int(spec["hidden_size"]), int(spec["intermediate_size"])
        up, down, act = cls.names(spec, prefix)
        out = [WeightSpec(up, (i, h)), WeightSpec(down, (h, i))]
        if spec["activation"] == "xielu":
            out.append(WeightSpec(act, (2,), kind="vector"))
        return out

    def load(self, weights, rt) -> None:
        up, down, act = self.names(self.spec, self.prefix)
        self.w_up = rt.matrix(weights.get(up))
        self.w_down = rt.matrix(weights.get(down))
        if self.activation == "xielu":
            p, q = weights.get(act).to(torch.float64).reshape(2).tolist()
            softplus = [max(v, 0.0) + math.log1p(math.exp(-abs(v))) for v in (p, q)]
            self.factors = rt.vector(torch.tensor([softplus[0], 0.5 + softplus[1]], dtype=torch.float64))

    def forward(self, ctx, x, out, accumulate: bool, defer: bool = False):
        from .base import project_out

        rt = ctx.rt
        k = rt.kernels
        act = ctx.buf("mlp.act", (ctx.n_tokens, self.inter), rt.dtype)
        if self.activation == "xielu":
            k.gemm_xielu(x, self.w_up, act, self.factors)
        else:
            wide = ctx.buf("mlp.up", (ctx.n_tokens, self.inter), torch.float32)
            k.gemm(x, self.w_up, wide, STORE_F32)
            k.bias_act(wide, None, act, self.activation)
        return project_out(ctx, act, self.w_down, out, accumulate, defer, "mlp.down_slices")


@register_part("clamped_gated_mlp")
class ClampedGatedMLP(FeedForward):
    """``down(g * sigmoid(alpha * g) * (u + 1))`` with ``g = min(gate(x), limit)`` and ``u = clamp(up(x),
    -limit, limit)``: a gated unit whose two branches are bounded before they meet.  Parameters:
    ``hidden_size``, ``intermediate_size``, ``limit``, ``alpha`` (the sigmoid's slope), and the tensor
    names below the prefix ``gate_name``, ``up_name``, ``down_name``.

    Gate and up are one matrix product over their rows one after the other, stored in float32; the
    unit is a pass of its own in 32-bit that rounds to the compute dtype for the down product."""

    graph_safe = True
    repeatable = True

    def __init__(self, spec: PartSpec, prefix: str = ""):
        super().__init__(spec, prefix)
        self.hidden = int(spec["hidden_size"])
        self.inter = int(spec["intermediate_size"])
        self.limit = float(spec["limit"])
        self.alpha = float(spec["alpha"])
        if not self.limit > 0:
            raise ValueError(f"the gated unit's limit must be positive, got {self.limit}")
        self.w_gate_up = self.w_down = None

    @classmethod
    def names(cls, spec: PartSpec, prefix: str):
        p = spec.params
        return tuple(f"{prefix}.{p.get(key, default)}" for key, default in
                     (("gate_name", "gate"), ("up_name", "up"), ("down_name", "down")))

    @classmethod
    def weight_specs(cls, spec: PartSpec, prefix: str) -> list[WeightSpec]:
        h, i = int(spec["hidden_size"]), int(spec["intermediate_size"])
        gate, up, down = cls.names(spec, prefix)
        return [WeightSpec(gate, (i, h)), WeightSpec(up, (i, h)), WeightSpec(down, (h, i))]

    def load(self, weights, rt) -> None:
        gate_name, up_name, down_name = self.names(self.spec, self.prefix)
        gate, up = weights.get(gate_name), weights.get(up_name)
        if gate.dtype != up.dtype:
            gate, up = gate.to(torch.float32), up.to(torch.float32)
        self.w_gate_up = rt.matrix(torch.cat([gate, up], dim=0))
        self.w_down = rt.matrix(weights.get(down_name))

    def forward(self, ctx, x, out, accumulate: bool, defer: bool = False):
        from .base import project_out

        rt = ctx.rt
        k = rt.kernels
        wide = ctx.buf("mlp.gate_up", (ctx.n_tokens, 2 * self.inter), torch.float32)
        k.gemm(x, self.w_gate_up, wide, STORE_F32)
        act = ctx.buf("mlp.act", (ctx.n_tokens, self.inter), rt.dtype)
        k.glu_clamped(wide, act, self.limit, self.alpha)
        return project_out(ctx, act, self.w_down, out, accumulate, defer, "mlp.down_slices")
