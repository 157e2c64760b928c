"""Mixers that keep a matrix a head whose gates are one number a head and token, and the part that runs
several mixers side by side.

    S_t = a_t S_(t-1) + b_t k_t v_t^T        S [rows, vdim] in float32, zero at the start
    o_t = S_t^T q_t

``state_space``     Mamba-2's recurrence: ``a = exp(-exp(A_log) dt)``, ``b = dt``; k, v and q pass a short convolution
``matrix_memory``   xLSTM's matrix memory: exponential gates under a running maximum, and a normaliser

Both walk a few tokens one by one and take longer portions in chunks (csrc/memory.hip); a step of single
tokens is one launch.  Everything between the products is computed in 32-bit; the state lives in the cache
manager's state slots.
"""

from __future__ import annotations

from dataclasses import replace

import numpy as np
import torch

from ..config.base import PartSpec
from ..ops import STORE_F32
from .base import ProjectedMixer, StateSpec, WeightSpec, build_part, part_class, project_out, register_part, stack_rows

#: portions of at most this many tokens walk token by token, longer ones go by chunks
WALK_TOKENS = int(__import__("os").environ.get("LOCKSTEP_MEMORY_WALK_TOKENS", "16"))


class _Memory(ProjectedMixer):
    """What both memories share: the step's work list, the order of the launches."""

    graph_safe = True
    norm = False             # whether the memory keeps a normaliser

    def __init__(self, spec: PartSpec, prefix: str = ""):
        super().__init__(spec, prefix)
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.heads, self.dv = int(p["num_heads"]), int(p["value_dim"])
        self.eps = float(p["eps"])
        self.out_scale = 1.0 if p.get("out_scale") is None else float(p["out_scale"])
        self.out_width = self.heads * self.dv
        self.w_in = self.w_o = self.norm_weight = None

    #: rows of a head's state
    rows = 0

    def _check(self, rt) -> None:
        most = rt.kernels.memory_max_rows()
        if self.rows > most:
            raise ValueError(f"a state of {self.rows} rows a head is not supported: the memory kernels take up to {most}")

    def mixing_flops(self, tokens: int, start: int) -> float:
        """Decay, write and read of every state element per token."""
        return 5.0 * self.heads * self.rows * self.dv * tokens

    def out_matrix(self, weights):
        return weights.get(f"{self.prefix}.o")

    def load(self, weights, rt) -> None:
        self.w_in = rt.matrix(stack_rows(self.in_matrices(weights)))
        self.w_o = rt.matrix(self.out_matrix(weights))
        self.load_own(weights, rt)

    def load_own(self, weights, rt) -> None:
        self._check(rt)
        self.norm_weight = rt.vector(weights.get(f"{self.prefix}.norm"))
        if self.out_scale != 1.0:
            self.norm_weight = self.norm_weight * self.out_scale
        rt.kernels.mixers_lib()

    def prepare_group(self):
        return ("memory", "work")

    def prepare(self, ctx) -> None:
        """The chunks of the step's longer portions: (request of the step, chunk) each, and per such request (request, first
        chunk in the list, chunks, 0).  All memories share them."""
        key = ("memory", "work")
        if ctx.single_tokens or key in ctx.notes:
            return
        chunk = ctx.rt.kernels.memory_chunk()
        longer = np.flatnonzero(ctx.q_len > WALK_TOKENS)
        counts = -(-ctx.q_len[longer] // chunk)
        first = np.cumsum(counts) - counts
        seq = np.repeat(longer, counts)
        items = np.stack([seq, np.arange(len(seq)) - np.repeat(first, counts)], axis=1)
        runs = np.stack([longer, first, counts, np.zeros_like(longer)], axis=1)
        ctx.notes[key] = (len(items), len(runs), len(longer) < ctx.n_seqs)
        if len(items):
            ctx.declare(key, np.concatenate([items.reshape(-1), runs.reshape(-1)]), signature=("memory", len(items)))

    def _memory(self, ctx, q, k, v, gates, q_scale, skip, state, out) -> None:
        """The memory over a step that is not one of single tokens."""
        key = ("memory", "work")
        n_items, n_runs, walks = ctx.notes[key]
        items = runs = states = decays = None
        floats = self.heads * self.rows * (self.dv + (1 if self.norm else 0))
        if n_items:
            work = ctx.block(key)
            items, runs = work[:2 * n_items], work[2 * n_items:]
            states = ctx.buf("memory.states", (n_items, floats), torch.float32)
            decays = ctx.buf("memory.decays", (n_items * self.heads,), torch.float32)
        ctx.rt.kernels.memory(q, k, v, gates, self.heads, self.rows, self.dv, q_scale, skip, self.norm, ctx.seqs, ctx.n_seqs,
                              WALK_TOKENS, walks, items, n_items, runs, n_runs, states, decays, state, out)

    def forward(self, ctx, run, x, out, accumulate: bool, defer: bool = False):
        rt = ctx.rt
        raw = ctx.buf("memory.in_f32", (ctx.n_tokens, self.w_in.shape[0]), torch.float32)
        rt.kernels.gemm(x, self.w_in, raw, STORE_F32)
        mixed = ctx.buf("memory.mixed", (ctx.n_tokens, self.out_width), rt.dtype)
        self.mix(ctx, run, raw, mixed)
        return project_out(ctx, mixed, self.w_o, out, accumulate, defer, "memory.out_slices")


@register_part("state_space")
class StateSpace(_Memory):
    """The state-space mixer of Mamba-2.  ``W_in h`` is laid out ``z (heads*vdim) | x (heads*vdim) | B (groups*state) | C
    (groups*state) | dt (heads)``; ``x``, ``B`` and ``C`` pass a causal convolution a channel (``conv [channels, taps]``, the last
    column is the current token's; bias ``conv.b``; zeros before the start) and SiLU; ``dt <- softplus(dt + dt_bias)``.  Head ``n``
    (``B`` and ``C`` of group ``n // (heads / groups)``): ``S <- exp(-exp(A_log) dt) S + dt B x^T``, ``y = S^T C + D x``.  ``y silu(z)`` is
    divided by its root mean square in ``norm_parts`` equal parts (``eps``), times ``norm``; then ``W_o``.

    Parameters: ``hidden_size``, ``num_heads``, ``value_dim``, ``state_size``, ``groups``, ``taps``, ``norm_parts``, ``eps``, ``out_scale``.
    Tensors below the prefix: ``in``, ``conv``, ``conv.b``, ``dt_bias``, ``A_log``, ``D`` (``[heads]`` each), ``norm [heads*vdim]``, ``o``.

    A request's state slot holds the matrices and, behind them, the convolution's last inputs: the input at position ``p`` in
    row ``p mod taps`` of a ring, so that a decoded token's input goes where no one of its step reads."""

    def __init__(self, spec: PartSpec, prefix: str = ""):
        super().__init__(spec, prefix)
        p = spec.params
        self.rows, self.groups, self.taps = int(p["state_size"]), int(p["groups"]), int(p["taps"])
        self.parts_of_norm = int(p["norm_parts"])
        self.inner = self.heads * self.dv
        if min(self.heads, self.dv, self.rows, self.groups, self.taps, self.parts_of_norm) <= 0 or self.heads % self.groups \
                or self.inner % self.parts_of_norm:
            raise ValueError(f"{self.heads} heads over {self.groups} groups with sizes {self.rows}, {self.dv}, {self.taps} taps and "
                             f"{self.parts_of_norm} parts are not a state-space mixer")
        self.channels = self.inner + 2 * self.groups * self.rows
        self.ring_at = self.heads * self.rows * self.dv
        self.conv = self.conv_bias = self.dt_bias = self.a_log = self.skip = None

    @classmethod
    def weight_specs(cls, spec: PartSpec, prefix: str) -> list[WeightSpec]:
        p = spec.params
        h, n, dv, s, g, m = (int(p[key]) for key in ("hidden_size", "num_heads", "value_dim", "state_size", "groups", "taps"))
        inner, channels = n * dv, n * dv + 2 * g * s
        return [WeightSpec(f"{prefix}.in", (inner + channels + n, h)),
                WeightSpec(f"{prefix}.conv", (channels, m), kind="vector", init="unit"),
                WeightSpec(f"{prefix}.conv.b", (channels,), kind="vector"), WeightSpec(f"{prefix}.dt_bias", (n,), kind="vector"),
                WeightSpec(f"{prefix}.A_log", (n,), kind="vector"), WeightSpec(f"{prefix}.D", (n,), kind="vector", init="unit"),
                WeightSpec(f"{prefix}.norm", (inner,), kind="vector", init="norm"), WeightSpec(f"{prefix}.o", (h, inner))]

    def cache_spec(self):
        floats = self.ring_at + self.taps * self.channels
        return StateSpec((-(-floats // 4) * 4,), "float32")

    def in_matrices(self, weights) -> list:
        return [weights.get(f"{self.prefix}.in")]

    def load_own(self, weights, rt) -> None:
        super().load_own(weights, rt)
        get = lambda name: weights.get(f"{self.prefix}.{name}")  # noqa: E731
        self.conv = rt.vector(get("conv").t().contiguous())         # [taps, channels]
        self.conv_bias, self.dt_bias = rt.vector(get("conv.b")), rt.vector(get("dt_bias"))
        self.a_log, self.skip = rt.vector(get("A_log")), rt.vector(get("D"))

    def mix(self, ctx, run, raw, out) -> None:
        k, t, n = ctx.rt.kernels, ctx.n_tokens, self.heads
        x_at, dt_at = self.inner, self.inner + self.channels
        state = ctx.cache.unit_state(run.cache)
        y = ctx.buf("memory.y", (t, self.inner), torch.float32)
        if ctx.single_tokens:
            k.space_token(raw, x_at, dt_at, self.groups, self.conv, self.conv_bias, self.a_log, self.dt_bias, self.skip, n, self.rows,
                          self.dv, ctx.seqs, ctx.n_seqs, state, self.ring_at, y)
        else:
            conv = ctx.buf("memory.conv", (t, self.channels), torch.float32)
            gates = ctx.buf("memory.gates", (t * n * k.GATE_FLOATS,), torch.float32)
            k.conv_gates(raw, x_at, dt_at, self.channels, n, self.conv, self.conv_bias, self.a_log, self.dt_bias, ctx.tok_seq,
                         ctx.tok_pos, ctx.seqs, ctx.n_seqs, state, self.ring_at, conv, gates)
            share, b_at = n // self.groups, self.inner
            self._memory(ctx, (conv, b_at + self.groups * self.rows, share), (conv, b_at, share), (conv, 0, 1), gates, 1.0, self.skip,
                         state, y)
        k.gated_parts_norm(y, raw[:, :self.inner], self.parts_of_norm, self.norm_weight, self.eps, out)


@register_part("matrix_memory")
class MatrixMemory(_Memory):
    """The matrix memory of xLSTM (mLSTM).  ``q = W_q h * head_dim^-1/2`` and ``k = W_k h`` (heads of ``head_dim``), ``v = W_v h`` (heads
    of ``value_dim``); per head a log input gate ``i = cap tanh((W_i h + i.b) / cap)`` and a log forget gate ``f = logsigmoid(cap
    tanh((W_f h + f.b) / cap))`` with ``cap = gate_cap``.  With a running maximum ``m`` from zero, ``m' = max(f + m, i)``:

        S <- exp(f + m - m') S + exp(i - m') k v^T;   n likewise with k alone
        o = S^T q / (max(|n . q|, exp(-m')) + denom_eps)

    Each head's ``o`` is divided by its root mean square (``eps``), times ``norm [heads*value_dim]`` and ``sigmoid(W_g h)``; then ``W_o``.

    Parameters: ``hidden_size``, ``num_heads``, ``head_dim``, ``value_dim``, ``gate_cap``, ``eps``, ``denom_eps``, ``out_scale``.  Tensors below
    the prefix: ``q``, ``k``, ``v``, ``g``, ``i``, ``i.b``, ``f``, ``f.b``, ``norm``, ``o``.  A request's state slot holds ``S``, ``n`` and, in two places a
    head of which the length's parity says the current one, the maximum, as the sum of two numbers (a slow forget gate is far
    below the maximum's last place in float32)."""

    norm = True

    def __init__(self, spec: PartSpec, prefix: str = ""):
        super().__init__(spec, prefix)
        p = spec.params
        self.rows, self.cap, self.denom_eps = int(p["head_dim"]), float(p["gate_cap"]), float(p["denom_eps"])
        if min(self.heads, self.dv, self.rows) <= 0 or not self.cap > 0:
            raise ValueError("heads, sizes and the gates' cap of a matrix memory must be positive")
        self.max_at = self.heads * self.rows * (self.dv + 1)
        self.i_bias = self.f_bias = None

    @classmethod
    def weight_specs(cls, spec: PartSpec, prefix: str) -> list[WeightSpec]:
        p = spec.params
        h, n, d, dv = (int(p[key]) for key in ("hidden_size", "num_heads", "head_dim", "value_dim"))
        return [WeightSpec(f"{prefix}.q", (n * d, h)), WeightSpec(f"{prefix}.k", (n * d, h)), WeightSpec(f"{prefix}.v", (n * dv, h)),
                WeightSpec(f"{prefix}.g", (n * dv, h)), WeightSpec(f"{prefix}.i", (n, h)), WeightSpec(f"{prefix}.i.b", (n,), kind="vector"),
                WeightSpec(f"{prefix}.f", (n, h)), WeightSpec(f"{prefix}.f.b", (n,), kind="vector"),
                WeightSpec(f"{prefix}.norm", (n * dv,), kind="vector", init="norm"), WeightSpec(f"{prefix}.o", (h, n * dv))]

    def cache_spec(self):
        return StateSpec((-(-(self.max_at + 4 * self.heads) // 4) * 4,), "float32")

    def in_matrices(self, weights) -> list:
        return [weights.get(f"{self.prefix}.{n}") for n in "qkvgif"]

    def load_own(self, weights, rt) -> None:
        super().load_own(weights, rt)
        self.i_bias = rt.vector(weights.get(f"{self.prefix}.i.b"))
        self.f_bias = rt.vector(weights.get(f"{self.prefix}.f.b"))

    def mix(self, ctx, run, raw, out) -> None:
        k, t, n, d, dv = ctx.rt.kernels, ctx.n_tokens, self.heads, self.rows, self.dv
        k_at, v_at = n * d, 2 * n * d
        g_at, i_at = v_at + n * dv, v_at + 2 * n * dv
        f_at = i_at + n
        state = ctx.cache.unit_state(run.cache)
        scale = d ** -0.5
        if ctx.single_tokens and dv <= k.exp_token_whole():           # the head's norm and gate in the same launch
            k.exp_token(raw, 0, k_at, v_at, i_at, f_at, self.i_bias, self.f_bias, self.cap, scale, n, d, dv, ctx.seqs, ctx.n_seqs, state,
                        self.max_at, None, out, normed=(self.norm_weight, g_at, self.eps, self.denom_eps))
            return
        o = ctx.buf("memory.y", (t, n * dv), torch.float32)
        gates = ctx.buf("memory.gates", (t * n * k.GATE_FLOATS,), torch.float32)
        if ctx.single_tokens:
            k.exp_token(raw, 0, k_at, v_at, i_at, f_at, self.i_bias, self.f_bias, self.cap, scale, n, d, dv, ctx.seqs, ctx.n_seqs, state,
                        self.max_at, gates, o)
        else:
            k.exp_gates(raw, i_at, f_at, n, self.i_bias, self.f_bias, self.cap, ctx.seqs, ctx.n_seqs, state, self.max_at, gates)
            self._memory(ctx, (raw, 0, 1), (raw, k_at, 1), (raw, v_at, 1), gates, scale, None, state, o)
        k.head_norm_gate(o, n, dv, self.norm_weight, raw[:, g_at:g_at + n * dv], self.eps, out, gate_act="sigmoid", denom=gates,
                         denom_eps=self.denom_eps)


@register_part("side_by_side")
class SideBySide(ProjectedMixer):
    """Several mixers that read the same input and whose outputs are added: ``sum_b branch_b(x)``.  Every branch is a
    ``ProjectedMixer``, so both products are one: the branches' input matrices one below the other, their output matrices side by
    side, each branch mixing its own columns (a branch's weight in the sum is its ``out_scale``).

    Parameters: ``branches``, a mapping from names to the branches' ``PartSpec``s; a branch's tensors stand below
    ``<prefix>.<name>``.  The first branch's cache unit is the schedule entry's ``cache``, the others' are its ``further`` ones."""

    graph_safe = True

    def __init__(self, spec: PartSpec, prefix: str = ""):
        super().__init__(spec, prefix)
        self.branches = [build_part(s, self.join(prefix, name)) for name, s in spec["branches"].items()]
        for branch in self.branches:
            if not isinstance(branch, ProjectedMixer) or getattr(branch, "out_bias", False):
                raise ValueError(f"{branch.kind!r} cannot be a branch: its input and output are not one product each")
        self.out_width = sum(b.out_width for b in self.branches)
        self.w_in = self.w_o = None
        self.in_widths: list[int] = []
        self._runs: dict = {}

    def parts(self):
        return tuple(self.branches)

    @classmethod
    def weight_specs(cls, spec: PartSpec, prefix: str) -> list[WeightSpec]:
        return [w for name, s in spec["branches"].items() for w in part_class(s.kind).weight_specs(s, cls.join(prefix, name))]

    def cache_spec(self):
        return self.branches[0].cache_spec()

    def further_specs(self) -> tuple:
        return tuple(b.cache_spec() for b in self.branches[1:])

    def mixing_flops(self, tokens: int, start: int) -> float:
        return sum(b.mixing_flops(tokens, start) for b in self.branches)

    def prepare_group(self):
        groups = tuple(b.prepare_group() for b in self.branches)
        return None if None in groups else ("side_by_side", *groups)

    def prepare(self, ctx) -> None:
        for branch in self.branches:
            branch.prepare(ctx)

    def in_matrices(self, weights) -> list:
        return [m for b in self.branches for m in b.in_matrices(weights)]

    def load(self, weights, rt) -> None:
        per_branch = [b.in_matrices(weights) for b in self.branches]
        self.in_widths = [sum(m.shape[0] for m in mats) for mats in per_branch]
        self.w_in = rt.matrix(stack_rows([m for mats in per_branch for m in mats]))
        self.w_o = rt.matrix(stack_rows([b.out_matrix(weights).t() for b in self.branches]).t().contiguous())
        for branch in self.branches:
            branch.load_own(weights, rt)

    def _branch_runs(self, run) -> list:
        """The schedule entry as every branch sees it: its own cache unit."""
        held = self._runs.get(run)
        if held is None:
            units = (run.cache, *run.further)
            held = self._runs[run] = [replace(run, cache=unit, further=()) for unit in units]
        return held

    def mix(self, ctx, run, raw, out) -> None:
        row = column = 0
        for branch, width, own in zip(self.branches, self.in_widths, self._branch_runs(run)):
            branch.mix(ctx, own, raw[:, row:row + width], out[:, column:column + branch.out_width])
            row += width
            column += branch.out_width

    def forward(self, ctx, run, x, out, accumulate: bool, defer: bool = False):
        rt = ctx.rt
        raw = ctx.buf("side.in_f32", (ctx.n_tokens, self.w_in.shape[0]), torch.float32)
        rt.kernels.gemm(x, self.w_in, raw, STORE_F32)
        mixed = ctx.buf("side.mixed", (ctx.n_tokens, self.out_width), rt.dtype)
        self.mix(ctx, run, raw, mixed)
        return project_out(ctx, mixed, self.w_o, out, accumulate, defer, "side.out_slices")
