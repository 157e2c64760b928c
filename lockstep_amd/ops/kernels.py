"""Python face of the HIP kernels: shape checks on the host, then the launch.

Every wrapper verifies what the kernel and its grid assume (device, dtype,
contiguity of rows, matching sizes) before it launches, because a kernel that
reads out of bounds can take the whole GPU down.  Launches go to torch's
current stream, so they order with torch's own copies and can be captured in
a HIP graph.  There is no fallback path: if the library cannot be loaded the
constructor raises.
"""

from __future__ import annotations

import ctypes
from ctypes import c_float, c_int, c_long, c_void_p

import torch

from . import build as _build

DTYPE_CODE = {torch.float32: 0, torch.bfloat16: 1}
STORE, STORE_F32, ADD_F32, SWIGLU = 0, 1, 2, 3


def interleave_gate_up(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """Rows of ``gate`` and ``up`` (``[I, K]`` each) interleaved in tiles of 16 rows:
    gate rows 0..15, up rows 0..15, gate rows 16..31, ...; the last tile of each is
    padded with zero rows.  This is the weight layout of the SwiGLU epilogue."""
    inter, k = gate.shape
    tiles = -(-inter // 16)
    out = torch.zeros((tiles, 2, 16, k), dtype=gate.dtype)
    pad = tiles * 16 - inter
    g = torch.cat([gate, gate.new_zeros((pad, k))]) if pad else gate
    u = torch.cat([up, up.new_zeros((pad, k))]) if pad else up
    out[:, 0] = g.view(tiles, 16, k)
    out[:, 1] = u.view(tiles, 16, k)
    return out.view(tiles * 32, k)
MAX_HEAD_DIM = 256


class KernelError(RuntimeError):
    pass


def _ptr(t) -> c_void_p:
    return c_void_p(t.data_ptr()) if t is not None else c_void_p(0)


_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)
_raw_device = getattr(torch._C, "_cuda_getDevice", None)


def _stream() -> c_void_p:
    """The current stream of the current device (asked through the raw call where torch has it:
    a kernel launch asks for it every time, and the Python stream object costs ten times as much)."""
    if _raw_stream is not None:
        return c_void_p(_raw_stream(_raw_device() if _raw_device is not None else torch.cuda.current_device()))
    return c_void_p(torch.cuda.current_stream().cuda_stream)


# The checks in front of a launch are plain conditionals whose message is made only when a check
# fails: a step runs some two thousand of them.
def _rows_ok(t: torch.Tensor, name: str) -> None:
    if not (t.is_cuda and t.dim() == 2 and t.stride(1) == 1):
        raise KernelError(f"{name} must be 2-D with contiguous rows on the GPU, got shape {tuple(t.shape)} "
                          f"strides {t.stride()} on {t.device}")


class Kernels:
    """The loaded libraries.  One instance per process (see ``kernels()``)."""

    def __init__(self, mutants: bool = False):
        """``mutants``: load the control libraries instead (built with their deliberately wrong
        variants compiled in, all switched off until ``set_mutants``); the tests' positive
        controls use them, the engine never does."""
        self.mutants = mutants
        self.core_path = _build.build_core_mutants() if mutants else _build.build_core()
        self.core = ctypes.CDLL(str(self.core_path))
        self.core.ls_last_error.restype = ctypes.c_char_p
        self.core.ls_sample_scratch_bytes.restype = ctypes.c_long
        self._attention: dict[int, ctypes.CDLL] = {}
        self.attention_paths: dict[int, str] = {}
        self._mixers = None
        self.mixers_path = None
        self._talking: dict[tuple, ctypes.CDLL] = {}
        self.talking_paths: dict[tuple, str] = {}
        self._sink: dict[tuple, ctypes.CDLL] = {}
        self.sink_paths: dict[tuple, str] = {}
        self._experts = None
        self.experts_path = None
        self._argmax_scratch: dict = {}
        self._sample_scratch: dict = {}
        self._sample_scratch_kept: list = []
        self._capabilities: dict = {}
        #: while this is a list, every launch is noted on it as (library, entry point, arguments):
        #: the engine repeats the launches of one layer for the next layers that are alike
        self.tape: list | None = None
        self._listed: dict = {}

    # -- helpers ------------------------------------------------------------
    @staticmethod
    def _check(lib, code: int) -> None:
        if code != 0:
            raise KernelError(lib.ls_last_error().decode())

    def _launch(self, lib, entry, args: tuple) -> None:
        if entry(*args) != 0:
            raise KernelError(lib.ls_last_error().decode())
        if self.tape is not None:
            self.tape.append((lib, entry, args))

    # -- launches handed over as one list ----------------------------------------
    def listed(self, lib, entry):
        """(address of the library's ``ls_call_listed``, the entry point's index there) for an entry point
        that ``run_list`` may name, or None."""
        key = (id(lib), entry.__name__)
        found = self._listed.get(key, False)
        if found is False:
            found = None
            if hasattr(lib, "ls_listed_index"):
                index = lib.ls_listed_index(entry.__name__.encode())
                if index >= 0:
                    found = (ctypes.cast(lib.ls_call_listed, c_void_p).value, index, lib)
            self._listed[key] = found
        return found

    def run_list(self, words, libs=(), period: int = 0) -> None:
        """Make the calls that ``words`` (a contiguous int64 array of records, see ``ls_run_list`` in
        csrc/core_api.h) lists, in order.  ``libs``: (word offset of a record, its library) pairs, for the
        message of a call that fails; with ``period`` the offsets repeat with that many words."""
        failed_at = ctypes.c_long(-1)
        code = self.core.ls_run_list(c_void_p(words.ctypes.data), c_long(words.size), ctypes.byref(failed_at))
        if code != 0:
            at = failed_at.value % period if period else failed_at.value
            lib = dict(libs).get(at, self.core)
            raise KernelError(lib.ls_last_error().decode())

    def attention_lib(self, head_dim: int):
        lib = self._attention.get(head_dim)
        if lib is None:
            path = _build.build_attention_mutants(head_dim) if self.mutants else _build.build_attention(head_dim)
            lib = ctypes.CDLL(str(path))
            lib.ls_last_error.restype = ctypes.c_char_p
            if not (lib.ls_attn_head_dim() == head_dim):
                raise KernelError(f"{path} was built for another head size")
            if self.mutants and getattr(self, "_attention_mask", 0):
                self._check(lib, lib.ls_set_mutants(c_int(self._attention_mask)))
            self._attention[head_dim] = lib
            self.attention_paths[head_dim] = str(path)
        return lib

    #: bits of ``set_mutants`` (csrc/common.h)
    MUTANT_KSLICE_BY_ROWS, MUTANT_NORM_BY_ROWS, MUTANT_SAMPLE_CHUNKS_BY_ROWS = 1, 2, 4      # core library
    MUTANT_REVERSED_FOLD_IN_PRODUCT = 8
    MUTANT_REVERSED_FOLD = 1                               # attention libraries

    def set_mutants(self, core: int = 0, attention: int = 0) -> None:
        """Switch wrong variants of the control libraries on (bit masks) or off (0)."""
        if not self.mutants:
            raise KernelError("these are the product libraries: they hold no mutants")
        self._check(self.core, self.core.ls_set_mutants(c_int(core)))
        for lib in self._attention.values():
            self._check(lib, lib.ls_set_mutants(c_int(attention)))
        self._attention_mask = attention

    def _memo(self, key, compute):
        """Capability queries do not change while the process runs: ask the library once."""
        have = self._capabilities.get(key)
        if have is None:
            have = self._capabilities[key] = compute()
        return have

    def coop_supported(self, head_dim: int, dtype: torch.dtype, page_size: int = 16) -> bool:
        """Whether the cooperative attention kernel can run (its tiles must fit into LDS)."""
        return self._memo(("coop", head_dim, dtype, page_size), lambda: page_size >= 8 and bool(
            self.attention_lib(head_dim).ls_attn_coop_supported(c_int(DTYPE_CODE[dtype]))))

    def decode_fused_supported(self, head_dim: int, dtype: torch.dtype, page_size: int) -> bool:
        """Whether ``attention_decode`` (norm, rotation and cache write inside the attention kernel) can run."""
        return self._memo(("decode_fused", head_dim, dtype, page_size), lambda: page_size >= 8 and bool(
            self.attention_lib(head_dim).ls_attn_decode_fused_supported(c_int(DTYPE_CODE[dtype]))))

    def compute_units(self) -> int:
        """Compute units of the current device."""
        return self._memo(("compute_units",), lambda: int(
            torch.cuda.get_device_properties(torch.cuda.current_device()).multi_processor_count))

    def wide_supported(self, head_dim: int, dtype: torch.dtype, page_size: int) -> bool:
        """Whether the wide attention kernel (variant 4, for prompt portions) can run."""
        return self._memo(("wide", head_dim, dtype, page_size), lambda: page_size >= 8 and bool(
            self.attention_lib(head_dim).ls_attn_wide_supported(c_int(DTYPE_CODE[dtype]))))

    def attention_block_rows(self, head_dim: int, variant: int) -> int:
        """Rows of the row blocks that work items of this variant count in."""
        return self._memo(("block_rows", head_dim, variant),
                          lambda: int(self.attention_lib(head_dim).ls_attn_block_rows(c_int(variant))))

    def attention_geometry(self, head_dim: int) -> tuple[int, int]:
        """(keys per tile, keys per split) of the attention kernels."""
        return self._memo(("geometry", head_dim), lambda: (self.attention_lib(head_dim).ls_attn_tile_keys(),
                                                           self.attention_lib(head_dim).ls_attn_split_keys()))

    # -- matrix product -------------------------------------------------------
    def gemm(self, x: torch.Tensor, w: torch.Tensor, out: torch.Tensor, epilogue: int = STORE,
             norm_weight: torch.Tensor | None = None, eps: float = 0.0) -> None:
        """``out (+)= x @ w.T``; ``x [M,K]``, ``w [N,K]`` contiguous, ``out [M,N]``.

        ``epilogue=SWIGLU``: ``w`` holds gate and up rows interleaved in tiles of
        16 (see ``interleave_gate_up``) and ``out [M, I]`` gets ``silu(gate) * up``.
        ``norm_weight`` (float32 ``[K]``): ``x`` is the float32 residual stream and is
        RMS-normalised on the fly with this weight and ``eps`` (at most 16 rows)."""
        _rows_ok(x, "gemm x"); _rows_ok(w, "gemm w"); _rows_ok(out, "gemm out")
        if not (w.dtype in DTYPE_CODE):
            raise KernelError(f"gemm weights must be float32 or bfloat16, got {w.dtype}")
        if norm_weight is None:
            if not (x.dtype == w.dtype):
                raise KernelError(f"gemm operands must share a dtype, got {x.dtype} and {w.dtype}")
        else:
            if not (x.dtype == torch.float32 and x.shape[0] <= 16):
                raise KernelError("the fused norm reads at most 16 float32 rows")
            if not (norm_weight.is_cuda and norm_weight.dtype == torch.float32 and norm_weight.is_contiguous()
                  and norm_weight.shape == (x.shape[1],)):
                raise KernelError(f"norm weight must be float32 [{x.shape[1]}]")
        m, k = x.shape
        n = w.shape[0]
        if not (w.shape[1] == k and w.is_contiguous()):
            raise KernelError(f"gemm w must be contiguous [N,{k}], got {tuple(w.shape)}")
        if epilogue == SWIGLU:
            cols = out.shape[1]
            if not (n % 32 == 0 and n // 2 - 16 < cols <= n // 2 and out.shape[0] == m):
                raise KernelError(f"SwiGLU output [{m},{cols}] does not fit {n} interleaved weight rows")
        else:
            cols = n
            if not (tuple(out.shape) == (m, n)):
                raise KernelError(f"gemm out must be [{m},{n}], got {tuple(out.shape)}")
        want = w.dtype if epilogue in (STORE, SWIGLU) else torch.float32
        if not (out.dtype == want):
            raise KernelError(f"gemm out dtype {out.dtype} does not fit epilogue {epilogue}")
        if m == 0:
            return
        self._launch(self.core, self.core.ls_gemm, (
            c_int(DTYPE_CODE[w.dtype]), c_int(epilogue), _ptr(x), _ptr(w), _ptr(out), c_int(m), c_int(n), c_int(k),
            c_long(x.stride(0)), c_long(out.stride(0)), _ptr(norm_weight), c_float(eps), c_int(cols), _stream()))

    def gemm_xielu(self, x: torch.Tensor, w: torch.Tensor, out: torch.Tensor, act: torch.Tensor) -> None:
        """``out = xielu(x @ w.T)`` in the compute dtype, element by element: ``act[0] z^2 + z/2`` above zero, ``act[1]
        (e^z - 1 - z) + z/2`` elsewhere; ``act`` two float32 numbers on the GPU."""
        _rows_ok(x, "gemm_xielu x"); _rows_ok(w, "gemm_xielu w"); _rows_ok(out, "gemm_xielu out")
        m, k = x.shape
        n = w.shape[0]
        if not (w.dtype in DTYPE_CODE and x.dtype == w.dtype == out.dtype and w.is_contiguous() and w.shape[1] == k
                and tuple(out.shape) == (m, n)):
            raise KernelError(f"gemm_xielu: operands {tuple(x.shape)} {x.dtype}, {tuple(w.shape)} {w.dtype} and output "
                              f"{tuple(out.shape)} {out.dtype} do not fit")
        self._f32_vector(act, 2, "gemm_xielu act")
        if m == 0:
            return
        self._launch(self.core, self.core.ls_gemm_xielu, (
            c_int(DTYPE_CODE[w.dtype]), _ptr(x), _ptr(w), _ptr(out), c_int(m), c_int(n), c_int(k), c_long(x.stride(0)),
            c_long(out.stride(0)), _ptr(act), _stream()))

    def gemm_slices_count(self, k: int) -> int:
        """K slices of a product over ``k`` (first dimension of ``gemm_slices``'s output)."""
        return self._memo(("slices", k), lambda: int(self.core.ls_gemm_slices_count(c_int(k))))

    def gemm_slices_max_rows(self, k: int, dtype: torch.dtype) -> int:
        """Most rows ``gemm_slices`` takes for a product over ``k``: 64, or 256 where the kernel that walks
        the column blocks with its rows in registers has an instance for the slice length."""
        return self._memo(("slices_rows", k, dtype),
                          lambda: int(self.core.ls_gemm_slices_max_rows(c_int(DTYPE_CODE[dtype]), c_int(k))))

    def gemm_slices(self, x: torch.Tensor, w: torch.Tensor, partials: torch.Tensor) -> None:
        """Slice sums of ``x @ w.T`` for at most ``gemm_slices_max_rows`` rows: ``partials [slices, M, N]``
        float32, to be added in ascending order by the consumer (``add_rmsnorm``).  The work is cut over K
        as well as over N."""
        _rows_ok(x, "gemm_slices x")
        m, k = x.shape
        n = w.shape[0]
        if not (w.is_cuda and w.dim() == 2 and w.is_contiguous() and w.shape[1] == k and w.dtype == x.dtype
              and w.dtype in DTYPE_CODE):
            raise KernelError("gemm_slices w must be [N, K] contiguous in the dtype of x")
        if not (partials.is_cuda and partials.dtype == torch.float32 and partials.is_contiguous()
              and partials.shape == (self.gemm_slices_count(k), m, n)):
            raise KernelError(f"gemm_slices partials must be float32 [{self.gemm_slices_count(k)}, {m}, {n}]")
        self._launch(self.core, self.core.ls_gemm_slices, (
            c_int(DTYPE_CODE[w.dtype]), _ptr(x), _ptr(w), _ptr(partials), c_int(m), c_int(n), c_int(k),
            c_long(x.stride(0)), _stream()))

    def gemm_slices_folded_ok(self, dtype: torch.dtype, m: int, n: int, k: int, head_dim: int, splits: int) -> bool:
        """Whether ``gemm_slices_folded`` takes a product of these sizes."""
        return self._memo(("slices_folded", dtype, m, n, k, head_dim, splits), lambda: bool(
            self.core.ls_gemm_slices_folded_ok(c_int(DTYPE_CODE[dtype]), c_int(m), c_int(n), c_int(k), c_int(head_dim),
                                               c_int(splits))))

    def gemm_slices_folded(self, part_acc: torch.Tensor, part_ml: torch.Tensor, splits: int, head_dim: int,
                           w: torch.Tensor, partials: torch.Tensor) -> None:
        """``gemm_slices`` for an operand that still lies as the per-split sums of an attention launch over
        single decoded tokens: row ``(m * heads + h) * splits + s`` of ``part_acc [., head_dim]`` and
        ``part_ml [., 2]`` holds split ``s`` of token ``m``, head ``h``.  The kernel folds them (ascending,
        from the empty state, then sum / weight rounded to the compute dtype: what the combine launch
        would write) on its way; ``partials [slices, M, N]`` gets the bits ``gemm_slices`` would leave."""
        slices, m, n = partials.shape
        k = w.shape[1]
        if not (w.is_cuda and w.dim() == 2 and w.is_contiguous() and w.dtype in DTYPE_CODE and w.shape[0] == n):
            raise KernelError("gemm_slices_folded w must be [N, K] contiguous")
        if not (partials.is_cuda and partials.dtype == torch.float32 and partials.is_contiguous()
                and slices == self.gemm_slices_count(k)):
            raise KernelError(f"gemm_slices_folded partials must be float32 [{self.gemm_slices_count(k)}, M, N]")
        if not self.gemm_slices_folded_ok(w.dtype, m, n, k, head_dim, splits):
            raise KernelError(f"gemm_slices_folded does not take M={m} N={n} K={k} head_dim={head_dim} splits={splits}")
        rows = m * (k // head_dim) * splits
        for name, t, width in (("part_acc", part_acc, head_dim), ("part_ml", part_ml, 2)):
            if not (t.is_cuda and t.dtype == torch.float32 and t.is_contiguous() and t.dim() == 2
                    and t.shape[1] == width and t.shape[0] >= rows):
                raise KernelError(f"gemm_slices_folded {name} must be float32 [>= {rows}, {width}]")
        self._launch(self.core, self.core.ls_gemm_slices_folded, (
            c_int(DTYPE_CODE[w.dtype]), _ptr(part_acc), _ptr(part_ml), c_int(splits), c_int(head_dim), _ptr(w),
            _ptr(partials), c_int(m), c_int(n), c_int(k), _stream()))

    def add_rmsnorm(self, h: torch.Tensor, partials: torch.Tensor, weight, out, eps: float = 0.0,
                    rows: torch.Tensor | None = None) -> None:
        """``h[row] += partials[0][row] + partials[1][row] + ...``; then, unless ``out`` is None,
        ``out = rmsnorm(h[row]) * weight`` as ``rmsnorm`` computes it.  ``rows`` selects rows of ``h``."""
        _rows_ok(h, "add_rmsnorm h")
        if not (h.dtype == torch.float32):
            raise KernelError("add_rmsnorm works on the float32 residual stream")
        if not (partials.is_cuda and partials.dtype == torch.float32 and partials.is_contiguous()
              and partials.dim() == 3 and partials.shape[2] == h.shape[1]):
            raise KernelError("add_rmsnorm partials [slices, rows, width]")
        n_rows = h.shape[0] if rows is None else rows.shape[0]
        if rows is not None:
            if not (rows.is_cuda and rows.dtype == torch.int32 and rows.is_contiguous()):
                raise KernelError("add_rmsnorm rows: int32 on the GPU")
        dtype = torch.float32
        ld_out = 0
        if out is not None:
            _rows_ok(out, "add_rmsnorm out")
            if not (out.dtype in DTYPE_CODE and out.shape == (n_rows, h.shape[1])):
                raise KernelError("add_rmsnorm out shape or dtype")
            if not (weight is not None and weight.dtype == torch.float32 and weight.is_contiguous()
                  and weight.numel() == h.shape[1]):
                raise KernelError("add_rmsnorm weight must be float32 [width]")
            dtype, ld_out = out.dtype, out.stride(0)
        if n_rows == 0:
            return
        self._launch(self.core, self.core.ls_add_rmsnorm, (
            c_int(DTYPE_CODE[dtype]), _ptr(h), _ptr(partials), c_int(partials.shape[0]), c_int(partials.shape[1]),
            _ptr(weight), _ptr(out), _ptr(rows), c_int(n_rows), c_int(h.shape[1]), c_long(h.stride(0)),
            c_long(ld_out), c_float(eps), _stream()))

    # -- rows -------------------------------------------------------------------
    def embed(self, tokens: torch.Tensor, table: torch.Tensor, out: torch.Tensor, scale: float = 1.0, copies: int = 1) -> None:
        """``out[t] = table[tokens[t]] * scale`` as float32 rows, ``copies`` times side by side."""
        if not (tokens.is_cuda and tokens.dtype == torch.int32 and tokens.dim() == 1 and tokens.is_contiguous()):
            raise KernelError("embed tokens must be a contiguous int32 vector on the GPU")
        _rows_ok(table, "embed table"); _rows_ok(out, "embed out")
        if not (table.is_contiguous() and table.dtype in DTYPE_CODE):
            raise KernelError("embed table must be contiguous float32/bfloat16")
        if not (copies >= 1 and out.dtype == torch.float32 and out.shape == (tokens.shape[0], copies * table.shape[1])):
            raise KernelError(f"embed out must be float32 [{tokens.shape[0]},{copies * table.shape[1]}]")
        if tokens.shape[0] == 0:
            return
        self._launch(self.core, self.core.ls_embed, (
            c_int(DTYPE_CODE[table.dtype]), _ptr(tokens), _ptr(table), _ptr(out), c_int(tokens.shape[0]),
            c_int(table.shape[0]), c_int(table.shape[1]), c_long(out.stride(0)), c_float(scale), c_int(copies), _stream()))

    def rmsnorm(self, x: torch.Tensor, weight: torch.Tensor, out: torch.Tensor, eps: float,
                rows: torch.Tensor | None = None) -> None:
        """Rows of float ``x`` (all, or those listed in ``rows``) normalised into ``out``."""
        _rows_ok(x, "rmsnorm x"); _rows_ok(out, "rmsnorm out")
        if not (x.dtype == torch.float32):
            raise KernelError("rmsnorm reads the float32 residual stream")
        if not (weight.is_cuda and weight.dtype == torch.float32 and weight.is_contiguous()
              and weight.shape == (x.shape[1],)):
            raise KernelError(f"rmsnorm weight must be float32 [{x.shape[1]}]")
        if not (out.dtype in DTYPE_CODE and out.shape[1] == x.shape[1]):
            raise KernelError("rmsnorm out has the wrong width or dtype")
        n = out.shape[0]
        if rows is not None:
            if not (rows.is_cuda and rows.dtype == torch.int32 and rows.is_contiguous() and rows.shape == (n,)):
                raise KernelError(f"rmsnorm rows must be int32 [{n}]")
        else:
            if not (x.shape[0] == n):
                raise KernelError("rmsnorm out must have as many rows as x")
        if n == 0:
            return
        self._launch(self.core, self.core.ls_rmsnorm, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(x), _ptr(weight), _ptr(out), _ptr(rows), c_int(n), c_int(x.shape[1]),
            c_long(x.stride(0)), c_long(out.stride(0)), c_float(eps), _stream()))

    def swiglu(self, gate_up: torch.Tensor, out: torch.Tensor) -> None:
        _rows_ok(gate_up, "swiglu input"); _rows_ok(out, "swiglu out")
        rows, inter = out.shape
        if not (gate_up.shape == (rows, 2 * inter) and gate_up.dtype == out.dtype and out.dtype in DTYPE_CODE):
            raise KernelError(f"swiglu input must be [{rows},{2 * inter}] of the output's dtype")
        if rows == 0:
            return
        self._launch(self.core, self.core.ls_swiglu, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(gate_up), _ptr(out), c_int(rows), c_int(inter),
            c_long(gate_up.stride(0)), c_long(out.stride(0)), _stream()))

    ACTIVATIONS = {"none": 0, "silu": 1, "gelu_tanh": 2, "gelu": 3, "relu": 4}

    def bias_act(self, x: torch.Tensor, bias, out: torch.Tensor, activation: str = "none", gated: bool = False) -> None:
        """``out = act(x + bias)`` on float32 rows ``x``; gated: ``x`` holds gates then ups and
        ``out = act(gate + bias_gate) * (up + bias_up)``.  ``bias`` float32 or None; ``out`` float32
        or bfloat16, and may be ``x`` itself when not gated."""
        _rows_ok(x, "bias_act x"); _rows_ok(out, "bias_act out")
        if activation not in self.ACTIVATIONS:
            raise KernelError(f"activation {activation!r} is not built; known: {', '.join(self.ACTIVATIONS)}")
        rows, width = out.shape
        if not (x.dtype == torch.float32 and x.shape == (rows, 2 * width if gated else width) and out.dtype in DTYPE_CODE):
            raise KernelError(f"bias_act reads float32 [{rows},{2 * width if gated else width}], got {tuple(x.shape)} {x.dtype}")
        if bias is not None:
            if not (bias.is_cuda and bias.dtype == torch.float32 and bias.is_contiguous() and bias.shape == (x.shape[1],)):
                raise KernelError(f"bias_act bias must be float32 [{x.shape[1]}]")
        if gated and x.data_ptr() == out.data_ptr():
            raise KernelError("a gated bias_act cannot work in place")
        if rows == 0:
            return
        self._launch(self.core, self.core.ls_bias_act, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(x), c_long(x.stride(0)), _ptr(bias), _ptr(out), c_long(out.stride(0)),
            c_int(rows), c_int(width), c_int(self.ACTIVATIONS[activation]), c_int(1 if gated else 0), _stream()))

    #: (row, chunk) pairs the library's static arg-max scratch holds (LS_ARGMAX_STATIC_PAIRS)
    ARGMAX_STATIC_PAIRS = 16384

    def argmax(self, logits: torch.Tensor, out: torch.Tensor) -> None:
        """Lowest index among the maxima of every float32 row.  Calls that fit the library's static
        scratch array go through the entry point that allocates nothing: that array never moves, so
        a captured graph that contains the launch stays valid whatever runs in between.  Larger
        calls bring a scratch buffer; a buffer that was outgrown is kept until the process ends,
        because a captured graph may still write into it.

        The static array is one per GPU and process: calls that overlap on one GPU (two streams, two
        engines in one process that do not order their work) race on it.  This engine launches
        everything on one stream, which orders them."""
        _rows_ok(logits, "argmax logits")
        if not (logits.dtype == torch.float32):
            raise KernelError("argmax reads float32 logits")
        if not (out.is_cuda and out.dtype == torch.int32 and out.is_contiguous() and out.shape == (logits.shape[0],)):
            raise KernelError(f"argmax out must be int32 [{logits.shape[0]}]")
        if logits.shape[0] == 0:
            return
        pairs = logits.shape[0] * self.core.ls_argmax_chunks(c_int(logits.shape[1]))
        if pairs <= self.ARGMAX_STATIC_PAIRS:
            self._launch(self.core, self.core.ls_argmax_static, (
                _ptr(logits), _ptr(out), c_int(logits.shape[0]), c_int(logits.shape[1]), c_long(logits.stride(0)),
                _stream()))
            return
        held = self._argmax_scratch.setdefault(logits.device, [])
        if not held or held[-1].numel() < 2 * pairs:
            held.append(torch.empty(max(2 * pairs, 2 * held[-1].numel() if held else 0), dtype=torch.int32,
                                    device=logits.device))
        scratch = held[-1]
        self._launch(self.core, self.core.ls_argmax, (
            _ptr(logits), _ptr(out), c_int(logits.shape[0]), c_int(logits.shape[1]), c_long(logits.stride(0)),
            _ptr(scratch), c_long(scratch.numel()), _stream()))

    #: one row's request as ``sample_top_p`` takes it (eight 4-byte words; csrc/sample.hip: SampleRow)
    SAMPLE_ROW = [("row", "<i4"), ("temperature", "<f4"), ("top_p", "<f8"), ("key0", "<u4"), ("key1", "<u4"),
                  ("pos_lo", "<u4"), ("pos_hi", "<u4")]
    SAMPLE_ROW_INTS = 8
    SAMPLE_POSITION_AT = 6          # the word of a record that holds the low half of the position

    @classmethod
    def pack_sample_requests(cls, requests, rows: int):
        """``requests``: (row of the logits, temperature > 0, top_p, seed XOR k(uid) as an int of 64 bits,
        position) each; the records as int32 words, eight a request."""
        import numpy as np

        packed = np.zeros(len(requests), dtype=cls.SAMPLE_ROW)
        for i, (row, temperature, top_p, mixed, position) in enumerate(requests):
            if not (0 <= row < rows and temperature > 0):
                raise KernelError(f"sample: row {row} of {rows} at temperature {temperature}")
            packed[i] = (row, temperature, top_p, mixed & 0xFFFFFFFF, (mixed >> 32) & 0xFFFFFFFF,
                         position & 0xFFFFFFFF, (position >> 32) & 0xFFFFFFFF)
        return packed.view(np.int32)

    def sample_top_p(self, logits: torch.Tensor, requests, out: torch.Tensor, records: torch.Tensor | None = None,
                     any_nucleus: bool | None = None, scatter: bool = False) -> None:
        """One token for each request: ``requests`` is a sequence of (row of the float32 ``logits``,
        temperature > 0, top_p, seed XOR k(uid) as an int of 64 bits, position); ``out`` int32 on the GPU
        gets request i's token at ``out[i]`` (with ``scatter`` at ``out[row]``).  Or ``records``: the same
        packed by ``pack_sample_requests`` and already on the GPU (int32, eight words a request), with
        ``any_nucleus`` saying whether any top_p is below one.  The host sampler's procedure in float64
        (sampling/sampler.py) without its sort, the draw included (Philox-4x32-10 keyed as
        sampling/philox.py keys it)."""
        _rows_ok(logits, "sample logits")
        if not (logits.dtype == torch.float32):
            raise KernelError("sample reads float32 logits")
        if records is None:
            n = len(requests)
            if n == 0:
                return
            records = torch.from_numpy(self.pack_sample_requests(requests, logits.shape[0])).to(logits.device)
            any_nucleus = any(top_p < 1.0 for _, _, top_p, _, _ in requests)
        else:
            if not (records.is_cuda and records.dtype == torch.int32 and records.is_contiguous()
                    and records.numel() % self.SAMPLE_ROW_INTS == 0 and any_nucleus is not None):
                raise KernelError("sample records: contiguous int32 on the GPU, eight words a request, and any_nucleus")
            n = records.numel() // self.SAMPLE_ROW_INTS
            if n == 0:
                return
        if not (out.is_cuda and out.dtype == torch.int32 and out.is_contiguous()
                and out.numel() >= (logits.shape[0] if scatter else n)):
            raise KernelError("sample out must be int32 on the GPU, one for every request (with scatter: every row)")
        vocab = logits.shape[1]
        need = int(self.core.ls_sample_scratch_bytes(c_int(n), c_int(vocab)))
        scratch = self._sample_scratch.get(logits.device)
        if scratch is None or scratch.numel() < need:
            # (a buffer that was outgrown is kept: a captured graph may still write into it)
            scratch = torch.empty(need, dtype=torch.uint8, device=logits.device)
            self._sample_scratch_kept.append(self._sample_scratch.get(logits.device))
            self._sample_scratch[logits.device] = scratch
        self._launch(self.core, self.core.ls_sample_top_p, (
            _ptr(logits), c_long(logits.stride(0)), _ptr(records), _ptr(out), _ptr(scratch), c_long(scratch.numel()),
            c_int(n), c_int(vocab), c_int(1 if any_nucleus else 0), c_int(1 if scatter else 0), _stream()))

    def advance_decode(self, meta: torch.Tensor, n_seqs: int, off_tokens: int, picked: torch.Tensor,
                       ring: torch.Tensor, counter: torch.Tensor, off_runs: int, n_runs: int) -> None:
        """Between two decode steps that run without the host: the picked tokens become the next
        inputs inside the uploaded metadata ``meta``, every value named by the ``n_runs`` runs
        (first, stride, count) of the table at ``meta[off_runs]`` moves on by one, and the tokens
        are appended to ``ring[counter]``.  The step's upload builds the table and checks it."""
        for t in (meta, picked, ring, counter):
            if not (t.is_cuda and t.dtype == torch.int32 and t.is_contiguous()):
                raise KernelError("advance_decode works on int32 GPU tensors")
        if not (picked.numel() >= n_seqs):
            raise KernelError("advance_decode: picked is too short")
        self._launch(self.core, self.core.ls_advance_decode, (
            _ptr(meta), c_long(meta.numel()), c_int(n_seqs), c_int(off_tokens), _ptr(picked), _ptr(ring),
            _ptr(counter), c_int(off_runs), c_int(n_runs), _stream()))

    # -- attention ----------------------------------------------------------------
    def qk_rope_kv(self, qkv: torch.Tensor, n_tokens: int, nq: int, nkv: int, d: int, q_weight, k_weight,
                   eps: float, cos, sin, rot: int, tok_seq, tok_pos, seqs, max_pos: int, table, k_pages,
                   v_pages, page_size: int, write_kv: bool) -> None:
        """Per-head norm, rotation and cache write on the fused projection ``qkv``.

        ``max_pos`` is the largest position in the step (checked against the
        tables); ``table`` is the group's block table ``[rows, stride]``.
        """
        _rows_ok(qkv, "qkv")
        if not (qkv.dtype in DTYPE_CODE and qkv.shape[0] >= n_tokens):
            raise KernelError("qkv has too few rows or a wrong dtype")
        heads = nq + 2 * nkv if write_kv else nq
        if not (qkv.shape[1] >= heads * d):
            raise KernelError(f"qkv rows hold {qkv.shape[1]} values, {heads} heads of {d} are needed")
        if not (d <= MAX_HEAD_DIM):
            raise KernelError(f"head size {d} exceeds the supported maximum {MAX_HEAD_DIM}")
        for name, w in (("q norm weight", q_weight), ("k norm weight", k_weight)):
            if w is not None:
                if not (w.is_cuda and w.dtype == torch.float32 and w.is_contiguous() and w.shape == (d,)):
                    raise KernelError(f"{name} must be float32 [{d}]")
        positions = 0
        if cos is not None:
            if not (sin is not None and cos.shape == sin.shape and cos.dim() == 2 and cos.shape[1] * 2 == rot
                  and cos.dtype == torch.float32 and cos.is_contiguous() and sin.is_contiguous() and cos.is_cuda):
                raise KernelError("rotation tables must be float32 [positions, rotary_dim/2]")
            positions = cos.shape[0]
            if not (max_pos < positions):
                raise KernelError(f"position {max_pos} is beyond the rotation tables ({positions})")
        for name, t in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
            if not (t.is_cuda and t.dtype == torch.int32 and t.is_contiguous() and t.numel() >= n_tokens):
                raise KernelError(f"{name} must be int32 with at least {n_tokens} entries")
        if write_kv:
            if not (table is not None and table.is_cuda and table.dtype == torch.int32 and table.dim() == 2
                  and table.is_contiguous()):
                raise KernelError("block table must be a contiguous int32 matrix")
            if not (max_pos // page_size < table.shape[1]):
                raise KernelError(f"position {max_pos} needs page {max_pos // page_size}, the block table has {table.shape[1]} columns")
            for name, pages in (("key pages", k_pages), ("value pages", v_pages)):
                if not (pages.is_cuda and pages.dtype == qkv.dtype and pages.is_contiguous() and pages.dim() == 4):
                    raise KernelError(f"{name} must be contiguous 4-D of the compute dtype")
            if not (k_pages.shape[1:] == (nkv, page_size, d) and v_pages.shape[1:] == (nkv, d, page_size)
                  and k_pages.shape[0] == v_pages.shape[0]):
                raise KernelError(f"cache pages do not have the layout [pages,{nkv},{page_size},{d}] / [pages,{nkv},{d},{page_size}]")
        if n_tokens == 0:
            return
        self._launch(self.core, self.core.ls_qk_rope_kv, (
            c_int(DTYPE_CODE[qkv.dtype]), _ptr(qkv), c_long(qkv.stride(0)), c_int(n_tokens), c_int(nq), c_int(nkv),
            c_int(d), _ptr(q_weight), _ptr(k_weight), c_float(eps), _ptr(cos), _ptr(sin), c_int(rot),
            c_int(positions), _ptr(tok_seq), _ptr(tok_pos), _ptr(seqs), _ptr(table), c_int(table.shape[1] if table
            is not None else 0), _ptr(k_pages), _ptr(v_pages), c_int(page_size), c_int(1 if write_kv else 0),
            _stream()))

    def attention(self, q: torch.Tensor, nq: int, nkv: int, d: int, k_pages, v_pages, page_size: int, table,
                  seqs, items, n_items: int, out: torch.Tensor, part_acc, part_ml, scale: float,
                  window: int, variant: int = 0, max_rows: int = 0, spans: bool = False,
                  single_tile: bool = False) -> None:
        """Launch the attention kernel over ``n_items`` work items (see attention.hip).
        ``variant``: 0 staged through LDS where it fits, 1 direct from global memory, 2 staged or
        error, 3 cooperative (every item has at most 16 rows; ``max_rows`` states the largest),
        4 wide (prompt portions; items count row blocks of ``attention_block_rows``), 5 the same
        with half the rows a block (for steps with few rows).  ``spans`` (cooperative only): items
        that leave partial results may hold several splits each.  ``single_tile`` (cooperative only): every
        item holds one key tile (a hint: such a launch needs one tile buffer a workgroup, not two)."""
        lib = self.attention_lib(d)
        _rows_ok(q, "attention q"); _rows_ok(out, "attention out")
        if not (q.dtype in DTYPE_CODE and out.dtype == q.dtype):
            raise KernelError("attention q/out dtype")
        if not (nq % nkv == 0):
            raise KernelError(f"{nq} query heads are not a multiple of {nkv} kv heads")
        if not (q.shape[1] >= nq * d and out.shape[1] >= nq * d):
            raise KernelError("attention q/out rows are too short")
        if not (k_pages.dtype == q.dtype and v_pages.dtype == q.dtype and k_pages.is_contiguous()
              and v_pages.is_contiguous() and k_pages.shape[1:] == (nkv, page_size, d)
              and v_pages.shape[1:] == (nkv, d, page_size)):
            raise KernelError("attention cache pages have the wrong layout or dtype")
        if not (table.dtype == torch.int32 and table.dim() == 2 and table.is_contiguous()):
            raise KernelError("attention block table")
        if not (items.dtype == torch.int32 and items.is_contiguous() and items.numel() >= ATTENTION_ITEM_INTS * n_items):
            raise KernelError("attention items must hold 32 int32 each (see pack_attention_items)")
        if n_items == 0:
            return
        self._launch(lib, lib.ls_attention, (
            c_int(DTYPE_CODE[q.dtype]), _ptr(q), c_long(q.stride(0)), _ptr(k_pages), _ptr(v_pages), c_int(nkv),
            c_int(page_size), _ptr(table), c_int(table.shape[1]), _ptr(seqs), _ptr(items), c_int(n_items),
            _ptr(out), c_long(out.stride(0)), _ptr(part_acc), _ptr(part_ml), c_int(nq // nkv), c_float(scale),
            c_int(window), c_int(variant), c_int(max_rows), c_int((1 if spans else 0) | (2 if single_tile else 0)),
            _stream()))

    def attention_decode(self, qkv: torch.Tensor, nq: int, nkv: int, d: int, k_pages, v_pages, page_size: int,
                         table, seqs, items, n_items: int, out: torch.Tensor, part_acc, part_ml, scale: float,
                         window: int, q_weight, k_weight, eps: float, cos, sin, rot: int, max_pos: int,
                         write_kv: bool, spans: bool = False, single_tile: bool = False) -> None:
        """A step of single decoded tokens: what ``qk_rope_kv`` and ``attention`` (cooperative items) do,
        in one launch.  ``qkv`` is the raw fused projection; every request brings exactly one token."""
        lib = self.attention_lib(d)
        _rows_ok(qkv, "attention_decode qkv"); _rows_ok(out, "attention_decode out")
        if not (qkv.dtype in DTYPE_CODE and out.dtype == qkv.dtype):
            raise KernelError("attention_decode qkv/out dtype")
        if not (nq % nkv == 0):
            raise KernelError(f"{nq} query heads are not a multiple of {nkv} kv heads")
        heads = nq + 2 * nkv if write_kv else nq
        if not (qkv.shape[1] >= heads * d and out.shape[1] >= nq * d):
            raise KernelError("attention_decode rows are too short")
        if not (k_pages.dtype == qkv.dtype and v_pages.dtype == qkv.dtype and k_pages.is_contiguous()
              and v_pages.is_contiguous() and k_pages.shape[1:] == (nkv, page_size, d)
              and v_pages.shape[1:] == (nkv, d, page_size)):
            raise KernelError("attention cache pages have the wrong layout or dtype")
        if not (table.dtype == torch.int32 and table.dim() == 2 and table.is_contiguous()):
            raise KernelError("attention block table")
        if not (items.dtype == torch.int32 and items.is_contiguous() and items.numel() >= ATTENTION_ITEM_INTS * n_items):
            raise KernelError("attention items must hold 32 int32 each (see pack_attention_items)")
        for w in (q_weight, k_weight):
            if not (w is None or (w.dtype == torch.float32 and w.is_contiguous() and w.numel() == d)):
                raise KernelError("per-head norm weights must be float32 [head_dim]")
        positions = 0
        if cos is not None:
            if not (sin is not None and cos.dtype == torch.float32 and sin.dtype == torch.float32
                  and cos.is_contiguous() and sin.is_contiguous() and cos.shape == sin.shape
                  and cos.shape[1] == rot // 2):
                raise KernelError("rotation tables must be float32 [positions, rot/2]")
            positions = cos.shape[0]
        if n_items == 0:
            return
        self._launch(lib, lib.ls_attention_decode, (
            c_int(DTYPE_CODE[qkv.dtype]), _ptr(qkv), c_long(qkv.stride(0)), _ptr(k_pages), _ptr(v_pages), c_int(nq),
            c_int(nkv), c_int(page_size), _ptr(table), c_int(table.shape[1]), _ptr(seqs), _ptr(items),
            c_int(n_items), _ptr(out), c_long(out.stride(0)), _ptr(part_acc), _ptr(part_ml), c_float(scale),
            c_int(window), _ptr(q_weight), _ptr(k_weight), c_float(eps), _ptr(cos), _ptr(sin), c_int(rot),
            c_int(positions), c_int(max_pos), c_int(1 if write_kv else 0),
            c_int((1 if spans else 0) | (2 if single_tile else 0)), _stream()))

    def attention_combine(self, d: int, seqs, items, n_items: int, nq: int, nkv: int, part_acc, part_ml,
                          out: torch.Tensor, max_rows: int = 0) -> None:
        """Fold the splits' partial results of the requests in ``items`` into ``out``.  ``max_rows``: the
        most rows (tokens times query heads a kv head) a request of an item brings, 0 if unknown; with
        at most 16 the fold that asks for many splits at a time is taken (same bits)."""
        lib = self.attention_lib(d)
        _rows_ok(out, "combine out")
        if not (out.dtype in DTYPE_CODE and out.shape[1] >= nq * d):
            raise KernelError("combine out rows are too short")
        if not (items.dtype == torch.int32 and items.is_contiguous() and items.numel() >= COMBINE_ITEM_INTS * n_items):
            raise KernelError("combine items must hold 8 int32 each (see pack_combine_items)")
        if n_items == 0:
            return
        self._launch(lib, lib.ls_attention_combine, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(seqs), _ptr(items), c_int(n_items), c_int(nkv), _ptr(part_acc),
            _ptr(part_ml), _ptr(out), c_long(out.stride(0)), c_int(nq // nkv), c_int(max_rows), _stream()))

    # -- mixers beyond softmax attention: norms, gated units, recurrences ----------------
    def mixers_lib(self):
        """The library of csrc/mixers.hip, built and loaded when a part first asks for it."""
        if self._mixers is None:
            self.mixers_path = _build.build_mixers()
            lib = ctypes.CDLL(str(self.mixers_path))
            lib.ls_last_error.restype = ctypes.c_char_p
            self._mixers = lib
        return self._mixers

    def talking_lib(self, heads: int, kv_heads: int, dim: int, vdim: int):
        """The talking-heads attention library of one shape."""
        shape = (heads, kv_heads, dim, vdim)
        lib = self._talking.get(shape)
        if lib is None:
            path = _build.build_talking(*shape)
            lib = ctypes.CDLL(str(path))
            lib.ls_last_error.restype = ctypes.c_char_p
            if (lib.ls_talk_heads(), lib.ls_talk_kv_heads(), lib.ls_talk_dim(), lib.ls_talk_vdim()) != shape:
                raise KernelError(f"{path} was built for another shape")
            self._talking[shape] = lib
            self.talking_paths[shape] = str(path)
        return lib

    @staticmethod
    def _f32_vector(t, n: int, name: str) -> None:
        if not (t.is_cuda and t.dtype == torch.float32 and t.is_contiguous() and t.numel() == n):
            raise KernelError(f"{name} must be float32 with {n} elements on the GPU")

    def dyt(self, h: torch.Tensor, weight, bias, alpha, out, rows: torch.Tensor | None = None,
            partials: torch.Tensor | None = None) -> None:
        """Dynamic Tanh norm: ``out = tanh(alpha * h[row]) * weight + bias`` on rows of the float32 stream
        ``h`` (all, or those listed in ``rows``); with ``partials [slices, rows, width]`` these are added
        to ``h`` first, in ascending order.  ``out`` None: the addition only."""
        _rows_ok(h, "dyt h")
        if not (h.dtype == torch.float32):
            raise KernelError("dyt reads the float32 residual stream")
        width = h.shape[1]
        n_rows = h.shape[0] if rows is None else rows.shape[0]
        if rows is not None and not (rows.is_cuda and rows.dtype == torch.int32 and rows.is_contiguous()):
            raise KernelError("dyt rows: int32 on the GPU")
        slices = p_rows = 0
        if partials is not None:
            if not (partials.is_cuda and partials.dtype == torch.float32 and partials.is_contiguous()
                    and partials.dim() == 3 and partials.shape[2] == width and partials.shape[1] >= (h.shape[0] if rows is None else 1)):
                raise KernelError("dyt partials [slices, rows, width] float32")
            slices, p_rows = partials.shape[0], partials.shape[1]
        dtype, ld_out = torch.float32, 0
        if out is not None:
            _rows_ok(out, "dyt out")
            if not (out.dtype in DTYPE_CODE and out.shape == (n_rows, width)):
                raise KernelError(f"dyt out must be [{n_rows},{width}]")
            self._f32_vector(weight, width, "dyt weight"); self._f32_vector(bias, width, "dyt bias")
            self._f32_vector(alpha, 1, "dyt alpha")
            dtype, ld_out = out.dtype, out.stride(0)
        if n_rows == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_dyt, (
            c_int(DTYPE_CODE[dtype]), _ptr(h), _ptr(partials), c_int(slices), c_int(p_rows), _ptr(weight), _ptr(bias),
            _ptr(alpha), _ptr(out), _ptr(rows), c_int(n_rows), c_int(width), c_long(h.stride(0)), c_long(ld_out),
            _stream()))

    def glu_clamped(self, x: torch.Tensor, out: torch.Tensor, limit: float, alpha: float) -> None:
        """``out = g * sigmoid(alpha * g) * (u + 1)`` with ``g = min(gate, limit)``, ``u = clamp(up, -limit,
        limit)``; ``x`` float32 ``[rows, 2 * width]`` holds the gates, then the ups."""
        _rows_ok(x, "glu_clamped x"); _rows_ok(out, "glu_clamped out")
        rows, width = out.shape
        if not (x.dtype == torch.float32 and x.shape == (rows, 2 * width) and out.dtype in DTYPE_CODE):
            raise KernelError(f"glu_clamped reads float32 [{rows},{2 * width}]")
        if rows == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_glu_clamped, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(x), c_long(x.stride(0)), _ptr(out), c_long(out.stride(0)), c_int(rows),
            c_int(width), c_float(limit), c_float(alpha), _stream()))

    def softcap(self, x: torch.Tensor, cap: float) -> None:
        """``x = cap * tanh(x / cap)`` in place on float32 rows."""
        _rows_ok(x, "softcap x")
        if not (x.dtype == torch.float32 and cap > 0):
            raise KernelError("softcap works on float32 rows with a positive cap")
        if x.shape[0] == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_softcap, (_ptr(x), c_long(x.stride(0)), c_int(x.shape[0]), c_int(x.shape[1]),
                                           c_float(cap), _stream()))

    @staticmethod
    def _rotation_tables(cos, sin, rot: int, max_pos: int) -> int:
        if rot == 0:
            return 0
        if not (cos is not None and sin is not None and cos.shape == sin.shape and cos.dim() == 2
                and cos.shape[1] * 2 == rot and cos.dtype == torch.float32 and sin.dtype == torch.float32
                and cos.is_contiguous() and sin.is_contiguous() and cos.is_cuda):
            raise KernelError("rotation tables must be float32 [positions, rotary_dim/2]")
        if not (max_pos < cos.shape[0]):
            raise KernelError(f"position {max_pos} is beyond the rotation tables ({cos.shape[0]})")
        return cos.shape[0]

    def _paged_ok(self, k_pages, v_pages, table, dtype, kv_heads: int, page_size: int, dim: int, vdim: int) -> None:
        if not (k_pages.dtype == dtype and v_pages.dtype == dtype and k_pages.is_contiguous() and v_pages.is_contiguous()
                and k_pages.dim() == 4 and k_pages.shape[1:] == (kv_heads, page_size, dim)
                and v_pages.shape[1:] == (kv_heads, vdim, page_size) and k_pages.shape[0] == v_pages.shape[0]):
            raise KernelError(f"cache pages do not have the layout [pages,{kv_heads},{page_size},{dim}] / "
                              f"[pages,{kv_heads},{vdim},{page_size}] of the compute dtype")
        if not (table.is_cuda and table.dtype == torch.int32 and table.dim() == 2 and table.is_contiguous()):
            raise KernelError("block table must be a contiguous int32 matrix")

    def talk_qkv(self, raw: torch.Tensor, n_tokens: int, heads: int, kv_heads: int, dim: int, vdim: int, bias, cos, sin,
                 rot: int, max_pos: int, tok_seq, tok_pos, seqs, table, q_out: torch.Tensor, k_pages, v_pages,
                 page_size: int, vmix_mode: int = 0, vmix=None, v_first=None) -> None:
        """Post pass of the fused projection ``raw`` (float32 ``[T, heads*dim + kv_heads*dim + kv_heads*vdim]``):
        biases, rotation of queries and keys, value mixing (1: keep the values in ``v_first``; 2: mix
        ``v_first`` in with the weight ``vmix``), queries to ``q_out``, keys and values to their pages."""
        _rows_ok(raw, "talk_qkv raw"); _rows_ok(q_out, "talk_qkv q_out")
        width = heads * dim + kv_heads * (dim + vdim)
        if not (raw.dtype == torch.float32 and raw.shape[0] >= n_tokens and raw.shape[1] == width):
            raise KernelError(f"talk_qkv raw must be float32 [>= {n_tokens}, {width}]")
        if not (q_out.dtype in DTYPE_CODE and q_out.shape[0] >= n_tokens and q_out.shape[1] == heads * dim):
            raise KernelError("talk_qkv q_out has the wrong shape or dtype")
        if bias is not None:
            self._f32_vector(bias, width, "talk_qkv bias")
        positions = self._rotation_tables(cos, sin, rot, max_pos)
        self._paged_ok(k_pages, v_pages, table, q_out.dtype, kv_heads, page_size, dim, vdim)
        if not (max_pos // page_size < table.shape[1]):
            raise KernelError(f"position {max_pos} needs page {max_pos // page_size}, the block table has {table.shape[1]} columns")
        for name, t in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
            if not (t.is_cuda and t.dtype == torch.int32 and t.is_contiguous() and t.numel() >= n_tokens):
                raise KernelError(f"{name} must be int32 with at least {n_tokens} entries")
        ldv = 0
        if vmix_mode:
            if not (v_first is not None and v_first.is_cuda and v_first.dtype == torch.float32 and v_first.dim() == 2
                    and v_first.stride(1) == 1 and v_first.shape[0] >= n_tokens and v_first.shape[1] == kv_heads * vdim):
                raise KernelError(f"talk_qkv v_first must be float32 [>= {n_tokens}, {kv_heads * vdim}]")
            ldv = v_first.stride(0)
            if vmix_mode == 2:
                self._f32_vector(vmix, 1, "talk_qkv vmix")
        if n_tokens == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_talk_qkv, (
            c_int(DTYPE_CODE[q_out.dtype]), _ptr(raw), c_long(raw.stride(0)), c_int(n_tokens), c_int(heads),
            c_int(kv_heads), c_int(dim), c_int(vdim), _ptr(bias), _ptr(cos), _ptr(sin), c_int(rot), c_int(positions),
            c_int(max_pos), _ptr(tok_seq), _ptr(tok_pos), _ptr(seqs), _ptr(table), c_int(table.shape[1]), _ptr(q_out),
            c_long(q_out.stride(0)), _ptr(k_pages), _ptr(v_pages), c_int(page_size), c_int(vmix_mode), _ptr(vmix),
            _ptr(v_first), c_long(ldv), _stream()))

    def talk_attention(self, q: torch.Tensor, heads: int, kv_heads: int, dim: int, vdim: int, k_pages, v_pages,
                       page_size: int, table, seqs, blocks: torch.Tensor, n_blocks: int, talk: torch.Tensor,
                       scale: float, window: int, keep_first: int, out: torch.Tensor, folds: torch.Tensor | None = None,
                       n_folds: int = 0, part: torch.Tensor | None = None, part_rows: int = 16,
                       mix_weights: bool = False, sink=None, stats: torch.Tensor | None = None, gate=None) -> None:
        """Talking-heads attention of the step's queries ``q [T, heads*dim]`` over the paged cache; ``blocks``
        lists ``n_blocks`` work items of four ints (request of the step, block of 16 of its rows, run, runs);
        ``talk [heads, heads]``.  A row block whose visible keys are dealt to several work items (runs > 1) has a
        fold item of four ints in ``folds`` (first work item, runs, first packed row, rows); their results wait in
        ``part`` (float32, ``n_blocks * part_rows * heads * (vdim + 2)`` elements; ``part_rows`` 16, or 1 for a step
        of single decoded tokens) until a second launch has folded them.  ``mix_weights``: the heads' weights are
        mixed after each head's own softmax instead of their scores before it (``stats``: float32 scratch of
        ``n_blocks * 16 * heads * 2`` elements), with ``sink [heads]`` (float32 or None) in every head's denominator
        and ``gate`` (float32 rows of ``heads*vdim`` logits or None) whose sigmoid multiplies the output."""
        lib = self.talking_lib(heads, kv_heads, dim, vdim)
        _rows_ok(q, "talk_attention q"); _rows_ok(out, "talk_attention out")
        if not (q.dtype in DTYPE_CODE and out.dtype == q.dtype and q.shape[1] == heads * dim
                and out.shape[1] == heads * vdim and out.shape[0] == q.shape[0]):
            raise KernelError("talk_attention q / out have the wrong shape or dtype")
        self._paged_ok(k_pages, v_pages, table, q.dtype, kv_heads, page_size, dim, vdim)
        if not (blocks.is_cuda and blocks.dtype == torch.int32 and blocks.is_contiguous() and blocks.numel() >= 4 * n_blocks):
            raise KernelError("talk_attention work items must hold four int32 each")
        if n_folds:
            if not (folds is not None and folds.is_cuda and folds.dtype == torch.int32 and folds.is_contiguous()
                    and folds.numel() >= 4 * n_folds and part_rows in (1, 16)
                    and part is not None and part.is_cuda and part.dtype == torch.float32 and part.is_contiguous()
                    and part.numel() >= n_blocks * part_rows * heads * (vdim + 2)):
                raise KernelError("talk_attention folds: four int32 each, and room for every work item's partial result")
        self._f32_vector(talk, heads * heads, "talk_attention talk")
        if not (window > 0 and keep_first >= 0):
            raise KernelError(f"talk_attention window {window} / kept first tokens {keep_first}")
        ldg = 0
        if mix_weights:
            if not (stats is not None and stats.is_cuda and stats.dtype == torch.float32 and stats.is_contiguous()
                    and stats.numel() >= n_blocks * 16 * heads * 2):
                raise KernelError("talk_attention stats: float32 with 32 * heads elements a work item")
            if sink is not None:
                self._f32_vector(sink, heads, "talk_attention sink")
            if gate is not None:
                _rows_ok(gate, "talk_attention gate")
                if not (gate.dtype == torch.float32 and gate.shape[0] >= q.shape[0] and gate.shape[1] == heads * vdim):
                    raise KernelError(f"talk_attention gate must be float32 [>= {q.shape[0]}, {heads * vdim}]")
                ldg = gate.stride(0)
        elif sink is not None or gate is not None:
            raise KernelError("talk_attention: a sink and a gate come with mixed weights only")
        if n_blocks == 0:
            return
        self._launch(lib, lib.ls_talk_attention, (
            c_int(DTYPE_CODE[q.dtype]), _ptr(q), c_long(q.stride(0)), _ptr(k_pages), _ptr(v_pages), c_int(page_size),
            _ptr(table), c_int(table.shape[1]), _ptr(seqs), _ptr(blocks), c_int(n_blocks), _ptr(talk), c_float(scale),
            c_int(window), c_int(keep_first), _ptr(out), c_long(out.stride(0)), _ptr(folds), c_int(n_folds), _ptr(part),
            c_int(part_rows), c_int(int(bool(mix_weights))), _ptr(sink), _ptr(stats), _ptr(gate), c_long(ldg), _stream()))

    LINREC_HGRN2, LINREC_RETENTION = 0, 1

    def linrec_max_dim(self) -> int:
        return self._memo(("linrec_max_dim",), lambda: int(self.mixers_lib().ls_linrec_max_dim()))

    def linrec_gate_floats(self, n_tokens: int, heads: int, dim: int) -> int:
        """Floats of the scratch buffer ``linrec`` needs for a step of ``n_tokens`` tokens."""
        lib = self.mixers_lib()
        lib.ls_linrec_gate_floats.restype = ctypes.c_long
        return int(lib.ls_linrec_gate_floats(c_int(n_tokens), c_int(heads), c_int(dim)))

    def linrec(self, mode: int, raw: torch.Tensor, q_at: int, ab_at: int, v_at: int, heads: int, dim: int, vdim: int,
               p0, p1, cos, sin, rot: int, max_pos: int, tok_pos, seqs, n_seqs: int, state: torch.Tensor,
               gates: torch.Tensor, out: torch.Tensor) -> None:
        """The linear recurrence ``S_t = diag(a_t) S_(t-1) + b_t v_t^T``, ``o_t = S_t^T q_t`` over the tokens of
        every request of the step; ``raw`` float32 holds the projections (q at column ``q_at``, the gate or key
        projection at ``ab_at``, v at ``v_at``), ``state`` float32 ``[slots, heads, dim, vdim]`` is read and
        left for the next step, ``out`` float32 ``[T, heads*vdim]`` gets ``o_t``.  Mode ``LINREC_HGRN2``:
        ``p0`` lower bounds ``[heads*dim]``, ``p1`` the gate's bias or None; ``LINREC_RETENTION``: ``p0`` the
        heads' decays, rotation tables for q and k at the positions ``tok_pos``.  ``gates``: float32 scratch of
        ``linrec_gate_floats`` elements (q, decay and write gate of every token, computed once a step)."""
        _rows_ok(raw, "linrec raw"); _rows_ok(out, "linrec out")
        if not (raw.dtype == torch.float32 and out.dtype == torch.float32 and out.shape[1] == heads * vdim
                and out.shape[0] == raw.shape[0]):
            raise KernelError("linrec reads and writes float32 rows, out [T, heads*vdim]")
        if not (0 <= q_at and q_at + heads * dim <= raw.shape[1] and 0 <= ab_at and ab_at + heads * dim <= raw.shape[1]
                and 0 <= v_at and v_at + heads * vdim <= raw.shape[1]):
            raise KernelError("linrec: the projections do not fit the rows of raw")
        if not (dim <= self.linrec_max_dim()):
            raise KernelError(f"linrec takes states of at most {self.linrec_max_dim()} rows, got {dim}")
        if not (state.is_cuda and state.dtype == torch.float32 and state.is_contiguous()
                and tuple(state.shape[1:]) == (heads, dim, vdim)):
            raise KernelError(f"linrec state must be float32 [slots,{heads},{dim},{vdim}]")
        positions = 0
        if mode == self.LINREC_HGRN2:
            self._f32_vector(p0, heads * dim, "linrec lower bounds")
            if p1 is not None:
                self._f32_vector(p1, heads * dim, "linrec gate bias")
        else:
            self._f32_vector(p0, heads, "linrec decays")
            positions = self._rotation_tables(cos, sin, rot, max_pos)
        if not (gates.is_cuda and gates.dtype == torch.float32 and gates.is_contiguous()
                and gates.numel() >= self.linrec_gate_floats(raw.shape[0], heads, dim)):
            raise KernelError("linrec gates: float32 scratch of linrec_gate_floats elements")
        if not (tok_pos.is_cuda and tok_pos.dtype == torch.int32 and tok_pos.is_contiguous() and tok_pos.numel() >= raw.shape[0]):
            raise KernelError("linrec tok_pos: int32, one position a token")
        if n_seqs == 0 or raw.shape[0] == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_linrec, (
            c_int(mode), _ptr(raw), c_long(raw.stride(0)), c_int(q_at), c_int(ab_at), c_int(v_at), c_int(raw.shape[0]),
            c_int(heads), c_int(dim), c_int(vdim), _ptr(p0), _ptr(p1), _ptr(cos), _ptr(sin), c_int(rot),
            c_int(positions), c_int(max_pos), _ptr(tok_pos), _ptr(seqs), c_int(n_seqs), _ptr(state), _ptr(gates),
            _ptr(out), c_long(out.stride(0)), _stream()))

    def head_norm_gate(self, x: torch.Tensor, heads: int, vdim: int, weight, gate, eps: float, out: torch.Tensor,
                       gate_act: str = "silu", denom=None, denom_eps: float = 0.0) -> None:
        """Per (token, head): ``x / sqrt(mean(x^2) + eps)`` over the head's ``vdim`` values, times ``weight
        [vdim]`` and ``silu(gate)`` or, with ``gate_act = "sigmoid"``, ``sigmoid(gate)`` (float32 rows like ``x``)
        where given; ``x`` float32 ``[T, heads*vdim]``.  A weight of ``heads*vdim`` elements is one vector a head.  ``denom``
        (float32 ``[T, heads, 4]``, its last two places a floor and a read-out): every head is first divided by ``max(|read-out|,
        floor) + denom_eps``."""
        if gate_act not in ("silu", "sigmoid"):
            raise KernelError(f"head_norm_gate: the gate's activation is silu or sigmoid, got {gate_act!r}")
        _rows_ok(x, "head_norm_gate x"); _rows_ok(out, "head_norm_gate out")
        if not (x.dtype == torch.float32 and x.shape[1] == heads * vdim and out.shape == x.shape and out.dtype in DTYPE_CODE):
            raise KernelError("head_norm_gate reads float32 [T, heads*vdim] and writes the same shape")
        each = 0
        if weight is not None:
            each = vdim if weight.numel() == heads * vdim else 0
            self._f32_vector(weight, heads * vdim if each else vdim, "head_norm_gate weight")
        if denom is not None:
            self._f32_vector(denom, x.shape[0] * heads * 4, "head_norm_gate denom")
        ldg = 0
        if gate is not None:
            if not (gate.is_cuda and gate.dtype == torch.float32 and gate.dim() == 2 and gate.stride(1) == 1
                    and gate.shape == x.shape):
                raise KernelError("head_norm_gate gate must be float32 rows of the shape of x")
            ldg = gate.stride(0)
        if x.shape[0] == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_head_norm_gate, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(x), c_long(x.stride(0)), c_int(x.shape[0]), c_int(heads), c_int(vdim),
            _ptr(weight), c_int(each), _ptr(gate), c_long(ldg), c_int(int(gate_act == "sigmoid")), _ptr(denom), c_float(denom_eps),
            c_float(eps), _ptr(out),
            c_long(out.stride(0)), _stream()))


    # -- attention with a sink, and what comes before it --------------------------------------
    def sink_lib(self, dim: int, vdim: int):
        """The sink attention library of one key size and one value size."""
        shape = (dim, vdim)
        lib = self._sink.get(shape)
        if lib is None:
            path = _build.build_sink(*shape)
            lib = ctypes.CDLL(str(path))
            lib.ls_last_error.restype = ctypes.c_char_p
            if (lib.ls_sink_dim(), lib.ls_sink_vdim()) != shape:
                raise KernelError(f"{path} was built for another shape")
            self._sink[shape] = lib
            self.sink_paths[shape] = str(path)
        return lib

    #: the value of ``row_tiles`` that asks ``sink_attention`` for its kernel with tiles staged in LDS
    SINK_STAGED = 8

    def sink_staged_keys(self, dim: int, vdim: int, dtype: torch.dtype) -> int:
        """Keys of a tile of the staged kernel for prompt portions; 0 where the sizes do not fit it."""
        return self._memo(("sink_staged_keys", dim, vdim, dtype),
                          lambda: int(self.sink_lib(dim, vdim).ls_sink_staged_keys(c_int(DTYPE_CODE[dtype]))))

    def sink_staged_rows(self, heads: int, kv_heads: int) -> int:
        """Rows of a work item's block in the staged kernel: four waves are min(group, 4) heads times groups of 32 rows."""
        group = heads // kv_heads
        return 32 * (4 // min(group, 4))

    def qkv_post(self, raw: torch.Tensor, n_tokens: int, heads: int, kv_heads: int, dim: int, vdim: int, bias, q_norm,
                 k_norm, eps: float, cos, sin, rot: int, neighbours: bool, max_pos: int, tok_seq, tok_pos, seqs, table,
                 q_out: torch.Tensor, k_pages, v_pages, page_size: int, keys_are_values: bool = False,
                 key_pad: int | None = None, per_head: bool = False, head_weights: bool = False, value_scale: float = 1.0) -> None:
        """Post pass of the fused projection ``raw`` (float32, ``q | k | v | ...``; no ``v`` with
        ``keys_are_values``, where the biased, unnormalised keys are stored as the values): biases, a
        root-mean-square norm over the whole of q and of k with the weights ``q_norm`` / ``k_norm``, rotation of
        the first ``rot`` dimensions of each head in pairs ``(i, i + rot/2)`` or of ``neighbours``, queries to
        ``q_out``, keys and values to their pages.  ``key_pad``: the size of a head in ``q_out`` and in the key
        pages where it exceeds ``dim`` (zeros beyond ``dim``).  ``per_head``: every head of q and of k is divided
        by its own root mean square over ``dim`` (``eps`` inside the root, no weights) instead; with
        ``head_weights`` as well, then multiplied by ``q_norm`` / ``k_norm`` of ``dim`` elements, which all heads share.
        Values are stored times ``value_scale``."""
        _rows_ok(raw, "qkv_post raw"); _rows_ok(q_out, "qkv_post q_out")
        key_pad = dim if key_pad is None else key_pad
        width = heads * dim + kv_heads * dim + (0 if keys_are_values else kv_heads * vdim)
        if not (raw.dtype == torch.float32 and raw.shape[0] >= n_tokens and raw.shape[1] >= width):
            raise KernelError(f"qkv_post raw must be float32 [>= {n_tokens}, >= {width}]")
        if not (key_pad >= dim and q_out.dtype in DTYPE_CODE and q_out.shape[0] >= n_tokens and q_out.shape[1] == heads * key_pad):
            raise KernelError("qkv_post q_out has the wrong shape or dtype")
        if keys_are_values and dim != vdim:
            raise KernelError(f"keys of {dim} elements cannot be values of {vdim}")
        if bias is not None:
            self._f32_vector(bias, width, "qkv_post bias")
        if (q_norm is None) != (k_norm is None):
            raise KernelError("qkv_post normalises both q and k or neither")
        if head_weights and not (per_head and q_norm is not None):
            raise KernelError("qkv_post: weights that the heads share belong to a norm a head, and both are needed")
        if q_norm is not None:
            self._f32_vector(q_norm, dim if head_weights else heads * dim, "qkv_post q_norm")
            self._f32_vector(k_norm, dim if head_weights else kv_heads * dim, "qkv_post k_norm")
        if per_head and ((q_norm is not None and not head_weights) or not eps > 0):
            raise KernelError("qkv_post: a norm a head takes no weights, or one vector for all heads, and needs a positive eps")
        positions = self._rotation_tables(cos, sin, rot, max_pos)
        self._paged_ok(k_pages, v_pages, table, q_out.dtype, kv_heads, page_size, key_pad, vdim)
        if not (max_pos // page_size < table.shape[1]):
            raise KernelError(f"position {max_pos} needs page {max_pos // page_size}, the block table has {table.shape[1]} columns")
        for name, t in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
            if not (t.is_cuda and t.dtype == torch.int32 and t.is_contiguous() and t.numel() >= n_tokens):
                raise KernelError(f"{name} must be int32 with at least {n_tokens} entries")
        if n_tokens == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_qkv_post, (
            c_int(DTYPE_CODE[q_out.dtype]), _ptr(raw), c_long(raw.stride(0)), c_int(n_tokens), c_int(heads),
            c_int(kv_heads), c_int(dim), c_int(key_pad), c_int(vdim), c_int(int(keys_are_values)), c_int(2 if head_weights else int(per_head)), _ptr(bias), _ptr(q_norm), _ptr(k_norm),
            c_float(eps), _ptr(cos), _ptr(sin), c_int(rot), c_int(int(neighbours)), c_int(positions), c_int(max_pos),
            _ptr(tok_seq), _ptr(tok_pos), _ptr(seqs), _ptr(table), c_int(table.shape[1]), _ptr(q_out),
            c_long(q_out.stride(0)), _ptr(k_pages), _ptr(v_pages), c_int(page_size), c_float(value_scale), _stream()))

    def sink_attention(self, q: torch.Tensor, heads: int, kv_heads: int, dim: int, vdim: int, k_pages, v_pages,
                       page_size: int, table, seqs, items: torch.Tensor, n_items: int, row_tiles: int, scale: float,
                       window: int, chunk: int, sink, dist_bias, gate, out: torch.Tensor,
                       folds: torch.Tensor | None = None, n_folds: int = 0, part: torch.Tensor | None = None,
                       keep_first: int = 0) -> None:
        """Attention of the step's queries ``q [T, heads*dim]`` over the paged cache with a sink in the softmax.
        ``items``: ``n_items`` work items of four ints (request of the step, block of ``16 * row_tiles`` of its
        rows, run, runs); ``row_tiles`` 1, 2 or 4, or 0 for a step of single decoded tokens, or ``SINK_STAGED`` for
        the kernel that stages key tiles in LDS (blocks of ``sink_staged_rows`` rows).  ``window`` /
        ``chunk``: 0 for none; ``keep_first``: with a window, the first that many tokens stay visible.  ``sink [heads]`` float32 or None; ``dist_bias [heads, distances]`` float32 or
        None (its last column serves every larger distance); ``gate``: float32 rows of ``heads*vdim`` logits
        whose sigmoid multiplies the output, or None.  Row blocks whose keys are dealt to several work items
        have a fold item in ``folds`` (first work item, runs, first packed row, rows) and their results wait in
        ``part`` (float32) until a second launch has folded them."""
        lib = self.sink_lib(dim, vdim)
        _rows_ok(q, "sink_attention q"); _rows_ok(out, "sink_attention out")
        if not (q.dtype in DTYPE_CODE and out.dtype == q.dtype and q.shape[1] == heads * dim
                and out.shape[1] == heads * vdim and out.shape[0] == q.shape[0]):
            raise KernelError("sink_attention q / out have the wrong shape or dtype")
        self._paged_ok(k_pages, v_pages, table, q.dtype, kv_heads, page_size, dim, vdim)
        if not (items.is_cuda and items.dtype == torch.int32 and items.is_contiguous() and items.numel() >= 4 * n_items):
            raise KernelError("sink_attention work items must hold four int32 each")
        if row_tiles not in (0, 1, 2, 4, self.SINK_STAGED):
            raise KernelError(f"sink_attention takes 0, 1, 2 or 4 row tiles or {self.SINK_STAGED} for its staged kernel, got {row_tiles}")
        if row_tiles == self.SINK_STAGED:
            if not (self.sink_staged_keys(dim, vdim, q.dtype) and page_size % (16 // q.element_size()) == 0):
                raise KernelError(f"the staged kernel does not take keys of {dim}, values of {vdim} on pages of {page_size}")
            part_rows = self.sink_staged_rows(heads, kv_heads)
        else:
            part_rows = 16 * row_tiles if row_tiles else 1
        if n_folds:
            if not (folds is not None and folds.is_cuda and folds.dtype == torch.int32 and folds.is_contiguous()
                    and folds.numel() >= 4 * n_folds and part is not None and part.is_cuda
                    and part.dtype == torch.float32 and part.is_contiguous()
                    and part.numel() >= n_items * part_rows * heads * (vdim + 2)):
                raise KernelError("sink_attention folds: four int32 each, and room for every work item's partial result")
        if sink is not None:
            self._f32_vector(sink, heads, "sink_attention sink")
        n_dist = 0
        if dist_bias is not None:
            if not (dist_bias.is_cuda and dist_bias.dtype == torch.float32 and dist_bias.is_contiguous()
                    and dist_bias.dim() == 2 and dist_bias.shape[0] == heads and dist_bias.shape[1] > 0):
                raise KernelError(f"sink_attention dist_bias must be float32 [{heads}, distances]")
            n_dist = dist_bias.shape[1]
        ldg = 0
        if gate is not None:
            _rows_ok(gate, "sink_attention gate")
            if not (gate.dtype == torch.float32 and gate.shape[0] >= q.shape[0] and gate.shape[1] == heads * vdim):
                raise KernelError(f"sink_attention gate must be float32 [>= {q.shape[0]}, {heads * vdim}]")
            ldg = gate.stride(0)
        if not (window >= 0 and chunk >= 0):
            raise KernelError(f"sink_attention window {window} / chunk {chunk}")
        if not (keep_first >= 0 and (keep_first == 0 or (window > 0 and chunk == 0))):
            raise KernelError(f"sink_attention: {keep_first} kept first tokens need a window and no chunks")
        if n_items == 0:
            return
        self._launch(lib, lib.ls_sink_attention, (
            c_int(DTYPE_CODE[q.dtype]), _ptr(q), c_long(q.stride(0)), _ptr(k_pages), _ptr(v_pages), c_int(page_size),
            _ptr(table), c_int(table.shape[1]), _ptr(seqs), _ptr(items), c_int(n_items), c_int(row_tiles), c_int(heads),
            c_int(kv_heads), c_float(scale), c_int(window), c_int(chunk), c_int(keep_first), _ptr(sink), _ptr(dist_bias), c_int(n_dist),
            _ptr(gate), c_long(ldg), _ptr(out), c_long(out.stride(0)), _ptr(folds), c_int(n_folds), _ptr(part),
            c_int(part_rows), _stream()))

    # -- many small experts --------------------------------------------------------------------
    def experts_lib(self):
        """The library of csrc/experts.hip, built and loaded when a part first asks for it."""
        if self._experts is None:
            self.experts_path = _build.build_experts()
            lib = ctypes.CDLL(str(self.experts_path))
            lib.ls_last_error.restype = ctypes.c_char_p
            self._experts = lib
        return self._experts

    def experts_max_top(self) -> int:
        return self._memo(("experts_max_top",), lambda: int(self.experts_lib().ls_experts_max_top()))

    def experts_tile_capacity(self, n_tokens: int, experts: int, top: int, rows_a_tile: int) -> int:
        """Tiles of ``rows_a_tile`` rows that the (token, choice) pairs of a step can need at most."""
        pairs = n_tokens * top
        return pairs // rows_a_tile + min(pairs, experts)

    @staticmethod
    def _i32(t, n: int, name: str) -> None:
        if not (t.is_cuda and t.dtype == torch.int32 and t.is_contiguous() and t.numel() >= n):
            raise KernelError(f"{name} must be int32 with at least {n} elements on the GPU")

    def experts_route(self, logits: torch.Tensor, bias, top: int, rows_a_tile: int, expert: torch.Tensor,
                      weight: torch.Tensor, order: torch.Tensor, tiles: torch.Tensor, counts: torch.Tensor,
                      scoring: str = "softmax", correction=None, groups: tuple[int, int] = (1, 1)) -> None:
        """From router ``logits [T, E]`` (float32) and ``bias [E]``: every token's ``top`` experts (largest logit
        first, the lower index wins a tie) into ``expert [T, top]``, the softmax over the chosen logits into
        ``weight [T, top]``; the pairs ``token * top + choice`` sorted by expert into ``order``, and every
        expert's pairs cut into ``tiles [capacity, 4]`` (expert or -1, first place in ``order``, rows, 0).
        ``scoring = "sigmoid"``: every chosen expert weighs the sigmoid of its own logit instead (the weights of a token need not add up to one).
        ``scoring = "softmax_all"``: scores are the softmax over all logits; the choice goes by score + ``correction [E]``, within
        the ``groups[1]`` best of ``groups[0]`` equal runs of neighbouring experts (a run counts by its largest choice
        score); the weights are the chosen experts' scores divided by their sum."""
        _rows_ok(logits, "experts_route logits")
        if scoring not in ("softmax", "sigmoid", "softmax_all"):
            raise KernelError(f"experts_route: scoring is softmax, sigmoid or softmax_all, got {scoring!r}")
        t, e = logits.shape
        count, keep = groups
        if scoring == "softmax_all":
            self._f32_vector(correction, e, "experts_route correction")
            if not (0 < keep <= count and e % count == 0 and top <= keep * (e // count)):
                raise KernelError(f"experts_route: {e} experts in {count} groups of which {keep} are kept, {top} a token")
        if not (logits.dtype == torch.float32 and 0 < top <= min(e, self.experts_max_top())):
            raise KernelError(f"experts_route: float32 logits and 1 <= top <= {min(e, self.experts_max_top())}, got {top}")
        if bias is not None:
            self._f32_vector(bias, e, "experts_route bias")
        cap = self.experts_tile_capacity(t, e, top, rows_a_tile)
        self._i32(expert, t * top, "experts_route expert"); self._i32(order, t * top, "experts_route order")
        self._i32(tiles, 4 * cap, "experts_route tiles"); self._i32(counts, e, "experts_route counts")
        if not (weight.is_cuda and weight.dtype == torch.float32 and weight.is_contiguous() and weight.numel() >= t * top):
            raise KernelError("experts_route weight must be float32 [T, top]")
        if t == 0:
            return
        lib = self.experts_lib()
        self._launch(lib, lib.ls_experts_route, (
            _ptr(logits), c_long(logits.stride(0)), _ptr(bias), c_int(t), c_int(e), c_int(top), c_int(rows_a_tile),
            _ptr(expert), _ptr(weight), _ptr(order), _ptr(tiles), c_int(cap), _ptr(counts), c_int(("softmax", "sigmoid", "softmax_all").index(scoring)),
            _ptr(correction), c_int(count), c_int(keep), _stream()))

    def experts_route_product_ok(self, dtype: torch.dtype, n_tokens: int, experts: int, top: int, k: int) -> bool:
        """Whether ``experts_route_product`` takes a step of this many tokens of ``k`` elements."""
        return self._memo(("route_product", dtype, n_tokens, experts, top, k), lambda: bool(self.experts_lib().ls_experts_route_product_ok(
            c_int(DTYPE_CODE[dtype]), c_int(n_tokens), c_int(experts), c_int(top), c_int(k))))

    def experts_route_product(self, x: torch.Tensor, w_router: torch.Tensor, bias, top: int, rows_a_tile: int, expert: torch.Tensor,
                              weight: torch.Tensor, order: torch.Tensor, tiles: torch.Tensor, scoring: str = "softmax", correction=None,
                              groups: tuple[int, int] = (1, 1)) -> None:
        """``experts_route`` of the logits ``x @ w_router.T`` (float32 sums) for a few tokens, the product in the same launch."""
        _rows_ok(x, "experts_route_product x")
        if scoring not in ("softmax", "sigmoid", "softmax_all"):
            raise KernelError(f"experts_route_product: scoring is softmax, sigmoid or softmax_all, got {scoring!r}")
        t, k = x.shape
        if not (w_router.is_cuda and w_router.dim() == 2 and w_router.is_contiguous() and w_router.shape[1] == k
                and w_router.dtype == x.dtype and x.dtype in DTYPE_CODE):
            raise KernelError("experts_route_product: the router's matrix must be [E, K] in the dtype of x")
        e = w_router.shape[0]
        if not (0 < top <= min(e, self.experts_max_top()) and self.experts_route_product_ok(x.dtype, t, e, top, k)):
            raise KernelError(f"experts_route_product does not take {t} tokens, {top} of {e} experts")
        count, keep = groups
        if bias is not None:
            self._f32_vector(bias, e, "experts_route_product bias")
        if scoring == "softmax_all":
            self._f32_vector(correction, e, "experts_route_product correction")
            if not (0 < keep <= count and e % count == 0 and top <= keep * (e // count)):
                raise KernelError(f"experts_route_product: {e} experts in {count} groups of which {keep} are kept, {top} a token")
        cap = self.experts_tile_capacity(t, e, top, rows_a_tile)
        self._i32(expert, t * top, "experts_route_product expert"); self._i32(order, t * top, "experts_route_product order")
        self._i32(tiles, 4 * cap, "experts_route_product tiles")
        if not (weight.is_cuda and weight.dtype == torch.float32 and weight.is_contiguous() and weight.numel() >= t * top):
            raise KernelError("experts_route_product weight must be float32 [T, top]")
        if t == 0:
            return
        lib = self.experts_lib()
        self._launch(lib, lib.ls_experts_route_product, (
            c_int(DTYPE_CODE[x.dtype]), _ptr(x), c_long(x.stride(0)), _ptr(w_router), c_int(k), _ptr(bias), c_int(t), c_int(e), c_int(top),
            c_int(rows_a_tile), _ptr(expert), _ptr(weight), _ptr(order), _ptr(tiles), c_int(cap),
            c_int(("softmax", "sigmoid", "softmax_all").index(scoring)), _ptr(correction), c_int(count), c_int(keep), _stream()))

    def experts_apply(self, x: torch.Tensor, w_gate: torch.Tensor, w_up: torch.Tensor, w_down: torch.Tensor, top: int,
                      rows_a_tile: int, order: torch.Tensor, tiles: torch.Tensor, weight: torch.Tensor, limit: float,
                      alpha: float, act: torch.Tensor, partials: torch.Tensor, shift: float = 1.0,
                      weigh_input: bool = False, identity: int = 0, shared=None) -> None:
        """``partials[k][t] = weight[t, k] * down_e(act(gate_e x[t], up_e x[t]))`` for every token's ``k``-th
        expert ``e``, with the clamped gated unit of ``glu_clamped`` as activation (``min(g, limit) sigmoid(alpha
        min(g, limit)) (clamp(u, -limit, limit) + shift)``; an infinite ``limit``, ``alpha`` 1 and ``shift`` 0 are the
        plain unit ``silu(g) u``).  ``w_gate``, ``w_up``
        ``[E, F, K]``, ``w_down [E, N, F]`` in the compute dtype; ``act``: scratch ``[T * top, F]`` of the
        compute dtype; ``partials [top, T, N]`` float32; the routing as ``experts_route`` left it.
        ``weigh_input``: the weight multiplies the expert's input instead, ``partials[k][t] = down_e(act(w gate_e
        x[t], w up_e x[t]))``.  ``identity``: that many experts behind those with weights return their input.
        ``shared`` (tiles of 16 rows only): an expert that every token uses, worked on in the same launches, as (its gate and
        up rows interleaved in tiles of 16, its down matrix ``[N, Fs]``, scratch ``[T, Fs]`` of the compute dtype, float32
        ``[T, N]`` for its output)."""
        _rows_ok(x, "experts_apply x"); _rows_ok(act, "experts_apply act")
        t, k = x.shape
        if not (w_gate.dim() == 3 and w_gate.shape == w_up.shape and w_gate.shape[2] == k and w_down.dim() == 3
                and w_down.shape[0] == w_gate.shape[0] and w_down.shape[2] == w_gate.shape[1]
                and w_gate.is_contiguous() and w_up.is_contiguous() and w_down.is_contiguous()
                and w_gate.dtype == x.dtype == w_up.dtype == w_down.dtype == act.dtype and x.dtype in DTYPE_CODE):
            raise KernelError("experts_apply weights must be [E, F, K], [E, F, K], [E, N, F] of the compute dtype")
        real, f, n = w_gate.shape[0], w_gate.shape[1], w_down.shape[1]
        e = real + identity
        if not (identity >= 0 and (identity == 0 or n == k)):
            raise KernelError(f"experts_apply: an expert that returns its input of {k} elements cannot stand beside outputs of {n}")
        cap = self.experts_tile_capacity(t, e, top, rows_a_tile)
        if not (act.shape[0] >= t * top and act.shape[1] == f):
            raise KernelError(f"experts_apply act must be [>= {t * top}, {f}]")
        if not (partials.is_cuda and partials.dtype == torch.float32 and partials.is_contiguous()
                and tuple(partials.shape) == (top, t, n)):
            raise KernelError(f"experts_apply partials must be float32 [{top}, {t}, {n}]")
        self._i32(order, t * top, "experts_apply order"); self._i32(tiles, 4 * cap, "experts_apply tiles")
        if not (weight.is_cuda and weight.dtype == torch.float32 and weight.is_contiguous() and weight.numel() >= t * top):
            raise KernelError("experts_apply weight must be float32 [T, top]")
        gate_up = down = sh_act = sh_out = None
        sh_f = sh_ld = 0
        if shared is not None:
            gate_up, down, sh_act, sh_out = shared
            sh_f = down.shape[1]
            _rows_ok(sh_act, "experts_apply shared act"); _rows_ok(sh_out, "experts_apply shared out")
            if not (rows_a_tile == 16 and gate_up.is_cuda and gate_up.is_contiguous() and down.is_contiguous() and gate_up.dtype == down.dtype
                    == sh_act.dtype == x.dtype and tuple(gate_up.shape) == (-(-sh_f // 16) * 32, k) and down.shape[0] == n
                    and sh_act.shape[0] >= t and sh_act.shape[1] == sh_f and sh_out.dtype == torch.float32 and sh_out.is_contiguous()
                    and tuple(sh_out.shape) == (t, n)):
                raise KernelError("experts_apply: the shared expert's operands do not fit, or the tiles have more than 16 rows")
            sh_ld = sh_act.stride(0)
        if t == 0:
            return
        lib = self.experts_lib()
        self._launch(lib, lib.ls_experts_apply, (
            c_int(DTYPE_CODE[x.dtype]), _ptr(x), c_long(x.stride(0)), _ptr(w_gate), _ptr(w_up), _ptr(w_down), c_int(t),
            c_int(e), c_int(top), c_int(k), c_int(f), c_int(n), c_int(rows_a_tile), _ptr(order), _ptr(tiles), c_int(cap),
            _ptr(weight), c_float(limit), c_float(alpha), c_float(shift), _ptr(act), c_long(act.stride(0)), _ptr(partials),
            c_int(int(bool(weigh_input))), c_int(real), _ptr(gate_up), _ptr(down), c_int(sh_f), _ptr(sh_act), c_long(sh_ld),
            _ptr(sh_out), _stream()))

    def experts_route_table(self, token_ids: torch.Tensor, table: torch.Tensor, experts: int, rows_a_tile: int,
                            expert: torch.Tensor, weight: torch.Tensor, order: torch.Tensor, tiles: torch.Tensor,
                            counts: torch.Tensor) -> None:
        """Routing without a router: token ``t`` uses the experts in row ``token_ids[t]`` of ``table [vocab, top]``
        (int32, entries in ``[0, experts)``, those of a row differ), each with the weight ``1 / top``.  The
        outputs are those of ``experts_route``."""
        if not (table.is_cuda and table.dtype == torch.int32 and table.dim() == 2 and table.is_contiguous()):
            raise KernelError("experts_route_table table must be int32 [vocab, top] on the GPU")
        t, top = token_ids.shape[0], table.shape[1]
        if not (0 < top <= experts):
            raise KernelError(f"experts_route_table: {top} experts a token of {experts}")
        self._i32(token_ids, t, "experts_route_table token_ids")
        cap = self.experts_tile_capacity(t, experts, top, rows_a_tile)
        self._i32(expert, t * top, "experts_route_table expert"); self._i32(order, t * top, "experts_route_table order")
        self._i32(tiles, 4 * cap, "experts_route_table tiles"); self._i32(counts, experts, "experts_route_table counts")
        if not (weight.is_cuda and weight.dtype == torch.float32 and weight.is_contiguous() and weight.numel() >= t * top):
            raise KernelError("experts_route_table weight must be float32 [T, top]")
        if t == 0:
            return
        lib = self.experts_lib()
        self._launch(lib, lib.ls_experts_route_table, (
            _ptr(token_ids), _ptr(table), c_int(t), c_int(experts), c_int(top), c_int(rows_a_tile), _ptr(expert),
            _ptr(weight), _ptr(order), _ptr(tiles), c_int(cap), _ptr(counts), _stream()))

    # -- a residual stream of several copies ------------------------------------------------------
    def streams_max(self) -> tuple[int, int]:
        """(the most copies, the widest row) that ``streams_step`` takes."""
        return self._memo(("streams_max",), lambda: (int(self.mixers_lib().ls_streams_max()),
                                                     int(self.mixers_lib().ls_streams_max_width())))

    def streams_step(self, x: torch.Tensor, copies: int, partials, mix, gain, take, weight, eps: float, out,
                     rows: torch.Tensor | None = None, bias=None, centred: bool = False) -> None:
        """One step of a residual stream of ``copies`` copies, ``x`` float32 ``[T, copies * width]``.  With
        ``partials [slices, T, width]`` (a sublayer's output as slice sums) the copies are rewritten:
        ``x'_t = sum_s mix[s, t] x_s + gain[t] y``, ``y`` the sum of the slices in ascending order.  With ``out
        [rows, width]`` the copies are then read: ``u = sum_t take[t] x'_t`` (``take`` None: their plain sum) and
        ``out = (u - m) / sqrt(mean((u - m)^2) + eps) * weight (+ bias)`` with ``m`` the row's mean if ``centred``, else 0.  ``rows`` selects rows of ``x`` (all without it)."""
        _rows_ok(x, "streams_step x")
        if not (x.dtype == torch.float32 and copies > 0 and x.shape[1] % copies == 0):
            raise KernelError("streams_step works on float32 rows of whole copies")
        width = x.shape[1] // copies
        most, widest = self.streams_max()
        if not (copies <= most and width <= widest):
            raise KernelError(f"streams_step takes up to {most} copies of up to {widest} elements, got {copies} of {width}")
        n_rows = x.shape[0] if rows is None else rows.shape[0]
        if rows is not None and not (rows.is_cuda and rows.dtype == torch.int32 and rows.is_contiguous()):
            raise KernelError("streams_step rows: int32 on the GPU")
        slices = p_rows = 0
        if partials is not None:
            if not (partials.is_cuda and partials.dtype == torch.float32 and partials.is_contiguous() and partials.dim() == 3
                    and partials.shape[2] == width and partials.shape[1] >= x.shape[0]):
                raise KernelError(f"streams_step partials must be float32 [slices, >= {x.shape[0]}, {width}]")
            slices, p_rows = partials.shape[0], partials.shape[1]
            self._f32_vector(mix, copies * copies, "streams_step mix"); self._f32_vector(gain, copies, "streams_step gain")
        if take is not None:
            self._f32_vector(take, copies, "streams_step take")
        dtype, ld_out = torch.float32, 0
        if out is not None:
            _rows_ok(out, "streams_step out")
            if not (out.dtype in DTYPE_CODE and tuple(out.shape) == (n_rows, width) and eps > 0):
                raise KernelError(f"streams_step out must be [{n_rows},{width}], eps positive")
            self._f32_vector(weight, width, "streams_step weight")
            if bias is not None:
                self._f32_vector(bias, width, "streams_step bias")
            dtype, ld_out = out.dtype, out.stride(0)
        elif partials is None:
            return
        if n_rows == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_streams_step, (
            c_int(DTYPE_CODE[dtype]), _ptr(x), c_long(x.stride(0)), c_int(copies), c_int(width), _ptr(partials),
            c_int(slices), c_int(p_rows), _ptr(mix), _ptr(gain), _ptr(take), _ptr(weight), _ptr(bias), c_int(int(centred)),
            c_float(eps), _ptr(out),
            c_long(ld_out), _ptr(rows), c_int(n_rows), _stream()))

    # -- attention over a cached latent: the passes around it ----------------------------------------
    def latent_post(self, raw: torch.Tensor, n_tokens: int, q_rank: int, kv_rank: int, rot_dim: int, key_pad: int,
                    has_kv: bool, q_weight, kv_weight, eps: float, cos, sin, rot: int, max_pos: int, tok_seq, tok_pos,
                    seqs, table, q_latent: torch.Tensor, k_pages, v_pages, page_size: int) -> None:
        """Post pass of the down projections ``raw`` (float32, ``a | c | r``): the query latent ``a`` normalised
        with ``q_weight`` (None: as it is) into ``q_latent``; with ``has_kv`` the latent ``c`` normalised with ``kv_weight`` into the
        key pages (dimensions ``0 .. kv_rank`` of the one key head of ``key_pad`` elements) and into the value
        pages, and the shared key part ``r``, rotated in neighbouring pairs on its first ``rot`` dimensions,
        behind it in the key pages."""
        _rows_ok(raw, "latent_post raw"); _rows_ok(q_latent, "latent_post q_latent")
        width = q_rank + (kv_rank + rot_dim if has_kv else 0)
        if not (raw.dtype == torch.float32 and raw.shape[0] >= n_tokens and raw.shape[1] >= width):
            raise KernelError(f"latent_post raw must be float32 [>= {n_tokens}, >= {width}]")
        if not (q_latent.dtype in DTYPE_CODE and q_latent.shape[0] >= n_tokens and q_latent.shape[1] == q_rank):
            raise KernelError("latent_post q_latent has the wrong shape or dtype")
        if q_weight is not None:
            self._f32_vector(q_weight, q_rank, "latent_post q_weight")
        positions = 0
        if has_kv:
            self._f32_vector(kv_weight, kv_rank, "latent_post kv_weight")
            positions = self._rotation_tables(cos, sin, rot, max_pos)
            self._paged_ok(k_pages, v_pages, table, q_latent.dtype, 1, page_size, key_pad, kv_rank)
            if not (key_pad >= kv_rank + rot_dim and max_pos // page_size < table.shape[1]):
                raise KernelError("latent_post: the key head is too short, or a position lies beyond the block table")
            for name, t in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
                if not (t.is_cuda and t.dtype == torch.int32 and t.is_contiguous() and t.numel() >= n_tokens):
                    raise KernelError(f"{name} must be int32 with at least {n_tokens} entries")
        if n_tokens == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_latent_post, (
            c_int(DTYPE_CODE[q_latent.dtype]), _ptr(raw), c_long(raw.stride(0)), c_int(n_tokens), c_int(q_rank),
            c_int(kv_rank), c_int(rot_dim), c_int(key_pad), c_int(int(has_kv)), _ptr(q_weight),
            _ptr(kv_weight if has_kv else None), c_float(eps), _ptr(cos if has_kv else None), _ptr(sin if has_kv else None),
            c_int(rot), c_int(positions), c_int(max_pos), _ptr(tok_seq), _ptr(tok_pos), _ptr(seqs),
            _ptr(table if has_kv else None), c_int(table.shape[1] if has_kv else 0), _ptr(q_latent),
            c_long(q_latent.stride(0)), _ptr(k_pages if has_kv else None), _ptr(v_pages if has_kv else None),
            c_int(page_size), _stream()))

    def latent_query(self, qf: torch.Tensor, n_tokens: int, heads: int, dim: int, rot_dim: int, kv_rank: int, key_pad: int,
                     cos, sin, rot: int, max_pos: int, tok_pos, plain: torch.Tensor, q_out: torch.Tensor) -> None:
        """Post pass of the queries' up projection ``qf`` (float32, heads of ``dim`` plain and ``rot_dim`` rotated
        dimensions): the plain parts into ``plain [T, heads*dim]``; the rotated parts, rotated in neighbouring
        pairs on their first ``rot`` dimensions, into ``q_out [T, heads*key_pad]`` behind the ``kv_rank``
        dimensions of each head that the product with the keys' up projection fills (zeros up to ``key_pad``)."""
        _rows_ok(qf, "latent_query qf"); _rows_ok(plain, "latent_query plain"); _rows_ok(q_out, "latent_query q_out")
        if not (qf.dtype == torch.float32 and qf.shape[0] >= n_tokens and qf.shape[1] == heads * (dim + rot_dim)):
            raise KernelError(f"latent_query qf must be float32 [>= {n_tokens}, {heads * (dim + rot_dim)}]")
        if not (plain.dtype in DTYPE_CODE and q_out.dtype == plain.dtype and plain.shape[0] >= n_tokens
                and plain.shape[1] == heads * dim and q_out.shape[0] >= n_tokens and q_out.shape[1] == heads * key_pad
                and key_pad >= kv_rank + rot_dim):
            raise KernelError("latent_query outputs have the wrong shape or dtype")
        positions = self._rotation_tables(cos, sin, rot, max_pos)
        if not (tok_pos.is_cuda and tok_pos.dtype == torch.int32 and tok_pos.is_contiguous() and tok_pos.numel() >= n_tokens):
            raise KernelError("latent_query tok_pos: int32, one position a token")
        if n_tokens == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_latent_query, (
            c_int(DTYPE_CODE[plain.dtype]), _ptr(qf), c_long(qf.stride(0)), c_int(n_tokens), c_int(heads), c_int(dim),
            c_int(rot_dim), c_int(kv_rank), c_int(key_pad), _ptr(cos), _ptr(sin), c_int(rot), c_int(positions),
            c_int(max_pos), _ptr(tok_pos), _ptr(plain), c_long(plain.stride(0)), _ptr(q_out), c_long(q_out.stride(0)),
            _stream()))

    def heads_product(self, x: torch.Tensor, x_stride: int, w: torch.Tensor, out: torch.Tensor, o_stride: int,
                      n_rows: int | None = None) -> None:
        """A product a head: ``out[t, h * o_stride + n] = sum_k w[h, n, k] x[t, h * x_stride + k]`` with
        ``w [heads, N, K]`` contiguous; ``x``, ``w`` and ``out`` in one compute dtype."""
        _rows_ok(x, "heads_product x"); _rows_ok(out, "heads_product out")
        n_rows = x.shape[0] if n_rows is None else n_rows
        if not (w.is_cuda and w.dim() == 3 and w.is_contiguous() and w.dtype in DTYPE_CODE and x.dtype == w.dtype == out.dtype):
            raise KernelError("heads_product w must be [heads, N, K] contiguous, all operands of one dtype")
        heads, n, k = w.shape
        if not (x.shape[0] >= n_rows and out.shape[0] >= n_rows and x.shape[1] >= (heads - 1) * x_stride + k
                and out.shape[1] >= (heads - 1) * o_stride + n and x_stride >= 0 and o_stride >= 0):
            raise KernelError("heads_product: the heads do not fit the rows")
        if n_rows == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_heads_product, (
            c_int(DTYPE_CODE[w.dtype]), _ptr(x), c_long(x.stride(0)), c_int(x_stride), _ptr(w), c_int(heads), c_int(n),
            c_int(k), c_int(n_rows), _ptr(out), c_long(out.stride(0)), c_int(o_stride), _stream()))

    # -- the gated delta rule -----------------------------------------------------------------------
    def delta_max_dim(self) -> int:
        return self._memo(("delta_max_dim",), lambda: int(self.mixers_lib().ls_delta_max_dim()))

    def delta_scratch_floats(self, n_tokens: int, kv_heads: int, heads: int, dim: int, vdim: int, channel: bool = False) -> int:
        lib = self.mixers_lib()
        entry = lib.ls_delta_scratch_floats_channel if channel else lib.ls_delta_scratch_floats
        entry.restype = ctypes.c_long
        return int(entry(c_int(n_tokens), c_int(kv_heads), c_int(heads), c_int(dim), c_int(vdim)))

    def delta_rule(self, raw: torch.Tensor, kv_heads: int, heads: int, dim: int, vdim: int, taps: torch.Tensor, a_log,
                   dt_bias, unit_eps: float, tok_seq, tok_pos, seqs, n_seqs: int, state: torch.Tensor,
                   scratch: torch.Tensor, out: torch.Tensor, channel_decay: torch.Tensor | None = None) -> None:
        """The gated delta rule over the tokens of every request of the step.  ``raw`` float32 holds the
        projections ``q | k`` (``kv_heads`` heads of ``dim``) ``| v`` (``heads`` of ``vdim``) ``| b | a``
        (``heads`` each); every channel of q, k and v passes a causal convolution with ``taps [channels, M]``
        (the last column is the current token's) and silu; q and k become unit vectors (``unit_eps`` inside
        the root), q also times ``dim^-1/2``; ``beta = sigmoid(b)``, ``decay = exp(-exp(a_log) softplus(a +
        dt_bias))``; per head ``S <- decay S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q``.  ``state``
        float32 ``[slots, heads*dim*vdim + (M-1)*channels]``: the matrices, then the convolutions' last inputs;
        read and left for the next step.  ``out`` float32 ``[T, heads*vdim]``.  ``channel_decay`` (float32 rows of
        ``heads*dim`` logits): a decay for every head and key channel instead, ``g = exp(-exp(a_log_h) softplus(logit +
        dt_bias))`` with ``dt_bias [heads*dim]``, which multiplies the rows of ``S``; ``raw`` then ends with ``b``."""
        _rows_ok(raw, "delta_rule raw"); _rows_ok(out, "delta_rule out")
        t = raw.shape[0]
        channels = 2 * kv_heads * dim + heads * vdim
        chan = channel_decay is not None
        ldc = 0
        if chan:
            _rows_ok(channel_decay, "delta_rule channel_decay")
            if not (channel_decay.dtype == torch.float32 and channel_decay.shape[0] >= t and channel_decay.shape[1] == heads * dim):
                raise KernelError(f"delta_rule channel_decay must be float32 [>= {t}, {heads * dim}]")
            ldc = channel_decay.stride(0)
        if not (raw.dtype == torch.float32 and raw.shape[1] >= channels + (1 if chan else 2) * heads and out.dtype == torch.float32
                and tuple(out.shape) == (t, heads * vdim)):
            raise KernelError("delta_rule reads and writes float32 rows, out [T, heads*vdim]")
        if not (heads % kv_heads == 0 and dim <= self.delta_max_dim()):
            raise KernelError(f"delta_rule: {heads} heads over {kv_heads} key heads, keys of at most {self.delta_max_dim()}")
        if not (taps.is_cuda and taps.dtype == torch.float32 and taps.is_contiguous() and taps.dim() == 2
                and taps.shape[0] == channels and taps.shape[1] >= 1):
            raise KernelError(f"delta_rule taps must be float32 [{channels}, M]")
        m = taps.shape[1]
        self._f32_vector(a_log, heads, "delta_rule a_log")
        self._f32_vector(dt_bias, heads * dim if chan else heads, "delta_rule dt_bias")
        if not (state.is_cuda and state.dtype == torch.float32 and state.is_contiguous() and state.dim() == 2
                and state.shape[1] == heads * dim * vdim + (m - 1) * channels):
            raise KernelError(f"delta_rule state must be float32 [slots, {heads * dim * vdim + (m - 1) * channels}]")
        if not (scratch.is_cuda and scratch.dtype == torch.float32 and scratch.is_contiguous()
                and scratch.numel() >= self.delta_scratch_floats(t, kv_heads, heads, dim, vdim, chan)):
            raise KernelError("delta_rule scratch: float32 of delta_scratch_floats elements")
        for name, v in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
            if not (v.is_cuda and v.dtype == torch.int32 and v.is_contiguous() and v.numel() >= t):
                raise KernelError(f"delta_rule {name}: int32, one entry a token")
        if n_seqs == 0 or t == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_delta_rule, (
            _ptr(raw), c_long(raw.stride(0)), c_int(t), c_int(kv_heads), c_int(heads), c_int(dim), c_int(vdim), c_int(m),
            _ptr(taps), _ptr(a_log), _ptr(dt_bias), c_float(unit_eps), _ptr(tok_seq), _ptr(tok_pos), _ptr(seqs),
            c_int(n_seqs), _ptr(state), c_long(state.stride(0)), _ptr(scratch), _ptr(out), c_long(out.stride(0)),
            _ptr(channel_decay), c_long(ldc), _stream()))

    # -- an embedding with a table of token pairs, and the shift of a sublayer's input by a token -------------
    def embed_pair(self, tokens: torch.Tensor, tok_seq, tok_pos, seqs, table: torch.Tensor, pairs: torch.Tensor,
                   mul_prev: int, mul_cur: int, state: torch.Tensor, out: torch.Tensor, scale: float = 1.0) -> None:
        """``out[t] = table[tokens[t]] * scale + pairs[(token before * mul_prev + tokens[t] * mul_cur) mod buckets]``
        as float32 rows, ``buckets = pairs.shape[0] - 1``; a request's first token takes the last row of ``pairs``.
        ``state`` int32 ``[slots, 1]``: the last token of every request so far, read for the first row of a portion
        and left as the portion's last token."""
        if not (tokens.is_cuda and tokens.dtype == torch.int32 and tokens.dim() == 1 and tokens.is_contiguous()):
            raise KernelError("embed_pair tokens must be a contiguous int32 vector on the GPU")
        t = tokens.shape[0]
        _rows_ok(table, "embed_pair table"); _rows_ok(pairs, "embed_pair pairs"); _rows_ok(out, "embed_pair out")
        if not (table.is_contiguous() and pairs.is_contiguous() and table.dtype in DTYPE_CODE and pairs.dtype == table.dtype
                and pairs.shape[1] == table.shape[1] and pairs.shape[0] >= 2):
            raise KernelError("embed_pair tables must be contiguous, of one dtype and one width, the pairs' with two rows or more")
        if not (out.dtype == torch.float32 and tuple(out.shape) == (t, table.shape[1])):
            raise KernelError(f"embed_pair out must be float32 [{t},{table.shape[1]}]")
        if not (state.is_cuda and state.dtype == torch.int32 and state.dim() == 2 and state.stride(1) == 1):
            raise KernelError("embed_pair state must be int32 [slots, 1] on the GPU")
        for name, v in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
            if not (v.is_cuda and v.dtype == torch.int32 and v.is_contiguous() and v.numel() >= t):
                raise KernelError(f"embed_pair {name}: int32, one entry a token")
        if t == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_embed_pair, (
            c_int(DTYPE_CODE[table.dtype]), _ptr(tokens), _ptr(tok_seq), _ptr(tok_pos), _ptr(seqs), _ptr(table),
            c_int(table.shape[0]), _ptr(pairs), c_int(pairs.shape[0] - 1), c_long(mul_prev), c_long(mul_cur), _ptr(state),
            c_long(state.stride(0)), _ptr(out), c_int(t), c_int(table.shape[1]), c_long(out.stride(0)), c_float(scale),
            _stream()))

    def add_rmsnorm_shift(self, h: torch.Tensor, partials, weight: torch.Tensor, eps: float, mu: torch.Tensor, tok_seq,
                          tok_pos, seqs, state: torch.Tensor, out: torch.Tensor) -> None:
        """For a step of single tokens, in one launch: ``h[t] += partials[0][t] + partials[1][t] + ...`` (``partials``
        may be None), ``n = rmsnorm(h[t]) * weight`` as ``rmsnorm`` computes it, ``out[t] = n + (kept - n) * mu`` with
        the request's row of ``state`` (zeros at its first token), which is then left as ``n``."""
        _rows_ok(h, "add_rmsnorm_shift h"); _rows_ok(out, "add_rmsnorm_shift out")
        t, width = h.shape
        if not (h.dtype == torch.float32 and out.dtype in DTYPE_CODE and tuple(out.shape) == (t, width) and width % 4 == 0):
            raise KernelError("add_rmsnorm_shift works on float32 rows of a multiple of four elements")
        self._f32_vector(weight, width, "add_rmsnorm_shift weight"); self._f32_vector(mu, width, "add_rmsnorm_shift mu")
        slices = p_rows = 0
        if partials is not None:
            if not (partials.is_cuda and partials.dtype == torch.float32 and partials.is_contiguous() and partials.dim() == 3
                    and partials.shape[2] == width and partials.shape[1] >= t):
                raise KernelError("add_rmsnorm_shift partials [slices, rows, width]")
            slices, p_rows = partials.shape[0], partials.shape[1]
        if not (state.is_cuda and state.dtype == torch.float32 and state.dim() == 2 and state.stride(1) == 1
                and state.shape[1] >= width):
            raise KernelError(f"add_rmsnorm_shift state must be float32 [slots, >= {width}]")
        for name, v in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
            if not (v.is_cuda and v.dtype == torch.int32 and v.is_contiguous() and v.numel() >= t):
                raise KernelError(f"add_rmsnorm_shift {name}: int32, one entry a token")
        if t == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_add_rmsnorm_shift, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(h), _ptr(partials), c_int(slices), c_int(p_rows), _ptr(weight), _ptr(mu),
            _ptr(tok_seq), _ptr(tok_pos), _ptr(seqs), _ptr(state), c_long(state.stride(0)), _ptr(out), c_int(t), c_int(width),
            c_long(h.stride(0)), c_long(out.stride(0)), c_float(eps), _stream()))

    def token_shift(self, normed: torch.Tensor, mu: torch.Tensor, tok_seq, tok_pos, seqs, state: torch.Tensor,
                    out: torch.Tensor) -> None:
        """``out[t] = n[t] + (n[t-1] - n[t]) * mu`` for the float32 rows ``normed`` of the step, ``n[t-1]`` being the row
        of the same request's token before (zeros at a request's first token); ``state`` float32 ``[slots, width]``
        holds that row for the first token of a portion and is left as the portion's last row."""
        _rows_ok(normed, "token_shift normed"); _rows_ok(out, "token_shift out")
        t, width = normed.shape
        if not (normed.dtype == torch.float32 and out.dtype in DTYPE_CODE and tuple(out.shape) == (t, width)):
            raise KernelError("token_shift reads float32 rows and writes rows of the same shape")
        self._f32_vector(mu, width, "token_shift mu")
        if not (state.is_cuda and state.dtype == torch.float32 and state.dim() == 2 and state.stride(1) == 1
                and state.shape[1] >= width):
            raise KernelError(f"token_shift state must be float32 [slots, >= {width}]")
        for name, v in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
            if not (v.is_cuda and v.dtype == torch.int32 and v.is_contiguous() and v.numel() >= t):
                raise KernelError(f"token_shift {name}: int32, one entry a token")
        if t == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_token_shift, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(normed), c_long(normed.stride(0)), _ptr(mu), _ptr(tok_seq), _ptr(tok_pos),
            _ptr(seqs), _ptr(state), c_long(state.stride(0)), _ptr(out), c_long(out.stride(0)), c_int(t), c_int(width),
            _stream()))

    # -- sublayers with norms on both sides, averages over depth ------------------------------------
    def residual_step(self, x: torch.Tensor, partials, post, results, keep: int, shares, norm, out,
                      rows: torch.Tensor | None = None) -> None:
        """One step of the float32 residual stream ``x [T, width]`` between two sublayers.  With ``partials [slices, T,
        width]`` (a sublayer's output as slice sums, added in ascending order to ``y``): ``x += y``, or, with ``post``,
        ``x += norm(y)``.  With ``results [layers + 1, T, width]``: ``results[keep] = x``; with ``shares [keep + 1]`` then
        ``x = sum_j shares[j] results[j]``.  With ``out [rows, width]``: ``out = norm(x)``.  ``post`` and ``norm`` are
        ``(weight, eps, centred)``, ``norm`` with an optional fourth entry, a bias (or None) that is added behind it; a norm is ``(v - m) / sqrt(mean((v - m)^2) + eps) * weight`` with ``m`` the row's mean
        if ``centred``, else 0.  ``rows`` selects rows of ``x``; then nothing but ``out`` is written."""
        _rows_ok(x, "residual_step x")
        t, width = x.shape
        lib = self.mixers_lib()
        widest = self._memo(("residual_step_max",), lambda: int(lib.ls_residual_step_max_width()))
        if not (x.dtype == torch.float32 and width <= widest):
            raise KernelError(f"residual_step works on float32 rows of up to {widest} elements")
        n_rows = t if rows is None else rows.shape[0]
        if rows is not None and not (rows.is_cuda and rows.dtype == torch.int32 and rows.is_contiguous() and out is not None):
            raise KernelError("residual_step rows: int32 on the GPU, and an output")
        slices = p_rows = r_rows = 0
        if partials is not None:
            if not (partials.is_cuda and partials.dtype == torch.float32 and partials.is_contiguous() and partials.dim() == 3
                    and partials.shape[2] == width and partials.shape[1] >= t):
                raise KernelError(f"residual_step partials must be float32 [slices, >= {t}, {width}]")
            slices, p_rows = partials.shape[0], partials.shape[1]
        post_weight, post_eps, post_centred = tuple(post)[:3] if post is not None else (None, 0.0, False)
        if post is not None and len(post) > 3 and post[3] is not None:
            raise KernelError("residual_step: a norm of the sublayer's output has no bias")
        if post is not None:
            if partials is None:
                raise KernelError("residual_step: a norm of the sublayer's output needs its slices")
            self._f32_vector(post_weight, width, "residual_step post weight")
        if results is not None:
            if not (results.is_cuda and results.dtype == torch.float32 and results.is_contiguous() and results.dim() == 3
                    and results.shape[2] == width and results.shape[1] >= t and 0 <= keep < results.shape[0]):
                raise KernelError(f"residual_step results must be float32 [> {keep}, >= {t}, {width}]")
            r_rows = results.shape[1]
        if shares is not None:
            if results is None:
                raise KernelError("residual_step: shares need results")
            self._f32_vector(shares, keep + 1, "residual_step shares")
        weight, eps, centred, bias, dtype, ld_out = None, 0.0, False, None, torch.float32, 0
        if out is not None:
            weight, eps, centred, bias = (tuple(norm) + (None,))[:4]
            if bias is not None:
                self._f32_vector(bias, width, "residual_step bias")
            _rows_ok(out, "residual_step out")
            if not (out.dtype in DTYPE_CODE and tuple(out.shape) == (n_rows, width) and eps > 0):
                raise KernelError(f"residual_step out must be [{n_rows},{width}], eps positive")
            self._f32_vector(weight, width, "residual_step weight")
            dtype, ld_out = out.dtype, out.stride(0)
        elif partials is None and results is None:
            return
        if n_rows == 0:
            return
        self._launch(lib, lib.ls_residual_step, (
            c_int(DTYPE_CODE[dtype]), _ptr(x), c_long(x.stride(0)), c_int(width), _ptr(partials), c_int(slices), c_int(p_rows),
            _ptr(post_weight), c_float(post_eps), c_int(int(post_centred)), _ptr(results), c_int(r_rows), c_int(keep),
            _ptr(shares), _ptr(weight), _ptr(bias), c_float(eps), c_int(int(centred)), _ptr(out), c_long(ld_out), _ptr(rows), c_int(n_rows),
            _stream()))

    def channel_recurrence(self, raw: torch.Tensor, a_at: int, u_at: int, g_at: int, a_bias, u_bias, seqs, n_seqs: int,
                           single_tokens: bool, state: torch.Tensor, out: torch.Tensor) -> None:
        """``S_t = (1 - z) S_(t-1) + z c``, ``out_t = S_t silu(g)`` element by element over the tokens of every request, with
        ``z = sigmoid(a + a_bias)`` and ``c = v + 1/2`` where ``v = u + u_bias >= 0``, else ``sigmoid(v)``.  ``raw`` float32
        rows that hold ``a``, ``u`` and ``g`` at the columns ``a_at``, ``u_at``, ``g_at``; ``state`` float32 ``[slots, width]``."""
        _rows_ok(raw, "channel_recurrence raw"); _rows_ok(out, "channel_recurrence out")
        t, width = out.shape
        if not (raw.dtype == torch.float32 and raw.shape[0] >= t and min(a_at, u_at, g_at) >= 0
                and raw.shape[1] >= max(a_at, u_at, g_at) + width and out.dtype in DTYPE_CODE):
            raise KernelError("channel_recurrence: the projections do not fit the float32 rows, or the output's dtype is wrong")
        self._f32_vector(a_bias, width, "channel_recurrence a_bias"); self._f32_vector(u_bias, width, "channel_recurrence u_bias")
        if not (state.is_cuda and state.dtype == torch.float32 and state.dim() == 2 and state.stride(1) == 1
                and state.shape[1] >= width):
            raise KernelError(f"channel_recurrence state must be float32 [slots, >= {width}]")
        if not (seqs.is_cuda and seqs.dtype == torch.int32 and seqs.is_contiguous() and seqs.numel() >= 8 * n_seqs):
            raise KernelError("channel_recurrence seqs: eight int32 a request")
        if t == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_channel_recurrence, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(raw), c_long(raw.stride(0)), c_int(a_at), c_int(u_at), c_int(g_at),
            _ptr(a_bias), _ptr(u_bias), c_int(width), _ptr(seqs), c_int(n_seqs), c_int(int(single_tokens)), _ptr(state),
            c_long(state.stride(0)), _ptr(out), c_long(out.stride(0)), _stream()))

    def embed_positions(self, tokens: torch.Tensor, tok_pos, table: torch.Tensor, freq: torch.Tensor, out: torch.Tensor,
                        scale: float = 1.0) -> None:
        """``out[t] = table[tokens[t]] * scale + v`` as float32 rows, ``v[2i] = sin(p freq[i])`` and ``v[2i + 1] = cos(p
        freq[i])`` at the token's position ``p``; ``freq`` float64 ``[(width + 1) // 2]``."""
        _rows_ok(table, "embed_positions table"); _rows_ok(out, "embed_positions out")
        t, width = out.shape
        for name, v in (("tokens", tokens), ("tok_pos", tok_pos)):
            if not (v.is_cuda and v.dtype == torch.int32 and v.dim() == 1 and v.is_contiguous() and v.shape[0] >= t):
                raise KernelError(f"embed_positions {name}: a contiguous int32 vector on the GPU, one entry a token")
        if not (table.is_contiguous() and table.dtype in DTYPE_CODE and table.shape[1] == width and out.dtype == torch.float32):
            raise KernelError("embed_positions: a contiguous float32/bfloat16 table and float32 rows of its width")
        if not (freq.is_cuda and freq.dtype == torch.float64 and freq.is_contiguous() and freq.numel() == (width + 1) // 2):
            raise KernelError(f"embed_positions freq must be float64 with {(width + 1) // 2} elements on the GPU")
        if t == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_embed_positions, (
            c_int(DTYPE_CODE[table.dtype]), _ptr(tokens), _ptr(tok_pos), _ptr(table), c_int(table.shape[0]), _ptr(freq),
            _ptr(out), c_int(t), c_int(width), c_long(out.stride(0)), c_float(scale), _stream()))

    # -- matrix memories with one gate a head and token ------------------------------------------------
    #: floats of a head's gates of a token (log a, b, floor, n . q)
    GATE_FLOATS = 4

    def memory_max_rows(self) -> int:
        return self._memo(("memory_max_rows",), lambda: int(self.mixers_lib().ls_memory_max_rows()))

    def memory_chunk(self) -> int:
        """Tokens of a chunk of ``memory_chunks``."""
        return self._memo(("memory_chunk",), lambda: int(self.mixers_lib().ls_memory_chunk()))

    def _memory_state(self, state, floats: int, what: str) -> None:
        if not (state.is_cuda and state.dtype == torch.float32 and state.dim() == 2 and state.stride(1) == 1 and state.shape[1] >= floats):
            raise KernelError(f"{what} state must be float32 [slots, >= {floats}]")

    def _gates_ok(self, gates, n_tokens: int, heads: int, what: str) -> None:
        if not (gates.is_cuda and gates.dtype == torch.float32 and gates.is_contiguous()
                and gates.numel() >= n_tokens * heads * self.GATE_FLOATS):
            raise KernelError(f"{what} gates: float32, four a token and head")

    def _tokens_ok(self, n_tokens: int, tok_seq, tok_pos, what: str) -> None:
        for name, v in (("tok_seq", tok_seq), ("tok_pos", tok_pos)):
            if not (v.is_cuda and v.dtype == torch.int32 and v.is_contiguous() and v.numel() >= n_tokens):
                raise KernelError(f"{what} {name}: int32, one entry a token")

    def _seqs_ok(self, seqs, n_seqs: int, what: str) -> None:
        self._i32(seqs, 8 * n_seqs, f"{what} seqs")

    def _space_ok(self, raw, x_at, dt_at, channels, heads, taps, conv_bias, a_log, dt_bias, what: str) -> int:
        _rows_ok(raw, f"{what} raw")
        if not (raw.dtype == torch.float32 and min(x_at, dt_at) >= 0 and raw.shape[1] >= max(x_at + channels, dt_at + heads)):
            raise KernelError(f"{what}: the projections do not fit the float32 rows")
        if not (taps.is_cuda and taps.dtype == torch.float32 and taps.is_contiguous() and taps.dim() == 2
                and taps.shape[1] == channels and taps.shape[0] >= 1):
            raise KernelError(f"{what} taps must be float32 [M, {channels}]")
        self._f32_vector(conv_bias, channels, f"{what} conv bias")
        self._f32_vector(a_log, heads, f"{what} a_log")
        self._f32_vector(dt_bias, heads, f"{what} dt_bias")
        return taps.shape[0]

    def conv_gates(self, raw: torch.Tensor, x_at: int, dt_at: int, channels: int, heads: int, taps: torch.Tensor, conv_bias, a_log,
                   dt_bias, tok_seq, tok_pos, seqs, n_seqs: int, state: torch.Tensor, ring_at: int, conv: torch.Tensor,
                   gates: torch.Tensor) -> None:
        """What a state-space mixer computes of a step's tokens before its memory.  Every one of the ``channels`` columns of
        the float32 rows ``raw`` from ``x_at`` on passes ``silu(bias + sum_m taps[m] in(p - M + 1 + m))`` into ``conv [T,
        channels]``; ``dt = softplus(raw[dt_at ..] + dt_bias)`` gives the gates ``log a = -exp(a_log) dt``, ``b = dt``.  ``taps [M,
        channels]``.  ``state``: at ``ring_at`` the ring ``[M, channels]`` of the request's last inputs, which this call moves on."""
        m = self._space_ok(raw, x_at, dt_at, channels, heads, taps, conv_bias, a_log, dt_bias, "conv_gates")
        t = raw.shape[0]
        self._memory_state(state, ring_at + m * channels, "conv_gates")
        self._gates_ok(gates, t, heads, "conv_gates")
        self._tokens_ok(t, tok_seq, tok_pos, "conv_gates")
        self._seqs_ok(seqs, n_seqs, "conv_gates")
        if not (conv.is_cuda and conv.dtype == torch.float32 and conv.is_contiguous() and tuple(conv.shape) == (t, channels)):
            raise KernelError(f"conv_gates conv must be float32 [{t}, {channels}]")
        if t == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_conv_gates, (
            _ptr(raw), c_long(raw.stride(0)), c_int(x_at), c_int(dt_at), c_int(t), c_int(channels), c_int(heads), c_int(m), _ptr(taps),
            _ptr(conv_bias), _ptr(a_log), _ptr(dt_bias), _ptr(tok_seq), _ptr(tok_pos), _ptr(seqs), c_int(n_seqs), _ptr(state),
            c_long(state.stride(0)), c_long(ring_at), _ptr(conv), _ptr(gates), _stream()))

    def exp_gates(self, raw: torch.Tensor, i_at: int, f_at: int, heads: int, i_bias, f_bias, cap: float, seqs, n_seqs: int,
                  state: torch.Tensor, max_at: int, gates: torch.Tensor) -> None:
        """Exponential gates: ``i = cap tanh((raw[i_at ..] + i_bias) / cap)``, ``f = logsigmoid(cap tanh((raw[f_at ..] + f_bias) /
        cap))``, a running maximum ``m = max(f + m, i)`` from zero; ``log a = f + m_before - m``, ``b = exp(i - m)``, floor
        ``exp(-m)``.  ``state``: at ``max_at`` two places of two floats a head, the maximum being the sum in the one of the length's parity."""
        _rows_ok(raw, "exp_gates raw")
        if not (raw.dtype == torch.float32 and cap > 0 and min(i_at, f_at) >= 0 and raw.shape[1] >= max(i_at, f_at) + heads):
            raise KernelError("exp_gates: the projections do not fit the float32 rows, or the cap is not positive")
        self._f32_vector(i_bias, heads, "exp_gates i_bias"); self._f32_vector(f_bias, heads, "exp_gates f_bias")
        self._memory_state(state, max_at + 4 * heads, "exp_gates")
        self._gates_ok(gates, raw.shape[0], heads, "exp_gates")
        self._seqs_ok(seqs, n_seqs, "exp_gates")
        if raw.shape[0] == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_exp_gates, (
            _ptr(raw), c_long(raw.stride(0)), c_int(i_at), c_int(f_at), c_int(heads), _ptr(i_bias), _ptr(f_bias), c_float(cap),
            _ptr(seqs), c_int(n_seqs), _ptr(state), c_long(state.stride(0)), c_long(max_at), _ptr(gates), _stream()))

    def _memory_rows(self, rows, heads: int, size: int, n_tokens: int, what: str):
        """``rows``: (float32 rows, column of head 0, heads that share one) of q, k or v; their pointer, strides and share."""
        t, at, share = rows
        _rows_ok(t, what)
        if not (t.dtype == torch.float32 and share > 0 and heads % share == 0 and at >= 0 and t.shape[0] >= n_tokens
                and t.shape[1] >= at + (heads // share) * size):
            raise KernelError(f"{what}: {heads // max(share, 1)} heads of {size} do not fit the float32 rows")
        return c_void_p(t.data_ptr() + 4 * at), c_long(t.stride(0)), c_int(size), c_int(share)

    def memory(self, q, k, v, gates: torch.Tensor, heads: int, rows: int, vdim: int, q_scale: float, skip, norm: bool, seqs,
               n_seqs: int, longest: int, walks: bool, items, n_items: int, runs, n_runs: int, states, decays, state: torch.Tensor,
               out: torch.Tensor) -> None:
        """A matrix memory over the tokens of every request of the step: per head ``S <- a S + b k v^T`` (``rows x vdim``),
        ``out = S^T q * q_scale + skip v``; with ``norm`` also ``n <- a n + b k`` and ``n . q`` into the gates' last place.  ``q``,
        ``k``, ``v``: (float32 rows ``[T, .]``, first column, heads that share one); ``gates`` as ``conv_gates`` or ``exp_gates``
        left them.  Requests of at most ``longest`` tokens walk token by token (``walks``: there are some); the others go
        by chunks of ``memory_chunk()`` tokens: ``items`` (request of the step, chunk) and ``runs`` (request, first item,
        items, 0) name them, ``states [n_items, floats]`` and ``decays [n_items, heads]`` are scratch.  ``state [slots, .]``: ``S``,
        then ``n``."""
        t = out.shape[0]
        floats = heads * rows * vdim + (heads * rows if norm else 0)
        if not (0 < rows <= self.memory_max_rows()):
            raise KernelError(f"memory: states of at most {self.memory_max_rows()} rows a head, got {rows}")
        _rows_ok(out, "memory out")
        if not (out.dtype == torch.float32 and out.shape[1] == heads * vdim):
            raise KernelError(f"memory out must be float32 [T, {heads * vdim}]")
        self._memory_state(state, floats, "memory")
        self._gates_ok(gates, t, heads, "memory")
        self._seqs_ok(seqs, n_seqs, "memory")
        if skip is not None:
            self._f32_vector(skip, heads, "memory skip")
        if v[2] != 1:
            raise KernelError("memory: every head has values of its own")
        qa = self._memory_rows(q, heads, rows, t, "memory q")
        ka = self._memory_rows(k, heads, rows, t, "memory k")
        va = self._memory_rows(v, heads, vdim, t, "memory v")[:3]
        if n_items:
            self._i32(items, 2 * n_items, "memory items"); self._i32(runs, 4 * n_runs, "memory runs")
            for name, s, n in (("states", states, n_items * floats), ("decays", decays, n_items * heads)):
                if not (s is not None and s.is_cuda and s.dtype == torch.float32 and s.is_contiguous() and s.numel() >= n):
                    raise KernelError(f"memory {name}: float32 scratch of {n} elements")
        if t == 0:
            return
        lib = self.mixers_lib()
        head = (*qa, *ka, *va, _ptr(gates), c_int(heads), c_int(rows), c_int(vdim), c_float(q_scale), _ptr(skip), c_int(int(norm)),
                _ptr(seqs))
        tail = (_ptr(state), c_long(state.stride(0)), _ptr(out), c_long(out.stride(0)), _stream())
        if walks:
            self._launch(lib, lib.ls_memory_walk, (*head, c_int(n_seqs), c_int(longest), *tail))
        if n_items:
            self._launch(lib, lib.ls_memory_chunks, (*head, _ptr(items), c_int(n_items), _ptr(runs), c_int(n_runs), _ptr(states),
                                                     c_long(floats), _ptr(decays), *tail))

    def space_token(self, raw: torch.Tensor, x_at: int, dt_at: int, groups: int, taps: torch.Tensor, conv_bias, a_log, dt_bias, skip,
                    heads: int, rows: int, vdim: int, seqs, n_seqs: int, state: torch.Tensor, ring_at: int, out: torch.Tensor) -> None:
        """A step of single tokens of a state-space mixer in one launch: what ``conv_gates`` and ``memory`` do (channels ``x``
        (heads x vdim) ``| B | C`` (groups x rows each) from ``x_at`` on)."""
        channels = heads * vdim + 2 * groups * rows
        m = self._space_ok(raw, x_at, dt_at, channels, heads, taps, conv_bias, a_log, dt_bias, "space_token")
        self._f32_vector(skip, heads, "space_token skip")
        self._memory_state(state, ring_at + m * channels, "space_token")
        self._seqs_ok(seqs, n_seqs, "space_token")
        _rows_ok(out, "space_token out")
        if not (out.dtype == torch.float32 and tuple(out.shape) == (n_seqs, heads * vdim) and raw.shape[0] >= n_seqs and heads % groups == 0):
            raise KernelError(f"space_token out must be float32 [{n_seqs}, {heads * vdim}], heads a multiple of the groups")
        if n_seqs == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_space_token, (
            _ptr(raw), c_long(raw.stride(0)), c_int(x_at), c_int(dt_at), c_int(channels), c_int(groups), c_int(m), c_long(ring_at),
            _ptr(taps), _ptr(conv_bias), _ptr(a_log), _ptr(dt_bias), _ptr(skip), c_int(heads), c_int(rows), c_int(vdim), _ptr(seqs),
            c_int(n_seqs), _ptr(state), c_long(state.stride(0)), _ptr(out), c_long(out.stride(0)), _stream()))

    def exp_token(self, raw: torch.Tensor, q_at: int, k_at: int, v_at: int, i_at: int, f_at: int, i_bias, f_bias, cap: float,
                  q_scale: float, heads: int, rows: int, vdim: int, seqs, n_seqs: int, state: torch.Tensor, max_at: int,
                  gates, out: torch.Tensor, normed=None) -> None:
        """A step of single tokens of a memory with exponential gates in one launch: what ``exp_gates`` and ``memory`` do.
        ``normed`` (heads of at most ``exp_token_whole()`` columns): (weight ``[heads*vdim]``, column of the gate's logits, eps,
        denom_eps); ``out`` then gets what ``head_norm_gate`` would leave, in its dtype, and there are no ``gates``."""
        _rows_ok(raw, "exp_token raw"); _rows_ok(out, "exp_token out")
        if not (raw.dtype == torch.float32 and cap > 0 and min(q_at, k_at, v_at, i_at, f_at) >= 0 and raw.shape[0] >= n_seqs
                and raw.shape[1] >= max(max(q_at, k_at) + heads * rows, v_at + heads * vdim, max(i_at, f_at) + heads)):
            raise KernelError("exp_token: the projections do not fit the float32 rows, or the cap is not positive")
        self._f32_vector(i_bias, heads, "exp_token i_bias"); self._f32_vector(f_bias, heads, "exp_token f_bias")
        self._memory_state(state, max_at + 4 * heads, "exp_token")
        self._seqs_ok(seqs, n_seqs, "exp_token")
        weight, g_at, eps, denom_eps = normed if normed is not None else (None, 0, 0.0, 0.0)
        if normed is None:
            self._gates_ok(gates, n_seqs, heads, "exp_token")
        else:
            self._f32_vector(weight, heads * vdim, "exp_token weight")
            if not (vdim <= self.exp_token_whole() and 0 <= g_at <= raw.shape[1] - heads * vdim and eps > 0):
                raise KernelError(f"exp_token: the norm behind takes heads of up to {self.exp_token_whole()} columns and a gate inside the rows")
        if not (out.dtype in DTYPE_CODE and (normed is not None or out.dtype == torch.float32) and tuple(out.shape) == (n_seqs, heads * vdim)):
            raise KernelError(f"exp_token out must be [{n_seqs}, {heads * vdim}], float32 without a norm behind")
        if n_seqs == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_exp_token, (
            _ptr(raw), c_long(raw.stride(0)), c_int(q_at), c_int(k_at), c_int(v_at), c_int(i_at), c_int(f_at), c_long(max_at),
            _ptr(i_bias), _ptr(f_bias), c_float(cap), c_float(q_scale), c_int(heads), c_int(rows), c_int(vdim), _ptr(seqs),
            c_int(n_seqs), _ptr(state), c_long(state.stride(0)), _ptr(gates if normed is None else None),
            _ptr(out if normed is None else None), c_long(out.stride(0)), c_int(DTYPE_CODE[out.dtype]), _ptr(weight), c_int(g_at),
            c_float(eps), c_float(denom_eps), _ptr(out if normed is not None else None), c_long(out.stride(0)), _stream()))

    def exp_token_whole(self) -> int:
        """Columns a head may have for ``exp_token`` to norm it in the same launch."""
        return self._memo(("exp_token_whole",), lambda: int(self.mixers_lib().ls_exp_token_whole()))

    def gated_parts_norm(self, y: torch.Tensor, z: torch.Tensor, parts: int, weight, eps: float, out: torch.Tensor) -> None:
        """``y * silu(z)``, divided by its root mean square in each of ``parts`` equal runs of a row (``eps`` inside the
        root), times ``weight``; ``y`` and ``z`` float32 rows."""
        _rows_ok(y, "gated_parts_norm y"); _rows_ok(z, "gated_parts_norm z"); _rows_ok(out, "gated_parts_norm out")
        t, inner = out.shape
        if not (y.dtype == torch.float32 and z.dtype == torch.float32 and tuple(y.shape) == (t, inner) and tuple(z.shape) == (t, inner)
                and out.dtype in DTYPE_CODE and parts > 0 and inner % parts == 0 and eps > 0):
            raise KernelError(f"gated_parts_norm: float32 rows of {inner} elements in {parts} equal parts, eps positive")
        self._f32_vector(weight, inner, "gated_parts_norm weight")
        if t == 0:
            return
        lib = self.mixers_lib()
        self._launch(lib, lib.ls_gated_parts_norm, (
            c_int(DTYPE_CODE[out.dtype]), _ptr(y), c_long(y.stride(0)), _ptr(z), c_long(z.stride(0)), c_int(t), c_int(inner),
            c_int(parts), _ptr(weight), c_float(eps), _ptr(out), c_long(out.stride(0)), _stream()))


ATTENTION_ITEM_INTS = 32
COMBINE_ITEM_INTS = 8


def pack_attention_items(items, seqs, pages=None) -> "np.ndarray":
    """Work items of the attention kernels as the device wants them.  ``items``:
    rows of (seq, row_block, split_begin, split_end, part_base, n_splits,
    split_lo, 0), seq -1 for an item that stands for no work; ``seqs``: the step's rows of (q_off, q_len, q_start, kv_len,
    table_row, 0, 0, 0).  Each item gets a copy of its request's row appended, so
    that a workgroup learns its work from one load, and sixteen more ints: with ``pages`` (an int array
    ``[items, 16]``, or None) the block-table entries of the item's one key tile, which the fused decode kernel
    then takes from the item instead of the block table (the eighth int of the item says so)."""
    import numpy as np

    items = np.asarray(items, dtype=np.int64).reshape(-1, 8)
    seqs = np.asarray(seqs, dtype=np.int64).reshape(-1, 8)
    if not len(items):
        return np.zeros(0, dtype=np.int64)
    null = items[:, 0] < 0
    rows = seqs[np.maximum(items[:, 0], 0)]
    rows[null] = 0                               # a null item is all zeros: a request of no rows, no splits
    items = np.where(null[:, None], 0, items)
    if pages is None:
        ids = np.zeros((len(items), 16), dtype=np.int64)
    else:
        ids = np.asarray(pages, dtype=np.int64).reshape(len(items), 16)
        ids = np.where(null[:, None], 0, ids)
        items = items.copy()
        items[:, 7] = np.where(null, 0, 1)
    return np.concatenate([items, rows, ids], axis=1).reshape(-1)


def pack_combine_items(items, seqs) -> "np.ndarray":
    """Combine items (seq, row_block, part_base, n_splits) with q_off and q_len of their request appended."""
    import numpy as np

    items = np.asarray(items, dtype=np.int64).reshape(-1, 4)
    seqs = np.asarray(seqs, dtype=np.int64).reshape(-1, 8)
    if not len(items):
        return np.zeros(0, dtype=np.int64)
    pad = np.zeros((len(items), 2), dtype=np.int64)
    null = items[:, 0] < 0
    rows = seqs[np.maximum(items[:, 0], 0), :2]
    rows[null] = 0
    items = np.where(null[:, None], 0, items)
    return np.concatenate([items, rows, pad], axis=1).reshape(-1)


_INSTANCE: Kernels | None = None


def kernels() -> Kernels:
    global _INSTANCE
    if _INSTANCE is None:
        _INSTANCE = Kernels()
    return _INSTANCE
