"""The kernel library as the parts see it: hand-written HIP kernels for gfx950,
called through a C ABI on torch tensors.  There is no CPU path and no
fallback: without the library, or without a GPU, construction fails.

Every wrapper checks on the host that shapes, dtypes and devices are what the
kernel and its grid assume before anything is launched.
"""
from __future__ import annotations

import contextlib
import ctypes
import os
from ctypes import c_float, c_int, c_void_p
from typing import Optional, Tuple

import torch

from . import build

F32, BF16 = 0, 1


class KernelError(RuntimeError):
    pass


class PendingProduct:
    """x W^T not run yet: what ``linear(..., deferred=True)`` returns for a decode step's
    few rows.  ``add_rmsnorm(..., lazy=True)`` runs it with the residual sum and the
    norm taken into the product; anything else runs it as it is (``resolve``)."""

    def __init__(self, x: torch.Tensor, matrix):
        self.x, self.matrix = x, matrix
        self.shape = (x.shape[0], _shape_of(matrix)[0])
        self.dtype = x.dtype


class NormedRows:
    """Rows of a norm whose scalar factor is still owed: ``xw`` = bfloat16(weight * h)
    [rows, n] and ``ssq`` [parts, rows], partial sums of h^2 in float32; the normed rows
    are xw / sqrt(sum(ssq) / n + eps).  ``linear`` and ``linear_swiglu`` take it as their
    input and apply the factor to their outputs."""

    def __init__(self, xw: torch.Tensor, ssq: torch.Tensor, eps: float):
        self.xw, self.ssq, self.eps = xw, ssq, float(eps)
        self.shape = tuple(xw.shape)
        self.dtype = xw.dtype


def _dtype_code(dtype: torch.dtype) -> int:
    if dtype == torch.float32:
        return F32
    if dtype == torch.bfloat16:
        return BF16
    raise KernelError(f"kernels take float32 or bfloat16 tensors, not {dtype}")


# what a product without a gate passes for the activation, the factor and the distance of the outputs' rows
_NO_GATE = (0, 1.0, 0)
_LIB = None


def load_library():
    """Load (building it first if nothing is built) the shared library."""
    global _LIB
    if _LIB is not None:
        return _LIB
    path = build.find_library() or build.build_library()
    try:
        lib = ctypes.CDLL(path)
    except OSError as exc:
        raise KernelError(f"cannot load the kernel library {path}: {exc}") from None
    lib.tli_last_error.restype = ctypes.c_char_p
    P, I, F = c_void_p, c_int, c_float
    sigs = {
        "tli_abi_version": [],
        "tli_device_compute_units": [],
        "tli_embed": [P, P, P, I, I, I, I, P],
        "tli_feed_tokens": [P, P, P, I, I, P],
        "tli_add_rmsnorm": [P, P, P, P, P, I, I, I, F, I, I, P],
        "tli_swiglu": [P, P, I, I, I, F, F, I, F, I, P],
        "tli_qkv_to_cache": [P, P, P, P, P, P, P, I, I, I, I, I, I, I, P, F, P, F, P, P, I, I, I, I, I, P],
        "tli_values_to_cache": [P, P, P, P, I, I, P, I, I, I, I, I, I, P],
        "tli_keys_values_to_cache": [P, P, P, P, P, I, I, P, I, I, I, I, I, I, P, F, P, P, I, P],
        "tli_attention_plain": [P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, I, P],
        "tli_gemm_plain": [P, P, P, I, I, I, I, I, I, P],
        "tli_gemm_skinny_bf16": [P, P, P, I, I, I, I, I, I, I, F, I, P],
        "tli_gemm_skinny_fused_bf16": [P, P, P, I, I, I, I, P, I, F, P, P, P, P, I, I, F, I, P],
        "tli_gemm_mid_bf16": [P, P, P, P, I, I, I, I, I, I, I, I, F, I, P],
        "tli_gemm_mid_splits": [I, I, I],
        "tli_gemm_mid_splits_rows": [I, I, I, I],
        "tli_gemm_mid_reduce": [P, P, I, I, I, I, P],
        "tli_gemm_rows_bf16": [P, P, P, P, I, I, I, I, I, I, I, F, I, P],
        "tli_gemm_rows_splits": [I, I, I],
        "tli_attention_decode_bf16": [P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, I, I, P],
        "tli_qkv_attention_decode_bf16": [P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, P, F, P, F, P, P, I,
                                          F, I, I, I, P, I, P],
        "tli_attention_prefill_bf16": [P, P, P, P, P, P, I, I, P, I, I, I, I, I, I, F, I, I, P, P],
        "tli_qkv_attention_prefill_bf16": [P, P, P, P, P, P, I, I, P, I, I, I, I, I, I, P, F, P, P, F, I, I, P],
        "tli_embed_scaled": [P, P, P, P, P, I, I, I, I, F, I, P],
        "tli_activation": [P, P, ctypes.c_longlong, I, I, P],
        "tli_softcap": [P, ctypes.c_longlong, F, P],
        "tli_streams_open": [P, P, I, I, I, P],
        "tli_streams_norm": [P, P, P, P, P, P, P, P, I, I, I, I, F, I, I, P, P, P, P, P, I, P],
        "tli_token_shift": [P, P, P, P, P, P, P, P, I, I, I, P],
        "tli_conv_heads": [P, P, P, P, P, P, P, P, P, P, I, I, P, I, I, I, I, I, I, I, I, I, P],
        "tli_attention_biased_plain": [P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, P, P, P, I, I, I, P],
        "tli_attention_biased_mfma_bf16": [P, P, P, P, P, P, I, I, I, P, I, I, I, I, I, I, F, P, P, P, I, I, I, P],
        "tli_add_layernorm": [P, P, P, P, P, P, P, P, I, I, I, F, I, P],
        "tli_delta_prepare": [P, I, P, P, P, ctypes.c_longlong, ctypes.c_longlong, P, P, P, P, P, P, P, P, P, P, P, P, P,
                              I, I, I, I, I, I, I, I, P],
        "tli_delta_recurrence": [P, P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, P],
        "tli_delta_state_floats": [I, I],
        "tli_gated_rmsnorm": [P, P, I, P, P, I, I, I, F, I, P],
        "tli_moe_route": [P, ctypes.c_longlong, ctypes.c_longlong, P, P, P, I, I, I, I, I, F, I, I, I, I, P, P],
        "tli_moe_router_bf16": [P, P, I, P, P, P, I, I, I, I, I, F, I, I, I, I, P, P],
        "tli_moe_experts": [P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, F, F, I, I, P],
        "tli_norm_add": [P, P, P, P, I, I, F, I, P],
        "tli_residual_rows": [P, P, ctypes.c_longlong, P],
        "tli_attention_sized_plain": [P, P, P, P, P, P, P, I, I, I, I, I, I, I, I, I, F, I, I, I, I, P, P],
        "tli_attention_sized_mfma_takes": [I, I, I, I],
        "tli_head_products_mfma_takes": [I, I] + [ctypes.c_longlong] * 4,
        "tli_head_products_mfma_bf16": [P, ctypes.c_longlong, ctypes.c_longlong, P, P, ctypes.c_longlong, ctypes.c_longlong,
                                        I, I, I, I, P, I, P],
        "tli_attention_sized_mfma_bf16": [P, P, P, P, P, P, I, I, P, I, I, I, I, I, I, I, I, F, I, I, I, I, P, I, P, P],
        "tli_diff_prepare": [P, I, P, P, P, P, P, P, I, I, I, I, I, I, I, I, P, P, F, I, P],
        "tli_diff_combine": [P, P, I, I, P, I, I, I, F, F, F, I, P],
        "tli_latent_prepare": [P, I, P, I, P, P, P, P, P, I, I, I, I, I, I, I, I, I, P, F, P, P, I, P],
        "tli_head_products_plain": [P, ctypes.c_longlong, ctypes.c_longlong, P, P, ctypes.c_longlong, ctypes.c_longlong,
                                    I, I, I, I, P, I, I, P],
        "tli_moe_grouped_tile": [I, I],
        "tli_moe_grouped_bf16": [P, P, P, P, P, P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, F, F, I, I, P],
        "tli_keyed_prepare": [P, I, P, P, P, P, P, P, P, I, I, I, I, I, I, I, I, P, P, I, I, I, P],
        "tli_add_bias": [P, P, I, I, I, P],
        "tli_lightning_recurrence": [P, I, P, P, P, P, P, P, P, I, I, I, I, I, I, I, I, P],
        "tli_lightning_norm": [P, P, I, P, P, I, I, F, I, P],
        "tli_retention": [P, I, P, P, P, P, P, P, P, P, P, P, I, I, I, F, I, I, I, I, I, I, I, I, P],
        "tli_retention_step": [P, I, P, P, P, I, P, P, P, P, P, I, I, I, F, F, F, I, I, I, I, I, P],
        "tli_mlstm_step": [P, I, P, P, I, P, I, F, P, F, F, P, P, P, P, I, P, P, F, F, I, I, I, I, I, P],
        "tli_chunked_takes": [I, I, I, I],
        "tli_retention_chunked_bf16": [P, I, P, P, P, I, P, P, P, P, P, P, I, I, I, F, F, F, I, I, I, I, I, P],
        "tli_mlstm_chunked_bf16": [P, I, P, ctypes.c_longlong, ctypes.c_longlong, P, I, I, F, P, F, F, P, P, P, P, I, P, P, P, P, P, F, F, I, I, I, I, I, P],
        "tli_mlstm": [P, I, P, ctypes.c_longlong, ctypes.c_longlong, P, I, I, F, P, F, F, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, I, I, P],
        "tli_head_norm_gate": [P, P, P, P, I, P, I, I, I, I, F, I, F, I, P],
        "tli_pooled_prepare": [P, I, P, P, P, P, P, P, P, P, I, P, I, I, I, I, I, I, I, I, P, P, F, P, P, I, I, I, P, P, P, I, I, I, I, I, P],
        "tli_attention_pooled_plain": [P, P, P, P, P, P, P, I, I, I, I, I, I, I, I, F, I, P, P, P, I, I, I, I, P, I, F, P],
        "tli_pooled_prefill_takes": [I, I, I, I, I, I],
        "tli_pooled_prefill_bf16": [P, P, P, P, P, P, I, I, P, I, I, I, I, I, I, I, F, I, P, P, P, I, I, I, I, P, I, F, P],
        "tli_attention_pooled_mfma_bf16": [P, P, P, P, P, P, I, I, P, I, I, I, I, I, I, I, F, I, P, P, P, I, I, I, I, P, I, F, I, P, P],
        "tli_norm_add_norm": [P, P, I, I, P, F, P, F, P, P, I, I, P, I, P, P, P, I, P],
        "tli_gemm_skinny_unit_bf16": [P, P, P, I, I, I, I, P, P, I, I, P],
        "tli_gemm_mid_unit_bf16": [P, P, P, I, I, I, I, P, P, I, I, P],
        "tli_gemm_reduce_unit_bf16": [P, P, I, I, I, I, P, P, I, I, P],
        "tli_token_mixes": [P, P, I, P, P, P, P, P, P, I, I, I, P],
        "tli_norm_rows": [P, I, P, P, I, I, F, I, P],
        "tli_token_gate": [P, P, P, P, I, I, I, I, I, I, I, P],
        "tli_wkv_decays": [P, ctypes.c_longlong, ctypes.c_longlong, P, P, P, I, I, I, I, P],
        "tli_gemm_skinny_groups_bf16": [P, P, P, I, I, I, I, I, ctypes.c_longlong, P],
        "tli_gemm_mid_groups_bf16": [P, P, P, P, I, I, I, I, I, I, ctypes.c_longlong, P],
        "tli_gemm_rows_groups_bf16": [P, P, P, P, I, I, I, I, I, ctypes.c_longlong, P],
        "tli_wkv_chunked_takes": [I, I, I],
        "tli_wkv_chunked_bf16": [P, I, P, ctypes.c_longlong, ctypes.c_longlong, P, P, I, P, P, P, I, P, P, P, P, P, F, I, I, I, I, I, P],
        "tli_wkv_step": [P, I, I, P, ctypes.c_longlong, ctypes.c_longlong, P, P, I, P, P, P, P, I, P, P, F, I, I, I, I, I, P],
        "tli_wkv_rows": [P, I, P, P, P, P, P, P, P, I, I, I, I, I, P],
        "tli_sample": [P, I, I, P, P, P, P, P, P],
        "tli_sample_scratch_bytes": [I],
        "tli_random_normal": [P, ctypes.c_longlong, ctypes.c_uint32, ctypes.c_uint32, ctypes.c_uint32, P, F, F, I, P],
    }
    for name, args in sigs.items():
        fn = getattr(lib, name)
        fn.argtypes = args
        fn.restype = c_int
    lib.tli_lightning_scratch_floats.argtypes = [I, I, I, I, I, I]
    lib.tli_lightning_scratch_floats.restype = ctypes.c_longlong
    lib.tli_wkv_chunked_scratch_floats.argtypes = [I, I, I, I, I]
    lib.tli_wkv_chunked_scratch_floats.restype = ctypes.c_longlong
    lib.tli_chunked_scratch_floats.argtypes = [I, I, I, I, I]
    lib.tli_chunked_scratch_floats.restype = ctypes.c_longlong
    lib.tli_sample_uniform.argtypes = [ctypes.c_uint32, ctypes.c_uint32, ctypes.c_uint32]
    lib.tli_sample_uniform.restype = c_float
    _LIB = lib
    return lib


def _shape_of(w) -> Tuple[int, int]:
    """(out, in) of a [out, in] tensor or of a matrix as the parts hold it, without asking for its
    row-major form (which such a matrix may have to put together first)."""
    shape = getattr(w, "shape", None)
    return tuple(shape) if shape is not None else tuple(w.w.shape)


def _ptr(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


class DeferredSum:
    """A matrix product whose k range was split, left as float32 partial sums
    [splits, rows, cols].  ``HipOps.linear(..., deferred=True)`` may return one
    instead of a tensor; ``add_rmsnorm`` takes it as the delta and adds the parts
    itself (rounding the sum to ``dtype`` as the product's own reduction would),
    anything else calls ``HipOps.resolve`` first."""

    def __init__(self, parts: torch.Tensor, dtype: torch.dtype):
        self.parts = parts
        self.dtype = dtype
        self.shape = tuple(parts.shape[1:])


class HipOps:
    name = "hip-gfx950"
    MAX_HEAD_DIM = 512
    SKINNY_ROWS = 64
    MID_ROWS_FROM = 17           # from this many rows the x-sharing kernel multiplies,
    MID_ROWS_TO = 128            # up to this many
    MID_ROWS_TO_PLAIN = 256      # a product without a gate: up to this many (two blocks of 128 rows side by side)
    DECODE_WORKGROUPS = 256      # the device's compute units (set to what the device reports when the library is loaded):
                                 # the decode attention splits a row's keys to come near one workgroup for each
    DECODE_SPLIT_KEYS = 1024     # a split walks at least this many keys
    # A step of prompt portions whose first sequences decode: the prefill kernel takes a row that decodes
    # as a sequence of one row, beside its other workgroups; the decode kernel is a second launch (8 to 10
    # us) that runs before it, but splits a long row's keys and puts four waves on a row.  Those rows go
    # to the decode kernel when they are few and much longer than the portions (up to 8 rows of 3,000
    # keys and more, twice the longest portion's sequence: 4 rows of 4,000 keys beside 256 / 1,024 /
    # 2,000 new tokens 62 / 110 / 126 us in the prefill kernel, 47 / 69 / 98 us with the decode kernel),
    # or many beside short portions (64 rows and more beside at most 512 new tokens: 64 rows of 200 keys
    # beside 256 tokens 50 against 42 us, 128 rows 75 against 53).  Measured at 4 to 128 rows of 200 to
    # 4,000 keys beside 256 to 2,000 new tokens behind up to 3,584 keys; elsewhere the prefill kernel
    # alone is as fast or up to a fifth faster.
    DECODE_BESIDE_FEW = (8, 3000, 2.0)       # at most so many rows, of at least so many keys and so many times the portions' longest
    DECODE_BESIDE_MANY = (64, 512)           # at least so many rows, beside at most so many new tokens

    def __init__(self, device):
        self.device = torch.device(device)
        if self.device.type != "cuda":
            raise KernelError(f"the kernels run on an AMD GPU ('cuda:N' in torch), not on '{device}'")
        if not torch.cuda.is_available():
            raise KernelError("no GPU is visible to torch; this engine has no CPU path")
        self.lib = load_library()
        with torch.cuda.device(self.device):
            self.DECODE_WORKGROUPS = int(self.lib.tli_device_compute_units())
        self._held_stream = None
        self.force_plain = False     # tests: run the plain attention kernel for bfloat16 too
        self.plain_products = False  # every matrix product through the plain kernel
        self.separate_norms = False  # tests: decode steps run their norms as kernels of their own
        self.unfused_decode = False  # tests: decode steps through qkv_to_cache and paged_attention too
        self.separate_cache_writes = False   # tests: the keys and the values of prompt portions by a kernel each
        self.decode_solo = "auto"    # the decode attention that gives a row's kv head a wave to itself: "auto" (where
                                     # the rows fill the chip), "always" (wherever its limits allow), "never"
        self.prefill_direct = 0      # tests: 1 = the prefill attention kernel without LDS staging; 2, 3 = with, 1 or 2 tiles a wave; 4..8 = a forced order of row blocks; 10, 11 = heads of 64 and 128 with two sets of waves a workgroup, with one; 13 = as 0 for rows with many keys before them
        self.mid_cfg = 0             # measurements: launch shape and k ranges of the 17..128-row kernel
        self.mid_splits = 0
        self.skinny_cfg = 0          # measurements: force a launch shape of the weight-streaming kernel
        # Products of more than 128 rows: "own" = gemm_rows; "library" = the BLAS library; "measure" = the
        # faster of the two for the shape, timed once when the shape first comes up.  The latter two
        # multiply with the row-major form of a matrix, which is then held beside its decode layout
        # (see keep_row_major): set this before the weights are loaded.
        self.many_rows = "own"
        self.measured = {}           # (rows rounded up to 128, N, K, gated) -> True where gemm_rows won
        self._cold = None            # what is written between two timed runs
        self.attention_tile_rows = 16   # measurements, tests: 32 = tiles of 32 rows in the biased attention kernel (heads up to 128)
        self.moe_tile = 0            # measurements, tests: force the slots of a tile of the routed experts' products (16, 32, 64, 128)
        self.rows_cfg = 0            # measurements: force a launch shape and the k ranges of gemm_rows
        self.sinks_in_prefill = os.environ.get("TLI_SINKS_IN_PREFILL", "1") != "0"   # measurements, tests: False sends portions of prompts with sinks through sized_attention too
        self.lightning_lanes = int(os.environ.get("TLI_LIGHTNING_LANES", "0"))   # measurements, tests: 16 or 64 lanes a column of the lightning recurrence's state (0: the launch rule)
        self.rows_splits = 0
        self.pooled_prefill = True       # measurements, tests: False sends portions of prompts over windows and pooled blocks through the kernels for sizes of their own
        self.sized_splits = None         # measurements, tests: the same of a decoding row's cached vectors that all heads read (None: the rule)
        self.pooled_splits = None        # measurements, tests: into how many splits a decoding row's keys over windows and pooled blocks go (None: the rule)
        self.recurrence_in_chunks = True    # measurements, tests: False sends the portions of prompts of retention, mLSTM and wkv through the recurrence row by row
        self.separate_activations = False   # measurements, tests: True leaves the activations of products without a gate to a pass of their own
        self.grouped_products = True        # measurements, tests: False multiplies stacked matrices with inputs of their own one by one

    @property
    def keep_row_major(self) -> bool:
        """Whether a bfloat16 matrix is to keep its row-major form beside its decode layout."""
        return self.many_rows != "own"

    def use_plain_kernels(self) -> None:
        """Every product, attention and norm through the plain kernels, bfloat16 too
        (what the float32 path runs): to tell a fault of a tuned kernel from one elsewhere."""
        self.force_plain = self.plain_products = self.separate_norms = self.unfused_decode = True

    # ---- helpers ----------------------------------------------------------
    def _stream(self):
        if self._held_stream is not None:
            return self._held_stream
        return torch.cuda.current_stream(self.device).cuda_stream

    @contextlib.contextmanager
    def hold_stream(self):
        """Inside, every kernel goes to the stream that was current on entry: one look-up for the
        hundreds of launches of a step instead of one each (a quarter of the host's time in a step
        that is not replayed from a recording)."""
        before = self._held_stream
        self._held_stream = torch.cuda.current_stream(self.device).cuda_stream
        try:
            yield
        finally:
            self._held_stream = before

    def _call(self, fn, *args):
        if fn(*args) != 0:
            raise KernelError(self.lib.tli_last_error().decode())

    def _want(self, t: torch.Tensor, what: str, dtype=None, shape=None):
        if t.device != self.device:
            raise KernelError(f"{what} is on {t.device}, expected {self.device}")
        if not t.is_contiguous():
            raise KernelError(f"{what} must be contiguous")
        if dtype is not None and t.dtype != dtype:
            raise KernelError(f"{what} has dtype {t.dtype}, expected {dtype}")
        if shape is not None and tuple(t.shape) != tuple(shape):
            raise KernelError(f"{what} has shape {tuple(t.shape)}, expected {tuple(shape)}")

    # ---- limits that parts ask about at build time --------------------------
    def check_attention_sizes(self, heads: int, kv_heads: int, head_dim: int) -> None:
        if head_dim % 16 or not 16 <= head_dim <= self.MAX_HEAD_DIM:
            raise KernelError(f"head_dim {head_dim} is not supported: the attention kernels take "
                              f"multiples of 16 from 16 to {self.MAX_HEAD_DIM}")
        if heads <= 0 or kv_heads <= 0 or heads % kv_heads:
            raise KernelError(f"{heads} heads cannot be grouped over {kv_heads} kv heads")

    def check_page_size(self, page_size: int) -> None:
        if page_size <= 0 or page_size > 256 or page_size & (page_size - 1):
            raise KernelError(f"page size {page_size} is not supported: powers of two up to 256")

    # ---- ops ------------------------------------------------------------------
    def feed_tokens(self, token_ids: torch.Tensor, token_from: torch.Tensor, src: torch.Tensor, rows: int):
        """token_ids[r] = src[token_from[r]] where token_from[r] >= 0 (all int32, on the device)."""
        for t, what in ((token_ids, "token ids"), (token_from, "token sources"), (src, "sampled tokens")):
            self._want(t, what, torch.int32)
        if token_ids.numel() < rows or token_from.numel() < rows:
            raise KernelError("fewer token ids than rows")
        self._call(self.lib.tli_feed_tokens, token_ids.data_ptr(), token_from.data_ptr(), src.data_ptr(),
                   rows, src.numel(), self._stream())

    def embed(self, table: torch.Tensor, token_ids: torch.Tensor, num_rows: int, scale: float = 1.0,
              positions: Optional[torch.Tensor] = None, pos_table: Optional[torch.Tensor] = None) -> torch.Tensor:
        """float32 rows [num_rows, hidden]: table[id], or scale * table[id] + pos_table[position]."""
        vocab, hidden = table.shape
        self._want(table, "embedding table")
        self._want(token_ids, "token ids", torch.int32)
        if token_ids.numel() < num_rows:
            raise KernelError("fewer token ids than rows")
        out = torch.empty((num_rows, hidden), dtype=torch.float32, device=self.device)
        if pos_table is not None or scale != 1.0:
            npos = 0
            if pos_table is not None:
                npos = pos_table.shape[0]
                self._want(pos_table, "position table", table.dtype, (npos, hidden))
                self._want(positions, "positions", torch.int32)
                if positions.numel() < num_rows:
                    raise KernelError("fewer positions than rows")
            self._call(self.lib.tli_embed_scaled, table.data_ptr(), token_ids.data_ptr(), _ptr(pos_table), _ptr(positions),
                       out.data_ptr(), num_rows, hidden, vocab, npos, float(scale), _dtype_code(table.dtype), self._stream())
            return out
        self._call(self.lib.tli_embed, table.data_ptr(), token_ids.data_ptr(), out.data_ptr(),
                   num_rows, hidden, vocab, _dtype_code(table.dtype), self._stream())
        return out

    def resolve(self, y):
        """The tensor of a product that ``linear(..., deferred=True)`` left unfinished."""
        if isinstance(y, PendingProduct):
            return self.linear(y.x, y.matrix)
        if isinstance(y, NormedRows):
            raise KernelError("normed rows that still owe their factor go to linear or linear_swiglu")
        if not isinstance(y, DeferredSum):
            return y
        splits, M, N = y.parts.shape
        out = torch.empty((M, N), dtype=y.dtype, device=self.device)
        self._call(self.lib.tli_gemm_mid_reduce, y.parts.data_ptr(), out.data_ptr(), M, N, splits,
                   _dtype_code(y.dtype), self._stream())
        return out

    def add_rmsnorm(self, resid, delta, weight, eps, out_dtype, rows=None, num_rows=None, lazy=False):
        """``lazy``: the caller hands the result to ``linear`` or ``linear_swiglu`` only and so
        also takes ``NormedRows``."""
        total, n = resid.shape
        self._want(resid, "residual", torch.float32)
        self._want(weight, "norm weight", torch.float32, (n,))
        if isinstance(delta, PendingProduct):
            if lazy and rows is None and not self.separate_norms:
                return self._product_into_residual(delta, resid, weight, eps)
            delta = self.resolve(delta)
        parts = 0
        if isinstance(delta, DeferredSum):
            if delta.dtype != out_dtype or out_dtype != torch.bfloat16:
                delta = self.resolve(delta)
            else:
                parts = delta.parts.shape[0]
                delta = delta.parts
                self._want(delta, "partial sums of the residual delta", torch.float32, (parts, total, n))
        if delta is not None and not parts:
            self._want(delta, "residual delta", out_dtype, (total, n))
        out_rows = total
        if rows is not None:
            self._want(rows, "row list", torch.int32)
            out_rows = rows.numel() if num_rows is None else num_rows
            if rows.numel() < out_rows:
                raise KernelError("row list is shorter than the rows asked for")
        out = torch.empty((out_rows, n), dtype=out_dtype, device=self.device)
        self._call(self.lib.tli_add_rmsnorm, resid.data_ptr(), _ptr(delta), weight.data_ptr(),
                   out.data_ptr(), _ptr(rows), out_rows, total, n, float(eps),
                   _dtype_code(out_dtype), parts, self._stream())
        return out

    def tile_matrix(self, w: torch.Tensor) -> Optional[torch.Tensor]:
        """The decode layout of a bfloat16 matrix W[N,K]: blocks of 16 rows x 128
        columns, zero-padded to whole blocks, stored [row block][column block][j][lane][8]
        with lane = 16*c + r holding W[16*row block + r][128*column block + 32*c + 8*j + e].
        A wave of the weight-streaming kernel then reads 4 KiB in a row per block, in the
        order its MFMA operands want.  None if the matrix cannot use that kernel."""
        N, K = w.shape
        if w.dtype != torch.bfloat16 or K % 8:
            return None
        n16, k128 = (N + 15) // 16 * 16, (K + 127) // 128 * 128
        if (n16, k128) != (N, K):
            padded = torch.zeros((n16, k128), dtype=w.dtype, device=w.device)
            padded[:N, :K] = w
            w = padded
        t = w.view(n16 // 16, 16, k128 // 128, 4, 4, 8)          # [nb, r, kb, c, j, e]
        return t.permute(0, 2, 4, 3, 1, 5).contiguous()           # [nb, kb, j, c, r, e]

    def untile_matrix(self, tiled: torch.Tensor, shape) -> torch.Tensor:
        """The row-major matrix [N, K] again from its decode layout (a new tensor)."""
        N, K = shape
        nb, kb = tiled.shape[0], tiled.shape[1]
        w = tiled.permute(0, 4, 1, 3, 2, 5).reshape(nb * 16, kb * 128)        # [nb, r, kb, c, j, e]
        return w[:N, :K].contiguous()

    def linear(self, x: torch.Tensor, w, out_dtype: Optional[torch.dtype] = None, deferred: bool = False,
               sums_only: bool = False):
        """y = x W^T.  ``w`` is a [N, K] tensor or a ``Matrix`` (row-major tensor plus
        its decode layout).  ``deferred``: the caller hands the result to ``add_rmsnorm``
        (or to ``resolve``) and so also takes a ``PendingProduct`` or a ``DeferredSum``;
        ``sums_only``: to ``qkv_attention`` (or to ``resolve``), which takes a ``DeferredSum``."""
        if isinstance(x, NormedRows):
            return self._linear_normed(x, w, getattr(w, "tiled", None), 0, out_dtype)
        if self.plain_products:
            return self.linear_plain(x, getattr(w, "w", w), out_dtype)
        tiled = getattr(w, "tiled", None)
        if (deferred and not sums_only and tiled is not None and x.dtype == torch.bfloat16
                and 0 < x.shape[0] <= 16 and out_dtype in (None, torch.bfloat16) and not self.separate_norms):
            return PendingProduct(x, w)
        matrix = w
        M, K = x.shape
        N, K2 = _shape_of(matrix)
        if K != K2:
            raise KernelError(f"linear: input has {K} columns, the matrix {K2}")
        self._want(x, "linear input")
        w_dtype = getattr(matrix, "dtype", None) or matrix.w.dtype
        if x.dtype != w_dtype:
            raise KernelError(f"linear: input is {x.dtype}, the matrix {w_dtype}")
        out_dtype = out_dtype or x.dtype
        y = torch.empty((M, N), dtype=out_dtype, device=self.device)
        if M == 0:
            return y
        if x.dtype == torch.bfloat16 and K % 8 == 0:
            # (beyond 128 rows only with bfloat16 results, and not where the library or a measurement was asked for)
            if tiled is not None and self.MID_ROWS_FROM <= M <= (
                    self.MID_ROWS_TO_PLAIN if out_dtype == torch.bfloat16 and self.many_rows == "own" else self.MID_ROWS_TO):
                return self._linear_mid(x, tiled, y, M, N, K, 0, deferred or sums_only)
            if tiled is not None and out_dtype == torch.float32 and M > self.MID_ROWS_TO:
                # float32 logits for many rows (a decode step of hundreds of requests, a replay that wants
                # every position): the x-sharing kernel, 256 rows (two row blocks side by side) at a time
                # (512 rows of the Qwen3-8B head: 8 x 363 us in the kernel below, 4 x 240 us in portions of
                # 128 rows).  The last rows too, however few: a row's sums are then the same bits whatever
                # the number of rows beside it in its block of 128, which a step replayed with rows that
                # only fill it up relies on.
                for m0 in range(0, M, self.MID_ROWS_TO_PLAIN):
                    m1 = min(M, m0 + self.MID_ROWS_TO_PLAIN)
                    self._linear_mid(x[m0:m1], tiled, y[m0:m1], m1 - m0, N, K, 0)
                return y
            if M <= self.SKINNY_ROWS or out_dtype == torch.float32:
                # few rows (decode), or float32 logits: the weight-streaming MFMA kernel,
                # 64 rows at a time
                wp = tiled
                if wp is None:
                    wp = getattr(matrix, "w", matrix)
                    self._want(wp, "linear matrix")
                for m0 in range(0, M, self.SKINNY_ROWS):
                    m1 = min(M, m0 + self.SKINNY_ROWS)
                    self._call(self.lib.tli_gemm_skinny_bf16, x[m0:m1].data_ptr(), wp.data_ptr(),
                               y[m0:m1].data_ptr(), m1 - m0, N, K, _dtype_code(out_dtype),
                               0 if tiled is None else 1, self.skinny_cfg, *_NO_GATE, self._stream())
                return y
            if tiled is not None and out_dtype == torch.bfloat16 and self._rows_kernel_wins(x, matrix, tiled, M, N, K, 0):
                return self._linear_rows(x, tiled, y, M, N, K, 0, deferred or sums_only)
            # many rows (prefill) where the library was asked for: its matrix product, as the
            # reference uses its library for more than one row (kernels/src/matmul_kernel_cuda.cu:84-91)
            w = getattr(matrix, "w", matrix)
            self._want(w, "linear matrix")
            torch.matmul(x, w.t(), out=y)
            return y
        w = getattr(matrix, "w", matrix)
        self._want(w, "linear matrix")
        self._call(self.lib.tli_gemm_plain, x.data_ptr(), w.data_ptr(), y.data_ptr(), M, N, K,
                   _dtype_code(x.dtype), _dtype_code(w.dtype), _dtype_code(out_dtype), self._stream())
        return y

    def _product_into_residual(self, p: PendingProduct, resid, weight, eps) -> NormedRows:
        """resid += x W^T, and the rows of the norm that follows, its factor still owed."""
        x, m = p.x, p.matrix
        M, K = x.shape
        N = _shape_of(m)[0]
        self._want(x, "linear input", torch.bfloat16, (M, _shape_of(m)[1]))
        if tuple(resid.shape) != (M, N):
            raise KernelError(f"the product gives {(M, N)}, the residual is {tuple(resid.shape)}")
        xw = torch.empty((M, N), dtype=torch.bfloat16, device=self.device)
        ssq = torch.empty(((N + 15) // 16, M), dtype=torch.float32, device=self.device)
        self._call(self.lib.tli_gemm_skinny_fused_bf16, x.data_ptr(), m.tiled.data_ptr(), None, M, N, K, 0,
                   None, 0, 0.0, resid.data_ptr(), weight.data_ptr(), xw.data_ptr(), ssq.data_ptr(), 0, *_NO_GATE,
                   self._stream())
        return NormedRows(xw, ssq, eps)

    def _linear_normed(self, x: NormedRows, m, tiled, gated: int, out_dtype=None, act: int = 0, scale: float = 1.0, into=None):
        """y = normed rows . W^T with the rows' factor applied to the outputs."""
        M, K = x.xw.shape
        if tiled is None:
            raise KernelError("normed rows that still owe their factor need a matrix in the decode layout")
        if out_dtype not in (None, torch.bfloat16):
            raise KernelError("normed rows that still owe their factor give bfloat16 products")
        rows_out = _shape_of(m)[0]
        if _shape_of(m)[1] != K:
            raise KernelError(f"linear: input has {K} columns, the matrix {_shape_of(m)[1]}")
        N = 2 * m.inter if gated else rows_out
        y, y_at, ld = self._rows_into(into, M, m.inter if gated else N, torch.bfloat16)
        self._call(self.lib.tli_gemm_skinny_fused_bf16, x.xw.data_ptr(), tiled.data_ptr(), y_at, M, N, K,
                   gated, x.ssq.data_ptr(), x.ssq.shape[0], x.eps, None, None, None, None, 0, act, float(scale), ld,
                   self._stream())
        return y

    def _linear_mid(self, x, tiled, y, M, N, K, gated, deferred=False, gate=None):
        """17..128 rows (without a gate: up to 256): the kernel that shares x through LDS, k cut into
        ranges when the output alone gives too few workgroups.  ``deferred``: the partial sums of the
        ranges are left for the consumer to add, which saves the pass that adds them.  ``gate``: (address of
        the output, activation, factor, distance of its rows) of a gated product."""
        splits = self.mid_splits or self.lib.tli_gemm_mid_splits_rows(M, N, K, gated)
        part = None
        if splits > 1:
            part = torch.empty((splits, M, N), dtype=torch.float32, device=self.device)
        leave = deferred and splits > 1 and not gated and y.dtype == torch.bfloat16
        y_at, *gate = gate or (y.data_ptr(), *_NO_GATE)
        self._call(self.lib.tli_gemm_mid_bf16, x.data_ptr(), tiled.data_ptr(), None if leave else y_at,
                   _ptr(part), M, N, K, _dtype_code(y.dtype), gated, splits, self.mid_cfg, *gate, self._stream())
        return DeferredSum(part, y.dtype) if leave else y

    def _rows_kernel_wins(self, x, matrix, tiled, M, N, K, gated) -> bool:
        """Whether this product of more than 128 rows goes to gemm_rows (else to the library).
        With ``many_rows`` = "measure": which one is faster changes with the shape by up to 10%
        either way (how well each one's tiles fill the compute units), so both are timed when a
        shape first comes up: three runs each after one to warm up, a few milliseconds, outside
        any graph capture."""
        if max(M, N + 15) * (K + 127) * 2 >= 1 << 32:
            return False                      # gemm_rows keeps 32-bit offsets into its operands
        if self.many_rows != "measure":
            return self.many_rows == "own"
        key = ((M + 127) // 128, N, K, gated)
        won = self.measured.get(key)
        if won is not None:
            return won
        if torch.cuda.is_current_stream_capturing():
            return False                      # (nothing can be timed now; the shape is measured when it next comes up eagerly)
        y = torch.empty((M, N // 2 if gated else N), dtype=torch.bfloat16, device=self.device)
        wide = torch.empty((M, N), dtype=torch.bfloat16, device=self.device) if gated else None
        w = getattr(matrix, "w", matrix)

        def library():
            if gated:
                torch.matmul(x, w.t(), out=wide)
                self.swiglu(wide)
            else:
                torch.matmul(x, w.t(), out=y)

        def own():
            self._linear_rows(x, tiled, y, M, N, K, gated)

        # (in a model the weights of a layer come from memory, not from the last-level cache where a
        # second run would find them: 384 MB are written between the runs)
        if self._cold is None:
            self._cold = torch.empty(96 << 20, dtype=torch.float32, device=self.device)
        times = []
        for fn in (library, own):
            fn()
            total = 0.0
            for _ in range(3):
                self._cold.fill_(0.0)
                start, stop = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
                start.record()
                fn()
                stop.record()
                stop.synchronize()
                total += start.elapsed_time(stop)
            times.append(total)
        won = times[1] < times[0]
        self.measured[key] = won
        return won

    def _linear_rows(self, x, tiled, y, M, N, K, gated, deferred=False, gate=None):
        """Any number of rows from the decode layout; k cut into ranges when the output
        alone gives too few workgroups.  ``deferred``: the partial sums of the ranges are
        left for the consumer to add.  ``gate`` as in ``_linear_mid``."""
        splits = self.rows_splits or self.lib.tli_gemm_rows_splits(M, N, K)
        part = None
        if splits > 1:
            part = torch.empty((splits, M, N), dtype=torch.float32, device=self.device)
        leave = deferred and splits > 1 and not gated
        y_at, *gate = gate or (y.data_ptr(), *_NO_GATE)
        self._call(self.lib.tli_gemm_rows_bf16, x.data_ptr(), tiled.data_ptr(), None if leave else y_at,
                   _ptr(part), M, N, K, gated, splits, self.rows_cfg, *gate, self._stream())
        return DeferredSum(part, y.dtype) if leave else y

    def linear_plain(self, x: torch.Tensor, w: torch.Tensor, out_dtype: Optional[torch.dtype] = None):
        """The plain tiled kernel for any sizes and dtypes: the reference beside the tuned ones."""
        M, K = x.shape
        N = w.shape[0]
        self._want(x, "linear input")
        self._want(w, "linear matrix", x.dtype, (N, K))
        out_dtype = out_dtype or x.dtype
        y = torch.empty((M, N), dtype=out_dtype, device=self.device)
        self._call(self.lib.tli_gemm_plain, x.data_ptr(), w.data_ptr(), y.data_ptr(), M, N, K,
                   _dtype_code(x.dtype), _dtype_code(w.dtype), _dtype_code(out_dtype), self._stream())
        return y

    GATE_ACTIVATIONS = {"silu": 0, "gelu_tanh": 1}

    def check_gate_activation(self, name: str) -> None:
        if name not in self.GATE_ACTIVATIONS:
            raise KernelError(f"gate activation '{name}' is not known; known: {', '.join(sorted(self.GATE_ACTIVATIONS))}")

    def _rows_into(self, into, rows: int, cols: int, dtype):
        """(tensor, address, distance of its rows) of ``rows`` x ``cols`` outputs: a new tensor, or, for ``into`` =
        (tensor, column), the columns from there on of the rows of that tensor, which other outputs share."""
        if into is None:
            y = torch.empty((rows, cols), dtype=dtype, device=self.device)
            return y, y.data_ptr(), cols
        y, at = into
        self._want(y, "shared rows of outputs", dtype)
        if y.dim() != 2 or y.shape[0] != rows or at < 0 or at % 8 or at + cols > y.shape[1] or (y.shape[1] % 8 and cols != y.shape[1]):
            raise KernelError(f"{cols} columns from {at} on (a multiple of 8) do not fit shared rows of shape {tuple(y.shape)}")
        return y, y.data_ptr() + at * y.element_size(), y.shape[1]

    def linear_swiglu(self, x: torch.Tensor, m, activation: str = "silu", scale: float = 1.0, into=None) -> torch.Tensor:
        """act(x gate^T) * (x up^T) * scale for a ``GatedMatrix``.  Few rows: one pass of
        the weight-streaming kernel over the interleaved layout, the activation in
        its epilogue.  Otherwise the stacked product, then the activation.  ``into`` (a tensor and a
        column of it): the outputs go there, beside what else its rows hold."""
        act = self.GATE_ACTIVATIONS[activation]
        if isinstance(x, NormedRows):
            return self._linear_normed(x, m, getattr(m, "gated", None), 1, act=act, scale=scale, into=into)
        M, K = x.shape
        gated = getattr(m, "gated", None) if not self.plain_products else None
        if gated is not None and 0 < M <= self.MID_ROWS_TO and x.dtype == torch.bfloat16:
            self._want(x, "linear input", torch.bfloat16, (M, _shape_of(m)[1]))
            y, y_at, ld = self._rows_into(into, M, m.inter, x.dtype)
            if M >= self.MID_ROWS_FROM:
                return self._linear_mid(x, gated, y, M, 2 * m.inter, K, 1, gate=(y_at, act, float(scale), ld))
            self._call(self.lib.tli_gemm_skinny_bf16, x.data_ptr(), gated.data_ptr(), y_at, M,
                       2 * m.inter, K, BF16, 2, self.skinny_cfg if self.skinny_cfg >= 20 else 0, act, float(scale), ld,
                       self._stream())
            return y
        if (gated is not None and x.dtype == torch.bfloat16 and K % 8 == 0
                and self._rows_kernel_wins(x, m, gated, M, 2 * m.inter, K, 1)):
            self._want(x, "linear input", torch.bfloat16, (M, _shape_of(m)[1]))
            y, y_at, ld = self._rows_into(into, M, m.inter, x.dtype)
            return self._linear_rows(x, gated, y, M, 2 * m.inter, K, 1, gate=(y_at, act, float(scale), ld))
        return self.swiglu(self.linear(x, m), activation=activation, scale=scale, into=into)

    def swiglu(self, gu: torch.Tensor, limit: float = 0.0, slope: float = 1.0, activation: str = "silu", scale: float = 1.0,
               into=None) -> torch.Tensor:
        """From gate and up sums side by side [rows, 2 n] to the hidden units [rows, n]: act(g) * u * scale, or with a
        positive ``limit`` the limited form g' * sigmoid(slope * g') * (u' + 1), g' = min(g, limit), u' = clamp(u,
        -limit, limit).  ``into`` as in ``linear_swiglu``."""
        rows, two = gu.shape
        if two % 2:
            raise KernelError("swiglu input must hold gate and up side by side")
        self._want(gu, "swiglu input")
        out, out_at, ld = self._rows_into(into, rows, two // 2, gu.dtype)
        self._call(self.lib.tli_swiglu, gu.data_ptr(), out_at, rows, two // 2,
                   _dtype_code(gu.dtype), float(limit), float(slope), self.GATE_ACTIVATIONS[activation], float(scale), ld,
                   self._stream())
        return out

    def qkv_to_cache(self, qkv, step, cache, heads, kv_heads, head_dim, q_norm, k_norm, rotary, queries=True):
        """Norms and rotation of q and k, k and v into the cache; returns q.  Without
        ``queries`` only the keys and values are done (bfloat16 heads of 64, 128, 256),
        the values by a kernel of their own that writes runs of slots."""
        T = step.num_rows
        q_dim, kv_dim = heads * head_dim, kv_heads * head_dim
        self._want(qkv, "qkv", None, (T, q_dim + 2 * kv_dim))
        q = torch.empty((T, q_dim), dtype=qkv.dtype, device=self.device) if queries else None
        qw, qe = q_norm if q_norm is not None else (None, 0.0)
        kw, ke = k_norm if k_norm is not None else (None, 0.0)
        for w in (qw, kw):
            if w is not None:
                self._want(w, "head norm weight", torch.float32, (head_dim,))
        cos = sin = None
        rd = npos = 0
        if rotary is not None:
            cos, sin, rd = self._rotary(rotary, step)
            npos = cos.shape[0]
        write = 1 if (cache is not None and cache.writes) else 0
        k_ptr = v_ptr = tab_ptr = None
        width = page = pages = 0
        if write:
            kc, vc = cache.record("k"), cache.record("v")
            g = cache.group
            self._check_cache(kc, vc, g, kv_heads, head_dim, qkv.dtype, step)
            k_ptr, v_ptr, tab_ptr = kc.data_ptr(), vc.data_ptr(), g.tables.data_ptr()
            width, page, pages = g.table_width, g.page_size, kc.shape[0]
        if (not queries and write and qkv.dtype == torch.bfloat16 and head_dim in (64, 128, 256) and page >= 8
                and (rotary is None or rd == head_dim) and not self.separate_cache_writes):
            # keys and values in one pass (prompt portions: the attention kernel takes q from qkv itself)
            self._call(self.lib.tli_keys_values_to_cache, qkv.data_ptr(), k_ptr, v_ptr, step.row_start.data_ptr(),
                       step.seq_start.data_ptr(), step.num_seqs, T, tab_ptr, width, page, pages, heads, kv_heads,
                       head_dim, _ptr(kw), float(ke), _ptr(cos), _ptr(sin), npos, self._stream())
            return None
        self._call(self.lib.tli_qkv_to_cache, qkv.data_ptr(), _ptr(q), k_ptr, v_ptr,
                   step.positions.data_ptr(), step.seq_of_row.data_ptr(), tab_ptr, width, page, pages,
                   T, heads, kv_heads, head_dim, _ptr(qw), float(qe), _ptr(kw), float(ke),
                   _ptr(cos), _ptr(sin), rd, npos, write, 0 if queries else 1, _dtype_code(qkv.dtype),
                   self._stream())
        if write and not queries:
            self._call(self.lib.tli_values_to_cache, qkv.data_ptr(), v_ptr, step.row_start.data_ptr(),
                       step.seq_start.data_ptr(), step.num_seqs, T, tab_ptr, width, page, pages, heads,
                       kv_heads, head_dim, self._stream())
        return q

    def _rotary(self, rotary, step):
        """(cos, sin, rotary_dim) of what a mixer passes as ``rotary``, checked.  The kernels turn
        the pairs (i, i + rotary_dim/2); a fourth element that names another pairing is refused."""
        cos, sin, rd = rotary[0], rotary[1], int(rotary[2])
        if len(rotary) > 3 and rotary[3] != "half":
            raise KernelError(f"the kernels rotate the pairs (i, i + rotary_dim/2) of a head, not the pairing "
                              f"'{rotary[3]}'; the attention part reorders a head's elements for that")
        npos = cos.shape[0]
        self._want(cos, "cos table", torch.float32, (npos, rd // 2))
        self._want(sin, "sin table", torch.float32, (npos, rd // 2))
        if step.max_seq_len > npos:
            raise KernelError(f"a position reaches {step.max_seq_len}, the rotation table has {npos}")
        return cos, sin, rd

    def _check_cache(self, kc, vc, g, kv_heads, head_dim, dtype, step):
        pages = kc.shape[0]
        self._want(kc, "key cache", dtype, (pages, kv_heads, g.page_size, head_dim))
        self._want(vc, "value cache", dtype, (pages, kv_heads, head_dim, g.page_size))
        self._want(g.tables, "block tables", torch.int32, (step.num_seqs, g.table_width))
        if (step.max_seq_len + g.page_size - 1) // g.page_size > g.table_width:
            raise KernelError("a block table is narrower than its sequence needs")

    def paged_attention(self, q, step, cache, heads, kv_heads, head_dim, scale, window, sinks=None):
        """Attention of ``q`` [T, heads * head_dim] over the cache.  ``sinks`` (float32 [heads]): a logit a head that the
        softmax's denominator also holds; only steps with portions of prompts in bfloat16 take them here (see
        ``takes_sinks``), everything else goes through ``sized_attention``."""
        T = step.num_rows
        if sinks is not None and not self.takes_sinks(q.dtype, step, cache, head_dim):
            raise KernelError("this step's attention kernel has no sink; sized_attention has")
        self._want(q, "queries", None, (T, heads * head_dim))
        if cache is None:
            raise KernelError("attention needs a cache layer")
        kc, vc, g = cache.record("k"), cache.record("v"), cache.group
        self._check_cache(kc, vc, g, kv_heads, head_dim, q.dtype, step)
        out = torch.empty_like(q)
        if q.dtype == torch.bfloat16 and head_dim <= 256 and g.page_size >= 4 and not self.force_plain:
            if step.max_rows_per_seq == 1 and g.page_size >= 8:
                return self._attention_decode(q, out, step, kc, vc, g, heads, kv_heads, head_dim, scale, window)
            self._call(self.lib.tli_attention_prefill_bf16, q.data_ptr(), out.data_ptr(), kc.data_ptr(),
                       vc.data_ptr(), step.row_start.data_ptr(), step.seq_start.data_ptr(), step.num_seqs,
                       T, g.tables.data_ptr(), g.table_width, g.page_size, kc.shape[0], heads, kv_heads,
                       head_dim, float(scale), int(window or 0), self._prefill_mode(step, T), _ptr(sinks),
                       self._stream())
            return out
        self._call(self.lib.tli_attention_plain, q.data_ptr(), out.data_ptr(), kc.data_ptr(),
                   vc.data_ptr(), step.positions.data_ptr(), step.seq_of_row.data_ptr(),
                   g.tables.data_ptr(), g.table_width, g.page_size, kc.shape[0], T, heads, kv_heads,
                   head_dim, float(scale), int(window or 0), _dtype_code(q.dtype), self._stream())
        return out

    def takes_sinks(self, dtype, step, cache, head_dim) -> bool:
        """Whether ``paged_attention`` runs this step through the kernel for portions of prompts, which takes sinks."""
        return (self.sinks_in_prefill and dtype == torch.bfloat16 and head_dim % 16 == 0 and 16 <= head_dim <= 256
                and cache.group.page_size >= 4 and not self.force_plain and not (step.max_rows_per_seq == 1 and cache.group.page_size >= 8))

    def qkv_attention(self, qkv, step, cache, heads, kv_heads, head_dim, q_norm, k_norm, rotary, scale, window):
        """From the raw projections to the attention output: norms and rotation of q
        and k, k and v into the cache, attention over the cache.  A decode step (one
        row a sequence) does all of it in the attention kernel where the sizes allow;
        other steps run qkv_to_cache and paged_attention.  ``qkv`` may be a ``DeferredSum``:
        the kernel of a decode step adds the partial sums itself."""
        sums = None
        if isinstance(qkv, DeferredSum):
            sums = qkv
            if not (step.max_rows_per_seq == 1 and qkv.dtype == torch.bfloat16 and cache is not None
                    and head_dim % 64 == 0 and head_dim <= 256 and heads // kv_heads <= 16
                    and cache.group.page_size >= 8 and not self.force_plain and not self.unfused_decode
                     and (rotary is None or rotary[2] == head_dim)):
                qkv, sums = self.resolve(qkv), None
        fusable = (qkv.dtype == torch.bfloat16 and cache is not None and head_dim % 64 == 0
                   and head_dim <= 256 and not self.force_plain and not self.unfused_decode
                   and (rotary is None or rotary[2] == head_dim))
        if (fusable and step.max_rows_per_seq > 1 and head_dim != 192 and cache.group.page_size >= 8
                and self.prefill_direct != 1):
            return self._qkv_attention_prefill(qkv, step, cache, heads, kv_heads, head_dim, q_norm, k_norm,
                                               rotary, scale, window)
        fused = (fusable and step.max_rows_per_seq == 1 and heads // kv_heads <= 16
                 and cache.group.page_size >= 8)
        if not fused:
            q = self.qkv_to_cache(qkv, step, cache, heads, kv_heads, head_dim, q_norm, k_norm, rotary)
            return self.paged_attention(q, step, cache, heads, kv_heads, head_dim, scale, window)
        T = step.num_rows
        if sums is not None:
            self._want(sums.parts, "partial sums of qkv", torch.float32,
                       (sums.parts.shape[0], T, (heads + 2 * kv_heads) * head_dim))
        else:
            self._want(qkv, "qkv", None, (T, (heads + 2 * kv_heads) * head_dim))
        kc, vc, g = cache.record("k"), cache.record("v"), cache.group
        self._check_cache(kc, vc, g, kv_heads, head_dim, qkv.dtype, step)
        qw, qe = q_norm if q_norm is not None else (None, 0.0)
        kw, ke = k_norm if k_norm is not None else (None, 0.0)
        for w in (qw, kw):
            if w is not None:
                self._want(w, "head norm weight", torch.float32, (head_dim,))
        cos = sin = None
        if rotary is not None:
            cos, sin, rd = self._rotary(rotary, step)
        out = torch.empty((T, heads * head_dim), dtype=qkv.dtype, device=self.device)
        splits, per_split, partial = self._decode_splits(step.num_rows, step.reach, g, heads, kv_heads, head_dim, window,
                                                         getattr(step, "skew", 1))
        if splits == 1 and self._a_wave_a_row(T, per_split, g, heads, kv_heads, head_dim):
            splits = 0
        self._call(self.lib.tli_qkv_attention_decode_bf16, None if sums is not None else qkv.data_ptr(),
                   out.data_ptr(), _ptr(partial),
                   kc.data_ptr(), vc.data_ptr(), step.positions.data_ptr(), step.seq_of_row.data_ptr(),
                   g.tables.data_ptr(), g.table_width, g.page_size, kc.shape[0], T, heads, kv_heads,
                   head_dim, _ptr(qw), float(qe), _ptr(kw), float(ke), _ptr(cos), _ptr(sin),
                   1 if cache.writes else 0, float(scale), int(window or 0), splits, per_split,
                   None if sums is None else sums.parts.data_ptr(), 0 if sums is None else sums.parts.shape[0],
                   self._stream())
        return out

    def _qkv_attention_prefill(self, qkv, step, cache, heads, kv_heads, head_dim, q_norm, k_norm, rotary,
                               scale, window):
        """Portions of prompts: keys and values go into the cache in one pass, the
        attention kernel norms and rotates its queries itself (a query is read by
        one wave only, so nothing is done twice and q is never written)."""
        T = step.num_rows
        self.qkv_to_cache(qkv, step, cache, heads, kv_heads, head_dim, q_norm, k_norm, rotary, queries=False)
        kc, vc, g = cache.record("k"), cache.record("v"), cache.group
        self._check_cache(kc, vc, g, kv_heads, head_dim, qkv.dtype, step)
        qw, qe = q_norm if q_norm is not None else (None, 0.0)
        cos, sin = (rotary[0], rotary[1]) if rotary is not None else (None, None)
        out = torch.empty((T, heads * head_dim), dtype=qkv.dtype, device=self.device)
        first = self._rows_for_the_decode_kernel(step, heads, kv_heads)
        if first:
            longest = max(step.h_seq_len[:first])
            kw, ke = k_norm if k_norm is not None else (None, 0.0)
            splits, per_split, partial = self._decode_splits(first, max(128, 1 << (longest - 1).bit_length()), g, heads,
                                                             kv_heads, head_dim, window)
            self._call(self.lib.tli_qkv_attention_decode_bf16, qkv.data_ptr(), out.data_ptr(), _ptr(partial),
                       kc.data_ptr(), vc.data_ptr(), step.positions.data_ptr(), step.seq_of_row.data_ptr(),
                       g.tables.data_ptr(), g.table_width, g.page_size, kc.shape[0], first, heads, kv_heads,
                       head_dim, _ptr(qw), float(qe), _ptr(kw), float(ke), _ptr(cos), _ptr(sin),
                       0, float(scale), int(window or 0), splits, per_split, None, 0, self._stream())
        direct = self._prefill_mode(step, T - first, first)
        self._call(self.lib.tli_qkv_attention_prefill_bf16, qkv.data_ptr(), out.data_ptr(), kc.data_ptr(),
                   vc.data_ptr(), step.row_start.data_ptr() + 4 * first, step.seq_start.data_ptr() + 4 * first,
                   step.num_seqs - first, T - first, g.tables.data_ptr() + 4 * first * g.table_width, g.table_width,
                   g.page_size, kc.shape[0], heads, kv_heads,
                   head_dim, _ptr(qw), float(qe), _ptr(cos), _ptr(sin), float(scale), int(window or 0),
                   direct, self._stream())
        return out

    def _rows_for_the_decode_kernel(self, step, heads, kv_heads) -> int:
        """How many of a mixed step's leading sequences go to the decode kernel.  The sequences that
        decode (one row each) stand first in a step that the scheduler made.  The prefill kernel gives
        each of them workgroups that walk all their keys with one row; where that is slower than a
        second launch (see DECODE_BESIDE_FEW, DECODE_BESIDE_MANY) they go to the decode kernel, which
        splits a row's keys over workgroups (their keys and values are in the cache by then)."""
        first = 0
        starts = step.h_row_start
        while first < step.num_seqs and starts[first + 1] - starts[first] == 1:
            first += 1
        if first == 0 or first == step.num_seqs or heads // kv_heads > 16 or self.prefill_direct:
            return 0
        longest = max(step.h_seq_len[:first])
        beside = max(step.h_seq_len[first:step.num_seqs])
        few, many = self.DECODE_BESIDE_FEW, self.DECODE_BESIDE_MANY
        if (first <= few[0] and longest >= few[1] and longest >= few[2] * beside) or \
                (first >= many[0] and step.num_rows - first <= many[1]):
            return first
        return 0

    def _prefill_mode(self, step, rows, first=0):
        """The mode argument of the prefill attention kernels for the sequences from ``first`` on
        (``rows`` rows in all).  Their launch rule wants to know whether the rows have many keys
        before them, and the lengths themselves are on the device: 13 says that they have (the
        longest of those sequences is a quarter longer than all the rows)."""
        longest = max(step.h_seq_len[first:step.num_seqs]) if step.h_seq_len else step.max_seq_len
        if not self.prefill_direct and longest > rows + rows // 4:
            return 13
        return int(self.prefill_direct)

    def _decode_splits(self, T, reach, g, heads, kv_heads, head_dim, window, skew=1):
        """How the keys of ``T`` rows that decode (``reach``: a power of two that the longest
        of their sequences fits) are split over workgroups: they are when the batch alone
        would leave most of the compute units idle and the rows are long enough for the split
        to pay for its merge.  ``skew``: the longest sequence has at least this many times the
        keys of the average one."""
        reach = reach if not window else min(reach, (window + 31) // 32 * 32 + 32)
        groups = T * kv_heads * ((heads // kv_heads + 15) // 16)
        # A split costs a pass that merges the parts (4 to 5 us) and a workgroup that walks no more than
        # 1,500 keys is done in the time of the shortest split run (13 to 17 us against 17.5), so: no split
        # up to a reach of 2,048 keys; beyond, towards one workgroup a compute unit, half of that for 16
        # (row, kv head) pairs and fewer (more parts than that cost more in the merge than they save in the
        # walk), and splits of at least 1,024 keys, of 4,096 from a quarter of the compute units on (there
        # the workgroups already share the memory's rate between them).  Measured at heads of 128, 1 to 64
        # rows of 600 to 32,768 keys, every power of two of splits: this rule is within 8% of the best
        # everywhere; the one before (256 workgroups, 512 keys) was up to 45% over it at 1,024 keys and 20%
        # over it at 1 and 2 rows of 16,384 keys and more.
        # Sequences of unequal lengths: the workgroups of the short ones are done early, so the step's
        # rows count as that many fewer of the longest one's length (32 rows, one of 4,000 keys and 31 of
        # 300: 40 us unsplit, 30 us in four splits; 16 rows of 64 to 2,304 keys: 24.3 and 22.5 us).  With a
        # window every row walks about as many keys.
        if skew > 1 and not window:
            groups = max(1, groups // skew)
        units = self.DECODE_WORKGROUPS
        splits = 1
        if reach > 2 * self.DECODE_SPLIT_KEYS and groups < units:
            aim = units // 2 if groups <= units // 16 else units
            least = self.DECODE_SPLIT_KEYS if groups <= units // 4 else 4 * self.DECODE_SPLIT_KEYS
            splits = max(1, min((aim + groups - 1) // groups, reach // least, 64))
        # (a split's block table entries are kept in LDS: at most 2046 pages a split)
        splits = max(splits, -(-reach // (2046 * g.page_size // 128 * 128)))
        per_split = ((reach + splits - 1) // splits + 127) // 128 * 128
        splits = (reach + per_split - 1) // per_split
        partial = None
        if splits > 1:
            partial = torch.empty((T * heads * splits * (head_dim + 2),), dtype=torch.float32,
                                  device=self.device)
        return splits, per_split, partial

    def _a_wave_a_row(self, T, keys, g, heads, kv_heads, head_dim) -> bool:
        """Whether a decode step of ``T`` rows that see at most ``keys`` keys each goes to the kernel that
        gives every (row, kv head) one wave to itself: when there are four such pairs for every compute
        unit (a wave on its own waits for every block of its keys, so it takes many waves a SIMD to keep
        the chip busy; then it wins because four waves that share out one row's work and merge their sums
        spend most of their instructions on each other.  Measured at Qwen3-8B sizes, 160 keys a row, a whole
        decode step: 32 rows 3.74 -> 3.93 ms, 64 rows 4.09 -> 4.18, 128 rows 5.38 -> 5.28, 256 rows 10.11 ->
        9.73), and a row's keys lie within the 60 pages whose table entries a wave keeps in its lanes."""
        if self.decode_solo == "never" or head_dim not in (64, 128, 256) or keys > 60 * g.page_size:
            return False
        groups = T * kv_heads * ((heads // kv_heads + 15) // 16)
        return self.decode_solo == "always" or groups >= 4 * self.DECODE_WORKGROUPS

    def _attention_decode(self, q, out, step, kc, vc, g, heads, kv_heads, head_dim, scale, window):
        """One row per sequence."""
        T = step.num_rows
        splits, per_split, partial = self._decode_splits(step.num_rows, step.reach, g, heads, kv_heads, head_dim, window,
                                                         getattr(step, "skew", 1))
        self._call(self.lib.tli_attention_decode_bf16, q.data_ptr(), out.data_ptr(), _ptr(partial),
                   kc.data_ptr(), vc.data_ptr(), step.positions.data_ptr(), step.seq_of_row.data_ptr(),
                   g.tables.data_ptr(), g.table_width, g.page_size, kc.shape[0], T, heads, kv_heads,
                   head_dim, float(scale), int(window or 0), splits, per_split, self._stream())
        return out

    # ---- feed-forward without a gate, soft cap -----------------------------------------
    ACTIVATIONS = {"relu2": 0, "relu": 1, "silu": 2, "gelu_tanh": 3, "gelu": 4}

    def check_activation(self, name: str) -> None:
        if name not in self.ACTIVATIONS:
            raise KernelError(f"activation '{name}' is not known; known: {', '.join(sorted(self.ACTIVATIONS))}")

    def activation(self, x: torch.Tensor, name: str) -> torch.Tensor:
        self.check_activation(name)
        self._want(x, "activation input")
        out = torch.empty_like(x)
        self._call(self.lib.tli_activation, x.data_ptr(), out.data_ptr(), x.numel(), self.ACTIVATIONS[name],
                   _dtype_code(x.dtype), self._stream())
        return out

    def linear_act(self, x, matrix, activation: str, token=None):
        """``activation`` of x W^T, one of ``ACTIVATIONS``; with ``token`` = (table, column, ids) times row ids[t] of the table from that
        column on (``token_gate``).  Products of up to 128 rows, and those whose k is cut into ranges, do it where they write
        their sums; others are followed by a pass."""
        self.check_activation(activation)
        tiled = getattr(matrix, "tiled", None)
        M, K = x.shape
        N = _shape_of(matrix)[0]
        kind = self.ACTIVATIONS[activation]
        if (tiled is not None and x.dtype == torch.bfloat16 and not self.plain_products and self.many_rows == "own" and K % 8 == 0 and M > 0
                and K == _shape_of(matrix)[1] and not self.separate_activations):
            self._want(x, "linear input")
            table, ids, width, vocab = None, None, 0, 0
            if token is not None:
                table, at, ids = token
                self._want(table, "tokens' vectors", torch.bfloat16)
                self._want(ids, "token ids", torch.int32)
                if ids.numel() < M or at < 0 or at + N > table.shape[1]:
                    raise KernelError("a token's vector lies outside the table")
                vocab, width = table.shape
                table, ids = table.data_ptr() + 2 * at, ids.data_ptr()
            unit = (kind, table, ids, width, vocab, self._stream())
            y = torch.empty((M, N), dtype=torch.bfloat16, device=self.device)
            if M < self.MID_ROWS_FROM:
                self._call(self.lib.tli_gemm_skinny_unit_bf16, x.data_ptr(), tiled.data_ptr(), y.data_ptr(), M, N, K, *unit)
                return y
            mid = M <= self.MID_ROWS_TO
            splits = int(self.lib.tli_gemm_mid_splits_rows(M, N, K, 0)) if mid else int(self.lib.tli_gemm_rows_splits(M, N, K))
            if mid and splits == 1:
                self._call(self.lib.tli_gemm_mid_unit_bf16, x.data_ptr(), tiled.data_ptr(), y.data_ptr(), M, N, K, *unit)
                return y
            if splits > 1:
                product = self._linear_mid(x, tiled, y, M, N, K, 0, True) if mid else self._linear_rows(x, tiled, y, M, N, K, 0, True)
                if isinstance(product, DeferredSum):
                    self._call(self.lib.tli_gemm_reduce_unit_bf16, product.parts.data_ptr(), y.data_ptr(), M, N, product.parts.shape[0], *unit)
                    return y
                z = product
            else:
                z = self._linear_rows(x, tiled, y, M, N, K, 0)
        else:
            z = self.linear(x, matrix)
        return self.activation(z, activation) if token is None else self.token_gate(z, token[0], token[1], token[2], activation)

    def softcap(self, logits: torch.Tensor, cap: float) -> torch.Tensor:
        """logits <- cap * tanh(logits / cap), in place (float32)."""
        self._want(logits, "logits", torch.float32)
        self._call(self.lib.tli_softcap, logits.data_ptr(), logits.numel(), float(cap), self._stream())
        return logits

    # ---- several residual streams (hyper-connections), token shift ---------------------------
    MAX_STREAMS = 8
    MAX_STREAM_WIDTH = 15360

    def check_streams(self, streams: int, width: int) -> None:
        if not 1 <= streams <= self.MAX_STREAMS or not 1 <= width <= self.MAX_STREAM_WIDTH:
            raise KernelError(f"{streams} residual streams of width {width}: the kernels take up to "
                              f"{self.MAX_STREAMS} streams of up to {self.MAX_STREAM_WIDTH}")

    def streams_open(self, x: torch.Tensor, streams: int) -> torch.Tensor:
        rows, n = x.shape
        self._want(x, "embedding rows", torch.float32)
        out = torch.empty((rows, streams, n), dtype=torch.float32, device=self.device)
        self._call(self.lib.tli_streams_open, x.data_ptr(), out.data_ptr(), rows, n, streams, self._stream())
        return out

    def streams_norm(self, resid, pending, w_in, weight, eps, out_dtype, rows=None, num_rows=None, shift=None):
        """The streams ``resid`` (float32 [T, S, n]) take what ``pending`` (y with its ``mix`` and
        ``out`` weights, or None) still owes them; returns norm(sum_s w_in[s] x_s) in ``out_dtype``.
        With ``rows`` only those rows are computed and the streams stay as they are.  ``shift``
        (mu, kept rows [slots, n], step): the normed rows are mixed with the row before them
        (``token_shift``) on their way out."""
        total, S, n = resid.shape
        self._want(resid, "residual streams", torch.float32)
        self._want(weight, "norm weight", torch.float32, (n,))
        self._want(w_in, "stream read weights", torch.float32, (S,))
        y = mix = out_w = None
        parts = 0
        if pending is not None:
            y = pending.y
            if isinstance(y, DeferredSum) and y.dtype == torch.bfloat16 and not self.separate_norms:
                # partial sums of a split k range: the kernel adds them itself (no pass that only adds)
                parts, y = y.parts.shape[0], y.parts
                self._want(y, "partial sums of the owed rows", torch.float32, (parts, total, n))
            else:
                y = self.resolve(y)
                self._want(y, "owed rows", None, (total, n))
            mix, out_w = pending.mix, pending.out
            self._want(mix, "stream mix weights", torch.float32, (S, S))
            self._want(out_w, "stream write weights", torch.float32, (S,))
        out_rows = total
        if rows is not None:
            if shift is not None:
                raise KernelError("a token shift takes every row of the step")
            self._want(rows, "row list", torch.int32)
            out_rows = rows.numel() if num_rows is None else num_rows
            if rows.numel() < out_rows:
                raise KernelError("row list is shorter than the rows asked for")
        fused = shift is not None and shift[2].max_rows_per_seq == 1 and not self.separate_norms
        mid_dtype = torch.float32 if (shift is not None and not fused) else out_dtype
        out = torch.empty((out_rows, n), dtype=mid_dtype, device=self.device)
        mu = kept = slots = seq_start = seq_of_row = None
        if fused:
            mu, kept, step = shift
            self._check_shift(mu, kept, step, total, n)
            slots, seq_start, seq_of_row = step.slots, step.seq_start, step.seq_of_row
        self._call(self.lib.tli_streams_norm, resid.data_ptr(), _ptr(y), _ptr(mix), _ptr(out_w), w_in.data_ptr(),
                   weight.data_ptr(), out.data_ptr(), _ptr(rows), out_rows, total, n, S, float(eps),
                   (BF16 if parts else _dtype_code(y.dtype)) if y is not None else 0, _dtype_code(mid_dtype), _ptr(mu), _ptr(kept),
                   _ptr(slots), _ptr(seq_start), _ptr(seq_of_row), parts, self._stream())
        if shift is not None and not fused:
            return self.token_shift(out, shift[0], shift[1], shift[2], out_dtype)
        return out

    def _check_shift(self, mu, kept, step, rows, n):
        self._want(mu, "shift weights", torch.float32, (n,))
        self._want(kept, "kept rows of the shift", torch.float32, (kept.shape[0], n))
        if step.num_rows != rows:
            raise KernelError(f"the step has {step.num_rows} rows, the shift got {rows}")
        if max(step.h_slots, default=0) >= kept.shape[0]:
            raise KernelError("a sequence's slot lies outside the kept rows")

    def token_shift(self, h, mu, kept, step, out_dtype):
        """out[r] = h[r] + (row before r of its sequence - h[r]) * mu; the row before a step's first
        row is the sequence's kept row (nothing at position 0), which the sequence's last row replaces."""
        rows, n = h.shape
        self._want(h, "rows to shift", torch.float32)
        self._check_shift(mu, kept, step, rows, n)
        out = torch.empty((rows, n), dtype=out_dtype, device=self.device)
        self._call(self.lib.tli_token_shift, h.data_ptr(), mu.data_ptr(), kept.data_ptr(), out.data_ptr(),
                   step.seq_of_row.data_ptr(), step.row_start.data_ptr(), step.seq_start.data_ptr(),
                   step.slots.data_ptr(), rows, n, _dtype_code(out_dtype), self._stream())
        return out

    # ---- attention with convolved queries and keys, values = keys ----------------------------
    MASK_KINDS = {None: 0, "window": 1, "chunk": 2}
    MAX_CONV_TAPS = 64

    def check_conv_attention_sizes(self, heads: int, kv_heads: int, head_dim: int, taps: int) -> None:
        if not 1 <= head_dim <= self.MAX_HEAD_DIM:
            raise KernelError(f"head_dim {head_dim} is not supported: 1 to {self.MAX_HEAD_DIM}")
        if heads <= 0 or kv_heads <= 0 or heads % kv_heads:
            raise KernelError(f"{heads} heads cannot be grouped over {kv_heads} kv heads")
        if not 1 <= taps <= self.MAX_CONV_TAPS:
            raise KernelError(f"a convolution of {taps} taps is not supported: 1 to {self.MAX_CONV_TAPS}")

    def conv_key_attention(self, qk, bias, conv, state, step, cache, heads, kv_heads, head_dim, taps, scale,
                           temp, penalty, mask):
        """From the raw q and k projections [T, (heads + kv_heads) * head_dim] to the attention's
        output [T, heads * head_dim]: bias, convolution over time (``conv``: its weights tap by tap,
        [taps, channels], oldest tap first; ``state``: the sequences' kept rows [slots, taps - 1,
        channels]), keys into the cache, attention with the keys as values."""
        T = step.num_rows
        q_dim, C = heads * head_dim, (heads + kv_heads) * head_dim
        self.check_conv_attention_sizes(heads, kv_heads, head_dim, taps)
        self._want(qk, "q and k projections", None, (T, C))
        self._want(bias, "projection bias", torch.float32, (C,))
        self._want(conv, "convolution weights", torch.float32, (taps, C))
        if cache is None or not cache.writes:
            raise KernelError("this attention writes its keys into a cache layer of its own")
        kc, g = cache.record("k"), cache.group
        self._want(kc, "key cache", qk.dtype, (kc.shape[0], kv_heads, g.page_size, head_dim))
        self._want(g.tables, "block tables", torch.int32, (step.num_seqs, g.table_width))
        if (step.max_seq_len + g.page_size - 1) // g.page_size > g.table_width:
            raise KernelError("a block table is narrower than its sequence needs")
        if taps > 1:
            if state is None:
                raise KernelError("the convolution needs the sequences' kept rows")
            self._want(state, "kept rows of the convolution", qk.dtype, (state.shape[0], taps - 1, C))
            if max(step.h_slots, default=0) >= state.shape[0]:
                raise KernelError("a sequence's slot lies outside the kept rows")
        kind = self.MASK_KINDS.get(mask[0] if mask is not None else None)
        if kind is None:
            raise KernelError(f"mask '{mask[0]}' is not known")
        size = int(mask[1]) if mask is not None else 0
        r1, r2 = penalty if penalty is not None else (None, None)
        for w, what in ((temp, "head temperatures"), (r1, "distance penalty"), (r2, "distance penalty")):
            if w is not None:
                self._want(w, what, torch.float32, (heads,))
        q = torch.empty((T, q_dim), dtype=qk.dtype, device=self.device)
        self._call(self.lib.tli_conv_heads, qk.data_ptr(), bias.data_ptr(), conv.data_ptr(), _ptr(state), q.data_ptr(),
                   kc.data_ptr(), step.positions.data_ptr(), step.seq_of_row.data_ptr(), step.row_start.data_ptr(),
                   step.slots.data_ptr(), T, step.num_seqs, g.tables.data_ptr(), g.table_width, g.page_size,
                   kc.shape[0], heads, kv_heads, head_dim, taps,
                   1 if (step.max_rows_per_seq == 1 and not self.unfused_decode) else 0, _dtype_code(qk.dtype), self._stream())
        out = torch.empty_like(q)
        if qk.dtype == torch.bfloat16 and head_dim % 16 == 0 and head_dim <= 256 and not self.force_plain:
            # tiles of 16 rows (tiles of 32, two sets of columns a wave sharing each key tile, were measured at
            # heads of 128 and 2,048 rows in blocks of 1,024 positions: 114 us against 94, fewer waves in flight)
            starts = step.h_row_start
            per = 32 if (self.attention_tile_rows == 32 and head_dim <= 128) else 16
            # single rows (decode steps): the heads of a kv head are one tile's columns and share its keys
            grouped = heads // kv_heads if (step.max_rows_per_seq == 1 and 1 < heads // kv_heads <= 16
                                            and not self.unfused_decode) else 0
            if grouped:
                per = 16
            tiles = step.num_rows if grouped else sum((starts[i + 1] - starts[i] + per - 1) // per for i in range(step.num_seqs))
            self._call(self.lib.tli_attention_biased_mfma_bf16, q.data_ptr(), out.data_ptr(), kc.data_ptr(), None,
                       step.row_start.data_ptr(), step.seq_start.data_ptr(), step.num_seqs, tiles, per, g.tables.data_ptr(),
                       g.table_width, g.page_size, kc.shape[0], heads, kv_heads, head_dim, float(scale), _ptr(temp),
                       _ptr(r1), _ptr(r2), kind, size, grouped, self._stream())
            return out
        self._call(self.lib.tli_attention_biased_plain, q.data_ptr(), out.data_ptr(), kc.data_ptr(), None,
                   step.positions.data_ptr(), step.seq_of_row.data_ptr(), g.tables.data_ptr(), g.table_width,
                   g.page_size, kc.shape[0], T, heads, kv_heads, head_dim, float(scale), _ptr(temp), _ptr(r1), _ptr(r2),
                   kind, size, _dtype_code(qk.dtype), self._stream())
        return out

    # ---- layer norm ------------------------------------------------------------------------------
    def add_layernorm(self, resid, deltas, weights, eps, out_dtype, rows=None, num_rows=None):
        """``resid`` (float32 [T, n]) takes the sum of ``deltas`` (none, one or two tensors [T, n] of
        ``out_dtype``: what the parts before still owe it); returns the layer norm (no bias) of its rows
        once for every weight vector of ``weights`` (one or two: norms of the same rows share their mean
        and variance).  With ``rows`` only those rows are computed and ``resid`` stays as it is."""
        total, n = resid.shape
        self._want(resid, "residual", torch.float32)
        deltas = tuple(deltas)
        if len(deltas) > 2 or not 1 <= len(weights) <= 2:
            raise KernelError("add_layernorm takes at most two deltas and one or two weight vectors")
        for d in deltas:
            self._want(d, "residual delta", out_dtype, (total, n))
        for w in weights:
            self._want(w, "norm weight", torch.float32, (n,))
        out_rows = total
        if rows is not None:
            self._want(rows, "row list", torch.int32)
            out_rows = rows.numel() if num_rows is None else num_rows
            if rows.numel() < out_rows:
                raise KernelError("row list is shorter than the rows asked for")
        outs = [torch.empty((out_rows, n), dtype=out_dtype, device=self.device) for _ in weights]
        d1 = deltas[0] if deltas else None
        d2 = deltas[1] if len(deltas) > 1 else None
        self._call(self.lib.tli_add_layernorm, resid.data_ptr(), _ptr(d1), _ptr(d2), weights[0].data_ptr(),
                   _ptr(weights[1]) if len(weights) > 1 else None, outs[0].data_ptr(),
                   outs[1].data_ptr() if len(weights) > 1 else None, _ptr(rows), out_rows, total, n, float(eps),
                   _dtype_code(out_dtype), self._stream())
        return outs

    # ---- the gated delta rule ----------------------------------------------------------------------
    MAX_DELTA_KEY_DIM = 256

    def check_delta_sizes(self, heads: int, kv_heads: int, dk: int, dv: int, taps: int) -> None:
        if heads <= 0 or kv_heads <= 0 or heads % kv_heads or heads > 256:
            raise KernelError(f"{heads} heads (at most 256) cannot be grouped over {kv_heads} key heads")
        if not 1 <= dk <= self.MAX_DELTA_KEY_DIM or dv < 1:
            raise KernelError(f"a state of {dk} x {dv} a head is not supported: key heads of 1 to {self.MAX_DELTA_KEY_DIM}")
        if not 1 <= taps <= self.MAX_CONV_TAPS:
            raise KernelError(f"a convolution of {taps} taps is not supported: 1 to {self.MAX_CONV_TAPS}")

    def small_product(self, x: torch.Tensor, w_rows: torch.Tensor):
        """x W^T in float32 for a matrix of few rows (a router, a few numbers a head): returns (y, transposed).
        In a bfloat16 run the roles are swapped, the few rows of W being the rows of a product that streams x as
        its matrix: one launch for any number of rows of x, and y comes out as [rows of W, rows of x]
        (``transposed``); otherwise y is [rows of x, rows of W] from the ordinary product."""
        M, K = x.shape
        N = w_rows.shape[0]
        self._want(x, "product input")
        self._want(w_rows, "matrix of few rows", x.dtype, (N, K))
        if x.dtype != torch.bfloat16 or K % 8 or self.plain_products or M == 0:
            return self.linear_plain(x, w_rows, torch.float32), False
        y = torch.empty((N, M), dtype=torch.float32, device=self.device)
        for n0 in range(0, N, self.SKINNY_ROWS):
            n1 = min(N, n0 + self.SKINNY_ROWS)
            self._call(self.lib.tli_gemm_skinny_bf16, w_rows[n0:n1].data_ptr(), x.data_ptr(), y[n0:n1].data_ptr(), n1 - n0, M, K,
                       F32, 0, 0, *_NO_GATE, self._stream())
        return y, True

    def delta_state_shape(self, heads: int, dk: int, dv: int):
        """The shape of one request's recurrent state (float32).  The recurrence kernel keeps a head's [dk, dv]
        matrix in the order its lanes hold it, padded to whole blocks, so that it reads and writes it in runs."""
        n = int(self.lib.tli_delta_state_floats(dk, dv))
        if n <= 0:
            raise KernelError(f"a state of {dk} x {dv} a head is not supported")
        return (heads, n)

    def delta_rule(self, proj, gates, conv, a_log, dt_bias, kept, state, step, heads, kv_heads, dk, dv, taps,
                   gates_transposed=False):
        """From the raw projections ``proj`` [T, >= channels] (q, k, v first) and ``gates`` (float32 [T, 2 H]:
        b, then a; [2 H, T] with ``gates_transposed``) to the heads' outputs of the recurrence, float32 [T, H dv].  ``conv``: float32 [taps,
        channels], oldest tap first; ``kept`` [slots, taps - 1, channels] and ``state`` (float32 [slots,
        *delta_state_shape]) are the sequences' state, read (unless a sequence starts at position 0) and replaced."""
        T = step.num_rows
        self.check_delta_sizes(heads, kv_heads, dk, dv, taps)
        qd, vd = kv_heads * dk, heads * dv
        C = 2 * qd + vd
        if proj.dim() != 2 or proj.shape[0] != T or proj.shape[1] < C:
            raise KernelError(f"the projections have shape {tuple(proj.shape)}, expected [{T}, >= {C}]")
        self._want(proj, "projections")
        self._want(gates, "b and a", torch.float32, (2 * heads, T) if gates_transposed else (T, 2 * heads))
        ba_row, ba_col = (1, T) if gates_transposed else (2 * heads, 1)
        self._want(conv, "convolution weights", torch.float32, (taps, C))
        self._want(a_log, "A_log", torch.float32, (heads,))
        self._want(dt_bias, "dt_bias", torch.float32, (heads,))
        self._want(state, "recurrent state", torch.float32, (state.shape[0],) + self.delta_state_shape(heads, dk, dv))
        slots = state.shape[0]
        if taps > 1:
            if kept is None:
                raise KernelError("the convolution needs the sequences' kept rows")
            self._want(kept, "kept rows of the convolution", proj.dtype, (slots, taps - 1, C))
        if max(step.h_slots, default=0) >= slots:
            raise KernelError("a sequence's slot lies outside the state")
        f32 = dict(dtype=torch.float32, device=self.device)
        qn, kn = torch.empty((T, qd), **f32), torch.empty((T, qd), **f32)
        vc, out = torch.empty((T, vd), **f32), torch.empty((T, vd), **f32)
        beta, decay, qk = torch.empty((T, heads), **f32), torch.empty((T, heads), **f32), torch.empty((T, kv_heads), **f32)
        self._call(self.lib.tli_delta_prepare, proj.data_ptr(), proj.shape[1], conv.data_ptr(), _ptr(kept), gates.data_ptr(),
                   ba_row, ba_col, a_log.data_ptr(), dt_bias.data_ptr(), step.positions.data_ptr(), step.seq_of_row.data_ptr(),
                   step.row_start.data_ptr(), step.seq_start.data_ptr(), step.slots.data_ptr(), qn.data_ptr(),
                   kn.data_ptr(), vc.data_ptr(), beta.data_ptr(), decay.data_ptr(), qk.data_ptr(), T, step.num_seqs,
                   heads, kv_heads, dk, dv, taps, _dtype_code(proj.dtype), self._stream())
        self._call(self.lib.tli_delta_recurrence, qn.data_ptr(), kn.data_ptr(), vc.data_ptr(), beta.data_ptr(),
                   decay.data_ptr(), qk.data_ptr(), state.data_ptr(), out.data_ptr(), step.row_start.data_ptr(),
                   step.seq_start.data_ptr(), step.slots.data_ptr(), step.num_seqs, heads, kv_heads, dk, dv, self._stream())
        return out

    def gated_rmsnorm(self, o, proj, gate_at, weight, eps, heads, dv, out_dtype):
        """y = o / sqrt(mean(o^2) + eps) * weight * silu(gate) per head; ``o`` float32 [T, H dv], the gate
        is columns ``gate_at`` .. ``gate_at + H dv`` of ``proj``."""
        T = o.shape[0]
        self._want(o, "heads' outputs", torch.float32, (T, heads * dv))
        self._want(proj, "projections", out_dtype)
        if proj.shape[0] != T or proj.shape[1] < gate_at + heads * dv:
            raise KernelError("the gate lies outside the projections")
        self._want(weight, "norm weight", torch.float32, (dv,))
        out = torch.empty((T, heads * dv), dtype=out_dtype, device=self.device)
        self._call(self.lib.tli_gated_rmsnorm, o.data_ptr(), proj.data_ptr() + gate_at * proj.element_size(), proj.shape[1],
                   weight.data_ptr(), out.data_ptr(), T, heads, dv, float(eps), _dtype_code(out_dtype), self._stream())
        return out

    # ---- routed experts ---------------------------------------------------------------------------------
    MAX_EXPERTS_TOP = 32

    def check_expert_sizes(self, experts, top, groups, keep, hidden, inter) -> None:
        if not 1 <= top <= min(experts, self.MAX_EXPERTS_TOP) or experts > 2048:
            raise KernelError(f"{top} of {experts} experts a row: at most {self.MAX_EXPERTS_TOP} of at most 2048")
        if not 1 <= groups <= 64 or experts % groups or not 1 <= keep <= groups or keep * (experts // groups) < top:
            raise KernelError(f"{experts} experts in {groups} groups (at most 64), {keep} kept: cannot give {top}")
        if hidden * 4 > 64 * 1024 or top * inter * 4 > 64 * 1024:
            raise KernelError("a row, or the hidden units of a row's experts, do not fit a workgroup's memory")

    def pack_experts(self, w_gate_up, w_down, gated=True):
        """The experts' matrices in the tiled layout that the matrix-core kernels read (``tile_matrix`` of every
        expert's gate, up and down matrix; ``gated`` false: ``w_gate_up`` is [E, ff, n], up matrices alone), or None
        where those kernels do not apply (float32, sizes that are no multiples of 8, the plain kernels asked for): then
        ``apply_experts`` works from the row-major matrices."""
        E, rows, n = w_gate_up.shape
        ff = rows // 2 if gated else rows
        if w_gate_up.dtype != torch.bfloat16 or n % 8 or ff % 8 or E > 2048 or self.plain_products:
            return None
        return {"gate": torch.stack([self.tile_matrix(w_gate_up[e, :ff]) for e in range(E)]) if gated else None,
                "up": torch.stack([self.tile_matrix(w_gate_up[e, ff:] if gated else w_gate_up[e]) for e in range(E)]),
                "down": torch.stack([self.tile_matrix(w_down[e]) for e in range(E)]),
                "experts": E, "hidden": n, "inter": ff}

    ROUTER_SCORES = ("sigmoid", "softmax")
    ROUTER_GROUP_SCORES = ("top2", "max")

    def check_router(self, score: str, group_score: str) -> None:
        if score not in self.ROUTER_SCORES or group_score not in self.ROUTER_GROUP_SCORES:
            raise KernelError(f"a router with '{score}' scores and groups scored by '{group_score}' is not known; known: "
                              f"{', '.join(self.ROUTER_SCORES)}; {', '.join(self.ROUTER_GROUP_SCORES)}")

    def route_experts(self, z, experts, top, groups, keep, scale, has_shared, transposed=False, score="sigmoid",
                      group_score="top2", normalize=True, correction=None):
        """From router logits ``z`` (float32 [T, E (+ 1)]; [E (+ 1), T] with ``transposed``) to the chosen experts (int32 [T, top]), their
        weights (float32 [T, top]) and, if the last column is a shared expert's gate, its sigmoid [T].  ``score``: the
        scores are the logits' sigmoid or their softmax over the E; ``correction`` (float32 [E]) is added to them for the
        choice only; ``group_score``: a group counts by its two largest choice scores or by its largest; ``normalize``:
        the chosen scores are divided by their sum."""
        self.check_router(score, group_score)
        if correction is not None:
            self._want(correction, "router correction", torch.float32, (experts,))
        T = z.shape[1] if transposed else z.shape[0]
        columns = experts + (1 if has_shared else 0)
        self._want(z, "router logits", torch.float32, (columns, T) if transposed else (T, columns))
        z_row, z_col = (1, T) if transposed else (columns, 1)
        ids = torch.empty((T, top), dtype=torch.int32, device=self.device)
        weights = torch.empty((T, top), dtype=torch.float32, device=self.device)
        gate = torch.empty((T,), dtype=torch.float32, device=self.device) if has_shared else None
        self._call(self.lib.tli_moe_route, z.data_ptr(), z_row, z_col, ids.data_ptr(), weights.data_ptr(), _ptr(gate), T,
                   experts, top, groups, keep, float(scale), 1 if has_shared else 0, self.ROUTER_SCORES.index(score),
                   self.ROUTER_GROUP_SCORES.index(group_score), 1 if normalize else 0, _ptr(correction), self._stream())
        return ids, weights, gate

    ROUTER_ROWS = 128            # up to so many rows the router's product and its choice are one launch

    def router(self, x, w_rows, experts, top, groups, keep, scale, has_shared, score="sigmoid", group_score="top2", normalize=True,
               correction=None):
        """``route_experts`` of the logits x w_rows^T (float32 sums); ``w_rows`` [E (+ 1), n]."""
        T, n = x.shape
        if x.dtype != torch.bfloat16 or n % 8 or not 0 < T <= self.ROUTER_ROWS or self.plain_products:
            z, transposed = self.small_product(x, w_rows)
            return self.route_experts(z, experts, top, groups, keep, scale, has_shared, transposed, score, group_score, normalize, correction)
        self.check_router(score, group_score)
        self._want(x, "router input")
        self._want(w_rows, "router rows", torch.bfloat16, (experts + (1 if has_shared else 0), n))
        if correction is not None:
            self._want(correction, "router correction", torch.float32, (experts,))
        ids = torch.empty((T, top), dtype=torch.int32, device=self.device)
        weights = torch.empty((T, top), dtype=torch.float32, device=self.device)
        gate = torch.empty((T,), dtype=torch.float32, device=self.device) if has_shared else None
        self._call(self.lib.tli_moe_router_bf16, x.data_ptr(), w_rows.data_ptr(), n, ids.data_ptr(), weights.data_ptr(), _ptr(gate), T,
                   experts, top, groups, keep, float(scale), 1 if has_shared else 0, self.ROUTER_SCORES.index(score),
                   self.ROUTER_GROUP_SCORES.index(group_score), 1 if normalize else 0, _ptr(correction), self._stream())
        return ids, weights, gate

    def apply_experts(self, x, ids, weights, w_gate_up, w_down, packed, shared, shared_gate, limit=0.0, slope=1.0,
                      activation=None, weight_on_input=False):
        """sum_j weights[t, j] * expert ids[t, j] (x[t])  (+ shared_gate[t] * shared[t], or + shared[t] without a
        gate);  ``w_gate_up`` [E, 2 ff, n] (an expert's gate rows, then its up rows), ``w_down`` [E, n, ff]; with
        ``packed`` (what ``pack_experts`` gave) the row-major matrices may be None.  An id from E on is an expert
        that hands its input on: its term is weights[t, j] * x[t].  ``limit`` > 0: the experts' hidden units are the
        limited form (see ``swiglu``) instead of silu(gate) * up.  ``activation`` (one of ``ACTIVATIONS``): experts
        without a gate matrix, down(act(up x)), ``w_gate_up`` being [E, ff, n]; with ``weight_on_input`` a pair's weight
        multiplies the expert's input and not its output."""
        T, n = x.shape
        top = ids.shape[1]
        act = -1
        if activation is not None:
            self.check_activation(activation)
            act = self.ACTIVATIONS[activation]
        elif weight_on_input:
            raise KernelError("weights on the experts' inputs are for experts without a gate")
        on_input = 1 if weight_on_input else 0
        self._want(x, "expert input")
        self._want(ids, "chosen experts", torch.int32, (T, top))
        self._want(weights, "experts' weights", torch.float32, (T, top))
        if shared is not None:
            self._want(shared, "shared expert's output", x.dtype, (T, n))
            if shared_gate is not None:
                self._want(shared_gate, "shared expert's gate", torch.float32, (T,))
        out = torch.empty((T, n), dtype=x.dtype, device=self.device)
        if T == 0:
            return out
        if packed is not None and x.dtype == torch.bfloat16 and not self.plain_products:
            E, ff = packed["experts"], packed["inter"]
            if packed["hidden"] != n:
                raise KernelError(f"the experts read rows of {packed['hidden']}, the input has {n}")
            nb, kb = (ff + 15) // 16, (n + 127) // 128
            for role, shape in (("gate", (E, nb, kb, 4, 4, 16, 8)), ("up", (E, nb, kb, 4, 4, 16, 8)),
                                ("down", (E, (n + 15) // 16, (ff + 127) // 128, 4, 4, 16, 8))):
                if role == "gate" and act >= 0:
                    continue
                self._want(packed[role], f"experts' {role} matrices (tiled)", torch.bfloat16, shape)
            a_call = max(1, (65535 - E) * 16 // top)                 # (a launch's grid holds 65,535 tiles)
            for t0 in range(0, T, a_call):
                t1 = min(T, t0 + a_call)
                pairs = (t1 - t0) * top
                RT = self.moe_tile or int(self.lib.tli_moe_grouped_tile(pairs, E))
                slots = (pairs // RT + E) * RT
                i32 = dict(dtype=torch.int32, device=self.device)
                order, pos = torch.empty((slots,), **i32), torch.empty((pairs,), **i32)
                tile_expert, num_tiles = torch.empty((slots // RT,), **i32), torch.empty((1,), **i32)
                hid = torch.empty((slots, ff), dtype=torch.bfloat16, device=self.device)
                part = torch.empty((slots, n), dtype=torch.float32, device=self.device)
                self._call(self.lib.tli_moe_grouped_bf16, x[t0:t1].data_ptr(), ids[t0:t1].data_ptr(), weights[t0:t1].data_ptr(),
                           None if act >= 0 else packed["gate"].data_ptr(), packed["up"].data_ptr(), packed["down"].data_ptr(), order.data_ptr(),
                           pos.data_ptr(), tile_expert.data_ptr(), num_tiles.data_ptr(), hid.data_ptr(), part.data_ptr(),
                           None if shared is None else shared[t0:t1].data_ptr(),
                           None if (shared is None or shared_gate is None) else shared_gate[t0:t1].data_ptr(),
                           out[t0:t1].data_ptr(), t1 - t0, top, E, n, ff, RT, float(limit), float(slope), act, on_input,
                           self._stream())
            return out
        if w_gate_up is None or w_down is None:
            raise KernelError("the experts' row-major matrices were not kept and the tiled ones do not apply here")
        E, rows, _ = w_gate_up.shape
        ff = rows if act >= 0 else rows // 2
        self._want(w_gate_up, "experts' gate and up matrices", x.dtype, (E, ff if act >= 0 else 2 * ff, n))
        self._want(w_down, "experts' down matrices", x.dtype, (E, n, ff))
        hid = torch.empty((T * top, ff), dtype=x.dtype, device=self.device)
        for t0 in range(0, T, 32768):
            t1 = min(T, t0 + 32768)
            self._call(self.lib.tli_moe_experts, x[t0:t1].data_ptr(), ids[t0:t1].data_ptr(), weights[t0:t1].data_ptr(),
                       w_gate_up.data_ptr(), w_down.data_ptr(), hid[t0 * top:].data_ptr(),
                       None if shared is None else shared[t0:t1].data_ptr(),
                       None if (shared is None or shared_gate is None) else shared_gate[t0:t1].data_ptr(),
                       out[t0:t1].data_ptr(), t1 - t0, top, n, ff, E, _dtype_code(x.dtype), float(limit), float(slope), act,
                       on_input, self._stream())
        return out

    # ---- blocks that norm what a sublayer gives ------------------------------------------------------------
    def residual_rows(self, resid: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
        """The float32 residual's rows in the run's type (the residual itself in a float32 run)."""
        self._want(resid, "residual", torch.float32)
        if dtype == torch.float32:
            return resid
        if dtype != torch.bfloat16:
            raise KernelError(f"kernels take float32 or bfloat16 tensors, not {dtype}")
        out = torch.empty(resid.shape, dtype=dtype, device=self.device)
        self._call(self.lib.tli_residual_rows, resid.data_ptr(), out.data_ptr(), resid.numel(), self._stream())
        return out

    def norm_add(self, resid, y, weight, eps, out_dtype):
        """resid (float32 [T, n]) += weight * y / sqrt(mean(y^2) + eps) with ``y`` [T, n] in the run's type (or an
        unfinished product); returns the new residual's rows in the run's type (the residual itself in a float32 run)."""
        if isinstance(y, DeferredSum) and y.dtype == out_dtype == torch.bfloat16 and resid.shape[1] <= 8192:
            return self._norm_add_norm(resid, y, weight, eps, None, 0.0, out_dtype, None, None, None, None)
        y = self.resolve(y)
        total, n = resid.shape
        self._want(resid, "residual", torch.float32)
        self._want(weight, "norm weight", torch.float32, (n,))
        self._want(y, "sublayer output", out_dtype, (total, n))
        out = resid if out_dtype == torch.float32 else torch.empty((total, n), dtype=out_dtype, device=self.device)
        self._call(self.lib.tli_norm_add, resid.data_ptr(), y.data_ptr(), weight.data_ptr(),
                   None if out is resid else out.data_ptr(), total, n, float(eps), _dtype_code(out_dtype), self._stream())
        return out

    # ---- blocks that norm what a sublayer reads and what it gives ---------------------------------------------
    def norm_add_norm(self, resid, y, w_out, eps_out, w_in, eps_in, out_dtype, rows=None, num_rows=None):
        """resid (float32 [T, n]) += w_out * y / sqrt(mean(y^2) + eps_out) for ``y`` [T, n] in the run's type or an unfinished
        product (None: nothing is added); returns w_in * resid / sqrt(mean(resid^2) + eps_in) in the run's type.  With
        ``rows`` (int32 on the device, the first ``num_rows`` of them) only those rows, and ``resid`` is left as it is."""
        return self._norm_add_norm(resid, y, w_out, eps_out, w_in, eps_in, out_dtype, rows, num_rows, None, None)

    def norm_add_norm_mixes(self, resid, y, w_out, eps_out, w_in, eps_in, out_dtype, mixes, step):
        """``norm_add_norm`` and the ``token_mixes`` of its rows in one pass, [mixes, T, n], for a step of one row a sequence;
        None for other steps, with nothing done.  ``mixes`` = (mu [m, n], kept rows)."""
        if not self._single_rows(step):
            return None
        return self._norm_add_norm(resid, y, w_out, eps_out, w_in, eps_in, out_dtype, None, None, mixes, step)

    def _norm_add_norm(self, resid, y, w_out, eps_out, w_in, eps_in, out_dtype, rows, num_rows, mixes, step):
        total, n = resid.shape
        self._want(resid, "residual", torch.float32)
        if w_in is not None:
            self._want(w_in, "norm weight", torch.float32, (n,))
        parts = 0
        if y is not None:
            if isinstance(y, DeferredSum) and y.dtype == out_dtype == torch.bfloat16:
                y, parts = y.parts, y.parts.shape[0]
                self._want(y, "partial sums of a sublayer's output", torch.float32, (parts, total, n))
            else:
                y = self.resolve(y)
                self._want(y, "sublayer output", out_dtype, (total, n))
            self._want(w_out, "norm weight", torch.float32, (n,))
        count = total
        if rows is not None:
            self._want(rows, "rows", torch.int32)
            count = int(num_rows)
            if count > rows.numel():
                raise KernelError(f"{count} rows wanted, {rows.numel()} are named")
        mu, kept, m, slots, starts = None, None, 0, None, None
        if mixes is not None:
            mu, kept = mixes
            m = mu.shape[0]
            self._check_mixes(mu, kept, step, total, n, out_dtype)
            slots, starts = step.slots.data_ptr(), step.seq_start.data_ptr()
        out = torch.empty((count, n) if mixes is None else (m, count, n), dtype=out_dtype, device=self.device)
        self._call(self.lib.tli_norm_add_norm, resid.data_ptr(), _ptr(y), parts, total, None if y is None else w_out.data_ptr(),
                   float(eps_out), _ptr(w_in), float(eps_in), out.data_ptr(), _ptr(rows), count, n, _ptr(mu), m, _ptr(kept), slots, starts,
                   _dtype_code(out_dtype), self._stream())
        return out

    def _check_mixes(self, mu, kept, step, rows, n, dtype):
        self._want(mu, "weights of the mixes", torch.float32, (mu.shape[0], n))
        self._want(kept, "kept rows", dtype, (kept.shape[0], n))
        if step.num_rows != rows:
            raise KernelError(f"the step has {step.num_rows} rows, the mixes got {rows}")
        if max(step.h_slots, default=0) >= kept.shape[0]:
            raise KernelError("a sequence's slot lies outside the kept rows")

    def token_mixes(self, h, mu, kept, step):
        """out[m, r] = h[r] + (row before r of its sequence - h[r]) * mu[m], [mixes, rows, n]; the row before a step's
        first row is the sequence's kept row (nothing at position 0), which the sequence's last row replaces."""
        rows, n = h.shape
        self._want(h, "rows to mix")
        self._check_mixes(mu, kept, step, rows, n, h.dtype)
        out = torch.empty((mu.shape[0], rows, n), dtype=h.dtype, device=self.device)
        self._call(self.lib.tli_token_mixes, h.data_ptr(), mu.data_ptr(), mu.shape[0], kept.data_ptr(), out.data_ptr(),
                   step.seq_of_row.data_ptr(), step.row_start.data_ptr(), step.seq_start.data_ptr(), step.slots.data_ptr(), rows, n,
                   _dtype_code(h.dtype), self._stream())
        return out

    def token_gate(self, z, table, at, token_ids, activation):
        """act(z[t]) * table[token_ids[t], at : at + n], [T, n] in the type of ``z`` [T, n]."""
        self.check_activation(activation)
        T, n = z.shape
        self._want(z, "gate's logits")
        self._want(table, "tokens' vectors", z.dtype)
        self._want(token_ids, "token ids", torch.int32)
        if token_ids.numel() < T or at < 0 or at + n > table.shape[1]:
            raise KernelError("a token's vector lies outside the table")
        out = torch.empty((T, n), dtype=z.dtype, device=self.device)
        self._call(self.lib.tli_token_gate, z.data_ptr(), table.data_ptr(), token_ids.data_ptr(), out.data_ptr(), T, n, table.shape[1],
                   at, table.shape[0], self.ACTIVATIONS[activation], _dtype_code(z.dtype), self._stream())
        return out

    # ---- attention whose keys and values have sizes of their own -------------------------------------------
    MAX_SIZED_DIM = 1024

    def check_sized_attention(self, heads: int, kv_heads: int, key_dim: int, value_dim: int) -> None:
        if not (1 <= key_dim <= self.MAX_SIZED_DIM and 1 <= value_dim <= self.MAX_SIZED_DIM):
            raise KernelError(f"heads of {key_dim} and {value_dim} elements are not supported: 1 to {self.MAX_SIZED_DIM}")
        if heads <= 0 or kv_heads <= 0 or heads % kv_heads:
            raise KernelError(f"{heads} heads cannot be grouped over {kv_heads} kv heads")

    def _check_tables(self, g, step):
        self._want(g.tables, "block tables", torch.int32, (step.num_seqs, g.table_width))
        if (step.max_seq_len + g.page_size - 1) // g.page_size > g.table_width:
            raise KernelError("a block table is narrower than its sequence needs")

    def sized_attention(self, q, step, g, kc, vc, heads, kv_heads, maps, key_dim, value_dim, scale, window, keep_first,
                        out_dtype, sinks=None):
        """Attention of ``q`` [T, heads * maps, key_dim] over the key cache ``kc`` [pages, kv_heads * maps, page, key_dim]
        and the value cache ``vc`` [pages, kv_heads, value_dim, page] (None: a key's first value_dim elements are its
        values); map m of head h reads key head (h // (heads / kv_heads)) * maps + m.  A row at p sees t <= p with
        p - t < window or t < keep_first (window None: all).  ``sinks`` (float32 [heads * maps]): the softmax's
        denominator of (head, map) also holds exp(sink), a logit with no key and no value.  Returns [T, heads * maps,
        value_dim] of ``out_dtype``."""
        T = step.num_rows
        self.check_sized_attention(heads, kv_heads, key_dim, value_dim)
        self._want(q, "queries", None, (T, heads * maps, key_dim))
        pages = kc.shape[0]
        self._want(kc, "key cache", q.dtype, (pages, kv_heads * maps, g.page_size, key_dim))
        if vc is not None:
            self._want(vc, "value cache", q.dtype, (pages, kv_heads, value_dim, g.page_size))
        elif value_dim > key_dim:
            raise KernelError("values that are the start of their keys cannot be longer than the keys")
        self._check_tables(g, step)
        if sinks is not None:
            self._want(sinks, "sinks", torch.float32, (heads * maps,))
        if out_dtype not in (q.dtype, torch.float32):
            raise KernelError(f"attention over {q.dtype} gives {q.dtype} or float32, not {out_dtype}")
        out = torch.empty((T, heads * maps, value_dim), dtype=out_dtype, device=self.device)
        keep = int(keep_first or 0) if window else 0
        if (q.dtype == torch.bfloat16 and not self.force_plain
                and self.lib.tli_attention_sized_mfma_takes(key_dim, value_dim, g.page_size, 0 if vc is None else 1)):
            # tiles of 16 rows of a sequence; in steps of single rows a tile is a row, its columns the heads of a key head
            grouped = 1 if step.max_rows_per_seq == 1 else 0
            starts = step.h_row_start
            tiles = T if grouped else sum((starts[i + 1] - starts[i] + 15) // 16 for i in range(step.num_seqs))
            splits, parts = 1, None
            if grouped and vc is None and out_dtype == torch.bfloat16 and step.num_seqs == T:
                splits = self._sized_splits(T, step.reach, heads * maps, kv_heads * maps, window, keep)
                if splits > 1:
                    parts = torch.empty((T * heads * maps * splits * (value_dim + 4),), dtype=torch.float32, device=self.device)
            self._call(self.lib.tli_attention_sized_mfma_bf16, q.data_ptr(), out.data_ptr(), kc.data_ptr(), _ptr(vc),
                       step.row_start.data_ptr(), step.seq_start.data_ptr(), step.num_seqs, tiles, g.tables.data_ptr(),
                       g.table_width, g.page_size, pages, heads, kv_heads, maps, key_dim, value_dim, float(scale),
                       int(window or 0), keep, grouped, 1 if out_dtype == torch.float32 else 0, _ptr(sinks), splits, _ptr(parts),
                       self._stream())
            return out
        self._call(self.lib.tli_attention_sized_plain, q.data_ptr(), out.data_ptr(), kc.data_ptr(), _ptr(vc),
                   step.positions.data_ptr(), step.seq_of_row.data_ptr(), g.tables.data_ptr(), g.table_width, g.page_size,
                   pages, T, heads, kv_heads, maps, key_dim, value_dim, float(scale), int(window or 0),
                   keep, _dtype_code(q.dtype), 1 if out_dtype == torch.float32 else 0, _ptr(sinks),
                   self._stream())
        return out

    def differential_attention(self, proj, step, cache, heads, kv_heads, dim, vdim, q_weight, k_weight, norm_eps, scale,
                               lam, after, window, keep_first):
        """Attention with two softmax maps a head, from the raw projections ``proj`` [T, q (heads * 2 * dim) | k
        (kv_heads * 2 * dim) | v (kv_heads * vdim) | one gate logit a head] to the heads' gated outputs [T, heads *
        vdim]: q and k normed per head and map (RMS norm, weights ``q_weight``, ``k_weight`` float32 [dim]), k and v
        into the cache (records "k" [kv_heads * 2, page, dim] and "v" [kv_heads, vdim, page]), a1 and a2 the maps'
        outputs over the same values, o = a1 - lam * a2, o / sqrt(mean(o^2) + norm_eps) * after * sigmoid(gate)."""
        T = step.num_rows
        width = (heads + kv_heads) * 2 * dim + kv_heads * vdim + heads
        self._want(proj, "projections", None, (T, width))
        for w in (q_weight, k_weight):
            self._want(w, "head norm weight", torch.float32, (dim,))
        if cache is None or not cache.writes:
            raise KernelError("this attention writes its keys and values into a cache layer of its own")
        kc, vc, g = cache.record("k"), cache.record("v"), cache.group
        pages = kc.shape[0]
        self._want(kc, "key cache", proj.dtype, (pages, kv_heads * 2, g.page_size, dim))
        self._want(vc, "value cache", proj.dtype, (pages, kv_heads, vdim, g.page_size))
        self._check_tables(g, step)
        q = torch.empty((T, heads * 2, dim), dtype=proj.dtype, device=self.device)
        self._call(self.lib.tli_diff_prepare, proj.data_ptr(), width, q.data_ptr(), kc.data_ptr(), vc.data_ptr(),
                   step.positions.data_ptr(), step.seq_of_row.data_ptr(), g.tables.data_ptr(), g.table_width, g.page_size,
                   pages, T, heads, kv_heads, dim, vdim, q_weight.data_ptr(), k_weight.data_ptr(), float(norm_eps),
                   _dtype_code(proj.dtype), self._stream())
        maps = self.sized_attention(q, step, g, kc, vc, heads, kv_heads, 2, dim, vdim, scale, window, keep_first,
                                    torch.float32)
        out = torch.empty((T, heads * vdim), dtype=proj.dtype, device=self.device)
        self._call(self.lib.tli_diff_combine, maps.data_ptr(), proj.data_ptr(), width, width - heads, out.data_ptr(), T,
                   heads, vdim, float(lam), float(after), float(norm_eps), _dtype_code(proj.dtype), self._stream())
        return out

    SIZED_WORKGROUPS = 256           # decoding rows whose keys are shared out: the workgroups aimed at,
    SIZED_SPLIT_KEYS = 32            # and the fewest keys of a split (two tiles of 16)

    def _sized_splits(self, T, reach, units, key_heads, window, keep) -> int:
        """Over how many workgroups the keys of one (row, key head) that decodes are shared out, where all heads read one cached
        vector; ``reach``: a power of two that the longest sequence fits.  A workgroup takes a row's tiles of 16 keys one
        after the other."""
        keys = min(reach, (window + 15 if window else reach) + keep)
        groups = T * key_heads * ((units // key_heads + 63) // 64)
        return max(1, self.sized_splits or min(self.SIZED_WORKGROUPS // groups, keys // self.SIZED_SPLIT_KEYS, 64))

    def head_products(self, x, x_stride, w, out=None, out_stride=None, x_at=0, out_at=0, gate=None):
        """y[t, h, :] = w[h] x[t, h, :] for a matrix a head, ``w`` [heads, N, K].  ``x`` is [T, columns]: the input of
        head h are the K columns from ``x_at + h * x_stride`` on; ``out`` likewise with ``out_stride`` and ``out_at``
        (made as [T, heads * N] if not given).  Float32 sums, results in the type of x.  ``gate`` = (tensor [T, columns],
        column): head h's results are multiplied by the sigmoid of that tensor's element h columns on."""
        T, ldx = x.shape
        heads, N, K = w.shape
        gate_ptr, gate_ld = None, 0
        if gate is not None:
            z, z_at = gate
            self._want(z, "heads' gates", x.dtype)
            if z.dim() != 2 or z.shape[0] != T or z_at < 0 or z_at + heads > z.shape[1]:
                raise KernelError("the heads' gates lie outside their rows")
            gate_ptr, gate_ld = z.data_ptr() + z_at * z.element_size(), z.shape[1]
        self._want(x, "heads' inputs")
        self._want(w, "matrices of the heads", x.dtype)
        if x_at < 0 or x_stride < K or x_at + (heads - 1) * x_stride + K > ldx:
            raise KernelError("a head's input lies outside its row")
        if out is None:
            out, out_stride, out_at = torch.empty((T, heads * N), dtype=x.dtype, device=self.device), N, 0
        self._want(out, "heads' outputs", x.dtype)
        if out.dim() != 2 or out.shape[0] != T or out_at < 0 or out_stride < N or out_at + (heads - 1) * out_stride + N > out.shape[1]:
            raise KernelError("a head's output lies outside its row")
        es = x.element_size()
        if (x.dtype == torch.bfloat16 and not self.plain_products and x_at % 4 == 0 and out_at % 4 == 0
                and self.lib.tli_head_products_mfma_takes(N, K, ldx, x_stride, out.shape[1], out_stride)):
            self._call(self.lib.tli_head_products_mfma_bf16, x.data_ptr() + x_at * es, ldx, x_stride, w.data_ptr(),
                       out.data_ptr() + out_at * es, out.shape[1], out_stride, T, heads, N, K, gate_ptr, gate_ld, self._stream())
            return out
        self._call(self.lib.tli_head_products_plain, x.data_ptr() + x_at * es, ldx, x_stride, w.data_ptr(),
                   out.data_ptr() + out_at * es, out.shape[1], out_stride, T, heads, N, K, gate_ptr, gate_ld, _dtype_code(x.dtype),
                   self._stream())
        return out

    def norm_rows(self, proj, at, n, weight, eps):
        """weight * x / sqrt(mean(x^2) + eps) of the ``n`` columns from ``at`` on of every row of ``proj``, [T, n]."""
        T = proj.shape[0]
        self._want(proj, "projections")
        self._want(weight, "norm weight", torch.float32, (n,))
        if at < 0 or at + n > proj.shape[1]:
            raise KernelError("the elements to norm lie outside their row")
        out = torch.empty((T, n), dtype=proj.dtype, device=self.device)
        self._call(self.lib.tli_norm_rows, proj.data_ptr() + at * proj.element_size(), proj.shape[1], weight.data_ptr(), out.data_ptr(),
                   T, n, float(eps), _dtype_code(proj.dtype), self._stream())
        return out

    def latent_attention(self, query, q_at, own, step, cache, heads, dim, rot, rank, vdim, rotary, scale, w_qk, w_v, window=None,
                         sinks=None, gate=None):
        """Attention whose keys and values are made from one latent vector a position, from the raw queries
        ``query[:, q_at:]`` [T, heads * (dim + rot)] to the heads' outputs [T, heads * vdim].  ``own`` = (projections, column,
        norm weight, eps): latent (rank) | key part (rot) of the step's rows, which are normed, turned and written to the
        cache here; None: another call of this step has written them.
        The cache (record "latent" [page, rank + rot]) keeps the normed latent vector and the turned key part; a
        head's score is q_plain . (W_uk c) + q_turned . k_turned, computed as (W_uk^T q_plain) . c with ``w_qk``
        [heads, rank, dim] = W_uk^T a head, so that all heads read the one cached vector; the weighted sum of the
        latent vectors then goes through ``w_v`` [heads, vdim, rank] = W_uv a head.  ``window``, ``sinks``: as in
        ``sized_attention``; ``gate``: one number a head, as in ``head_products``."""
        T = step.num_rows
        self._want(query, "queries")
        if query.dim() != 2 or query.shape[0] != T or q_at < 0 or q_at + heads * (dim + rot) > query.shape[1]:
            raise KernelError(f"the queries have shape {tuple(query.shape)}, expected [{T}, >= {q_at + heads * (dim + rot)}]")
        if cache is None or cache.writes != (own is not None):
            raise KernelError("this attention either writes latent vectors of its own or reads those of another layer")
        es = query.element_size()
        down_ptr, down_ld, norm_ptr, norm_eps = None, 0, None, 0.0
        if own is not None:
            proj, at, norm_weight, norm_eps = own
            self._want(proj, "projections", query.dtype)
            if proj.dim() != 2 or proj.shape[0] != T or at < 0 or at + rank + rot > proj.shape[1]:
                raise KernelError("the latent vector lies outside the projections")
            self._want(norm_weight, "latent norm weight", torch.float32, (rank,))
            down_ptr, down_ld, norm_ptr = proj.data_ptr() + at * es, proj.shape[1], norm_weight.data_ptr()
        kc, g = cache.record("latent"), cache.group
        pages = kc.shape[0]
        key = rank + rot
        self._want(kc, "latent cache", query.dtype, (pages, g.page_size, key))
        self._check_tables(g, step)
        cos, sin, rd = self._rotary(rotary, step)
        if rd > rot:
            raise KernelError(f"{rd} turned elements do not fit a key part of {rot}")
        q = torch.empty((T, heads, key), dtype=query.dtype, device=self.device)
        self._call(self.lib.tli_latent_prepare, query.data_ptr() + q_at * es, query.shape[1], down_ptr, down_ld, q.data_ptr(),
                   kc.data_ptr(), step.positions.data_ptr(),
                   step.seq_of_row.data_ptr(), g.tables.data_ptr(), g.table_width, g.page_size, pages, T, heads, dim, rot,
                   rank, rd, norm_ptr, float(norm_eps), cos.data_ptr(), sin.data_ptr(),
                   _dtype_code(query.dtype), self._stream())
        self._want(w_qk, "matrices into the latent space", query.dtype, (heads, rank, dim))
        self._want(w_v, "matrices out of the latent space", query.dtype, (heads, vdim, rank))
        self.head_products(query, dim + rot, w_qk, out=q.view(T, heads * key), out_stride=key, x_at=q_at)
        o = self.sized_attention(q, step, g, kc.view(pages, 1, g.page_size, key), None, heads, 1, 1, key, rank, scale,
                                 window, 0, query.dtype, sinks=sinks)
        return self.head_products(o.view(T, heads * rank), rank, w_v, gate=gate)

    # ---- attention with biases and a sink whose values may be its keys ------------------------------------
    def sink_attention(self, proj, step, cache, heads, kv_heads, head_dim, bias, rotary, scale, sinks, window,
                       values_are_keys):
        """From the raw projections ``proj`` [T, q (heads * head_dim) | k (kv_heads * head_dim) (| v likewise, unless
        ``values_are_keys``)] to the heads' outputs [T, heads * head_dim]: ``bias`` (float32 over the projections' row,
        or None) is added, q and k are turned (``rotary``: cos, sin, turned elements; pairs (i, i + n/2)), the turned
        keys and the values (the keys before they are turned, or their own projection) go into the cache (records
        "k" [kv_heads, page, head_dim] and "v" [kv_heads, head_dim, page]), attention with ``sinks`` (float32 [heads]
        or None) over the cache."""
        T = step.num_rows
        width = (heads + (1 if values_are_keys else 2) * kv_heads) * head_dim
        self._want(proj, "projections", None, (T, width))
        if bias is not None:
            self._want(bias, "projections' bias", torch.float32, (width,))
        if cache is None or not cache.writes:
            raise KernelError("this attention writes its keys and values into a cache layer of its own")
        kc, vc, g = cache.record("k"), cache.record("v"), cache.group
        self._check_cache(kc, vc, g, kv_heads, head_dim, proj.dtype, step)
        cos = sin = None
        rd = npos = 0
        if rotary is not None:
            cos, sin, rd = self._rotary(rotary, step)
            npos = cos.shape[0]
        q = torch.empty((T, heads, head_dim), dtype=proj.dtype, device=self.device)
        self._call(self.lib.tli_keyed_prepare, proj.data_ptr(), width, _ptr(bias), q.data_ptr(), kc.data_ptr(), vc.data_ptr(),
                   step.positions.data_ptr(), step.seq_of_row.data_ptr(), g.tables.data_ptr(), g.table_width, g.page_size,
                   kc.shape[0], T, heads, kv_heads, head_dim, -1 if values_are_keys else (heads + kv_heads) * head_dim,
                   _ptr(cos), _ptr(sin), rd, npos, _dtype_code(proj.dtype), self._stream())
        if self.takes_sinks(proj.dtype, step, cache, head_dim):
            # portions of prompts: the kernel that the stock attention runs them through (keys and values through LDS)
            return self.paged_attention(q.view(T, heads * head_dim), step, cache, heads, kv_heads, head_dim, scale, window,
                                        sinks=sinks)
        o = self.sized_attention(q, step, g, kc, vc, heads, kv_heads, 1, head_dim, head_dim, scale, window, 0, proj.dtype,
                                 sinks=sinks)
        return o.view(T, heads * head_dim)

    def add_bias(self, y, bias):
        """y [T, n] += bias (float32 [n]), in place; ``y`` may be an unfinished product."""
        y = self.resolve(y)
        T, n = y.shape
        self._want(y, "rows")
        self._want(bias, "bias", torch.float32, (n,))
        self._call(self.lib.tli_add_bias, y.data_ptr(), bias.data_ptr(), T, n, _dtype_code(y.dtype), self._stream())
        return y

    # ---- lightning attention -----------------------------------------------------------------------------
    def check_lightning_sizes(self, heads: int, dk: int, dv: int) -> None:
        if heads <= 0 or not 1 <= dk <= 256 or dv < 1:
            raise KernelError(f"lightning attention with {heads} heads of keys of {dk} (1 to 256) and values of {dv} is not supported")

    def lightning_state_shape(self, heads: int, dk: int, dv: int):
        """The shape of one request's recurrent state (float32): a head's matrix is kept transposed, so that the
        elements of a column, which one DPP row of lanes holds, lie together."""
        return (heads, dv, dk)

    def lightning_attention(self, proj, decay, state, step, heads, dk, dv):
        """From the raw projections ``proj`` [T, >= q (H dk) | k (H dk) | v (H dv)] to the heads' outputs of the
        recurrence S <- decay_h S + silu(k) silu(v)^T, o = S^T silu(q), float32 [T, H dv].  ``decay``: float32 [H];
        ``state``: float32 [slots, H, dv, dk], read (unless a sequence starts at position 0) and replaced."""
        T = step.num_rows
        self.check_lightning_sizes(heads, dk, dv)
        need = 2 * heads * dk + heads * dv
        if proj.dim() != 2 or proj.shape[0] != T or proj.shape[1] < need:
            raise KernelError(f"the projections have shape {tuple(proj.shape)}, expected [{T}, >= {need}]")
        self._want(proj, "projections")
        self._want(decay, "decays", torch.float32, (heads,))
        self._want(state, "recurrent state", torch.float32, (state.shape[0], heads, dv, dk))
        if max(step.h_slots, default=0) >= state.shape[0]:
            raise KernelError("a sequence's slot lies outside the state")
        out = torch.empty((T, heads * dv), dtype=torch.float32, device=self.device)
        # (silu(q), silu(k), silu(v) of the step in float32, padded as the recurrence's lanes hold them,
        # and, where long portions are walked in segments side by side, the segments' states)
        longest = int(step.max_rows_per_seq)
        scratch = torch.empty((int(self.lib.tli_lightning_scratch_floats(T, step.num_seqs, longest, heads, dk, dv)),),
                              dtype=torch.float32, device=self.device)
        self._call(self.lib.tli_lightning_recurrence, proj.data_ptr(), proj.shape[1], decay.data_ptr(), state.data_ptr(),
                   out.data_ptr(), scratch.data_ptr(), step.row_start.data_ptr(), step.seq_start.data_ptr(),
                   step.slots.data_ptr(), T, step.num_seqs, longest, heads, dk, dv, _dtype_code(proj.dtype),
                   int(self.lightning_lanes), self._stream())
        return out

    def lightning_norm(self, o, proj, gate_at, weight, eps, out_dtype):
        """y = o / sqrt(mean(o^2) + eps) * weight * sigmoid(gate) over a whole row; ``o`` float32 [T, n], the gate's
        logits are columns ``gate_at`` .. ``gate_at + n`` of ``proj``."""
        T, n = o.shape
        self._want(o, "heads' outputs", torch.float32)
        self._want(proj, "projections", out_dtype)
        if proj.shape[0] != T or proj.shape[1] < gate_at + n:
            raise KernelError("the gate lies outside the projections")
        self._want(weight, "norm weight", torch.float32, (n,))
        out = torch.empty((T, n), dtype=out_dtype, device=self.device)
        self._call(self.lib.tli_lightning_norm, o.data_ptr(), proj.data_ptr() + gate_at * proj.element_size(), proj.shape[1],
                   weight.data_ptr(), out.data_ptr(), T, n, float(eps), _dtype_code(out_dtype), self._stream())
        return out

    # ---- attention over a window and pooled blocks --------------------------------------------------------
    def _pairs(self, rotary, step):
        """(cos, sin, turned elements, pairing code, positions) of a ``RotaryTables`` or None, for kernels that turn
        either kind of pairs."""
        if rotary is None:
            return None, None, 0, 0, 0
        codes = {"half": 0, "interleaved": 1}
        if rotary[3] not in codes:
            raise KernelError(f"the pairing '{rotary[3]}' of a rotation is not known")
        cos, sin, rd = self._rotary(rotary[:3], step)
        return cos, sin, rd, codes[rotary[3]], cos.shape[0]

    def pooled_window_attention(self, proj, at, step, cache, heads, kv_heads, key_dim, value_dim, bias, q_weight, k_weight,
                                eps, rotary, scale, sinks, window, pool, out, out_at, out_scale):
        """From the raw projections ``proj[:, at:]`` (q (heads key_dim) | k (kv_heads key_dim) | v (kv_heads value_dim))
        to the heads' outputs times ``out_scale`` in ``out[:, out_at : out_at + heads value_dim]``: biases, RMS norms of q
        and of k over all their elements (weights float32 or None), rotation of either pairing, keys and values into
        the cache (records "k", "v"), the means of every ``pool`` positions' keys and values into ``cache.further[0]``, and
        attention over the window's tokens and the blocks before it with ``sinks`` (float32 [heads] or None)."""
        T = step.num_rows
        self.check_sized_attention(heads, kv_heads, key_dim, value_dim)
        qn, kn, vn = heads * key_dim, kv_heads * key_dim, kv_heads * value_dim
        self._want(proj, "projections", out.dtype)
        if proj.dim() != 2 or proj.shape[0] != T or at < 0 or proj.shape[1] < at + qn + kn + vn:
            raise KernelError(f"the projections have shape {tuple(proj.shape)}, expected [{T}, >= {at + qn + kn + vn}]")
        for w, n, what in ((bias, qn + kn + vn, "projections' bias"), (q_weight, qn, "norm weight of q"),
                           (k_weight, kn, "norm weight of k"), (sinks, heads, "sinks")):
            if w is not None:
                self._want(w, what, torch.float32, (n,))
        if cache is None or not cache.writes or len(cache.further) != 1:
            raise KernelError("this attention writes its keys and their means into cache layers of its own")
        if window <= 0 or pool <= 0:
            raise KernelError("a window and blocks of at least one position each")
        blocks = cache.further[0]
        kc, vc, g = cache.record("k"), cache.record("v"), cache.group
        bk, bv, bg = blocks.record("k"), blocks.record("v"), blocks.group
        for k, v, gr, what in ((kc, vc, g, "cache"), (bk, bv, bg, "cache of blocks")):
            self._want(k, f"key {what}", proj.dtype, (k.shape[0], kv_heads, gr.page_size, key_dim))
            self._want(v, f"value {what}", proj.dtype, (k.shape[0], kv_heads, value_dim, gr.page_size))
        if bg.page_size != g.page_size or bg.stride != pool or g.stride != 1:
            raise KernelError(f"the cache of blocks has one slot for {bg.stride} positions, the blocks have {pool}")
        self._check_tables(g, step)
        self._want(bg.tables, "block tables of the blocks", torch.int32, (step.num_seqs, bg.table_width))
        if -(-step.max_seq_len // (bg.page_size * pool)) > bg.table_width:
            raise KernelError("a block table is narrower than its sequence needs")
        _, out_ptr, out_ld = self._rows_into((out, out_at), T, heads * value_dim, proj.dtype)
        cos, sin, dims, pairing, npos = self._pairs(rotary, step)
        if dims > key_dim:
            raise KernelError(f"{dims} turned elements do not fit a head of {key_dim}")
        q = torch.empty((T, heads, key_dim), dtype=proj.dtype, device=self.device)
        single = 1 if step.max_rows_per_seq == 1 and step.num_seqs == T else 0
        pooled = (bk.data_ptr(), bv.data_ptr(), bg.tables.data_ptr(), bg.table_width, bk.shape[0], pool)
        self._call(self.lib.tli_pooled_prepare, proj.data_ptr() + at * proj.element_size(), proj.shape[1], _ptr(bias), q.data_ptr(),
                   kc.data_ptr(), vc.data_ptr(), step.positions.data_ptr(), step.seq_of_row.data_ptr(), step.row_start.data_ptr(),
                   step.seq_start.data_ptr(), step.num_seqs, g.tables.data_ptr(), g.table_width, g.page_size, kc.shape[0], T,
                   heads, kv_heads, key_dim, value_dim, _ptr(q_weight), _ptr(k_weight), float(eps), _ptr(cos), _ptr(sin), dims,
                   pairing, npos, *pooled, single, _dtype_code(proj.dtype), self._stream())
        starts = step.h_row_start
        if (proj.dtype == torch.bfloat16 and not self.force_plain and not single and self.pooled_prefill
                and self.lib.tli_pooled_prefill_takes(key_dim, value_dim, g.page_size, int(step.max_seq_len), int(window), pool)):
            tiles = sum((starts[i + 1] - starts[i] + 31) // 32 for i in range(step.num_seqs))
            self._call(self.lib.tli_pooled_prefill_bf16, q.data_ptr(), out_ptr, kc.data_ptr(), vc.data_ptr(),
                       step.row_start.data_ptr(), step.seq_start.data_ptr(), step.num_seqs, tiles, g.tables.data_ptr(),
                       g.table_width, g.page_size, kc.shape[0], heads, kv_heads, key_dim, value_dim, float(scale), int(window),
                       *pooled, int(step.max_seq_len), _ptr(sinks), out_ld, float(out_scale), self._stream())
            return
        if (proj.dtype == torch.bfloat16 and not self.force_plain
                and self.lib.tli_attention_sized_mfma_takes(key_dim, value_dim, g.page_size, 1)):
            tiles = T if single else sum((starts[i + 1] - starts[i] + 15) // 16 for i in range(step.num_seqs))
            splits, parts = self._pooled_splits(T, step.reach, heads, kv_heads, value_dim, window, pool) if single else (1, None)
            self._call(self.lib.tli_attention_pooled_mfma_bf16, q.data_ptr(), out_ptr, kc.data_ptr(), vc.data_ptr(),
                       step.row_start.data_ptr(), step.seq_start.data_ptr(), step.num_seqs, tiles, g.tables.data_ptr(),
                       g.table_width, g.page_size, kc.shape[0], heads, kv_heads, key_dim, value_dim, float(scale), int(window),
                       *pooled, single, _ptr(sinks), out_ld, float(out_scale), splits, _ptr(parts), self._stream())
            return
        self._call(self.lib.tli_attention_pooled_plain, q.data_ptr(), out_ptr, kc.data_ptr(), vc.data_ptr(),
                   step.positions.data_ptr(), step.seq_of_row.data_ptr(), g.tables.data_ptr(), g.table_width, g.page_size,
                   kc.shape[0], T, heads, kv_heads, key_dim, value_dim, float(scale), int(window), *pooled,
                   _dtype_code(proj.dtype), _ptr(sinks), out_ld, float(out_scale), self._stream())

    POOLED_WORKGROUPS = 768          # a split of decoding rows over windows and blocks: the workgroups aimed at,
    POOLED_SPLIT_KEYS = 128          # and the fewest keys of a split (two rounds of tiles of 16 over four waves)

    def _pooled_splits(self, T, reach, heads, kv_heads, value_dim, window, pool):
        """Over how many workgroups the keys of one (row, key head) that decodes are shared out, and the room for
        their sums; ``reach``: a power of two that the longest sequence fits.  A wave's tiles follow one another, each
        with its wait for memory (3 us), so a split pays for its merge where workgroups are few.  Measured at heads of
        128 on 8 key heads, 1,060 keys, a whole step of 4 layers (2 of them with this attention): 8 rows in 1, 2, 4, 8
        splits 0.585, 0.550, 0.532, 0.509 ms, 64 rows in 1, 2, 3, 4 splits 1.046, 1.006, 1.038, 1.009; at 700 keys 64
        rows 0.972, 0.989 and 0.984 in 1, 2 and 4; below 256 keys the same in 1 and 2."""
        keys = min(reach, window + 15) + max(0, reach - window) // pool
        groups = T * kv_heads * ((heads // kv_heads + 15) // 16)
        most = keys // self.POOLED_SPLIT_KEYS if keys >= 4 * self.POOLED_SPLIT_KEYS else 1
        splits = self.pooled_splits or min(self.POOLED_WORKGROUPS // groups, most, 64)
        if splits <= 1:
            return 1, None
        return splits, torch.empty((T * heads * splits * (value_dim + 4),), dtype=torch.float32, device=self.device)

    # ---- retention, mLSTM --------------------------------------------------------------------------------
    def _recurrent_inputs(self, proj, at, state, shape, step, heads, dk, dv):
        T = step.num_rows
        self.check_lightning_sizes(heads, dk, dv)
        need = at + 2 * heads * dk + heads * dv
        self._want(proj, "projections")
        if proj.dim() != 2 or proj.shape[0] != T or at < 0 or proj.shape[1] < need:
            raise KernelError(f"the projections have shape {tuple(proj.shape)}, expected [{T}, >= {need}]")
        self._want(state, "recurrent state", torch.float32, (state.shape[0],) + tuple(shape))
        if max(step.h_slots, default=0) >= state.shape[0]:
            raise KernelError("a sequence's slot lies outside the state")

    def _recurrence_scratch(self, step, heads, dk, dv, more=0):
        n = int(self.lib.tli_lightning_scratch_floats(step.num_rows, step.num_seqs, int(step.max_rows_per_seq), heads, dk, dv))
        return torch.empty((n + more,), dtype=torch.float32, device=self.device), n

    def _single_rows(self, step) -> bool:
        """Whether every sequence of the step brings one row, and such a step may run through kernels of its own."""
        return step.max_rows_per_seq == 1 and step.num_seqs == step.num_rows and not self.unfused_decode

    def _in_chunks(self, proj, at, dk, dv, dims=0, pairing=0) -> bool:
        """Whether rows go through the recurrence in chunks (csrc/chunked.hip), else row by row."""
        return (self.recurrence_in_chunks and proj.dtype == torch.bfloat16 and not self.force_plain
                and (proj.data_ptr() + 2 * at) % 16 == 0 and proj.shape[1] % 8 == 0
                and bool(self.lib.tli_chunked_takes(dk, dv, dims, pairing)))

    def _chunked_scratch(self, step, heads, dk, columns, more=0):
        n = int(self.lib.tli_chunked_scratch_floats(step.num_rows, step.num_seqs, heads, dk, columns))
        return torch.empty((n + more,), dtype=torch.float32, device=self.device), n

    def retention(self, proj, at, decay, state, step, heads, dk, dv, rotary, k_scale, eps, scale, out, out_at):
        """From the raw projections ``proj[:, at:]`` (q (H dk) | k (H dk) | v (H dv) | gate (H dv)) to the layer's rows in
        ``out[:, out_at : out_at + H dv]``: the recurrence S <- decay_h S + k v^T, o = S^T q with q and k turned
        (``rotary``, of either pairing, or None) and k times ``k_scale``, then o / sqrt(mean(o^2) + eps) * silu(gate) * scale
        head by head.  ``state``: float32 [slots, H, dv, dk], read (unless a sequence starts at position 0) and replaced."""
        T = step.num_rows
        self._recurrent_inputs(proj, at, state, (heads, dv, dk), step, heads, dk, dv)
        self._want(decay, "decays", torch.float32, (heads,))
        cos, sin, dims, pairing, npos = self._pairs(rotary, step)
        if dims > dk:
            raise KernelError(f"{dims} turned elements do not fit a head of {dk}")
        _, out_ptr, out_ld = self._rows_into((out, out_at), T, heads * dv, proj.dtype)
        proj_ptr = proj.data_ptr() + at * proj.element_size()
        if self._single_rows(step):
            self._call(self.lib.tli_retention_step, proj_ptr, proj.shape[1], decay.data_ptr(), state.data_ptr(), out_ptr, out_ld,
                       step.positions.data_ptr(), step.seq_start.data_ptr(), step.slots.data_ptr(), _ptr(cos), _ptr(sin), dims,
                       pairing, npos, float(k_scale), float(eps), float(scale), T, heads, dk, dv, _dtype_code(proj.dtype),
                       self._stream())
            return
        if self._in_chunks(proj, at, dk, dv, dims, pairing):
            scratch, _ = self._chunked_scratch(step, heads, dk, dv)
            self._call(self.lib.tli_retention_chunked_bf16, proj_ptr, proj.shape[1], decay.data_ptr(), state.data_ptr(), out_ptr, out_ld,
                       scratch.data_ptr(), step.row_start.data_ptr(), step.seq_start.data_ptr(),
                       step.slots.data_ptr(), _ptr(cos), _ptr(sin), dims, pairing, npos, float(k_scale), float(eps), float(scale),
                       T, step.num_seqs, heads, dk, dv, self._stream())
            return
        o = torch.empty((T, heads, dv), dtype=torch.float32, device=self.device)
        scratch, _ = self._recurrence_scratch(step, heads, dk, dv)
        self._call(self.lib.tli_retention, proj_ptr, proj.shape[1], decay.data_ptr(),
                   state.data_ptr(), o.data_ptr(), scratch.data_ptr(), step.positions.data_ptr(), step.row_start.data_ptr(),
                   step.seq_start.data_ptr(), step.slots.data_ptr(), _ptr(cos), _ptr(sin), dims, pairing, npos, float(k_scale),
                   T, step.num_seqs, int(step.max_rows_per_seq), heads, dk, dv, _dtype_code(proj.dtype),
                   int(self.lightning_lanes), self._stream())
        self.head_norm_gate(o, None, None, proj, at + 2 * heads * dk + heads * dv, heads, dv, eps, "silu", scale, out, out_at)

    def mlstm_state_shape(self, heads: int, dk: int, dv: int):
        """The shape of one request's S beside its n: a head's matrix is kept transposed, n is its column dv."""
        return (heads, dv + 1, dk)

    def mlstm(self, proj, at, x, w_gates, gate_bias, cap, state, m_state, step, heads, dk, dv, q_scale, weight, eps, scale, out,
              out_at):
        """From the raw projections ``proj[:, at:]`` (q (H dk) | k (H dk) | v (H dv) | gate (H dv)) and the layer's input
        ``x`` (a tensor or ``NormedRows``) to the layer's rows in ``out[:, out_at : out_at + H dv]``: the gates' logits x
        w_gates^T + gate_bias (``w_gates`` [2 H, n]: input gates, then forget gates; float32 sums), the matrix memory, and
        o / sqrt(mean(o^2) + eps) * weight * sigmoid(gate) * scale head by head.  ``state``: float32 [slots,
        *mlstm_state_shape]; ``m_state``: float32 [slots, H]."""
        T = step.num_rows
        self._recurrent_inputs(proj, at, state, self.mlstm_state_shape(heads, dk, dv), step, heads, dk, dv)
        self._want(m_state, "running maxima", torch.float32, (state.shape[0], heads))
        self._want(gate_bias, "gate biases", torch.float32, (2 * heads,))
        self._want(weight, "norm weight", torch.float32, (heads * dv,))
        rows, ssq, x_eps = (x.xw, x.ssq, x.eps) if isinstance(x, NormedRows) else (x, None, 0.0)
        n = rows.shape[1]
        self._want(rows, "layer input", proj.dtype, (T, n))
        self._want(w_gates, "gate rows", proj.dtype, (2 * heads, n))
        parts = 0 if ssq is None else ssq.shape[0]
        if ssq is not None:
            self._want(ssq, "sums of squares", torch.float32, (parts, T))
        _, out_ptr, out_ld = self._rows_into((out, out_at), T, heads * dv, proj.dtype)
        gate_at = at + 2 * heads * dk + heads * dv
        if proj.shape[1] < gate_at + heads * dv:
            raise KernelError("the gate lies outside the projections")
        proj_ptr = proj.data_ptr() + at * proj.element_size()
        if self._single_rows(step):
            self._call(self.lib.tli_mlstm_step, proj_ptr, proj.shape[1], rows.data_ptr(), w_gates.data_ptr(), n, _ptr(ssq), parts,
                       float(x_eps), gate_bias.data_ptr(), float(cap), float(q_scale), weight.data_ptr(), m_state.data_ptr(),
                       state.data_ptr(), out_ptr, out_ld, step.seq_start.data_ptr(), step.slots.data_ptr(), float(eps),
                       float(scale), T, heads, dk, dv, _dtype_code(proj.dtype), self._stream())
            return
        gates, transposed = self.small_product(rows, w_gates)
        z_row, z_col = (1, T) if transposed else (2 * heads, 1)
        if self._in_chunks(proj, at, dk, dv):
            scratch, size = self._chunked_scratch(step, heads, dk, dv + 1, more=4 * heads * T)
            self._call(self.lib.tli_mlstm_chunked_bf16, proj_ptr, proj.shape[1], gates.data_ptr(), z_row, z_col, _ptr(ssq), parts, n,
                       float(x_eps), gate_bias.data_ptr(), float(cap), float(q_scale), weight.data_ptr(), m_state.data_ptr(),
                       state.data_ptr(), out_ptr, out_ld, scratch.data_ptr(), scratch.data_ptr() + 4 * size,
                       step.row_start.data_ptr(), step.seq_start.data_ptr(), step.slots.data_ptr(), float(eps), float(scale), T,
                       step.num_seqs, heads, dk, dv, self._stream())
            return
        single = 1 if step.max_rows_per_seq == 1 and step.num_seqs == T else 0
        o = torch.empty((T, heads, dv + 1), dtype=torch.float32, device=self.device)
        floors = torch.empty((heads, T), dtype=torch.float32, device=self.device)
        scratch, size = self._recurrence_scratch(step, heads, dk, dv + 1, more=3 * heads * T)
        self._call(self.lib.tli_mlstm, proj_ptr, proj.shape[1], gates.data_ptr(), z_row, z_col, _ptr(ssq), parts, n, float(x_eps),
                   gate_bias.data_ptr(), float(cap), float(q_scale), m_state.data_ptr(), state.data_ptr(), o.data_ptr(),
                   floors.data_ptr(), scratch.data_ptr(), scratch.data_ptr() + 4 * size, step.row_start.data_ptr(),
                   step.seq_start.data_ptr(), step.slots.data_ptr(), T, step.num_seqs, int(step.max_rows_per_seq), single,
                   heads, dk, dv, _dtype_code(proj.dtype), int(self.lightning_lanes), self._stream())
        self.head_norm_gate(o, floors, weight, proj, gate_at, heads, dv, eps, "sigmoid", scale, out, out_at)

    # ---- the RWKV's time mixing --------------------------------------------------------------------------------
    def check_wkv_sizes(self, heads: int, dk: int, dv: int, rank: int) -> None:
        if heads <= 0 or not 1 <= dk <= 256 or dv < 1 or not 1 <= rank <= 8192:
            raise KernelError(f"time mixing with {heads} heads of keys of {dk} (1 to 256) and values of {dv}, decays through {rank}, "
                              "is not supported")

    def wkv_state_shape(self, heads: int, dk: int, dv: int):
        """The shape of one request's recurrent state (float32): a head's matrix is kept transposed."""
        return (heads, dv, dk)

    def stacks_groups(self, sizes, cols: int, dtype) -> bool:
        """Whether matrices of these rows, each with an input of its own, are held stacked in one (``linear_groups``)."""
        return (dtype == torch.bfloat16 and cols % 8 == 0 and len(set(sizes)) == 1 and sizes[0] % 128 == 0
                and self.many_rows == "own" and not self.plain_products)

    def linear_groups(self, xs, groups, step=None):
        """``xs`` [G + 1, T, n] and a ``GroupedMatrix`` of G matrices and one of few rows: (the G products side by side,
        [T, >= sum of their rows] in the run's type, the last one's float32 sums, the distances of their rows and columns).
        Where the matrices are stacked one launch multiplies the G; in a ``step`` of one row a sequence it takes the last
        one with it and the products are float32."""
        count = len(groups.sizes)
        if xs.dim() != 3 or xs.shape[0] != count + 1 or xs.shape[2] != groups.cols:
            raise KernelError(f"{tuple(xs.shape)} are not the inputs of {count} matrices of {groups.cols} columns and one of few rows")
        self._want(xs, "inputs of several matrices", groups.dtype)
        M, K = int(xs.shape[1]), groups.cols
        proj = None
        if groups.stacked is not None and self.grouped_products and not self.plain_products and M > 0:
            every, few, apart = groups.sizes[0], groups.few.shape[0], M * K
            tiled = groups.stacked.tiled
            together = step is not None and self._single_rows(step) and M <= self.MID_ROWS_TO and few <= every
            N = count * every + (few if together else 0)
            dtype = torch.float32 if together else torch.bfloat16
            if M <= self.MID_ROWS_TO or every % 256 == 0:
                proj = torch.empty((M, N), dtype=dtype, device=self.device)
                if M < self.MID_ROWS_FROM:
                    self._call(self.lib.tli_gemm_skinny_groups_bf16, xs.data_ptr(), tiled.data_ptr(), proj.data_ptr(), M, N, K,
                               _dtype_code(dtype), every, apart, self._stream())
                else:
                    mid = M <= self.MID_ROWS_TO
                    splits = int(self.lib.tli_gemm_mid_splits_rows(M, N, K, 0) if mid else self.lib.tli_gemm_rows_splits(M, N, K))
                    part = torch.empty((splits, M, N), dtype=torch.float32, device=self.device) if splits > 1 else None
                    if mid:
                        self._call(self.lib.tli_gemm_mid_groups_bf16, xs.data_ptr(), tiled.data_ptr(), proj.data_ptr(), _ptr(part), M, N, K,
                                   _dtype_code(dtype), splits, every, apart, self._stream())
                    else:
                        self._call(self.lib.tli_gemm_rows_groups_bf16, xs.data_ptr(), tiled.data_ptr(), proj.data_ptr(), _ptr(part), M, N, K,
                                   splits, every, apart, self._stream())
                if together:
                    return proj, proj[:, count * every:], (N, 1)
        if proj is None:
            if groups.stacked is not None:
                w, at = groups.stacked.w, 0
                mats = []
                for n in groups.sizes:
                    mats.append(w[at:at + n])
                    at += n
            else:
                mats = groups.each
            proj = torch.cat([self.linear(xs[i], m) for i, m in enumerate(mats)], dim=1)
        z, transposed = self.small_product(xs[count], groups.few)
        return proj, z, ((1, M) if transposed else (groups.few.shape[0], 1))

    def wkv(self, proj, z, z_strides, w2, w0, u, state, step, heads, dk, dv, weight, eps, out_dtype):
        """From the projections ``proj`` [T, r (H dk) | k (H dk) | v (H dv) | g (H dv) | ..] and the decays' inner rows ``z``
        (float32, ``z_strides`` the distances of its rows and columns) to the layer's rows [T, H dv]: decays
        d = exp(-exp(w2 tanh(z) + w0)), o = (S + diag(u) k v^T)^T r, S <- diag(d) S + k v^T, then o / sqrt(mean(o^2) + eps) *
        weight * silu(g), the mean head by head.  ``state``: float32 [slots, H, dv, dk], read (unless a sequence starts at
        position 0) and replaced."""
        T = step.num_rows
        self._recurrent_inputs(proj, 0, state, (heads, dv, dk), step, heads, dk, dv)
        if proj.shape[1] < 2 * heads * (dk + dv):
            raise KernelError("the gate lies outside the projections")
        rank = w2.shape[1]
        z_row, z_col = z_strides

        def lies(shape, strides):            # (the distance of a dimension of one element says nothing)
            return tuple(z.shape) == shape and all(n == 1 or a == b for n, a, b in zip(shape, z.stride(), strides))
        if z.dtype != torch.float32 or z.device.type != "cuda" \
                or not (lies((T, rank), (z_row, z_col)) or lies((rank, T), (z_col, z_row))):
            raise KernelError(f"the decays' inner rows have shape {tuple(z.shape)} and strides {tuple(z.stride())}, not {rank} a row")
        self._want(w2, "decays' matrix", out_dtype, (heads * dk, rank))
        self._want(w0, "decays' bias", torch.float32, (heads * dk,))
        self._want(u, "current token's bonus", torch.float32, (heads, dk))
        self._want(weight, "norm weight", torch.float32, (heads * dv,))
        out = torch.empty((T, heads * dv), dtype=out_dtype, device=self.device)
        if self._single_rows(step):
            self._call(self.lib.tli_wkv_step, proj.data_ptr(), proj.shape[1], _dtype_code(proj.dtype), z.data_ptr(), z_row, z_col,
                       w2.data_ptr(), w0.data_ptr(), rank, u.data_ptr(), weight.data_ptr(), state.data_ptr(), out.data_ptr(), heads * dv,
                       step.seq_start.data_ptr(), step.slots.data_ptr(), float(eps), T, heads, dk, dv, _dtype_code(out_dtype),
                       self._stream())
            return out
        if (self.recurrence_in_chunks and proj.dtype == torch.bfloat16 and not self.force_plain and proj.shape[1] % 8 == 0
                and self.lib.tli_wkv_chunked_takes(dk, dv, rank)):
            scratch = torch.empty((int(self.lib.tli_wkv_chunked_scratch_floats(T, step.num_seqs, heads, dk, dv)),), dtype=torch.float32,
                                  device=self.device)
            self._call(self.lib.tli_wkv_chunked_bf16, proj.data_ptr(), proj.shape[1], z.data_ptr(), z_row, z_col, w2.data_ptr(), w0.data_ptr(),
                       rank, u.data_ptr(), state.data_ptr(), out.data_ptr(), heads * dv, weight.data_ptr(), scratch.data_ptr(),
                       step.row_start.data_ptr(), step.seq_start.data_ptr(), step.slots.data_ptr(), float(eps), T, step.num_seqs, heads,
                       dk, dv, self._stream())
            return out
        decay = torch.empty((T, heads * dk), dtype=torch.float32, device=self.device)
        self._call(self.lib.tli_wkv_decays, z.data_ptr(), z_row, z_col, w2.data_ptr(), w0.data_ptr(), decay.data_ptr(), T, rank,
                   heads * dk, _dtype_code(out_dtype), self._stream())
        o = torch.empty((T, heads, dv), dtype=torch.float32, device=self.device)
        self._call(self.lib.tli_wkv_rows, proj.data_ptr(), proj.shape[1], decay.data_ptr(), u.data_ptr(), state.data_ptr(), o.data_ptr(),
                   step.row_start.data_ptr(), step.seq_start.data_ptr(), step.slots.data_ptr(), step.num_seqs, heads, dk, dv,
                   _dtype_code(proj.dtype), self._stream())
        self.head_norm_gate(o, None, weight, proj, 2 * heads * dk + heads * dv, heads, dv, eps, "silu", 1.0, out, 0)
        return out

    OUTPUT_GATES = {"silu": 0, "sigmoid": 1}

    def head_norm_gate(self, o, floors, weight, proj, gate_at, heads, dv, eps, gate, scale, out, out_at):
        """x = o of a head, float32 [T, H, dv]; with ``floors`` (float32 [H, T]; ``o`` is then [T, H, dv + 1]) divided by
        max(|o[dv]|, floor) + 1e-6; then x / sqrt(mean(x^2) + eps) * weight * gate(proj[:, gate_at:]) * scale in
        ``out[:, out_at : out_at + H dv]``.  ``weight``: float32 [H dv] or None; ``gate``: "silu" or "sigmoid"."""
        T = o.shape[0]
        self._want(o, "heads' outputs", torch.float32, (T, heads, dv + (1 if floors is not None else 0)))
        if floors is not None:
            self._want(floors, "normalisers' floors", torch.float32, (heads, T))
        if weight is not None:
            self._want(weight, "norm weight", torch.float32, (heads * dv,))
        self._want(proj, "projections", out.dtype)
        if proj.shape[0] != T or gate_at < 0 or proj.shape[1] < gate_at + heads * dv:
            raise KernelError("the gate lies outside the projections")
        if gate not in self.OUTPUT_GATES:
            raise KernelError(f"gate '{gate}' is not known; known: {', '.join(sorted(self.OUTPUT_GATES))}")
        _, out_ptr, out_ld = self._rows_into((out, out_at), T, heads * dv, proj.dtype)
        self._call(self.lib.tli_head_norm_gate, o.data_ptr(), _ptr(floors), _ptr(weight),
                   proj.data_ptr() + gate_at * proj.element_size(), proj.shape[1], out_ptr, out_ld, T, heads, dv, float(eps),
                   self.OUTPUT_GATES[gate], float(scale), _dtype_code(proj.dtype), self._stream())

    def sample(self, logits: torch.Tensor, temperatures: Optional[torch.Tensor] = None,
               seeds: Optional[torch.Tensor] = None, top_p: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Token ids int32 [rows].  ``temperatures`` float32 [rows] (None: greedy);
        ``seeds`` int64 [rows], one draw seed per row; ``top_p`` float32 [rows] or None."""
        rows, vocab = logits.shape
        self._want(logits, "logits", torch.float32)
        if temperatures is not None:
            self._want(temperatures, "temperatures", torch.float32, (rows,))
            if seeds is None:
                raise KernelError("sampling with a temperature needs seeds")
            self._want(seeds, "seeds", torch.int64, (rows,))
        if top_p is not None:
            self._want(top_p, "top_p", torch.float32, (rows,))
        out = torch.empty((rows,), dtype=torch.int32, device=self.device)
        scratch = torch.empty((self.lib.tli_sample_scratch_bytes(rows),), dtype=torch.uint8, device=self.device)
        self._call(self.lib.tli_sample, logits.data_ptr(), rows, vocab, _ptr(temperatures),
                   _ptr(seeds) if temperatures is not None else None,
                   _ptr(top_p) if temperatures is not None else None, out.data_ptr(), scratch.data_ptr(),
                   self._stream())
        return out


def sample_uniform(seed: int, token: int) -> float:
    """The uniform number the sampling kernel draws for (seed, token)."""
    lib = load_library()
    seed &= (1 << 64) - 1
    return float(lib.tli_sample_uniform(seed & 0xFFFFFFFF, seed >> 32, token))
