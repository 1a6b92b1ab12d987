"""Python faces of the bf16 MFMA kernels (library ``fast``).

Each function returns ``False`` when the kernels do not cover the operands (the
caller then takes the generic kernel) and raises when they do but the call fails.
"""

from __future__ import annotations

import ctypes
from typing import Dict, NamedTuple, Optional

import torch

from ..csrc import build as _build
from . import core
from .core import KA_BF16, KA_F32, KernelError, _ptr, stream_ptr

_c_void_p, _c_int, _c_long, _c_float = ctypes.c_void_p, ctypes.c_int, ctypes.c_long, ctypes.c_float

_SIGNATURES = {
    "ka_linear_skinny_bf16": [_c_void_p, _c_long, _c_void_p, _c_long, _c_void_p, _c_void_p, _c_int, _c_long, _c_int,
                              _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p, _c_long, _c_void_p],
    "ka_linear_skinny_fused": [
        _c_void_p, _c_long, _c_int,                                   # A1, lda1, K1
        _c_void_p, _c_long, _c_int, _c_void_p, _c_long, _c_void_p,    # A2, lda2, K2, W2, ldw2, bias2
        _c_void_p, _c_void_p, _c_void_p, _c_float,                    # ln_x, gamma, beta, eps
        _c_void_p, _c_long, _c_void_p, _c_void_p, _c_int, _c_long, _c_int, _c_int, _c_int,   # target a
        _c_void_p, _c_long, _c_void_p, _c_void_p, _c_int, _c_long, _c_int, _c_int,           # target b
        _c_int, _c_int, _c_void_p, _c_long, _c_void_p],               # M, target_waves, partial sums and how many, stream
    "ka_linear_skinny_fused_rms": [_c_void_p, _c_void_p, _c_float, _c_int, _c_void_p, _c_long, _c_void_p, _c_void_p, _c_int, _c_long,
                                   _c_int, _c_int, _c_void_p, _c_long, _c_void_p, _c_void_p, _c_int, _c_long, _c_int, _c_int, _c_int,
                                   _c_int, _c_void_p],
    "ka_linear_skinny_pair_norm": [
        _c_void_p, _c_long, _c_int, _c_void_p, _c_long, _c_int,                  # A1, lda1, K1, A2, lda2, K2
        _c_void_p, _c_long, _c_void_p, _c_void_p, _c_long, _c_void_p,            # W1, ldw1, bias1, W2, ldw2, bias2
        _c_void_p, _c_long, _c_int, _c_int, _c_int, _c_int, _c_void_p, _c_long,  # out, ldo, N, accumulate, M, target_waves, partial sums
        _c_void_p, _c_void_p, _c_float, _c_void_p, _c_int, _c_long, _c_void_p],  # gamma, beta, eps, normed, its type and stride, stream
    "ka_linear_skinny_pair_in_parts": [_c_int, _c_int],
    "ka_linear_library_bf16": [_c_void_p, _c_long, _c_void_p, _c_long, _c_void_p, _c_void_p, _c_int, _c_long, _c_int,
                               _c_int, _c_int, _c_int, _c_int, _c_void_p, _c_long, _c_void_p],
    "ka_linear_tiled_bf16": [_c_void_p, _c_long, _c_void_p, _c_long, _c_void_p, _c_void_p, _c_int, _c_long, _c_int,
                             _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p, _c_long, _c_void_p],
    "ka_attention_prefill_bf16": [_c_void_p, _c_long, _c_void_p, _c_void_p, _c_void_p, _c_int, _c_void_p, _c_void_p,
                                  _c_int, _c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_long, _c_float,
                                  _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p],
    "ka_rope_cache_pages_bf16": [_c_void_p, _c_long, _c_void_p, _c_void_p, _c_void_p, _c_int, _c_void_p, _c_void_p,
                                 _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p, _c_void_p, _c_int, _c_void_p],
    "ka_attention_decode_bf16": [_c_void_p, _c_long, _c_void_p, _c_void_p, _c_void_p, _c_int, _c_void_p, _c_void_p,
                                 _c_void_p, _c_void_p, _c_long, _c_float, _c_int, _c_int, _c_int, _c_int, _c_int,
                                 _c_int, _c_int, _c_void_p, _c_long,
                                 _c_void_p, _c_void_p, _c_long, _c_void_p, _c_int, _c_void_p, _c_void_p, _c_void_p,
                                 _c_void_p],
    "ka_attention_decode_beside_bf16": [
        _c_void_p, _c_long, _c_void_p, _c_void_p, _c_void_p, _c_int, _c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_long,
        _c_float, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p, _c_long,                # ..., splits, partial sums
        _c_void_p, _c_void_p, _c_long, _c_void_p, _c_int, _c_void_p, _c_void_p, _c_void_p,          # the tokens' own keys and values
        _c_void_p, _c_long, _c_int,                                                                  # A, lda, K
        _c_void_p, _c_long, _c_void_p, _c_void_p, _c_int, _c_long, _c_int, _c_int, _c_void_p],      # W, ldw, bias, out, ..., stream
    "ka_attention_biased_bf16": [_c_void_p, _c_long, _c_void_p, _c_void_p, _c_void_p, _c_int, _c_void_p, _c_void_p, _c_int,
                                 _c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_long, _c_float,
                                 _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _c_void_p, _c_int, _c_void_p, _c_long,
                                 _c_void_p, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p, _c_float, _c_int, _c_int, _c_int, _c_void_p],
    "ka_latent_expand_supported": [_c_int, _c_int, _c_int, _c_int, _c_long],
    "ka_latent_expand_plan": [_c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p,
                              _c_void_p, _c_void_p, _c_void_p, _c_void_p],
    "ka_latent_expand_bf16": [_c_void_p, _c_long, _c_void_p, _c_void_p, _c_void_p, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p,
                              _c_void_p, _c_void_p],
    "ka_heads_linear_bf16": [_c_void_p, _c_long, _c_int, _c_void_p, _c_void_p, _c_long, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p,
                             _c_long, _c_void_p, _c_void_p],
    "ka_heads_linear_supported": [_c_long, _c_int, _c_long, _c_int, _c_int, _c_int],
    "ka_experts_gemm_supported": [_c_long, _c_int, _c_int, _c_long, _c_int, _c_int],
    "ka_experts_gemm_bf16": [_c_void_p, _c_long, _c_int, _c_void_p, _c_void_p, _c_void_p, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float,
                             _c_float, _c_float, _c_void_p, _c_long, _c_int, _c_int, _c_void_p],
    "ka_experts_few_supported": [_c_int, _c_long, _c_int, _c_int, _c_int],
    "ka_experts_few_bf16": [_c_void_p, _c_long, _c_int, _c_void_p, _c_void_p, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _c_float,
                            _c_float, _c_void_p, _c_long, _c_int, _c_void_p],
    "ka_matrix_memory_chunks_bf16": [_c_void_p, _c_void_p, _c_void_p, _c_void_p, _c_long, _c_void_p, _c_void_p, _c_void_p, _c_void_p,
                                     _c_void_p, _c_void_p, _c_long, _c_int, _c_int, _c_int, _c_int, _c_float, _c_float, _c_float,
                                     _c_void_p, _c_int, _c_void_p],
    "ka_gated_chunks_supported": [_c_int, _c_int],
    "ka_gated_chunks_scratch": [_c_int, _c_int, _c_int, _c_int, _c_int],
    "ka_gated_chunks_bf16": [_c_void_p, _c_void_p, _c_void_p, _c_long, _c_void_p, _c_float, _c_float, _c_void_p, _c_long, _c_void_p, _c_void_p,
                             _c_void_p, _c_void_p, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p],
    "ka_linear_chunks_bf16": [_c_void_p, _c_void_p, _c_void_p, _c_long, _c_void_p, _c_void_p, _c_long, _c_void_p, _c_void_p, _c_void_p,
                              _c_void_p, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_void_p],
    "ka_linear_skinny_norm_store": [_c_void_p, _c_void_p, _c_void_p, _c_float, _c_int, _c_void_p, _c_long, _c_void_p, _c_void_p,
                                    _c_int, _c_long, _c_int, _c_int, _c_int, _c_void_p, _c_long, _c_void_p],
}

# Rows up to which the weight-streaming kernel is used instead of the tiled one.
SKINNY_MAX_ROWS = 64
# Rows (and their width) up to which the weight-streaming kernel can normalise its input itself.
SKINNY_LN_MAX_ROWS = 16
SKINNY_LN_MAX_WIDTH = 4096
# Width of rows up to which a norm can follow a pair of skinny linears in their own launches.
NORM_AFTER_MAX_WIDTH = 8192
# Whether blocks let the weight-streaming kernel normalise its input itself. Every workgroup of
# the persistent kernel then repeats the LayerNorm of all rows once; with a few hundred workgroups
# that is cheaper than a launch of its own (measured on MI355X: 3 % of a decode step at batch 8).
FUSE_LAYERNORM_PROLOGUE = True
# Whether the matrix-core attention with further terms deals a row's keys out over several workgroups in decode steps
# of few rows (``attention_biased_bf16``).
SPLIT_DECODE_KEYS = True
# Whether the decode attention of a few rows (whose workgroups fill at most a quarter of the chip)
# takes the feed-forward's first linear into its own launch instead of leaving it to the launch of
# the q|k|v projection before it (measured on MI355X at Moondream 2's sizes: 3 to 5 % of a decode
# step at batch 1 to 4).
ATTENTION_TAKES_LINEAR = True
# Tile of the tiled kernels: 0 lets them choose by size; 221, 211 (any K), 12222, 23212, 22224, 22232, 13122
# (K in steps of 64 or 32, loads straight into LDS) force one, and 1000000 * parts + 23212 forces K to be cut into
# that many parts as well (for measurements and tests).
TILED_CONFIG = 0
# Whether linears of more than SKINNY_MAX_ROWS rows go to the vendor library (hipBLASLt) where it has
# a kernel for the case, bias, activation and the sum into the residual being its epilogues; the
# tiled kernels of this package then take what it declines. Measured on MI355X at Moondream 2's
# four linears: 201 against 242 us a layer at 2,048 rows, 112 against 151 at 730, 64 against 72 at 96.
LIBRARY_LINEAR = True
LIBRARY_WORKSPACE_BYTES = 128 << 20
# Activations that the library has no epilogue for (relu squared: ops.linear.ACT_RELU_SQUARED), and the size of an output from
# which the library's product and a pass over it are faster than this package's tiled kernel with the activation in its
# epilogue (2,048 rows of 2,048 by 4,224: 75 us).
_ACTIVATIONS_APART = (4,)
ACTIVATION_APART_FROM_ROWS = 256
ACTIVATION_APART_FROM_COLUMNS = 1024
_library_space = {}
SCRATCH_FLOATS = 8 << 20
WIDE_FLOATS = 8 << 20              # 32 MB of partial sums for the wide skinny kernel
_wide_scratch = {}
# Keys of one row a workgroup of the decode attention kernel takes before the row is split.
DECODE_KEYS_PER_WORKGROUP = 4096
# Longest row for which workgroups of four waves run with tiles of 32 keys, eight to a CU (the kernel goes by the
# width of the block table: 128 pages).
DECODE_SMALL_TILE_KEYS = 2048


class ChipSizes(NamedTuple):
    """What the choices between kernel forms need to know of the GPU at hand, all of it following
    from its number of compute units (four SIMDs each)."""

    compute_units: int
    # waves the split weight-streaming kernel aims to have on the chip: 8 per compute unit (one workgroup
    # of 8 waves per strip where there are as many strips as compute units; measured best on an MI355X
    # for an output projection + second feed-forward linear of 2048 outputs)
    skinny_target_waves: int
    # waves of the decode attention kernel that the chip holds at once (16 per compute unit: four per
    # SIMD at the registers the kernel needs), its workgroups of four waves (five per compute unit), and
    # its workgroups of four waves with tiles of two pages, which the kernel takes where all of them then
    # fit on the chip at once (eight per compute unit)
    decode_wave_slots: int
    decode_four_wave_places: int
    decode_small_tile_places: int


_chips: Dict[int, ChipSizes] = {}


def chip_sizes(device=None) -> ChipSizes:
    """The sizes for ``device`` (default: the current one), asked from the driver once per device."""
    index = torch.cuda.current_device() if device is None else _device_index(device)
    if index not in _chips:
        units = int(torch.cuda.get_device_properties(index).multi_processor_count)
        _chips[index] = ChipSizes(units, 8 * units, 16 * units, 5 * units, 8 * units)
    return _chips[index]


ACT_GATED = 0x100                  # (ops.linear.ACT_GATED)

_lib = None
_scratch: Dict[int, torch.Tensor] = {}
_OUT_CODE = {torch.float32: KA_F32, torch.bfloat16: KA_BF16}


def lib():
    global _lib
    if _lib is None:
        handle = _build.load("fast")
        for name, argtypes in _SIGNATURES.items():
            fn = getattr(handle, name)
            fn.argtypes = argtypes
            fn.restype = _c_int
        handle.ka_last_error.restype = ctypes.c_char_p
        handle.ka_linear_library_stats.argtypes = [ctypes.POINTER(ctypes.c_long)] * 5
        handle.ka_linear_library_set_tuning.argtypes = [_c_int]
        handle.ka_linear_library_set_tuning.restype = None
        handle.ka_linear_library_stats.restype = None
        handle.ka_skinny_set_persistent.argtypes = [_c_int]
        handle.ka_skinny_set_persistent.restype = None
        handle.ka_rope_cache_pages_supported.argtypes = [_c_int, _c_int, _c_int]
        handle.ka_rope_cache_pages_supported.restype = _c_int
        for name in ("ka_attention_prefill_supported", "ka_attention_decode_supported"):
            getattr(handle, name).argtypes = [_c_int, _c_int]
            getattr(handle, name).restype = _c_int
        handle.ka_attention_biased_supported.argtypes = [_c_int] * 3
        handle.ka_attention_biased_supported.restype = _c_int
        handle.ka_experts_gemm_tile.argtypes = []
        handle.ka_experts_gemm_tile.restype = _c_int
        handle.ka_attention_biased_query_block.argtypes = []
        handle.ka_attention_biased_query_block.restype = _c_int
        handle.ka_attention_decode_beside_supported.argtypes = [_c_int] * 6
        handle.ka_attention_decode_beside_supported.restype = _c_int
        for name in ("ka_attention_prefill_max_keys", "ka_attention_prefill_query_block"):
            getattr(handle, name).argtypes = [_c_int]
            getattr(handle, name).restype = _c_int
        _lib = handle
    return _lib


def set_skinny_persistent(enabled: int) -> None:
    """Whether one-segment skinny linears may use the persistent kernel where it fits (1, the
    default) or all go to the split kernel (0): for measurements, and for tests of the split kernel
    on sizes that it otherwise never sees."""
    lib().ka_skinny_set_persistent(int(enabled))


def set_skinny_wide(enabled: int) -> None:
    """Where skinny linears use the kernel that shares the activations through LDS and cuts K
    into parts: 1 (the default) where it was measured faster (two K-segments at 17 to 64 rows or
    with more strips than CUs at 5 to 16 rows; one segment too long for the persistent kernel's
    registers at 17 to 64 rows), 2 wherever it can run (for tests), 0 nowhere."""
    lib().ka_skinny_set_wide(int(enabled))


def _check(status: int) -> None:
    if status != 0:
        raise KernelError(lib().ka_last_error().decode())


def _device_index(device) -> int:
    """One key per GPU, whether or not the device's name carries its index."""
    device = torch.device(device)
    return torch.cuda.current_device() if device.index is None else device.index


def scratch(device: torch.device) -> torch.Tensor:
    """Partial results that the parts of a row's keys meet through in decode attention (one
    buffer per device). Calls on one device must not overlap."""
    key = _device_index(device)
    if key not in _scratch:
        _scratch[key] = torch.zeros(SCRATCH_FLOATS, dtype=torch.float32, device=device)
    return _scratch[key]


def _wide_args(device: torch.device, rows: int):
    """Scratch memory for the parts of K of a skinny linear that goes to the wide kernel: fp32
    partial sums, one buffer per device, made at the first skinny call (a step's first run is
    never inside a graph capture). Calls on one device must not overlap."""
    buf = _wide_scratch_buffer(device)
    return buf.data_ptr(), buf.numel()


def _wide_scratch_buffer(device: torch.device) -> torch.Tensor:
    key = _device_index(device)
    if key not in _wide_scratch:
        _wide_scratch[key] = torch.empty(WIDE_FLOATS, dtype=torch.float32, device=device)
    return _wide_scratch[key]


def _library_workspace(device: torch.device) -> torch.Tensor:
    """Scratch memory the vendor library's kernels may use (parts of K that meet in it), one buffer
    per device, made at the first call (a step's first run is never inside a graph capture).
    Calls on one device must not overlap."""
    key = _device_index(device)
    if key not in _library_space:
        _library_space[key] = torch.empty(LIBRARY_WORKSPACE_BYTES, dtype=torch.uint8, device=device)
    return _library_space[key]


def prepare(device: torch.device) -> int:
    """Everything these kernels keep per device, made now instead of at the first call that needs it
    (which may be the first step of a live request): the partial results of decode attention, the
    partial sums of the wide skinny kernel and the vendor library's workspace. Returns their bytes."""
    buffers = (scratch(device), _library_workspace(device), _wide_scratch_buffer(device))
    return sum(b.numel() * b.element_size() for b in buffers)


def library_stats() -> Dict[str, int]:
    """Plans the vendor-library linears keep, how often the library's heuristic was asked for an
    algorithm, how many plans had to make room, how many were tuned and how many of those took another
    algorithm than the first named (all since the process started)."""
    handle = lib()
    values = [ctypes.c_long(0) for _ in range(5)]
    handle.ka_linear_library_stats(*[ctypes.byref(v) for v in values])
    return dict(zip(("plans", "heuristic_calls", "evicted", "tuned", "tuned_other"), (int(v.value) for v in values)))


def set_library_tuning(runs: int) -> None:
    """``runs`` > 0: a plan of the vendor-library linears that is made from now on times, at its first call, every
    algorithm the library's heuristic named (``runs`` products each, on that call's operands, whose content is
    run over several times: a warm-up's) and keeps the fastest. 0 (the default): the first named."""
    lib().ka_linear_library_set_tuning(int(runs))


def _operand_ok(t: torch.Tensor, k: int) -> bool:
    return (t.dtype == torch.bfloat16 and t.dim() == 2 and t.shape[1] == k and t.stride(1) == 1 and t.stride(0) % 8 == 0
            and t.data_ptr() % 16 == 0)


def _bias_ok(bias: Optional[torch.Tensor], n: int) -> bool:
    return bias is None or (bias.dtype == torch.float32 and bias.numel() == n and bias.is_contiguous())


def _out_ok(out: torch.Tensor, m: int, n: int, act: int = 0) -> bool:
    """``out`` is ``[m, columns]`` of a linear of ``n`` weight rows (half of them if ``act`` says gated)."""
    n_out = n // 2 if act & ACT_GATED else n
    return (out.dtype in _OUT_CODE and tuple(out.shape) == (m, n_out) and out.stride(1) == 1 and out.data_ptr() % 16 == 0)


def linear_bf16(a, weight, bias, out, act, accumulate) -> bool:
    m, k = a.shape
    n = weight.shape[0]
    if m == 0:
        return True
    if k % 8 or not _operand_ok(a, k) or not _operand_ok(weight, k) or out.dtype not in _OUT_CODE \
            or out.data_ptr() % 16 or out.stride(1) != 1:
        return False
    if act & ACT_GATED and (n % 2 or accumulate):
        raise KernelError("linear: a gated linear needs an even number of weight rows and no accumulation")
    if tuple(out.shape) != (m, n // 2 if act & ACT_GATED else n):
        raise KernelError(f"linear: shapes a {tuple(a.shape)}, weight {tuple(weight.shape)}, out {tuple(out.shape)}")
    if not _bias_ok(bias, n):
        raise KernelError("linear: bias must be fp32 [N]")
    if accumulate and out.dtype != torch.float32:
        raise KernelError("linear: accumulate needs an fp32 output")
    handle = lib()
    if m <= SKINNY_MAX_ROWS:
        _check(handle.ka_linear_skinny_bf16(a.data_ptr(), a.stride(0), weight.data_ptr(), weight.stride(0), _ptr(bias),
                                            out.data_ptr(), _OUT_CODE[out.dtype], out.stride(0), m, n, k, act,
                                            int(accumulate), chip_sizes(a.device).skinny_target_waves, *_wide_args(a.device, m), stream_ptr()))
    else:
        if LIBRARY_LINEAR and TILED_CONFIG == 0:
            space = _library_workspace(a.device)
            # (an activation the library has no epilogue for: a pass of its own over the products)
            apart = act in _ACTIVATIONS_APART and m >= ACTIVATION_APART_FROM_ROWS and n >= ACTIVATION_APART_FROM_COLUMNS \
                and out.dtype == torch.bfloat16 and n % 8 == 0 and out.stride(0) % 8 == 0 and m <= 65535
            status = handle.ka_linear_library_bf16(a.data_ptr(), a.stride(0), weight.data_ptr(), weight.stride(0),
                                                   _ptr(bias), out.data_ptr(), _OUT_CODE[out.dtype], out.stride(0), m, n, k,
                                                   0 if apart else act, int(accumulate), space.data_ptr(), space.numel(), stream_ptr())
            if status == 0:
                if apart:
                    core.activate_rows(out, act)
                return True
            if status < 0:
                _check(status)
        _check(handle.ka_linear_tiled_bf16(a.data_ptr(), a.stride(0), weight.data_ptr(), weight.stride(0), _ptr(bias),
                                           out.data_ptr(), _OUT_CODE[out.dtype], out.stride(0), m, n, k, act,
                                           int(accumulate), TILED_CONFIG, *_wide_args(a.device, m), stream_ptr()))
    return True


def linear_pair_accumulate(a1, w1, b1, a2, w2, b2, out, then_norm=None, accumulate: bool = True) -> bool:
    """``out += a1 @ w1.T + b1 + a2 @ w2.T + b2`` in one launch (few rows, fp32 ``out``); with ``accumulate`` off
    the sum replaces ``out``.
    ``then_norm = (gamma, beta or None, eps, normed)``: also ``normed = LayerNorm(out)``, in the kernel
    that finishes the rows where there is one (more than 8 rows), else in a launch behind it. False:
    not covered, nothing was run (with ``then_norm``: try without)."""
    m, k1 = a1.shape
    k2 = a2.shape[1]
    n = w1.shape[0]
    if not (0 < m <= SKINNY_MAX_ROWS) or k1 % 8 or k2 % 8 or a2.shape[0] != m or w2.shape[0] != n:
        return False
    if not (_operand_ok(a1, k1) and _operand_ok(w1, k1) and _operand_ok(a2, k2) and _operand_ok(w2, k2)):
        return False
    if out.dtype != torch.float32 or not _out_ok(out, m, n) or not _bias_ok(b1, n) or not _bias_ok(b2, n):
        return False
    if then_norm is not None:
        gamma, beta, eps, normed = then_norm
        if n % 4 or n > NORM_AFTER_MAX_WIDTH or out.stride(0) % 4 or normed.dtype not in _OUT_CODE or not _out_ok(normed, m, n) \
                or normed.stride(0) % 4 or gamma.dtype != torch.float32 or gamma.numel() != n or gamma.data_ptr() % 16:
            return False
        if beta is not None and (beta.dtype != torch.float32 or beta.numel() != n or beta.data_ptr() % 16):
            return False
        if any(b is not None and b.data_ptr() % 16 for b in (b1, b2)):
            return False
        _check(lib().ka_linear_skinny_pair_norm(
            a1.data_ptr(), a1.stride(0), k1, a2.data_ptr(), a2.stride(0), k2, w1.data_ptr(), w1.stride(0), _ptr(b1),
            w2.data_ptr(), w2.stride(0), _ptr(b2), out.data_ptr(), out.stride(0), n, int(bool(accumulate)), m, chip_sizes(a1.device).skinny_target_waves,
            *_wide_args(a1.device, m), gamma.data_ptr(), _ptr(beta), float(eps), normed.data_ptr(), _OUT_CODE[normed.dtype],
            normed.stride(0), stream_ptr()))
        return True
    _check(lib().ka_linear_skinny_fused(
        a1.data_ptr(), a1.stride(0), k1, a2.data_ptr(), a2.stride(0), k2, w2.data_ptr(), w2.stride(0), _ptr(b2),
        None, None, None, 0.0,
        w1.data_ptr(), w1.stride(0), _ptr(b1), out.data_ptr(), KA_F32, out.stride(0), n, 0, int(bool(accumulate)),
        None, 0, None, None, 0, 0, 0, 0, m, chip_sizes(a1.device).skinny_target_waves, *_wide_args(a1.device, m), stream_ptr()))
    return True


def pair_finishes_rows(m: int, n: int) -> bool:
    """Whether ``linear_pair_accumulate`` of ``m`` rows and ``n`` outputs ends in a kernel that finishes
    whole rows (K cut into parts): that kernel normalises them as well at no launch of its own."""
    return bool(lib().ka_linear_skinny_pair_in_parts(int(m), int(n)))


def linear_two_outputs(a, wa, ba, out_a, act_a, wb, bb, out_b, act_b) -> bool:
    """``out_a = act_a(a @ wa.T + ba)`` and ``out_b = act_b(a @ wb.T + bb)`` in one launch (few rows)."""
    m, k = a.shape
    na, nb = wa.shape[0], wb.shape[0]
    if not (0 < m <= SKINNY_MAX_ROWS) or k % 8:
        return False
    if not (_operand_ok(a, k) and _operand_ok(wa, k) and _operand_ok(wb, k) and _out_ok(out_a, m, na, act_a)
            and _out_ok(out_b, m, nb, act_b) and _bias_ok(ba, na) and _bias_ok(bb, nb)):
        return False
    _check(lib().ka_linear_skinny_fused(
        a.data_ptr(), a.stride(0), k, None, 0, 0, None, 0, None,
        None, None, None, 0.0,
        wa.data_ptr(), wa.stride(0), _ptr(ba), out_a.data_ptr(), _OUT_CODE[out_a.dtype], out_a.stride(0), na, act_a, 0,
        wb.data_ptr(), wb.stride(0), _ptr(bb), out_b.data_ptr(), _OUT_CODE[out_b.dtype], out_b.stride(0), nb, act_b,
        m, chip_sizes(a.device).skinny_target_waves, *_wide_args(a.device, m), stream_ptr()))
    return True


def layernorm_linear(x, gamma, beta, eps, wa, ba, out_a, act_a, wb=None, bb=None, out_b=None, act_b=0, store=None,
                     centred: bool = True) -> bool:
    """``h = LayerNorm(x)``; ``out_a = act_a(h @ wa.T + ba)`` and, if a second target is given,
    ``out_b = act_b(h @ wb.T + bb)`` in one launch: the kernel normalises the fp32 rows itself
    (at most 16 of them, at most 4096 wide, and no more than fit in 96 KB of LDS as bf16).
    ``store`` (one target only): bf16 ``[m, k]`` that also receives ``h``, for launches that follow.
    ``centred`` ``False``: the norm is a root-mean-square norm, ``h = x / sqrt(mean(x^2) + eps) * gamma`` (no ``beta``,
    no ``store``)."""
    if not centred and (beta is not None or store is not None):
        return False
    m, k = x.shape
    if not (0 < m <= SKINNY_LN_MAX_ROWS) or k % 8 or k > SKINNY_LN_MAX_WIDTH or x.dtype != torch.float32 \
            or not x.is_contiguous():
        return False
    if x.data_ptr() % 16 or gamma.dtype != torch.float32 or gamma.numel() != k or gamma.data_ptr() % 16:
        return False
    if beta is not None and (beta.dtype != torch.float32 or beta.numel() != k or beta.data_ptr() % 16):
        return False
    na = wa.shape[0]
    if not (_operand_ok(wa, k) and _out_ok(out_a, m, na, act_a) and _bias_ok(ba, na)):
        return False
    two = wb is not None
    nb = wb.shape[0] if two else 0
    if two and not (_operand_ok(wb, k) and _out_ok(out_b, m, nb, act_b) and _bias_ok(bb, nb)):
        return False
    if m * (k + 8) * 2 > 96 * 1024:
        return False
    for bias, n in ((ba, na), (bb, nb)):
        if bias is not None and (n % 4 or bias.data_ptr() % 16):
            return False
    if store is not None:
        if two or store.dtype != torch.bfloat16 or not _out_ok(store, m, k) or store.stride(0) % 8:
            return False
        _check(lib().ka_linear_skinny_norm_store(
            x.data_ptr(), gamma.data_ptr(), _ptr(beta), float(eps), k, wa.data_ptr(), wa.stride(0), _ptr(ba),
            out_a.data_ptr(), _OUT_CODE[out_a.dtype], out_a.stride(0), na, act_a, m, store.data_ptr(), store.stride(0),
            stream_ptr()))
        return True
    if not centred:
        _check(lib().ka_linear_skinny_fused_rms(
            x.data_ptr(), gamma.data_ptr(), float(eps), k, wa.data_ptr(), wa.stride(0), _ptr(ba), out_a.data_ptr(),
            _OUT_CODE[out_a.dtype], out_a.stride(0), na, act_a, _ptr(wb), wb.stride(0) if two else 0, _ptr(bb) if two else None,
            _ptr(out_b), _OUT_CODE[out_b.dtype] if two else 0, out_b.stride(0) if two else 0, nb, act_b, m,
            chip_sizes(x.device).skinny_target_waves, stream_ptr()))
        return True
    _check(lib().ka_linear_skinny_fused(
        None, 0, k, None, 0, 0, None, 0, None,
        x.data_ptr(), gamma.data_ptr(), _ptr(beta), float(eps),
        wa.data_ptr(), wa.stride(0), _ptr(ba), out_a.data_ptr(), _OUT_CODE[out_a.dtype], out_a.stride(0), na, act_a, 0,
        _ptr(wb), wb.stride(0) if two else 0, _ptr(bb) if two else None, _ptr(out_b),
        _OUT_CODE[out_b.dtype] if two else 0, out_b.stride(0) if two else 0, nb, act_b,
        m, chip_sizes(x.device).skinny_target_waves, None, 0, stream_ptr()))
    return True


def rope_cache_bf16(qkv, positions, slots, table, k_cache, v_cache, n_heads, n_kv_heads, head_dim, page_size,
                    runs=None) -> bool:
    """Rotary encoding of q (in place) and k, and the cache write of k and v, a page's worth of
    tokens per workgroup (``ops.core.rope_cache`` says what the operands are). ``runs``: (int32 first
    token, int32 count) of the runs the tokens are cut into, every token in exactly one and none longer
    than a page (``StepBatch.page_runs``); without them every 16 tokens are a run. False: not covered
    (another page size, a rotary size that is no multiple of 16, rows that are not 16-byte aligned)."""
    if table is None or qkv.dtype != torch.bfloat16 or qkv.stride(1) != 1 or qkv.stride(0) % 8 or qkv.data_ptr() % 16:
        return False
    rot = int(table.shape[1])
    handle = lib()
    if not handle.ka_rope_cache_pages_supported(head_dim, rot, page_size) or table.data_ptr() % 16:
        return False
    if slots is not None and (k_cache.data_ptr() % 16 or v_cache.data_ptr() % 16):
        return False
    first, count = runs if runs is not None else (None, None)
    _check(handle.ka_rope_cache_pages_bf16(qkv.data_ptr(), qkv.stride(0), positions.data_ptr(), _ptr(slots), table.data_ptr(),
                                           int(table.shape[0]), _ptr(k_cache), _ptr(v_cache), qkv.shape[0], n_heads,
                                           n_kv_heads, head_dim, rot, page_size, _ptr(first), _ptr(count),
                                           int(first.numel()) if first is not None else 0, stream_ptr()))
    return True


def decode_shape(max_kv: int, workgroups: int = 1, head_dim: int = 64):
    """``(splits, waves)`` of the decode attention kernel: a workgroup of up to 16 waves takes a
    64-key tile per wave and round; rows longer than 4096 keys are cut into parts whose sums
    a second kernel merges (cutting the keys of a few short rows further, to put more CUs to
    work, was measured and changes nothing: 0.887 ms a step at batch 1 either way). With many
    workgroups (rows x heads) each gets fewer waves, so that they all fit on the chip at once.
    Head sizes up to 64 (measured at 32 heads and 1,024 keys): 16 waves up to 256 workgroups, 4
    beyond, which the kernel runs with tiles of 32 keys, eight workgroups to a CU, while the chip
    holds them all at once (four waves against eight: 6.70k against 6.53k tok/s at 9 rows, 10.6k
    against 10.4k at 16, 12.8k against 11.9k at 24, 16.5k against 15.9k at 48, 18.0k against 16.5k at
    64; rows of up to 2,048 keys: behind 4,096 keys the larger tile is 2 to 3 % ahead at 24 and 32
    rows). Larger head sizes, whose registers leave a CU eight waves, and longer rows: 16 waves up to
    256 workgroups, 8 up to 512, 4 beyond. Workgroups of four waves with tiles of 64 keys fit five to a CU; where they
    would end in a round that leaves much of the chip idle, eight waves again."""
    chip = chip_sizes()
    splits = max(1, -(-max_kv // DECODE_KEYS_PER_WORKGROUP))
    tiles = -(-max_kv // (64 * splits))
    waves = 4 if tiles <= 4 else 8 if tiles <= 8 else 16
    groups = workgroups * splits
    if groups <= chip.decode_wave_slots // 16:
        fit = 16
    elif head_dim <= 64 and groups <= chip.decode_small_tile_places and max_kv <= DECODE_SMALL_TILE_KEYS:
        fit = 4
    elif groups <= chip.decode_wave_slots // 8:
        fit = 8
    else:
        # workgroups of four waves run in rounds of as many as the chip has places for; where the last round
        # would leave much of the chip idle, workgroups of eight waves come out better (48 rows x 32 heads are
        # 1.2 rounds of the one, 3 rounds of the other: 14.9k against 15.2k tok/s)
        fit = 4
        rounds = -(-groups // chip.decode_four_wave_places)
        if groups < 0.7 * rounds * chip.decode_four_wave_places:
            fit = 8
    return splits, min(waves, fit)


def _attention_operands_ok(q, out) -> bool:
    return not (q.data_ptr() % 16 or q.stride(0) % 8 or out.data_ptr() % 16 or out.stride(0) % 4)


def _side_linear_ok(job) -> bool:
    """Operands of a ``parts.SideLinear`` that the persistent skinny kernel takes."""
    a, w, out = job.a, job.weight, job.out
    if a.dim() != 2 or a.dtype != torch.bfloat16 or w.dtype != torch.bfloat16:
        return False
    m, k = a.shape
    n = w.shape[0]
    if k % 8 or not (_operand_ok(a, k) and _operand_ok(w, k) and _out_ok(out, m, n, int(job.act)) and _bias_ok(job.bias, n)):
        return False
    return job.bias is None or (n % 4 == 0 and job.bias.data_ptr() % 16 == 0)


def attention_decode_takes(job, n: int, n_heads: int, head_dim: int, page_size: int, max_kv: int) -> bool:
    """Whether ``attention_decode_bf16`` runs ``job`` (a ``parts.SideLinear``) in its own launch: a few
    rows whose attention leaves most of the chip idle."""
    if not ATTENTION_TAKES_LINEAR or n == 0 or not _side_linear_ok(job) or job.a.shape[0] != n:
        return False
    splits = decode_shape(max_kv, n * n_heads, head_dim)[0]
    return bool(lib().ka_attention_decode_beside_supported(n, n_heads, splits, head_dim, page_size, job.a.shape[1]))


def attention_decode_bf16(q, k_cache, v_cache, block_table, token_row, kv_lo, kv_hi, out, scale, n_heads,
                          n_kv_heads, head_dim, batch, fuse=None, beside=None) -> bool:
    """One token per row. ``fuse = (k_new, v_new, table, slots)``: the kernel also rotates q and the
    token's key and stores key and value in the cache (the rotary kernel is then not run).
    ``beside``: a ``parts.SideLinear`` for which ``attention_decode_takes`` said yes; the launch
    computes it on the side (False: it does not after all, and nothing was run)."""
    n = q.shape[0]
    page_size = k_cache.shape[2]
    if n == 0:
        return beside is None
    handle = lib()
    if batch is None or not batch.decode_only or not _attention_operands_ok(q, out) \
            or not handle.ka_attention_decode_supported(head_dim, page_size):
        return False
    if beside is not None and not attention_decode_takes(beside, n, n_heads, head_dim, page_size, batch.max_kv):
        return False
    splits, waves = decode_shape(batch.max_kv, n * n_heads, head_dim)
    partial = scratch(q.device)
    if n * n_heads * splits * (head_dim + 2) > partial.numel():
        return False
    k_new = v_new = table = slots = None
    new_stride = rot = 0
    if fuse is not None:
        k_new, v_new, table, slots = fuse
        rot = int(table.shape[1])
        new_stride = k_new.stride(0)
        if rot % 16 or rot > head_dim or k_new.data_ptr() % 16 or v_new.data_ptr() % 16 \
                or new_stride % 8 or v_new.stride(0) != new_stride:
            return False
    if beside is not None:
        w, lin_out = beside.weight, beside.out
        _check(handle.ka_attention_decode_beside_bf16(
            q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(), block_table.data_ptr(),
            block_table.shape[1], token_row.data_ptr(), _ptr(kv_lo), kv_hi.data_ptr(), out.data_ptr(), out.stride(0),
            float(scale), n, n_heads, n_kv_heads, head_dim, page_size, splits, partial.data_ptr(), partial.numel(),
            _ptr(k_new), _ptr(v_new), new_stride, _ptr(table), rot, _ptr(slots), k_cache.data_ptr(), v_cache.data_ptr(),
            beside.a.data_ptr(), beside.a.stride(0), beside.a.shape[1], w.data_ptr(), w.stride(0), _ptr(beside.bias),
            lin_out.data_ptr(), _OUT_CODE[lin_out.dtype], lin_out.stride(0), w.shape[0], int(beside.act), stream_ptr()))
        return True
    _check(handle.ka_attention_decode_bf16(
        q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(), block_table.data_ptr(),
        block_table.shape[1], token_row.data_ptr(), _ptr(kv_lo), kv_hi.data_ptr(), out.data_ptr(), out.stride(0),
        float(scale), n, n_heads, n_kv_heads, head_dim, page_size, splits, waves, partial.data_ptr(), partial.numel(),
        _ptr(k_new), _ptr(v_new), new_stride, _ptr(table), rot, _ptr(slots),
        k_cache.data_ptr(), v_cache.data_ptr(), stream_ptr()))
    return True


def prefill_query_block(head_dim: int) -> int:
    """Queries of one row that a workgroup of the prompt attention kernel takes at this head size:
    the size the step's lists of blocks of queries must be cut to for it."""
    return int(lib().ka_attention_prefill_query_block(head_dim))


def _query_blocks(batch, head_dim: int):
    """``(rows, first tokens, size)`` of the blocks of queries of a step, at the size the kernel likes
    best among those the step lists (``batch.query_blocks``: size -> lists), else at 32."""
    listed = getattr(batch, "query_blocks", None) or {}
    best = prefill_query_block(head_dim)
    if best in listed:
        return (*listed[best], best)
    if 32 in listed:
        return (*listed[32], 32)
    if getattr(batch, "qblk_row", None) is not None:
        return batch.qblk_row, batch.qblk_tok, 32
    return None


def attention_bf16(q, k_cache, v_cache, block_table, token_row, kv_lo, kv_hi, out, scale, n_heads, n_kv_heads,
                   head_dim, batch) -> bool:
    n = q.shape[0]
    page_size = k_cache.shape[2]
    if n == 0:
        return True
    if batch is None or not _attention_operands_ok(q, out):
        return False
    if attention_decode_bf16(q, k_cache, v_cache, block_table, token_row, kv_lo, kv_hi, out, scale, n_heads,
                             n_kv_heads, head_dim, batch):
        return True
    handle = lib()
    # the longest row's block table must fit in LDS (the whole table's width where the length is not known)
    longest = int(batch.max_kv) if batch.max_kv > 1 else block_table.shape[1] * page_size
    blocks = _query_blocks(batch, head_dim) if handle.ka_attention_prefill_supported(head_dim, page_size) else None
    # (the prompt kernel is written for a positive scale; any other goes to the generic kernel)
    if blocks is not None and longest <= handle.ka_attention_prefill_max_keys(head_dim) and 0.0 < scale < float("inf"):
        rows, first_tokens, size = blocks
        _check(handle.ka_attention_prefill_bf16(
            q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(), block_table.data_ptr(),
            block_table.shape[1], rows.data_ptr(), first_tokens.data_ptr(), int(rows.numel()),
            batch.cu_q.data_ptr(), batch.kv_len.data_ptr(), _ptr(kv_lo), kv_hi.data_ptr(), out.data_ptr(),
            out.stride(0), float(scale), n_heads, n_kv_heads, head_dim, page_size,
            int(batch.max_kv) if batch.max_kv > 1 else 0, size, stream_ptr()))
        return True
    return False


def biased_query_block(head_dim: int, value_dim: int) -> Optional[int]:
    """Queries of one row that a workgroup of the MFMA kernel for attention with distance slopes, a sink and values of
    a size of their own takes, or ``None`` where that kernel does not cover the sizes."""
    handle = lib()
    if not handle.ka_attention_biased_supported(int(head_dim), int(value_dim), 16):
        return None
    return int(handle.ka_attention_biased_query_block())


def attention_biased_bf16(q, k_cache, v_cache, block_table, token_row, kv_lo, kv_hi, out, scale, n_heads, n_kv_heads,
                          head_dim, value_dim, positions, slopes, sink, batch, bias_table=None, gate=None, sinks=None,
                          keep_first: int = 0, maps: int = 1, values_in_keys: bool = False, softcap: Optional[float] = None,
                          gate_per_head: bool = False, row_tokens=None) -> bool:
    """Attention with the further terms of ``ops.core.attention_generic`` (values of ``value_dim`` channels, ``slopes``
    times the distance taken off the scores, a ``sink`` in the softmax's denominator or one per head in ``sinks``, kept
    first keys before the window, several maps per head over shared values, values that are the first channels of the
    keys, fp32 outputs where ``out`` is fp32) on the matrix cores, for prompt portions, mixed steps and decode steps
    alike. ``row_tokens`` ``(from, below)``: of a step that is no decode step, only rows of that many tokens are taken, the others'
    outputs are left alone. False: not covered (head sizes, page size, alignment, no list of blocks of 32 queries with the step),
    nothing was run."""
    n = q.shape[0]
    page_size = k_cache.shape[2]
    if n == 0:
        return True
    handle = lib()
    if batch is None or not handle.ka_attention_biased_supported(int(head_dim), int(value_dim), int(page_size)):
        return False
    out_f32 = out.dtype == torch.float32
    if q.dtype != torch.bfloat16 or q.data_ptr() % 16 or q.stride(0) % 8 or q.stride(1) != 1 or out.data_ptr() % (16 if out_f32 else 8) \
            or out.stride(0) % 4 or out.stride(1) != 1 or k_cache.data_ptr() % 16 or (v_cache is not None and v_cache.data_ptr() % 16):
        return False
    if (v_cache is None) != bool(values_in_keys) or (values_in_keys and (maps != 1 or value_dim > head_dim)) or (out_f32 and gate is not None):
        return False
    if n_heads % maps or n_kv_heads % maps:
        raise KernelError("attention: the maps must divide the heads")
    if sinks is not None and (sinks.dtype != torch.float32 or sinks.numel() != n_heads or not sinks.is_contiguous()):
        raise KernelError("attention: sink scores must be fp32 [H]")
    if slopes is not None and (slopes.dtype != torch.float32 or slopes.numel() != n_heads or positions is None):
        raise KernelError("attention: slopes must be fp32 [H] and come with the queries' positions")
    gate_cols = n_heads if gate_per_head else n_heads * value_dim
    if gate is not None and (gate.dtype != torch.bfloat16 or gate.dim() != 2 or gate.stride(1) != 1
                             or tuple(gate.shape) != (n, gate_cols)):
        raise KernelError("attention: the output gate must be bf16 [n, H hdv] (or [n, H])")
    if softcap is not None and not softcap > 0:
        raise KernelError("attention: a cap on the scores must be positive")
    if bias_table is not None and (bias_table.dtype != torch.float32 or bias_table.dim() != 2 or bias_table.shape[0] != n_heads
                                   or not bias_table.is_contiguous() or positions is None):
        raise KernelError("attention: the distance table must be contiguous fp32 [H, T] and come with the queries' positions")
    n_splits, partial = 1, None
    if batch.decode_only:
        rows = first = None
        n_blocks = 0
        groups = n_heads // n_kv_heads
        workgroups = n * n_kv_heads * -(-groups // 32)
        waves = 4 if workgroups >= 2 * chip_sizes(q.device).compute_units else 8
        # few rows: a row's keys are dealt out over several workgroups, whose partial results a second launch merges
        # (the number depends on the rows alone, so a captured step keeps its layout)
        units = chip_sizes(q.device).compute_units
        scratch_of = getattr(batch, "workspace", None)
        # (measured on MI355X: with more than an eighth of the chip's units busy, or more than four runs of keys a row,
        # the second launch costs more than the split gains)
        if SPLIT_DECODE_KEYS and scratch_of is not None and 8 * workgroups <= units:
            n_splits = 4
            partial = scratch_of.get("attention.partials", (n, n_heads, n_splits, value_dim + 2), torch.float32)
    else:
        size = int(handle.ka_attention_biased_query_block())
        listed = (getattr(batch, "query_blocks", None) or {}).get(size)
        if listed is None:
            return False
        rows, first = listed
        n_blocks = int(rows.numel())
        if n_blocks == 0 or n_blocks > 65535:
            return False
        waves = 4
    if n > 65535:
        return False
    _check(handle.ka_attention_biased_bf16(
        q.data_ptr(), q.stride(0), k_cache.data_ptr(), _ptr(v_cache), block_table.data_ptr(), block_table.shape[1],
        _ptr(rows), _ptr(first), n_blocks, batch.cu_q.data_ptr(), token_row.data_ptr(), _ptr(kv_lo), kv_hi.data_ptr(),
        _ptr(positions), _ptr(slopes), out.data_ptr(), out.stride(0), float(scale), n, n_heads, n_kv_heads, head_dim,
        value_dim, page_size, waves, int(sink is not None or sinks is not None), float(sink or 0.0), _ptr(bias_table),
        int(bias_table.shape[1]) if bias_table is not None else 0, _ptr(gate),
        (gate.stride(0) if n > 1 else gate_cols) if gate is not None else 0, _ptr(sinks), int(keep_first), int(maps),
        int(bool(values_in_keys)), int(out_f32), n_splits, _ptr(partial), float(softcap or 0.0), int(bool(gate_per_head)),
        *(row_tokens if row_tokens is not None else (0, 0x7fffffff)), stream_ptr()))
    return True


def attention_maps_bf16(q, k_cache, v_cache, block_table, token_row, kv_lo, kv_hi, out, scale, n_heads, n_kv_heads, head_dim,
                        value_dim, keep_first, maps, batch) -> bool:
    """``maps`` attentions per head over shared values behind a window that keeps the first keys (``n_heads`` and
    ``n_kv_heads`` count maps), outputs in fp32 ``[n, n_heads value_dim]``, on the matrix cores. False: not covered."""
    return attention_biased_bf16(q, k_cache, v_cache, block_table, token_row, kv_lo, kv_hi, out, scale, n_heads, n_kv_heads,
                                 head_dim, value_dim, None, None, None, batch, keep_first=keep_first, maps=maps)


def attention_latent_bf16(q, cache, block_table, token_row, kv_hi, out, scale, n_heads, row_dim, rank, sinks, batch, kv_lo=None,
                          head_gate=None, row_tokens=None) -> bool:
    """``n_heads`` query heads of ``row_dim`` channels over one cached row per key whose first ``rank`` channels are its
    value, with a sink score per head (``sinks`` ``None``: no sinks), behind a window (``kv_lo``), times the sigmoid of one number
    per head (``head_gate`` ``[n, H]``), on the matrix cores (rows above 128 channels: the kernel's wide form). False: not
    covered (rows that are no multiple of 16 channels among others)."""
    return attention_biased_bf16(q, cache, None, block_table, token_row, kv_lo, kv_hi, out, scale, n_heads, 1, row_dim, rank,
                                 None, None, None, batch, sinks=sinks, values_in_keys=True, gate=head_gate,
                                 gate_per_head=head_gate is not None, row_tokens=row_tokens)


class LiftPlan(NamedTuple):
    """What of a step's cached latents is lifted to keys and values per head (``latent_expand_plan``)."""

    capacity: int               # lifted pages there is room for
    list: torch.Tensor          # int32 [capacity * 16]: place in the cache of every lifted place, -1: none
    table: torch.Tensor         # int32 [rows, max_pages]: lifted page of a row's logical page
    used: torch.Tensor          # int32 [1]: lifted places in use
    lifted: torch.Tensor        # int32 [tokens]: 1 for the tokens of a lifted row
    row_tokens: int             # rows of at least this many tokens are lifted


def latent_expand_supported(n_heads: int, head_dim: int, value_dim: int, rank: int, row_dim: int) -> bool:
    """Whether latents of ``rank`` channels (in cached rows of ``row_dim``) can be lifted to keys and values of these heads and
    attended to on the matrix cores with keys and values in registers."""
    handle = lib()
    return bool(handle.ka_latent_expand_supported(int(n_heads), int(head_dim), int(value_dim), int(rank), int(row_dim))) \
        and head_dim <= 128 and value_dim <= 128 and bool(handle.ka_attention_biased_supported(int(head_dim), int(value_dim), 16))


def latent_expand_plan(batch, group, name: str, window: int, row_tokens: int, pool_pages: int) -> Optional[LiftPlan]:
    """Which rows of the step are lifted (those of at least ``row_tokens`` tokens), made by one launch from what the step holds. The
    room it is made for follows from the step's numbers of tokens and rows alone. ``None``: too many rows or pages."""
    handle = lib()
    n, rows = batch.n_tokens, batch.n_rows
    if rows > int(handle.ka_latent_expand_max_rows()) or batch.workspace is None:
        return None
    # a row of q tokens behind a window of w reads at most w - 1 + q keys, which touch one page more at either end
    most = n // 16 + min(rows, n // row_tokens) * (window // 16 + 3)
    capacity = -(-min(most, pool_pages) // 8) * 8
    if capacity <= 0 or capacity // 8 > 65535:
        return None
    ws = batch.workspace
    max_pages = group.block_table.shape[1]
    plan = LiftPlan(capacity, ws.get(f"latent.lift_list.{name}", (capacity * 16,), torch.int32),
                    ws.get(f"latent.lift_table.{name}", (rows, max_pages), torch.int32),
                    ws.get(f"latent.lift_used.{name}", (1,), torch.int32), ws.get(f"latent.lifted.{name}", (n,), torch.int32), int(row_tokens))
    _check(handle.ka_latent_expand_plan(batch.cu_q.data_ptr(), batch.kv_len.data_ptr(), _ptr(group.kv_lo), batch.token_row.data_ptr(),
                                        group.block_table.data_ptr(), max_pages, n, rows, int(row_tokens), capacity, plan.list.data_ptr(),
                                        plan.table.data_ptr(), plan.used.data_ptr(), plan.lifted.data_ptr(), stream_ptr()))
    return plan


def latent_expand_bf16(cache, weights, plan: LiftPlan, n_heads: int, head_dim: int, value_dim: int, rank: int, workspace):
    """The latents that ``plan`` lists lifted by ``weights`` ``[H head_dim + H value_dim, rank]``: keys ``[pages, H, 16, head_dim]`` and
    values ``[pages, H, value_dim, 16]`` of the workspace."""
    if cache.dtype != torch.bfloat16 or not cache.is_contiguous() or cache.dim() != 4 or cache.shape[1] != 1 or cache.shape[2] != 16 \
            or weights.dtype != torch.bfloat16 or not weights.is_contiguous() \
            or tuple(weights.shape) != (n_heads * (head_dim + value_dim), rank) or cache.shape[3] < rank:
        raise KernelError("latents to lift: cache bf16 [pages, 1, 16, >= rank], weights bf16 [H (d + dv), rank]")
    keys = workspace.get("latent.lift_keys", (plan.capacity, n_heads, 16, head_dim), torch.bfloat16)
    values = workspace.get("latent.lift_values", (plan.capacity, n_heads, value_dim, 16), torch.bfloat16)
    _check(lib().ka_latent_expand_bf16(cache.data_ptr(), cache.shape[3], weights.data_ptr(), plan.list.data_ptr(), plan.used.data_ptr(),
                                       plan.capacity, n_heads, head_dim, value_dim, rank, keys.data_ptr(), values.data_ptr(), stream_ptr()))
    return keys, values


def heads_linear_bf16(a, a_head: int, k: int, weights, out, out_head: int, n_out: int, gate=None, skip=None) -> bool:
    """``out[:, h, :n_out] = a[:, h, :k] @ weights[h].T`` for every head in one launch on the matrix cores: ``a`` ``[n, H a_head]``,
    ``weights`` ``[H, n_out, k]``, ``out`` ``[n, H out_head]``, all bf16; with ``gate`` (bf16, laid out as ``out``) times the
    sigmoid of it. ``skip`` (int32 ``[n]``): rows whose number is not 0 are left alone. False: not covered (``k`` no multiple of 16, heads that are not aligned), nothing was run."""
    n = a.shape[0]
    if n == 0:
        return True
    heads = int(weights.shape[0])
    if a.dtype != torch.bfloat16 or out.dtype != torch.bfloat16 or weights.dtype != torch.bfloat16 or a.stride(1) != 1 \
            or out.stride(1) != 1 or not weights.is_contiguous() or tuple(weights.shape) != (heads, n_out, k) \
            or a.shape[1] < heads * a_head or out.shape[1] < heads * out_head or n > 64 * 65535:
        return False
    lda, ldo = (a.stride(0), out.stride(0)) if n > 1 else (heads * a_head, heads * out_head)
    if gate is not None and (gate.dtype != torch.bfloat16 or gate.dim() != 2 or gate.stride(1) != 1 or gate.shape[0] != n
                             or gate.shape[1] < heads * out_head):
        return False
    handle = lib()
    if a.data_ptr() % 16 or out.data_ptr() % 8 or weights.data_ptr() % 16 \
            or not handle.ka_heads_linear_supported(lda, a_head, ldo, out_head, n_out, k):
        return False
    _check(handle.ka_heads_linear_bf16(a.data_ptr(), lda, a_head, weights.data_ptr(), out.data_ptr(), ldo, out_head, n, heads,
                                       n_out, k, _ptr(gate), (gate.stride(0) if n > 1 else heads * out_head) if gate is not None else 0,
                                       _ptr(skip), stream_ptr()))
    return True


def matrix_memory_chunks_scratch(n: int, n_rows: int, n_heads: int, head_dim: int, value_dim: int) -> int:
    """fp32 numbers of scratch that ``matrix_memory_chunks_bf16`` needs to run a step of ``n`` tokens in ``n_rows`` rows in
    three passes (all chunks at once, a scan, all chunks at once); 0: the kernel does not cover the head sizes."""
    handle = lib()
    handle.ka_matrix_memory_chunks_scratch.restype = ctypes.c_long
    if not handle.ka_matrix_memory_chunks_supported(int(head_dim), int(value_dim)):
        return 0
    return int(handle.ka_matrix_memory_chunks_scratch(int(n), int(n_rows), int(n_heads), int(head_dim), int(value_dim)))


def matrix_memory_chunks_bf16(projected, offsets, pre, state, cu_q, row_slot, gain, out, n_heads, head_dim, value_dim,
                              q_scale, cap, eps, scratch=None) -> bool:
    """``ops.core.matrix_memory`` for prompt portions on the matrix cores: the recurrence unrolled over chunks of 64 tokens
    (operands as for ``ops.core.matrix_memory``, which has checked them). ``scratch`` (fp32, at least
    ``matrix_memory_chunks_scratch`` numbers): the chunks of every row run at once, in three passes, instead of in turn.
    False: head sizes or alignment not covered, nothing was run."""
    handle = lib()
    n = projected.shape[0]
    if n == 0:
        return True
    if projected.dtype != torch.bfloat16 or not handle.ka_matrix_memory_chunks_supported(int(head_dim), int(value_dim)):
        return False
    oq, ok, ov, og = offsets
    size, base = projected.element_size(), projected.data_ptr()
    stride = projected.stride(0) if n > 1 else projected.shape[1]
    if base % 16 or stride % 8 or any(o % 8 for o in (oq, ok, ov)) or (n_heads * head_dim) % 8:
        return False
    if scratch is not None:
        need = matrix_memory_chunks_scratch(n, int(row_slot.numel()), n_heads, head_dim, value_dim)
        if scratch.dtype != torch.float32 or not scratch.is_contiguous() or scratch.numel() < need:
            raise KernelError(f"matrix memory: the passes' scratch must be contiguous fp32 of at least {need} numbers")
    _check(handle.ka_matrix_memory_chunks_bf16(base + oq * size, base + ok * size, base + ov * size,
                                               None if og is None else base + og * size, stride, pre.data_ptr(), state.data_ptr(),
                                               cu_q.data_ptr(), row_slot.data_ptr(), _ptr(gain), out.data_ptr(),
                                               out.stride(0) if n > 1 else n_heads * value_dim, int(row_slot.numel()), n_heads,
                                               head_dim, value_dim, float(q_scale), float(cap), float(eps), _ptr(scratch), n, stream_ptr()))
    return True


def linear_attention_chunks_scratch(n: int, n_rows: int, n_heads: int, head_dim: int, value_dim: int) -> int:
    """fp32 numbers of scratch that ``linear_attention_chunks_bf16`` needs for a step of ``n`` tokens in ``n_rows`` rows; 0: the
    kernels do not cover the head sizes."""
    handle = lib()
    handle.ka_linear_chunks_scratch.restype = ctypes.c_long
    if not handle.ka_linear_chunks_supported(int(head_dim), int(value_dim)):
        return 0
    return int(handle.ka_linear_chunks_scratch(int(n), int(n_rows), int(n_heads), int(head_dim), int(value_dim)))


def linear_attention_chunks_bf16(projected, offsets, log2_decay, state, cu_q, row_slot, raw, n_heads, head_dim, value_dim, act, scratch) -> bool:
    """``ops.core.linear_attention`` for prompt portions on the matrix cores: the recurrence unrolled over chunks of 64 tokens, all
    chunks at once in three launches (operands as there, with the decays' logarithms to base 2; ``scratch``: contiguous fp32 of
    at least ``linear_attention_chunks_scratch`` numbers). False: sizes or alignment not covered, nothing was run."""
    handle = lib()
    n = projected.shape[0]
    if n == 0:
        return True
    n_rows = int(row_slot.numel())
    if projected.dtype != torch.bfloat16 or not handle.ka_linear_chunks_supported(int(head_dim), int(value_dim)):
        return False
    oq, ok, ov = (int(o) for o in offsets)
    size, base = projected.element_size(), projected.data_ptr()
    stride = projected.stride(0) if n > 1 else projected.shape[1]
    if base % 16 or stride % 8 or any(o % 8 for o in (oq, ok, ov)) or projected.stride(1) != 1 or state.stride(0) % 4 \
            or n // 64 + n_rows > 65535:
        return False
    need = linear_attention_chunks_scratch(n, n_rows, n_heads, head_dim, value_dim)
    for t, numbers, what in ((scratch, need, "scratch"), (raw, n * n_heads * value_dim, "read-outs"), (log2_decay, n_heads, "decays")):
        if t.dtype != torch.float32 or not t.is_contiguous() or t.numel() < numbers or not t.is_cuda:
            raise KernelError(f"linear attention: the {what} must be contiguous fp32 of at least {numbers} numbers")
    if max(oq + n_heads * head_dim, ok + n_heads * head_dim, ov + n_heads * value_dim) > projected.shape[1] \
            or state.dtype != torch.float32 or state.shape[1] != n_heads * head_dim * value_dim \
            or cu_q.dtype != torch.int32 or cu_q.numel() != n_rows + 1 or row_slot.dtype != torch.int32:
        raise KernelError("linear attention: operands do not fit the head sizes")
    _check(handle.ka_linear_chunks_bf16(base + oq * size, base + ok * size, base + ov * size, stride, log2_decay.data_ptr(), state.data_ptr(),
                                        state.stride(0), cu_q.data_ptr(), row_slot.data_ptr(), raw.data_ptr(), scratch.data_ptr(), n, n_rows,
                                        n_heads, head_dim, value_dim, int(act), stream_ptr()))
    return True


def gated_chunks_scratch(n: int, n_rows: int, n_heads: int, head_dim: int, value_dim: int) -> int:
    """fp32 numbers of scratch that ``gated_chunks_bf16`` needs for a step of ``n`` tokens in ``n_rows`` rows; 0: the kernels do not
    cover the head sizes."""
    handle = lib()
    handle.ka_gated_chunks_scratch.restype = ctypes.c_long
    if not handle.ka_gated_chunks_supported(int(head_dim), int(value_dim)):
        return 0
    return int(handle.ka_gated_chunks_scratch(int(n), int(n_rows), int(n_heads), int(head_dim), int(value_dim)))


def gated_chunks_bf16(projected, offsets, pre, tau, q_scale, state, cu_q, row_slot, raw, n_heads, head_dim, value_dim, scratch) -> bool:
    """``ops.core.gated_linear_attention`` for prompt portions on the matrix cores: the recurrence unrolled over chunks of 64 tokens, all
    chunks at once in three launches (operands as there; ``scratch``: contiguous fp32 of at least ``gated_chunks_scratch`` numbers).
    False: sizes or alignment not covered, nothing was run."""
    handle = lib()
    n = projected.shape[0]
    if n == 0:
        return True
    n_rows = int(row_slot.numel())
    if projected.dtype != torch.bfloat16 or not handle.ka_gated_chunks_supported(int(head_dim), int(value_dim)):
        return False
    oq, ok, ov = (int(o) for o in offsets)
    size, base = projected.element_size(), projected.data_ptr()
    stride = projected.stride(0) if n > 1 else max(projected.stride(0), projected.shape[1])
    if base % 16 or stride % 8 or any(o % 8 for o in (oq, ok, ov)) or projected.stride(1) != 1 or state.stride(0) % 4 or state.data_ptr() % 16 \
            or n // 64 + n_rows > 65535:
        return False
    need = gated_chunks_scratch(n, n_rows, n_heads, head_dim, value_dim)
    for t, numbers, what in ((scratch, need, "scratch"), (raw, n * n_heads * value_dim, "read-outs"), (pre, n * n_heads * head_dim, "pre-activations")):
        if t.dtype != torch.float32 or not t.is_contiguous() or t.numel() < numbers or not t.is_cuda:
            raise KernelError(f"gated linear attention: the {what} must be contiguous fp32 of at least {numbers} numbers")
    if max(oq + n_heads * head_dim, ok + n_heads * head_dim, ov + n_heads * value_dim) > projected.shape[1] or not tau > 0 \
            or state.dtype != torch.float32 or state.dim() != 2 or state.stride(1) != 1 or state.shape[1] != n_heads * head_dim * value_dim \
            or cu_q.dtype != torch.int32 or cu_q.numel() != n_rows + 1 or row_slot.dtype != torch.int32:
        raise KernelError("gated linear attention: operands do not fit the head sizes")
    _check(handle.ka_gated_chunks_bf16(base + oq * size, base + ok * size, base + ov * size, stride, pre.data_ptr(), float(tau), float(q_scale),
                                       state.data_ptr(), state.stride(0), cu_q.data_ptr(), row_slot.data_ptr(), raw.data_ptr(), scratch.data_ptr(),
                                       n, n_rows, n_heads, head_dim, value_dim, stream_ptr()))
    return True


def experts_few_bf16(h, pairs, down, chosen, hidden, y, act, clamp=None) -> bool:
    """Both linears of the chosen experts for a step of few pairs on the matrix cores, every chosen expert's weights read once: operands as
    ``experts_feed_forward_bf16`` takes them, with ``hidden`` bf16 ``[n top, hidden]`` (the pairs' own rows). False: not covered, nothing was run."""
    n, top = chosen.shape
    n_experts, n_pair_rows, dim = pairs.shape
    ff = down.shape[2]
    handle = lib()
    lda = h.stride(0) if n > 1 else max(h.stride(0), dim)
    core._dev(h, pairs, down, chosen, hidden, y)
    if h.dtype != torch.bfloat16 or h.data_ptr() % 16 or pairs.data_ptr() % 16 or down.data_ptr() % 16 or hidden.data_ptr() % 16 \
            or not handle.ka_experts_few_supported(n * top, lda, n_pair_rows, dim, act) or not handle.ka_experts_few_supported(n * top, ff, dim, ff, 0):
        return False
    if tuple(down.shape) != (n_experts, dim, ff) or n_pair_rows != (2 * ff if act & 0x100 else ff) or pairs.dtype != torch.bfloat16 or down.dtype != torch.bfloat16:
        raise KernelError("experts: weights of the two linears do not belong together")
    if y.dtype != torch.float32 or tuple(y.shape) != (n * top, dim) or not y.is_contiguous() or chosen.dtype != torch.int32 or not chosen.is_contiguous() \
            or hidden.dtype != torch.bfloat16 or tuple(hidden.shape) != (n * top, ff) or not hidden.is_contiguous():
        raise KernelError("experts: fp32 outputs [pairs, dim], bf16 hidden rows [pairs, hidden] and int32 choices [n, top] expected")
    _check(handle.ka_experts_few_bf16(h.data_ptr(), lda, top, pairs.data_ptr(), chosen.data_ptr(), n * top, n_experts, n_pair_rows, dim, act,
                                      *core._clamp_args(clamp, act), hidden.data_ptr(), ff, 0, stream_ptr()))
    _check(handle.ka_experts_few_bf16(hidden.data_ptr(), ff, 1, down.data_ptr(), chosen.data_ptr(), n * top, n_experts, dim, ff, 0,
                                      *core._clamp_args(None, 0), y.data_ptr(), dim, 1, stream_ptr()))
    return True


def experts_feed_forward_bf16(h, pairs, down, chosen, hidden, y, act, workspace, clamp=None) -> bool:
    """Both linears of the chosen experts for all pairs of a step on the matrix cores, an expert's pairs together: the pairs
    are listed by expert (``ops.core.experts_sort``), the first linear (gated or not, as ``act`` says) gathers every pair's token from ``h`` ``[n, dim]`` and
    leaves the hidden rows in list order, the second writes fp32 ``y`` ``[n top, dim]`` at the pairs' own rows. ``pairs``
    ``[E, 2 hidden, dim]`` (not gated: ``[E, hidden, dim]``), ``down`` ``[E, dim, hidden]``, ``chosen`` int32 ``[n, top]``; ``hidden`` is not used (the list's hidden rows
    live in the workspace). ``clamp`` (a ``GateClamp``): the pair's product is the clamped one. False: not covered (sizes that are no multiple of 16, alignment), nothing was run."""
    n, top = chosen.shape
    n_experts, n_pair_rows, dim = pairs.shape
    ff = down.shape[2]
    handle = lib()
    if h.dtype != torch.bfloat16 or pairs.dtype != torch.bfloat16 or down.dtype != torch.bfloat16 or y.dtype != torch.float32 \
            or h.stride(1) != 1 or not pairs.is_contiguous() or not down.is_contiguous() or not y.is_contiguous() \
            or h.data_ptr() % 16 or pairs.data_ptr() % 16 or down.data_ptr() % 16 or y.data_ptr() % 16:
        return False
    lda = h.stride(0) if n > 1 else dim
    act = int(act)
    if n_pair_rows != (2 * ff if act & ACT_GATED else ff):
        raise KernelError("experts: the first linear's rows do not fit the hidden size")
    if not handle.ka_experts_gemm_supported(lda, n_pair_rows, dim, ff, act, 0) or not handle.ka_experts_gemm_supported(ff, dim, ff, dim, 0, 1):
        return False
    tile = int(handle.ka_experts_gemm_tile())
    # (sized by the step's tokens alone: the same for every replay of a captured step)
    capacity = -(-(n * top + n_experts * (tile - 1)) // tile) * tile
    if capacity // tile > 65535:
        return False
    listed = workspace.get("experts.sorted", (capacity,), torch.int32)
    tile_expert = workspace.get("experts.tile_expert", (capacity // tile,), torch.int32)
    rows = workspace.get("experts.hidden_listed", (capacity, ff), torch.bfloat16)
    core.experts_sort(chosen.view(-1), n_experts, tile, listed, tile_expert)
    _check(handle.ka_experts_gemm_bf16(h.data_ptr(), lda, top, pairs.data_ptr(), listed.data_ptr(), tile_expert.data_ptr(), capacity // tile,
                                       n_pair_rows, dim, act, *core._clamp_args(clamp, act), rows.data_ptr(), ff, 0, 0, stream_ptr()))
    _check(handle.ka_experts_gemm_bf16(rows.data_ptr(), ff, 0, down.data_ptr(), listed.data_ptr(), tile_expert.data_ptr(), capacity // tile,
                                       dim, ff, 0, *core._clamp_args(None, 0), y.data_ptr(), dim, 1, 1, stream_ptr()))
    return True
