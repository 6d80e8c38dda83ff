"""Python face of the gfx950 kernel library: one function per kernel entry point.

Each function checks devices, dtypes and shapes on the host, then calls the flat C ABI
through ctypes on the current HIP stream. There is no CPU fallback: without the library
or without a GPU these functions raise.
"""

from __future__ import annotations

import ctypes
import os
import time
from typing import Dict, Optional

import torch

from . import build as _build

# (the last two: a storing product leaves gelu of its float32 sums; a gated product gelu_tanh(gate) * up)
F32, BF16, BF16_GELU, BF16_GEGLU = 0, 1, 2, 3
PAGE_SIZE = 64          # tokens per cache page: the width of a wavefront
MAX_HEAD_DIM = 256          # of the matrix-core attention kernels
MAX_PLAIN_HEAD_DIM = 1024   # of the plain attention kernels, which serve what the others do not take
ABI_VERSION = 18

_lib = None


class KernelError(RuntimeError):
    pass


class _ProfiledLibrary:
    """The kernel library with every call bracketed by two events on the current stream.
    Nothing is waited for at a launch (a host that waits lets the GPU's clock drop, which would
    rescale every figure): the events are read when the report is asked for, as the reference's
    per-kernel profile does (native/src/v2_runtime.cpp:27590-27728)."""
    CAPACITY = 1 << 16

    def __init__(self, lib):
        self._library = lib
        self._pending = []          # (name, first event, second event)
        self._totals: Dict[str, Dict[str, float]] = {}
        self.overflow = 0

    def __getattr__(self, name):
        entry = getattr(self._library, name)
        if not name.startswith("fw_") or name in ("fw_last_error", "fw_abi_version") or name.endswith(("_plan", "_fits", "_tiles")):
            return entry

        def timed(*args):
            if len(self._pending) >= self.CAPACITY or torch.cuda.is_current_stream_capturing():
                self.overflow += 1
                return entry(*args)
            first, second = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            first.record()
            began = time.perf_counter()
            status = entry(*args)
            host_ms = (time.perf_counter() - began) * 1e3
            second.record()
            self._pending.append((name, first, second))
            total = self._totals.setdefault(name, {"calls": 0, "gpu_ms": 0.0, "host_launch_ms": 0.0, "max_us": 0.0})
            total["calls"] += 1
            total["host_launch_ms"] += host_ms
            return status
        return timed

    def report(self) -> Dict[str, Dict[str, float]]:
        torch.cuda.synchronize()
        for name, first, second in self._pending:
            ms = first.elapsed_time(second)
            total = self._totals[name]
            total["gpu_ms"] += ms
            total["max_us"] = max(total["max_us"], ms * 1e3)
        self._pending = []
        return {name: dict(total) for name, total in sorted(self._totals.items(), key=lambda item: -item[1]["gpu_ms"])}


_profiled: Optional[_ProfiledLibrary] = None


def kernel_profile(enable: bool = True) -> None:
    """Switches the per-kernel profile on or off (also switched on by FLYWEIGHT_KERNEL_PROFILE=1
    in the environment, as in the reference). While it is on, steps are not recorded into graphs."""
    global _profiled
    if enable and _profiled is None:
        _profiled = _ProfiledLibrary(library())
    elif not enable:
        _profiled = None


def kernel_profile_active() -> bool:
    return _profiled is not None


def kernel_profile_report() -> Dict[str, Dict[str, float]]:
    """Entry point -> calls, GPU milliseconds between its two events, host milliseconds inside
    the launching call, the longest single call in microseconds; sorted by GPU time."""
    return _profiled.report() if _profiled is not None else {}


def library():
    """Loads (building first if nothing is built) the kernel library."""
    global _lib
    if _profiled is not None:
        return _profiled
    if _lib is None:
        path = _build.ensure_built()
        lib = ctypes.CDLL(path)
        lib.fw_last_error.restype = ctypes.c_char_p
        lib.fw_abi_version.restype = ctypes.c_int
        if lib.fw_abi_version() != ABI_VERSION:
            raise KernelError(f"{path}: kernel library ABI {lib.fw_abi_version()} != {ABI_VERSION}; rebuild it")
        _lib = lib
        if os.environ.get("FLYWEIGHT_KERNEL_PROFILE", "")[:1] == "1":
            kernel_profile(True)
            return _profiled
    return _lib


def library_path() -> str:
    library()
    return _lib._name


def _check(status: int) -> None:
    if status != 0:
        raise KernelError(library().fw_last_error().decode("utf-8", "replace"))


def _code(dtype: torch.dtype) -> int:
    if dtype == torch.float32:
        return F32
    if dtype == torch.bfloat16:
        return BF16
    raise KernelError(f"kernels take float32 or bfloat16, not {dtype}")


def _dev(*tensors: Optional[torch.Tensor]) -> None:
    for t in tensors:
        if t is None:
            continue
        if not t.is_cuda:
            raise KernelError("kernels run on the GPU only; got a CPU tensor")
        if not t.is_contiguous():
            raise KernelError("kernels need contiguous tensors")


def _dev_rows(t: torch.Tensor, name: str) -> None:
    """A matrix whose rows may lie apart (a view of some columns of wider rows), each row contiguous."""
    if not t.is_cuda:
        raise KernelError("kernels run on the GPU only; got a CPU tensor")
    if t.dim() != 2 or t.stride(1) != 1:
        raise KernelError(f"{name} must be a matrix with contiguous rows")


def _stride(t: torch.Tensor) -> int:
    """Elements between the rows of a matrix (of a single row: its width)."""
    return t.stride(0) if t.shape[0] > 1 else max(t.shape[1], t.stride(0))


def _p(t: Optional[torch.Tensor]) -> ctypes.c_void_p:
    return ctypes.c_void_p(0 if t is None else t.data_ptr())


_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)


def _stream() -> ctypes.c_void_p:
    """The current HIP stream of the current device (asked for at every launch: a graph
    capture or a caller's stream context changes it)."""
    if _raw_stream is not None:
        return ctypes.c_void_p(_raw_stream(torch.cuda.current_device()))
    return ctypes.c_void_p(torch.cuda.current_stream().cuda_stream)


def _want(t: torch.Tensor, dtype: torch.dtype, name: str) -> None:
    if t.dtype != dtype:
        raise KernelError(f"{name} must be {dtype}, found {t.dtype}")


# ---------------------------------------------------------------------------------------
def embed_rows(table: torch.Tensor, ids: torch.Tensor, out: Optional[torch.Tensor] = None, scale: float = 1.0,
               places_table: Optional[torch.Tensor] = None, places: Optional[torch.Tensor] = None, copies: int = 1) -> torch.Tensor:
    """table[ids] * scale as float32 rows (``copies`` > 1: [rows, copies, hidden], every row that many times); with ``places_table`` and ``places`` (int32, one per row, checked against
    the table by the caller) plus places_table[places], not scaled."""
    _dev(table, ids, out, places_table, places)
    _want(ids, torch.int32, "ids")
    vocab, hidden = table.shape
    if (places_table is None) != (places is None):
        raise KernelError("embed_rows: a table of places and the rows' places come together")
    if places is not None:
        _want(places, torch.int32, "places")
        if places_table.dim() != 2 or places_table.shape[1] != hidden or places.numel() < ids.numel():
            raise KernelError(f"embed_rows: the table of places is {tuple(places_table.shape)} beside rows of {hidden}, {places.numel()} places for {ids.numel()} rows")
    rows = ids.numel()
    if out is None:
        out = torch.empty((rows, hidden) if copies == 1 else (rows, copies, hidden), dtype=torch.float32, device=table.device)
    _want(out, torch.float32, "out")
    if copies < 1 or out.shape != ((rows, hidden) if copies == 1 else (rows, copies, hidden)):
        raise KernelError(f"embed_rows: out is {tuple(out.shape)}, expected {(rows, hidden)} ({copies} copies)")
    _check(library().fw_embed_rows(_p(table), _code(table.dtype), _p(ids), _p(out), rows, hidden, vocab,
                                   ctypes.c_float(scale), _p(places_table), _code(places_table.dtype) if places_table is not None else F32,
                                   _p(places), places_table.shape[0] if places_table is not None else 0, int(copies), _stream()))
    return out


def scale_softcap_(x: torch.Tensor, scale: float = 1.0, cap: float = 0.0) -> torch.Tensor:
    """In place on float32: x * scale, then with ``cap`` > 0 cap * tanh(x / cap)."""
    _dev(x)
    _want(x, torch.float32, "x")
    if cap < 0:
        raise KernelError("scale_softcap: the cap must not be negative")
    _check(library().fw_scale_softcap(_p(x), ctypes.c_longlong(x.numel()), ctypes.c_float(scale), ctypes.c_float(cap), _stream()))
    return x


def rmsnorm_rows(x: torch.Tensor, weight: torch.Tensor, eps: float, out_dtype: torch.dtype,
                 row_index: Optional[torch.Tensor] = None, one_centered: bool = False,
                 out: Optional[torch.Tensor] = None) -> torch.Tensor:
    _dev(x, weight, row_index, out)
    _want(x, torch.float32, "x")
    _want(weight, torch.float32, "weight")
    hidden = x.shape[-1]
    if weight.shape != (hidden,):
        raise KernelError(f"rmsnorm: weight is {tuple(weight.shape)}, row width is {hidden}")
    rows = x.numel() // hidden if row_index is None else row_index.numel()
    if row_index is not None:
        _want(row_index, torch.int32, "row_index")
    if out is None:
        out = torch.empty((rows, hidden), dtype=out_dtype, device=x.device)
    if out.shape != (rows, hidden) or out.dtype != out_dtype:
        raise KernelError("rmsnorm: out has the wrong shape or dtype")
    _check(library().fw_rmsnorm_rows(_p(x), _p(weight), _p(out), _code(out_dtype), _p(row_index), rows, hidden,
                                     ctypes.c_float(eps), int(one_centered), _stream()))
    return out


def gemm_generic(a: torch.Tensor, w: torch.Tensor, bias: Optional[torch.Tensor] = None,
                 out_dtype: Optional[torch.dtype] = None, accumulate_into: Optional[torch.Tensor] = None,
                 out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """a [M, K] . w [N, K]^T (+ bias). With ``accumulate_into`` (float32 [M, N]) the
    product is added to it in place: the residual sum in float32."""
    _dev(a, w, bias, accumulate_into, out)
    M, K = a.shape
    N, K2 = w.shape
    if K != K2:
        raise KernelError(f"gemm: a is {tuple(a.shape)} but w is {tuple(w.shape)}")
    if bias is not None:
        _want(bias, torch.float32, "bias")
        if bias.shape != (N,):
            raise KernelError(f"gemm: bias is {tuple(bias.shape)}, expected {(N,)}")
    if accumulate_into is not None:
        _want(accumulate_into, torch.float32, "accumulate_into")
        if accumulate_into.shape != (M, N):
            raise KernelError(f"gemm: destination is {tuple(accumulate_into.shape)}, expected {(M, N)}")
        target, mode, code = accumulate_into, 1, F32
    else:
        out_dtype = out_dtype or a.dtype
        if out is None:
            out = torch.empty((M, N), dtype=out_dtype, device=a.device)
        if out.shape != (M, N) or out.dtype != out_dtype:
            raise KernelError("gemm: out has the wrong shape or dtype")
        target, mode, code = out, 0, _code(out_dtype)
    _check(library().fw_gemm_generic(_p(a), _code(a.dtype), _p(w), _code(w.dtype), _p(bias), _p(target), code, mode,
                                     M, N, K, _stream()))
    return target


def swiglu(gate_up: torch.Tensor, out_dtype: Optional[torch.dtype] = None,
           out: Optional[torch.Tensor] = None, gelu: bool = False) -> torch.Tensor:
    """silu(gate) * up of [rows, gate | up] (``gelu``: the tanh form of gelu in place of silu); the input may be float32
    beside a bfloat16 output."""
    _dev(gate_up, out)
    out_dtype = out_dtype or gate_up.dtype
    rows, width = gate_up.shape
    if width % 2:
        raise KernelError("swiglu: the input holds gate and up halves; its width must be even")
    inter = width // 2
    if out is None:
        out = torch.empty((rows, inter), dtype=out_dtype, device=gate_up.device)
    if out.shape != (rows, inter) or out.dtype != out_dtype:
        raise KernelError("swiglu: out has the wrong shape or dtype")
    _check(library().fw_swiglu(_p(gate_up), _code(gate_up.dtype), _p(out), _code(out_dtype), rows, inter, int(gelu), _stream()))
    return out


def rope_table(positions: torch.Tensor, inv_freq: torch.Tensor):
    """cos and sin [rows, half] (float32) of position * inv_freq (float64)."""
    _dev(positions, inv_freq)
    _want(positions, torch.int32, "positions")
    _want(inv_freq, torch.float64, "inv_freq")
    rows, half = positions.numel(), inv_freq.numel()
    cos = torch.empty((rows, half), dtype=torch.float32, device=positions.device)
    sin = torch.empty_like(cos)
    _check(library().fw_rope_table(_p(positions), _p(inv_freq), _p(cos), _p(sin), rows, half, _stream()))
    return cos, sin


def query_temperature(positions: torch.Tensor, coef: float, every: int) -> torch.Tensor:
    """float32 [rows]: 1 + coef * ln(floor((position + 1) / every) + 1)."""
    _dev(positions)
    _want(positions, torch.int32, "positions")
    out = torch.empty((positions.numel(),), dtype=torch.float32, device=positions.device)
    _check(library().fw_query_temperature(_p(positions), _p(out), positions.numel(), ctypes.c_float(coef), int(every), _stream()))
    return out


def shortconv(bcx: torch.Tensor, taps: torch.Tensor, conv_bias: Optional[torch.Tensor], state: torch.Tensor,
              row_seg: torch.Tensor, seg_row0: torch.Tensor, seg_slot: torch.Tensor, segments: int,
              out_dtype: Optional[torch.dtype] = None, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """state [slots, H, L-1] is read and updated in place. ``bcx`` may be float32 beside a
    bfloat16 output."""
    _dev(bcx, taps, conv_bias, state, row_seg, seg_row0, seg_slot, out)
    out_dtype = out_dtype or bcx.dtype
    rows, width = bcx.shape
    hidden, kernel = taps.shape
    if width != 3 * hidden:
        raise KernelError(f"shortconv: input width {width} is not 3 x {hidden}")
    _want(taps, torch.float32, "taps")
    _want(state, torch.float32, "state")
    if state.dim() != 3 or state.shape[1:] != (hidden, kernel - 1):
        raise KernelError(f"shortconv: state is {tuple(state.shape)}, expected [slots, {hidden}, {kernel - 1}]")
    if conv_bias is not None:
        _want(conv_bias, torch.float32, "conv_bias")
        if conv_bias.shape != (hidden,):
            raise KernelError("shortconv: bias has the wrong shape")
    for name, t, n in (("row_seg", row_seg, rows), ("seg_row0", seg_row0, segments + 1), ("seg_slot", seg_slot, segments)):
        _want(t, torch.int32, name)
        if t.numel() < n:
            raise KernelError(f"shortconv: {name} holds {t.numel()} entries, needs {n}")
    if out is None:
        out = torch.empty((rows, hidden), dtype=out_dtype, device=bcx.device)
    if out.shape != (rows, hidden) or out.dtype != out_dtype:
        raise KernelError("shortconv: out has the wrong shape or dtype")
    _check(library().fw_shortconv(_p(bcx), _code(bcx.dtype), _p(out), _code(out_dtype), _p(taps), _p(conv_bias), _p(state), _p(row_seg),
                                  _p(seg_row0), _p(seg_slot), rows, segments, hidden, kernel, state.shape[0], _stream()))
    return out


def _check_pages(k_pages: torch.Tensor, v_pages: torch.Tensor, kv_heads: int, head_dim: int, dtype: torch.dtype,
                 v_dim: Optional[int] = None):
    pages = k_pages.shape[0]
    v_dim = head_dim if v_dim is None else v_dim
    if k_pages.shape != (pages, kv_heads, PAGE_SIZE, head_dim):
        raise KernelError(f"K pages are {tuple(k_pages.shape)}, expected [pages, {kv_heads}, {PAGE_SIZE}, {head_dim}]")
    if v_pages.shape != (pages, kv_heads, v_dim, PAGE_SIZE):
        raise KernelError(f"V pages are {tuple(v_pages.shape)}, expected [pages, {kv_heads}, {v_dim}, {PAGE_SIZE}]")
    if k_pages.dtype != dtype or v_pages.dtype != dtype:
        raise KernelError(f"cache pages are {k_pages.dtype}/{v_pages.dtype} but activations are {dtype}")
    return pages


def qk_norm_rope_kv_write(qkv: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int,
                          q_norm_weight: Optional[torch.Tensor], k_norm_weight: Optional[torch.Tensor], eps: float,
                          cos: Optional[torch.Tensor], sin: Optional[torch.Tensor], rotary_dim: int,
                          k_pages: torch.Tensor, v_pages: torch.Tensor, block_table: torch.Tensor,
                          row_seg: torch.Tensor, row_pos: torch.Tensor, write_kv: bool = True,
                          v_dim: Optional[int] = None, interleaved: bool = False, q_only: bool = False,
                          q_row_scale: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The output and the cache take the pages' dtype; ``qkv`` may be float32 beside bfloat16 pages, and its rows may lie
    apart (some columns of wider rows).
    ``q_row_scale`` (float32 [rows]): a factor on each row's finished queries.
    ``v_dim``: the size of a value head where it is not ``head_dim``. ``interleaved``: channel 2i turns
    with channel 2i + 1 instead of channel i with channel i + rotary_dim / 2."""
    _dev(q_norm_weight, k_norm_weight, cos, sin, k_pages, v_pages, block_table, row_seg, row_pos)
    _dev_rows(qkv, "qkv")
    rows, width = qkv.shape
    v_dim = head_dim if v_dim is None else int(v_dim)
    expected = num_heads * head_dim if q_only else (num_heads + num_kv_heads) * head_dim + num_kv_heads * v_dim
    if width != expected or (q_only and write_kv):
        raise KernelError(f"qk_norm_rope: qkv width {width} != {expected} (queries alone: {q_only}; they bring nothing to store)")
    pages = _check_pages(k_pages, v_pages, num_kv_heads, head_dim, k_pages.dtype, v_dim)
    for w in (q_norm_weight, k_norm_weight):
        if w is not None:
            _want(w, torch.float32, "norm weight")
            if w.shape != (head_dim,):
                raise KernelError("qk_norm_rope: a head norm weight must be [head_dim]")
    if rotary_dim:
        for t in (cos, sin):
            _want(t, torch.float32, "rotation table")
            if t.shape != (rows, rotary_dim // 2):
                raise KernelError(f"qk_norm_rope: rotation table is {tuple(t.shape)}, expected {(rows, rotary_dim // 2)}")
    _want(block_table, torch.int32, "block_table")
    _want(row_seg, torch.int32, "row_seg")
    _want(row_pos, torch.int32, "row_pos")
    if block_table.dim() != 2 or row_seg.numel() < rows or row_pos.numel() < rows:
        raise KernelError("qk_norm_rope: batch index arrays are too short")
    q_out = torch.empty((rows, num_heads * head_dim), dtype=k_pages.dtype, device=qkv.device)
    _row_scale(q_row_scale, rows)
    _check(library().fw_qk_norm_rope_kv_write(
        _p(qkv), _code(qkv.dtype), _stride(qkv), _p(q_out), _code(k_pages.dtype), _p(q_norm_weight), _p(k_norm_weight), ctypes.c_float(eps), _p(cos), _p(sin),
        rotary_dim, _p(k_pages), _p(v_pages), _p(block_table), block_table.shape[1], _p(row_seg), _p(row_pos), rows,
        num_heads, num_kv_heads, head_dim, v_dim, PAGE_SIZE, pages, int(write_kv), int(interleaved), int(q_only), _p(q_row_scale), _stream()))
    return q_out


def _row_scale(q_row_scale: Optional[torch.Tensor], rows: int) -> None:
    if q_row_scale is not None:
        _dev(q_row_scale)
        _want(q_row_scale, torch.float32, "q_row_scale")
        if q_row_scale.numel() < rows:
            raise KernelError(f"a factor per row: {q_row_scale.numel()} for {rows} rows")


def _sinks(sinks: Optional[torch.Tensor], num_heads: int, keep_first: int, window: int, chunk: int,
           slopes: Optional[torch.Tensor] = None):
    """Checks what the mask and the softmax take beyond a window: ``keep_first`` first keys that stay seen
    (beside a window only), one more term exp(sinks[head]) in the denominator (float32 [heads]) and a bias by
    distance (``slopes`` float32 [heads]: slopes[head] * (row's position - key's position) is taken off a score)."""
    if slopes is not None:
        _dev(slopes)
        _want(slopes, torch.float32, "slopes")
        if slopes.shape != (num_heads,):
            raise KernelError(f"attention: slopes are {tuple(slopes.shape)}, expected one per head ({num_heads})")
    if keep_first < 0 or (keep_first and chunk):
        raise KernelError(f"attention: {keep_first} first keys are kept beside a window, not beside chunks")
    if sinks is not None:
        _dev(sinks)
        _want(sinks, torch.float32, "sinks")
        if sinks.shape != (num_heads,):
            raise KernelError(f"attention: sinks are {tuple(sinks.shape)}, expected one per head ({num_heads})")
    return int(keep_first) if window else 0, _p(sinks), _p(slopes)


def attention_generic(q: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int, k_pages: torch.Tensor,
                      v_pages: torch.Tensor, block_table: torch.Tensor, row_seg: torch.Tensor, row_pos: torch.Tensor,
                      scale: float, window: int = 0, v_dim: Optional[int] = None, chunk: int = 0,
                      softcap: float = 0.0, keep_first: int = 0, sinks: Optional[torch.Tensor] = None,
                      slopes: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``v_dim``: the size of a value head (and of a head's output) where it is not ``head_dim``.
    ``chunk`` > 0: a row sees only the keys of its own chunk of that many positions; ``softcap`` c > 0:
    score <- c tanh(score / c)."""
    _dev(q, k_pages, v_pages, block_table, row_seg, row_pos)
    rows = q.shape[0]
    v_dim = head_dim if v_dim is None else int(v_dim)
    if q.shape != (rows, num_heads * head_dim):
        raise KernelError(f"attention: q is {tuple(q.shape)}, expected {(rows, num_heads * head_dim)}")
    pages = _check_pages(k_pages, v_pages, num_kv_heads, head_dim, q.dtype, v_dim)
    _want(block_table, torch.int32, "block_table")
    _want(row_seg, torch.int32, "row_seg")
    _want(row_pos, torch.int32, "row_pos")
    if block_table.dim() != 2 or row_seg.numel() < rows or row_pos.numel() < rows:
        raise KernelError("attention: batch index arrays are too short")
    out = torch.empty((rows, num_heads * v_dim), dtype=q.dtype, device=q.device)
    _check(library().fw_attention_generic(
        _p(q), _p(out), _code(q.dtype), _p(k_pages), _p(v_pages), _p(block_table), block_table.shape[1], _p(row_seg),
        _p(row_pos), rows, num_heads, num_kv_heads, head_dim, v_dim, ctypes.c_float(scale), int(window), int(chunk),
        ctypes.c_float(softcap), *_sinks(sinks, num_heads, keep_first, window, chunk, slopes), PAGE_SIZE, pages, _stream()))
    return out


def argmax_rows(logits: torch.Tensor, out: Optional[torch.Tensor] = None, also: Optional[torch.Tensor] = None,
                advance: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The id of each row's largest logit (ties: the lowest id), int32 [rows], into ``out`` if
    given and into ``also`` as well; ``advance[r]`` goes up by one (all contiguous int32 of at
    least ``rows`` elements)."""
    _dev(logits)
    _want(logits, torch.float32, "logits")
    rows, vocab = logits.shape
    ids = out if out is not None else torch.empty((rows,), dtype=torch.int32, device=logits.device)
    for name, target in (("out", out), ("also", also), ("advance", advance)):
        if target is not None:
            _dev(target)
            _want(target, torch.int32, name)
            if target.numel() < rows or not target.is_contiguous():
                raise KernelError(f"argmax_rows: {name} must be contiguous and hold {rows} ids")
    workspace = torch.empty((max(rows, 1), 64), dtype=torch.int64, device=logits.device)       # best key of each part
    _check(library().fw_argmax_rows(_p(logits), _p(ids), _p(also), _p(advance), _p(workspace), rows, vocab, _stream()))
    return ids


def sample_rows(logits: torch.Tensor, settings: torch.Tensor, states: torch.Tensor, out: Optional[torch.Tensor] = None,
                also: Optional[torch.Tensor] = None, advance: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The next token of every row, drawn on the device (fw_sample_rows): ``settings`` float32
    [rows, 4] = temperature (0: greedy), top_k (0: all), top_p, min_p; ``states`` int64 [rows], the
    rows' xorshift64* generators, moved on in place by the rows that draw. ``out`` / ``also`` /
    ``advance`` as for ``argmax_rows``."""
    _dev(logits, settings, states)
    _want(logits, torch.float32, "logits")
    _want(settings, torch.float32, "settings")
    _want(states, torch.int64, "states")
    rows, vocab = logits.shape
    if settings.numel() < 4 * rows or states.numel() < rows or not settings.is_contiguous() or not states.is_contiguous():
        raise KernelError(f"sample_rows: settings must hold [{rows}, 4] and states [{rows}], contiguous")
    ids = out if out is not None else torch.empty((rows,), dtype=torch.int32, device=logits.device)
    for name, target in (("out", out), ("also", also), ("advance", advance)):
        if target is not None:
            _dev(target)
            _want(target, torch.int32, name)
            if target.numel() < rows or not target.is_contiguous():
                raise KernelError(f"sample_rows: {name} must be contiguous and hold {rows} ids")
    _check(library().fw_sample_rows(_p(logits), _p(settings), _p(states), _p(ids), _p(also), _p(advance), rows, vocab, _stream()))
    return ids


def fill_zero(t: torch.Tensor) -> None:
    _dev(t)
    _check(library().fw_fill_zero(_p(t), ctypes.c_longlong(t.numel() * t.element_size()), _stream()))


def fill_zero_pieces(first: torch.Tensor, pieces: int, stride_bytes: int) -> None:
    """Clears ``pieces`` runs of memory the size of ``first`` (contiguous), ``stride_bytes`` apart,
    beginning with ``first`` itself: the caller vouches that all of them lie in one allocation."""
    _dev(first)
    _check(library().fw_fill_zero_pieces(_p(first), int(pieces), ctypes.c_longlong(first.numel() * first.element_size()),
                                         ctypes.c_longlong(int(stride_bytes)), _stream()))


def gather_rows(rows: torch.Tensor, index: torch.Tensor) -> torch.Tensor:
    """rows[index] for float32 rows and an int32 index on the device (the embedding kernel: a
    table of rows is a table of rows)."""
    return embed_rows(rows, index)


def _fast_gemm(a: torch.Tensor, w: torch.Tensor, bias, target: torch.Tensor, out_code: int, mode: int, N: int,
               w_tiled: Optional[torch.Tensor] = None) -> None:
    """bfloat16 operands on the matrix cores: the skinny kernel for up to 16 rows, the medium one
    (K split over workgroups) for up to 64, the tiled ones beyond (large tiles where they fill the
    chip, K cut into slices where even the small tiles are too few)."""
    M, K = a.shape
    if SKINNY_MAX_ROWS < M <= MEDIUM_MAX_ROWS or (M <= SKINNY_MAX_ROWS and w.numel() >= MEDIUM_LARGE and K % 8 == 0):
        # also a few rows of a large W (a vocabulary's head: 65,536 x 2,048 at 8 rows 52 against 61 us)
        if out_code == BF16_GEGLU:      # that product is told by its unit, not by the output's type
            gemm_medium_into(a, w, bias, target, BF16, mode, N, w_tiled=w_tiled, glu=GEGLU)
        else:
            gemm_medium_into(a, w, bias, target, out_code, mode, N, w_tiled=w_tiled)
        return
    if M <= SKINNY_MAX_ROWS:
        entry = library().fw_gemm_skinny
    elif M > BIG_MIN_ROWS and library().fw_gemm_mfma_big_tiles(mode, M, N, K) >= BIG_TILES_MIN:
        entry = library().fw_gemm_mfma_big      # enough 256 x 256 tiles to fill the chip
    elif K >= (DEEP_MIN_K if mode == 1 else DEEP_MIN_K_STORE) and _deep_columns(mode, M, N, K):
        # whole rounds of one tile per compute unit: the waves split K
        _check(library().fw_gemm_mfma_deep(_p(a), _p(w), _p(bias), _p(target), out_code, mode, M, N, K,
                                           _deep_columns(mode, M, N, K), _stream()))
        return
    elif _deep_columns_few_rows(mode, M, N, K, one_round=True):
        _check(library().fw_gemm_mfma_deep(_p(a), _p(w), _p(bias), _p(target), out_code, mode, M, N, K,
                                           _deep_columns_few_rows(mode, M, N, K), _stream()))
        return
    elif M > BIG_MIN_ROWS and _big_tiles_store_well(mode, M, N, K):
        entry = library().fw_gemm_mfma_big      # fewer large tiles than compute units, but every other way takes two rounds
    elif _deep_columns_few_rows(mode, M, N, K):
        _check(library().fw_gemm_mfma_deep(_p(a), _p(w), _p(bias), _p(target), out_code, mode, M, N, K,
                                           _deep_columns_few_rows(mode, M, N, K), _stream()))
        return
    else:
        need_bytes, need_counters = ctypes.c_size_t(0), ctypes.c_int(0)
        _check(library().fw_gemm_mfma_split_plan(mode, M, N, K, ctypes.byref(need_bytes), ctypes.byref(need_counters)))
        if need_bytes.value:                    # fewer tiles than compute units: K is cut into slices
            workspace = torch.empty(need_bytes.value // 4, dtype=torch.float32, device=a.device)
            counters = _medium_counters(a.device, need_counters.value)
            _check(library().fw_gemm_mfma_split(_p(a), _p(w), _p(bias), _p(target), out_code, mode, M, N, K, _p(workspace),
                                                ctypes.c_size_t(need_bytes.value), _p(counters), counters.numel(), _stream()))
            return
        entry = library().fw_gemm_mfma
    _check(entry(_p(a), _p(w), _p(bias), _p(target), out_code, mode, M, N, K, _stream()))


SKINNY_MAX_ROWS = 16
MEDIUM_MAX_ROWS = 64
MEDIUM_LARGE = 1 << 25    # weights from which the medium product beats the skinny one at any number of rows
BIG_TILES_MIN = 192      # 256 x 256 tiles from which the large-tile prompt product is used (256 compute units)
DEEP_MIN_K = 1024         # adding into the residual (2,048 x 2,048 x 2,048: 31 vs 39 us; x 8,192: 83 vs 118 us; 2,048 x 1,024 x 1,024: 13 vs 15 us)
DEEP_MIN_K_STORE = 4096   # storing: no old values travel during the exchange at a tile's end, a short K gains nothing
DEEP_ROUND = 256          # tiles of a round: one per compute unit
DEEP_FILL = 0.85          # least share of the rounds' places that the tiles must fill (640 narrow tiles, 0.83: 193 vs 189 us)
# adding into the residual, 2,048 features: 144 wide tiles (1,152 rows) K 8,192 72 vs 103 us, K 2,048 28 vs 35 us; 160
# narrow tiles (576 rows) 46 vs 65 us and 16.5 vs 27 us; 576 narrow (2,304 rows) 120 vs 135 us; 128 narrow tiles lose
DEEP_FILL_ADDING = 0.55


def _round_fill(tiles: int) -> float:
    """The share of the places in whole rounds over the chip that the tiles fill."""
    rounds = -(-tiles // DEEP_ROUND)
    return tiles / (rounds * DEEP_ROUND) if tiles > 0 else 0.0


def _deep_columns(mode: int, M: int, N: int, K: int) -> int:
    """The width of the tiles whose waves split K that serves this shape: the width (128 or 64
    columns) whose tiles fill their rounds over the chip better, the wider at a tie, if they fill
    enough of them; else 0. A product that adds into the residual needs less (the other kernels
    ask for the old values at the end of a tile, where nothing hides the read)."""
    fills = {columns: _round_fill(library().fw_gemm_mfma_deep_tiles(mode, M, N, K, columns)) for columns in (128, 64)}
    columns = 128 if fills[128] >= fills[64] else 64
    return columns if fills[columns] >= (DEEP_FILL_ADDING if mode == 1 else DEEP_FILL) else 0


DEEP_FEW_ROWS = 512       # up to here the tiles whose waves split K also serve a short K, if they are not too few
DEEP_FEW_TILES_WIDE = 192   # tiles of 128 columns from which those are taken, else
DEEP_FEW_TILES = 96       # tiles of 64 columns from which those are


BIG_TILES_MIN_STORE = 96      # large tiles from which a storing product takes them, if the output fills
BIG_FILL_STORE = 0.95         # at least this share of them


def _big_tiles_store_well(mode: int, M: int, N: int, K: int) -> bool:
    """A storing product that no kernel serves in one round of small tiles takes the large
    tiles from 96 of them on if they are well filled: 768 x 3,072 (K 1,024) 18.7 -> 14.9 us,
    512 x 4,608 21.1 -> 14.6 us, 1,024 x 3,072 (K 2,048) 29.5 -> 25.0 us; 2,048 x 1,024 (96 tiles
    of 192 columns, an eighth of them outside the output) would lose, 14.1 -> 17.5 us."""
    if mode != 0:
        return False
    rows, columns = ctypes.c_int(0), ctypes.c_int(0)
    tiles = library().fw_gemm_mfma_big_plan(mode, M, N, K, ctypes.byref(rows), ctypes.byref(columns))
    return tiles >= BIG_TILES_MIN_STORE and M * N >= BIG_FILL_STORE * tiles * rows.value * columns.value


def _deep_columns_few_rows(mode: int, M: int, N: int, K: int, one_round: bool = False) -> int:
    """A few hundred rows (decode steps of that many requests, short prompts) give the 128 x 128
    tiles of the register-staged product less than a round over the chip; the tiles whose waves
    split K bring their operands straight into LDS, three slabs ahead, and a workgroup alone on
    its compute unit keeps them coming. Measured against the products they replace, 8 in a row:
    storing 6,144 features at 256 rows 16.0 vs 21.0 us, at 128 rows 15.0 vs 18.6; 3,072 features at
    256 rows 15.0 vs 18.6, at 512 rows 15.9 vs 21.0 us; adding 2,048 features (K 2,048) at 512 rows
    16.2 vs 23.0 us, at 320 rows 15.7 vs 21.5 us. With a long K (8,192) the product that cuts K over
    workgroups is level with them."""
    if mode not in (0, 1) or M > DEEP_FEW_ROWS or K > (LONG_K if mode == 1 else 1 << 30):
        return 0
    wide = library().fw_gemm_mfma_deep_tiles(mode, M, N, K, 128)
    narrow = library().fw_gemm_mfma_deep_tiles(mode, M, N, K, 64)
    if mode == 0 and DEEP_FEW_TILES_WIDE <= wide <= DEEP_ROUND:
        return 128
    if DEEP_FEW_TILES <= narrow <= (1 if one_round else 2) * DEEP_ROUND:
        return 64
    return 0


BIG_MIN_ROWS = 128       # up to here a 256-row tile would be at least half empty (the head at 128 rows: 110 vs 78 us)
_MEDIUM_COUNTERS = {}


TICKET_COUNTERS = 1 << 20      # 4 MB per device


def _medium_counters(device: torch.device, count: int) -> torch.Tensor:
    """Zeroed int32 counters for the tickets of the kernels whose last workgroup finishes the
    work of the others (the medium product, decode attention), one set per device: each kernel
    leaves them at zero, and calls on one device follow each other in stream order (work on
    several streams of one device at once would need a set per stream). The set is allocated
    once and never replaced: recorded graphs hold its address."""
    have = _MEDIUM_COUNTERS.get(device.index)
    if have is None:
        if torch.cuda.is_current_stream_capturing():
            raise KernelError("the ticket counters must exist before a graph is captured (prepare_device)")
        have = _MEDIUM_COUNTERS[device.index] = torch.zeros(TICKET_COUNTERS, dtype=torch.int32, device=device)
    if count > have.numel():
        raise KernelError(f"a kernel asks for {count} ticket counters; the device's set holds {have.numel()}")
    return have


def prepare_device(device: torch.device) -> None:
    """Allocates what kernels keep between calls on this device; a model does this when its
    weights arrive, so that nothing is allocated for the first time inside a graph capture."""
    _medium_counters(torch.device(device), 0)


def tile_weights(w: torch.Tensor) -> Optional[torch.Tensor]:
    """``w`` [rows, K] bfloat16 once more in operand tiles, [ceil(rows / 16), K / 32, 4, 16, 8]: what the
    decode products read as whole contiguous kilobytes per wave (see fw_gemm_decode). None where the
    layout does not apply (K no multiple of 32, another dtype)."""
    if w.dtype != torch.bfloat16 or w.dim() != 2 or w.shape[1] % 32 or not w.is_cuda:
        return None
    rows, K = w.shape
    padded = (rows + 15) // 16 * 16
    if padded != rows:
        w = torch.cat([w, torch.zeros((padded - rows, K), dtype=w.dtype, device=w.device)])
    return w.view(padded // 16, 16, K // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous()


def _tiled_for(w: torch.Tensor, w_tiled: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
    """``w_tiled`` if it is ``w`` in operand tiles (checked by its shape), else an error."""
    if w_tiled is None:
        return None
    rows, K = w.shape
    if (w_tiled.dtype != torch.bfloat16 or K % 32 or tuple(w_tiled.shape) != ((rows + 15) // 16, K // 32, 4, 16, 8)
            or not w_tiled.is_contiguous() or w_tiled.device != w.device):
        raise KernelError(f"weights in operand tiles for w {tuple(w.shape)} are bfloat16 [{(rows + 15) // 16}, {K // 32}, 4, 16, 8], "
                          f"found {tuple(w_tiled.shape)}")
    return w_tiled


def gemm_medium_into(a: torch.Tensor, w: torch.Tensor, bias, target: torch.Tensor, out_code: int, mode: int, N: int,
                     next_norm_weight: Optional[torch.Tensor] = None, next_one_centered: bool = False,
                     squares: Optional[torch.Tensor] = None, eps: float = 0.0, w_tiled: Optional[torch.Tensor] = None,
                     glu: Optional[tuple] = None):
    """The product for 1..64 rows with K split over workgroups (fw_gemm_medium). With
    ``squares`` ``a`` holds prepared activations (x * w of an RMS norm) and the rows' 1/rms is
    formed from those sums. With ``next_norm_weight`` (accumulating product) returns what the
    norm after it needs: (activations x * w_next, sums of squares)."""
    M, K = a.shape
    need_bytes, need_counters, squares_rows = ctypes.c_size_t(0), ctypes.c_int(0), ctypes.c_int(0)
    _check(library().fw_gemm_medium_plan(M, N, K, mode, ctypes.byref(need_bytes), ctypes.byref(need_counters),
                                         ctypes.byref(squares_rows)))
    workspace = counters = next_activations = next_squares = None
    if need_bytes.value:
        workspace = torch.empty(need_bytes.value // 4, dtype=torch.float32, device=a.device)
        counters = _medium_counters(a.device, need_counters.value)
    stride = 16 if M <= DECODE_MAX_ROWS else 64
    if next_norm_weight is not None:
        next_activations = torch.empty((M, N), dtype=torch.bfloat16, device=a.device)
        next_squares = torch.empty((squares_rows.value, stride), dtype=torch.float32, device=a.device)
    if squares is not None and (squares.dtype != torch.float32 or squares.dim() != 2 or squares.shape[1] != stride
                                or not squares.is_contiguous()):
        raise KernelError(f"gemm_medium: sums of squares for {M} rows are float32 [n, {stride}]")
    w_tiled = _tiled_for(w, w_tiled)
    _check(library().fw_gemm_medium(_p(a), _p(w if w_tiled is None else w_tiled), int(w_tiled is not None), _p(bias), _p(target), out_code, mode, M, N, K, _p(workspace),
                                    ctypes.c_size_t(need_bytes.value), _p(counters),
                                    0 if counters is None else counters.numel(), _p(next_norm_weight),
                                    int(next_one_centered), _p(next_activations), _p(next_squares), _p(squares),
                                    0 if squares is None else squares.shape[0], ctypes.c_float(eps), *_glu(glu), _stream()))
    if next_norm_weight is not None:
        return next_activations, next_squares
    return None


def gemm_medium(a: torch.Tensor, w: torch.Tensor, epilogue: int, *, bias: Optional[torch.Tensor] = None,
                out_dtype: Optional[torch.dtype] = None, accumulate_into: Optional[torch.Tensor] = None,
                squares: Optional[torch.Tensor] = None, eps: float = 0.0,
                next_norm_weight: Optional[torch.Tensor] = None, next_one_centered: bool = False,
                w_tiled: Optional[torch.Tensor] = None, glu: Optional[tuple] = None, gelu: bool = False):
    """The medium product with the fused decode product's conventions (EPILOGUE_STORE /
    ACCUMULATE / SWIGLU): returns the output, or for an accumulation with ``next_norm_weight``
    what the norm after it needs. ``glu`` (with EPILOGUE_SWIGLU): (limit, alpha, shift) of a gated
    unit with clamped halves instead of SwiGLU."""
    _dev(a, w, bias, accumulate_into, squares, next_norm_weight)
    _want(a, torch.bfloat16, "a")
    _want(w, torch.bfloat16, "w")
    M, K = a.shape
    kinds = 2 if epilogue == EPILOGUE_SWIGLU else 1
    if not 1 <= M <= MEDIUM_MAX_ROWS or w.shape[1] != K or w.shape[0] % kinds or K % 8 or epilogue not in (0, 1, 2):
        raise KernelError(f"gemm_medium: a is {tuple(a.shape)}, w is {tuple(w.shape)}, epilogue {epilogue}")
    N = w.shape[0] // kinds
    if bias is not None and (bias.dtype != torch.float32 or bias.shape != (w.shape[0],)):
        raise KernelError("gemm_medium: bias must be float32, one entry per row of w")
    if next_norm_weight is not None and (epilogue != EPILOGUE_ACCUMULATE or next_norm_weight.dtype != torch.float32
                                         or next_norm_weight.shape != (N,)):
        raise KernelError("gemm_medium: only the accumulating product prepares the next norm, whose weight is float32 [N]")
    if epilogue == EPILOGUE_ACCUMULATE:
        _want(accumulate_into, torch.float32, "accumulate_into")
        if accumulate_into.shape != (M, N):
            raise KernelError(f"gemm_medium: destination is {tuple(accumulate_into.shape)}, expected {(M, N)}")
        left = gemm_medium_into(a, w, bias, accumulate_into, F32, 1, N, next_norm_weight, next_one_centered, squares, eps, w_tiled=w_tiled)
        return accumulate_into if left is None else left
    out_dtype = torch.bfloat16 if epilogue == EPILOGUE_SWIGLU else (out_dtype or torch.bfloat16)
    out = torch.empty((M, N), dtype=out_dtype, device=a.device)
    if gelu and (epilogue != EPILOGUE_STORE or out_dtype != torch.bfloat16):
        raise KernelError("gemm_medium: gelu goes with a storing product of bfloat16")
    gemm_medium_into(a, w, bias, out, BF16_GELU if gelu else _code(out_dtype), epilogue, N, squares=squares, eps=eps, w_tiled=w_tiled, glu=glu)
    return out


def gemm_deep(a: torch.Tensor, w: torch.Tensor, bias: Optional[torch.Tensor] = None,
              out_dtype: Optional[torch.dtype] = None, accumulate_into: Optional[torch.Tensor] = None,
              columns: int = 128) -> torch.Tensor:
    """a [M, K] . w [N, K]^T (+ bias) on 128 x 128 tiles whose waves split K (fw_gemm_mfma_deep),
    whatever the dispatch of ``gemm`` would choose: bfloat16 operands, K a multiple of 64."""
    _dev(a, w, bias, accumulate_into)
    _want(a, torch.bfloat16, "a")
    _want(w, torch.bfloat16, "w")
    M, K = a.shape
    N = w.shape[0]
    if w.shape[1] != K or (bias is not None and (bias.dtype != torch.float32 or bias.shape != (N,))):
        raise KernelError(f"gemm_deep: a is {tuple(a.shape)}, w is {tuple(w.shape)}; bias is float32 [N]")
    if accumulate_into is not None:
        _want(accumulate_into, torch.float32, "accumulate_into")
        if accumulate_into.shape != (M, N):
            raise KernelError(f"gemm_deep: destination is {tuple(accumulate_into.shape)}, expected {(M, N)}")
        target, mode = accumulate_into, 1
    else:
        target, mode = torch.empty((M, N), dtype=out_dtype or a.dtype, device=a.device), 0
    _check(library().fw_gemm_mfma_deep(_p(a), _p(w), _p(bias), _p(target), _code(target.dtype), mode, M, N, K, int(columns), _stream()))
    return target


def _fast_ok(a: torch.Tensor, w: torch.Tensor) -> bool:
    return (a.dtype == torch.bfloat16 and w.dtype == torch.bfloat16 and a.shape[0] >= 1 and a.shape[1] % 8 == 0
            and a.data_ptr() % 16 == 0 and w.data_ptr() % 16 == 0)


# ---- dispatch: which kernel serves a call ------------------------------------------------
def gemm(a: torch.Tensor, w: torch.Tensor, bias: Optional[torch.Tensor] = None,
         out_dtype: Optional[torch.dtype] = None, accumulate_into: Optional[torch.Tensor] = None,
         w_tiled: Optional[torch.Tensor] = None, gelu: bool = False) -> torch.Tensor:
    """a [M, K] . w [N, K]^T (+ bias): bfloat16 operands go to the matrix-core kernels,
    everything else (float32, mixed) to the generic float32 one. ``w_tiled``: ``w`` once more in
    operand tiles (``tile_weights``), for the kernels of few rows that read it so. ``gelu``: the error-function gelu of
    the float32 sums, rounded once (the matrix-core products form it as they store)."""
    if gelu and accumulate_into is not None:
        raise KernelError("gemm: gelu goes with a product that stores")
    if gelu and (not _fast_ok(a, w) or (out_dtype or a.dtype) != torch.bfloat16):
        return gelu_rows(gemm(a, w, bias, out_dtype=torch.float32, w_tiled=w_tiled), out_dtype or a.dtype)
    if not _fast_ok(a, w):
        return gemm_generic(a, w, bias, out_dtype=out_dtype, accumulate_into=accumulate_into)
    _dev(a, w, bias, accumulate_into)
    M, K = a.shape
    N, K2 = w.shape
    if K != K2:
        raise KernelError(f"gemm: a is {tuple(a.shape)} but w is {tuple(w.shape)}")
    if bias is not None and (bias.dtype != torch.float32 or bias.shape != (N,)):
        raise KernelError("gemm: bias must be float32 [N]")
    if accumulate_into is not None:
        _want(accumulate_into, torch.float32, "accumulate_into")
        if accumulate_into.shape != (M, N):
            raise KernelError(f"gemm: destination is {tuple(accumulate_into.shape)}, expected {(M, N)}")
        _fast_gemm(a, w, bias, accumulate_into, F32, 1, N, w_tiled)
        return accumulate_into
    out_dtype = out_dtype or a.dtype
    out = torch.empty((M, N), dtype=out_dtype, device=a.device)
    _fast_gemm(a, w, bias, out, BF16_GELU if gelu else _code(out_dtype), 0, N, w_tiled)
    return out


def gemm_swiglu(a: torch.Tensor, w_gate_up: torch.Tensor, w_tiled: Optional[torch.Tensor] = None, gelu: bool = False) -> torch.Tensor:
    """silu(a . gate^T) * (a . up^T) with w_gate_up = [gate rows; up rows]: [M, I] in a's dtype (``gelu``: the tanh form of gelu
    in place of silu).
    On the bfloat16 path the activation is formed from the float32 sums inside the product's
    kernel; otherwise the [M, 2I] intermediate is float32 and a second kernel forms it."""
    rows2, K = w_gate_up.shape
    if rows2 % 2:
        raise KernelError("gemm_swiglu: the operand holds gate and up rows; their number must be even")
    if _fast_ok(a, w_gate_up):
        _dev(a, w_gate_up)
        if a.shape[1] != K:
            raise KernelError(f"gemm_swiglu: a is {tuple(a.shape)} but w is {tuple(w_gate_up.shape)}")
        out = torch.empty((a.shape[0], rows2 // 2), dtype=torch.bfloat16, device=a.device)
        _fast_gemm(a, w_gate_up, None, out, BF16_GEGLU if gelu else BF16, 2, rows2 // 2, w_tiled)
        return out
    return swiglu(gemm_generic(a, w_gate_up, out_dtype=torch.float32), out_dtype=a.dtype, gelu=gelu)


# ---- fused products for decode steps of up to 16 rows --------------------------------------------
EPILOGUE_STORE, EPILOGUE_ACCUMULATE, EPILOGUE_SWIGLU, EPILOGUE_CONV = 0, 1, 2, 3


GEGLU = "gelu_tanh"       # in place of a clamped unit's three numbers


def _glu(glu):
    """The three numbers a gated epilogue takes: (0, 1, 0) is SwiGLU, (-1, 1, 0) the same around the tanh form of gelu
    (``GEGLU``); else (limit > 0, alpha, shift)."""
    if glu is None or glu == GEGLU:
        return ctypes.c_float(0.0 if glu is None else -1.0), ctypes.c_float(1.0), ctypes.c_float(0.0)
    limit, alpha, shift = glu
    if not limit > 0:
        raise KernelError("a gated unit with clamped halves needs a positive limit")
    return ctypes.c_float(limit), ctypes.c_float(alpha), ctypes.c_float(shift)
DECODE_MAX_ROWS = 16
LONG_K = 4096
LONG_K_TILED_ROWS = 8


def gemm_decode_fits(rows: int, features: int, k: int, epilogue: int) -> bool:
    return bool(library().fw_gemm_decode_fits(int(rows), int(features), int(k), int(epilogue)))


def gemm_decode(a: torch.Tensor, w: torch.Tensor, epilogue: int, *, bias: Optional[torch.Tensor] = None,
                norm_weight: Optional[torch.Tensor] = None, eps: float = 0.0, one_centered: bool = False,
                row_index: Optional[torch.Tensor] = None, out_dtype: Optional[torch.dtype] = None,
                accumulate_into: Optional[torch.Tensor] = None, taps: Optional[torch.Tensor] = None,
                conv_bias: Optional[torch.Tensor] = None, state: Optional[torch.Tensor] = None,
                seg_slot: Optional[torch.Tensor] = None, squares: Optional[torch.Tensor] = None,
                next_norm_weight: Optional[torch.Tensor] = None, next_one_centered: bool = False,
                w_tiled: Optional[torch.Tensor] = None, glu: Optional[tuple] = None, gelu: bool = False):
    """One kernel for (optional RMS norm of float32 rows) -> product with bfloat16 ``w`` -> epilogue.
    ``glu`` (with EPILOGUE_SWIGLU): (limit, alpha, shift) of a gated unit with clamped halves. ``gelu`` (EPILOGUE_STORE,
    bfloat16, no norm in front): the error-function gelu of the sums is stored.
    With ``norm_weight`` ``a`` holds float32 rows (gathered through ``row_index`` if given), else
    bfloat16 activations. With ``next_norm_weight`` the accumulating epilogue also leaves what
    the norm after it needs, and the call returns (activations x * w_next, sums of squares);
    a later call takes those as ``a`` and ``squares`` (with ``eps``) and skips the norm's
    arithmetic. See fw_gemm_decode in fw_kernels.h for the epilogues."""
    _dev(a, w, bias, norm_weight, row_index, accumulate_into, taps, conv_bias, state, seg_slot, squares, next_norm_weight)
    _want(w, torch.bfloat16, "w")
    normed = norm_weight is not None
    if squares is not None and (normed or squares.dtype != torch.float32 or squares.dim() != 2 or squares.shape[1] != 16
                                or not squares.is_contiguous()):
        raise KernelError("gemm_decode: sums of squares are float32 [tiles, 16] and replace the norm")
    rows = row_index.numel() if (normed and row_index is not None) else a.shape[0]
    K = a.shape[1]
    tiles = {EPILOGUE_SWIGLU: 2, EPILOGUE_CONV: 3}.get(epilogue, 1)
    if w.shape[1] != K or w.shape[0] % tiles:
        raise KernelError(f"gemm_decode: a is {tuple(a.shape)} but w is {tuple(w.shape)}")
    N = w.shape[0] // tiles
    if normed:
        _want(a, torch.float32, "a")
        _want(norm_weight, torch.float32, "norm_weight")
        if norm_weight.shape != (K,):
            raise KernelError("gemm_decode: the norm weight must be [K]")
        if row_index is not None:
            _want(row_index, torch.int32, "row_index")
    else:
        _want(a, torch.bfloat16, "a")
    if bias is not None and (bias.dtype != torch.float32 or bias.shape != (w.shape[0],)):
        raise KernelError("gemm_decode: bias must be float32, one entry per row of w")
    kernel_size = 0
    if epilogue == EPILOGUE_CONV:
        _want(taps, torch.float32, "taps")
        _want(state, torch.float32, "state")
        _want(seg_slot, torch.int32, "seg_slot")
        kernel_size = taps.shape[1]
        if taps.shape != (N, kernel_size) or state.dim() != 3 or state.shape[1:] != (N, kernel_size - 1):
            raise KernelError("gemm_decode: taps must be [N, L] and state [slots, N, L - 1]")
        if seg_slot.numel() < rows or (conv_bias is not None and conv_bias.shape != (N,)):
            raise KernelError("gemm_decode: seg_slot or the convolution bias has the wrong size")
    if epilogue == EPILOGUE_ACCUMULATE:
        _want(accumulate_into, torch.float32, "accumulate_into")
        if accumulate_into.shape != (rows, N):
            raise KernelError(f"gemm_decode: destination is {tuple(accumulate_into.shape)}, expected {(rows, N)}")
        target, out_dtype = accumulate_into, torch.float32
    else:
        out_dtype = out_dtype or torch.bfloat16
        target = torch.empty((rows, N), dtype=out_dtype, device=a.device)
    next_activations = next_squares = None
    if next_norm_weight is not None and (epilogue != EPILOGUE_ACCUMULATE or next_norm_weight.dtype != torch.float32
                                         or next_norm_weight.shape != (N,)):
        raise KernelError("gemm_decode: only the accumulating product prepares the next norm, whose weight is float32 [N]")
    if epilogue == EPILOGUE_ACCUMULATE and K >= LONG_K and N <= 4096 and not (w_tiled is not None and rows <= LONG_K_TILED_ROWS):
        # few features and a long K: the kernel that splits K over workgroups streams W faster (from operand
        # tiles only beyond eight rows: 2,048 features over K 8,192 at 8 rows 11.4 against 11.0 us, at 16
        # rows 11.3 against 13.4)
        left = gemm_medium_into(a, w, bias, target, F32, 1, N, next_norm_weight, next_one_centered, w_tiled=w_tiled)
        return target if left is None else left
    if next_norm_weight is not None:
        next_activations = torch.empty((rows, N), dtype=torch.bfloat16, device=a.device)
        next_squares = torch.empty((library().fw_gemm_decode_accumulate_tiles(N), 16), dtype=torch.float32, device=a.device)
    prologue = 1 if normed else (2 if squares is not None else 0)
    if gelu and (epilogue != EPILOGUE_STORE or out_dtype != torch.bfloat16 or prologue):
        raise KernelError("gemm_decode: gelu goes with a plain storing product of bfloat16")
    w_tiled = _tiled_for(w, w_tiled)
    _check(library().fw_gemm_decode(
        prologue, _p(a), _p(norm_weight), _p(row_index), ctypes.c_float(eps), int(one_centered),
        _p(w if w_tiled is None else w_tiled), int(w_tiled is not None), _p(bias),
        _p(target), BF16_GELU if gelu else _code(out_dtype), int(epilogue), rows, N, K, _p(taps), _p(conv_bias), _p(state), _p(seg_slot),
        int(kernel_size), _p(next_norm_weight), int(next_one_centered), _p(next_activations), _p(next_squares),
        _p(squares), 0 if squares is None else squares.shape[0], *_glu(glu), _stream()))
    if next_norm_weight is not None:
        return next_activations, next_squares
    return target


DECODE_SPLIT_PAGES = 4


QUERY_TILE = 64


def query_tiles(seg_row0):
    """Cuts the rows of each segment into tiles of up to 64 that never span two segments:
    (segment of each tile, first row of each tile), as lists."""
    tile_seg, tile_row0 = [], []
    for seg in range(len(seg_row0) - 1):
        for row in range(seg_row0[seg], seg_row0[seg + 1], QUERY_TILE):
            tile_seg.append(seg)
            tile_row0.append(row)
    return tile_seg, tile_row0


def decode_splits(max_context: int, window: int = 0, chunk: int = 0, keep_first: int = 0) -> int:
    """Into how many workgroups at most the keys that a row sees are cut: runs of 4 pages."""
    blocks = (max_context + PAGE_SIZE - 1) // PAGE_SIZE
    span = min((n for n in (window, chunk) if n > 0), default=0)     # the most keys a row sees, where bounded
    if span > 0:
        blocks = min(blocks, (span + PAGE_SIZE - 2) // PAGE_SIZE + 1 + (keep_first + PAGE_SIZE - 1) // PAGE_SIZE)
    return max(1, (blocks + DECODE_SPLIT_PAGES - 1) // DECODE_SPLIT_PAGES)


def attention_prefill(q: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int, k_pages: torch.Tensor,
                      v_pages: torch.Tensor, block_table: torch.Tensor, tile_seg: torch.Tensor, tile_row0: torch.Tensor,
                      seg_row0: torch.Tensor, row_pos: torch.Tensor, scale: float, window: int = 0,
                      heads_together: int = 0, out: Optional[torch.Tensor] = None, v_dim: Optional[int] = None,
                      chunk: int = 0, softcap: float = 0.0, keep_first: int = 0, sinks: Optional[torch.Tensor] = None,
                      slopes: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``heads_together``: query heads of a kv group per workgroup (1, or 4 up to head_dim 64), 0: the
    kernel's choice. Only the rows of the given tiles are written (into ``out`` if given)."""
    _dev(q, k_pages, v_pages, block_table, tile_seg, tile_row0, seg_row0, row_pos)
    _want(q, torch.bfloat16, "q")
    rows = q.shape[0]
    v_dim = head_dim if v_dim is None else int(v_dim)
    if q.shape != (rows, num_heads * head_dim):
        raise KernelError(f"attention: q is {tuple(q.shape)}, expected {(rows, num_heads * head_dim)}")
    pages = _check_pages(k_pages, v_pages, num_kv_heads, head_dim, torch.bfloat16, v_dim)
    for name, t in (("block_table", block_table), ("tile_seg", tile_seg), ("tile_row0", tile_row0),
                    ("seg_row0", seg_row0), ("row_pos", row_pos)):
        _want(t, torch.int32, name)
    if block_table.dim() != 2 or row_pos.numel() < rows or tile_seg.numel() != tile_row0.numel():
        raise KernelError("attention: batch index arrays are inconsistent")
    if out is None:
        out = torch.empty((rows, num_heads * v_dim), dtype=q.dtype, device=q.device)
    elif out.shape != (rows, num_heads * v_dim) or out.dtype != q.dtype or not out.is_contiguous():
        raise KernelError("attention: out must be bfloat16 [rows, heads * v_dim]")
    _check(library().fw_attention_prefill(
        _p(q), _p(out), _p(k_pages), _p(v_pages), _p(block_table), block_table.shape[1], _p(tile_seg), _p(tile_row0),
        tile_seg.numel(), _p(seg_row0), _p(row_pos), rows, num_heads, num_kv_heads, head_dim, v_dim, ctypes.c_float(scale),
        int(window), int(chunk), ctypes.c_float(softcap), *_sinks(sinks, num_heads, keep_first, window, chunk, slopes), PAGE_SIZE, pages,
        int(heads_together), _stream()))
    return out


def _work(decode_work: Optional[torch.Tensor]):
    if decode_work is not None:
        _dev(decode_work)
        _want(decode_work, torch.int32, "decode_work")
        if decode_work.numel() < 1:
            raise KernelError("attention_decode: decode_work holds one int32")
    return _p(decode_work)


def attention_decode(q: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int, k_pages: torch.Tensor,
                     v_pages: torch.Tensor, block_table: torch.Tensor, row_seg: torch.Tensor, row_pos: torch.Tensor,
                     scale: float, max_context: int, window: int = 0, out: Optional[torch.Tensor] = None,
                     decode_work: Optional[torch.Tensor] = None, v_dim: Optional[int] = None, chunk: int = 0,
                     softcap: float = 0.0, keep_first: int = 0, sinks: Optional[torch.Tensor] = None,
                      slopes: Optional[torch.Tensor] = None) -> torch.Tensor:
    """One row per request; ``max_context`` bounds position + 1 of every row (the host knows it).
    ``decode_work``: one int32 on the device, the runs of 4 pages that the rows see together (the
    sum of ceil((position + 1) / 256)): the kernel shares the work out by it (fewer, longer
    workgroups once there are more than about 512); without it, one run per workgroup."""
    _dev(q, k_pages, v_pages, block_table, row_seg, row_pos)
    _want(q, torch.bfloat16, "q")
    rows = q.shape[0]
    v_dim = head_dim if v_dim is None else int(v_dim)
    if q.shape != (rows, num_heads * head_dim):
        raise KernelError(f"attention: q is {tuple(q.shape)}, expected {(rows, num_heads * head_dim)}")
    pages = _check_pages(k_pages, v_pages, num_kv_heads, head_dim, torch.bfloat16, v_dim)
    for name, t in (("block_table", block_table), ("row_seg", row_seg), ("row_pos", row_pos)):
        _want(t, torch.int32, name)
    if block_table.dim() != 2 or row_seg.numel() < rows or row_pos.numel() < rows:
        raise KernelError("attention: batch index arrays are too short")
    keep_first, sinks_at, slopes_at = _sinks(sinks, num_heads, keep_first, window, chunk, slopes)
    splits = decode_splits(max_context, window, chunk, keep_first)
    partial = torch.empty((rows, num_heads, splits, v_dim + 4), dtype=torch.float32, device=q.device)
    if out is None:
        out = torch.empty((rows, num_heads * v_dim), dtype=q.dtype, device=q.device)
    elif out.shape != (rows, num_heads * v_dim) or out.dtype != q.dtype or not out.is_contiguous():
        raise KernelError("attention: out must be bfloat16 [rows, heads * v_dim]")
    group = num_heads // num_kv_heads
    tickets = _medium_counters(q.device, rows * num_kv_heads * ((group + 15) // 16))
    _check(library().fw_attention_decode(
        _p(q), _p(out), _p(partial), splits, int(max_context), _work(decode_work), _p(tickets), tickets.numel(), _p(k_pages), _p(v_pages),
        _p(block_table),
        block_table.shape[1], _p(row_seg), _p(row_pos), rows, num_heads, num_kv_heads, head_dim, v_dim, ctypes.c_float(scale),
        int(window), int(chunk), ctypes.c_float(softcap), keep_first, sinks_at, slopes_at, PAGE_SIZE, pages, _stream()))
    return out


def attention_decode_fused(qkv: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int,
                           q_norm_weight: Optional[torch.Tensor], k_norm_weight: Optional[torch.Tensor], eps: float,
                           cos: Optional[torch.Tensor], sin: Optional[torch.Tensor], rotary_dim: int, k_pages: torch.Tensor,
                           v_pages: torch.Tensor, block_table: torch.Tensor, row_seg: torch.Tensor, row_pos: torch.Tensor,
                           scale: float, max_context: int, window: int = 0, write_kv: bool = True,
                           decode_work: Optional[torch.Tensor] = None, v_dim: Optional[int] = None, chunk: int = 0,
                           softcap: float = 0.0, interleaved: bool = False, q_only: bool = False, keep_first: int = 0,
                           sinks: Optional[torch.Tensor] = None, slopes: Optional[torch.Tensor] = None,
                           q_row_scale: Optional[torch.Tensor] = None) -> torch.Tensor:
    """One row per request, from the step's raw projections ``qkv`` (float32 [rows, (heads + 2 kv
    heads) * head_dim]): per-head norm and rotation of queries and keys, the new keys and values
    into their pages, and the split-key attention, in one kernel. Returns bfloat16 [rows, heads *
    head_dim]; the same numbers as ``qk_norm_rope_kv_write`` followed by ``attention_decode``."""
    _dev(qkv, q_norm_weight, k_norm_weight, cos, sin, k_pages, v_pages, block_table, row_seg, row_pos)
    _want(qkv, torch.float32, "qkv")
    rows, width = qkv.shape
    v_dim = head_dim if v_dim is None else int(v_dim)
    expected = num_heads * head_dim if q_only else (num_heads + num_kv_heads) * head_dim + num_kv_heads * v_dim
    if width != expected or (q_only and write_kv):
        raise KernelError(f"attention_decode_fused: qkv width {width} != {expected} (queries alone: {q_only}; they bring nothing to store)")
    pages = _check_pages(k_pages, v_pages, num_kv_heads, head_dim, torch.bfloat16, v_dim)
    for w in (q_norm_weight, k_norm_weight):
        if w is not None:
            _want(w, torch.float32, "norm weight")
            if w.shape != (head_dim,):
                raise KernelError("attention_decode_fused: a head norm weight must be [head_dim]")
    if rotary_dim:
        for t in (cos, sin):
            _want(t, torch.float32, "rotation table")
            if t.shape != (rows, rotary_dim // 2):
                raise KernelError(f"attention_decode_fused: rotation table is {tuple(t.shape)}, expected {(rows, rotary_dim // 2)}")
    for name, t in (("block_table", block_table), ("row_seg", row_seg), ("row_pos", row_pos)):
        _want(t, torch.int32, name)
    if block_table.dim() != 2 or row_seg.numel() < rows or row_pos.numel() < rows:
        raise KernelError("attention: batch index arrays are too short")
    keep_first, sinks_at, slopes_at = _sinks(sinks, num_heads, keep_first, window, chunk, slopes)
    splits = decode_splits(max_context, window, chunk, keep_first)
    partial = torch.empty((rows, num_heads, splits, v_dim + 4), dtype=torch.float32, device=qkv.device)
    out = torch.empty((rows, num_heads * v_dim), dtype=torch.bfloat16, device=qkv.device)
    group = num_heads // num_kv_heads
    tickets = _medium_counters(qkv.device, rows * num_kv_heads * ((group + 15) // 16))
    _row_scale(q_row_scale, rows)
    _check(library().fw_attention_decode_fused(
        _p(qkv), _p(q_norm_weight), _p(k_norm_weight), ctypes.c_float(eps), _p(cos), _p(sin), int(rotary_dim), int(write_kv), _p(out),
        _p(partial), splits, int(max_context), _work(decode_work), _p(tickets), tickets.numel(), _p(k_pages), _p(v_pages), _p(block_table),
        block_table.shape[1], _p(row_seg), _p(row_pos), rows, num_heads, num_kv_heads, head_dim, v_dim, ctypes.c_float(scale), int(window),
        int(chunk), ctypes.c_float(softcap), int(interleaved), int(q_only), keep_first, sinks_at, slopes_at, _p(q_row_scale), PAGE_SIZE, pages,
        _stream()))
    return out


def attention_is_tiled(head_dim: int) -> bool:
    """Whether bfloat16 attention with this head size runs on the matrix-core kernels (which
    work on tiles of QUERY_TILE rows)."""
    return head_dim % 16 == 0 and 16 <= head_dim <= MAX_HEAD_DIM


def attention(q: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int, k_pages: torch.Tensor,
              v_pages: torch.Tensor, block_table: torch.Tensor, ctx, scale: float, window: int = 0,
              tile_seg: Optional[torch.Tensor] = None, tile_row0: Optional[torch.Tensor] = None,
              decode_work: Optional[torch.Tensor] = None, v_dim: Optional[int] = None, chunk: int = 0,
              softcap: float = 0.0, keep_first: int = 0, sinks: Optional[torch.Tensor] = None,
                      slopes: Optional[torch.Tensor] = None) -> torch.Tensor:
    """bfloat16 with a head size in steps of 16 runs on the matrix cores: the split-key decode
    kernel for segments of one row (all of them, or those a mixed step begins with: a single row
    would hold a 64-row tile of the prompt kernel and walk its whole context alone), the tiled
    kernel for the rest (``tile_seg``, ``tile_row0``: the tiles of ``query_tiles`` in the order
    workgroups take them, those of the leading single rows in front; ``decode_work``: see
    ``attention_decode``); float32 and everything else on the generic kernel. ``v_dim``: the size of a
    value head (and of a head's output) where it is not ``head_dim``."""
    v_dim = head_dim if v_dim is None else int(v_dim)
    fast = q.dtype == torch.bfloat16 and attention_is_tiled(head_dim) and attention_is_tiled(v_dim)
    if fast and ctx.all_decode:
        return attention_decode(q, num_heads, num_kv_heads, head_dim, k_pages, v_pages, block_table, ctx.row_seg,
                                ctx.row_pos, scale, ctx.max_context, window, decode_work=decode_work, v_dim=v_dim,
                                chunk=chunk, softcap=softcap, keep_first=keep_first, sinks=sinks, slopes=slopes)
    if fast:
        if tile_seg is None or tile_row0 is None:
            raise KernelError("attention: the tiled kernel needs the step's query tiles")
        single = getattr(ctx, "decode_prefix", 0)       # leading segments of one row: rows and tiles 0 .. single - 1
        # four query heads of a kv group per workgroup pay where the rows sit behind a long context
        # (a page is read once for the four); from the start of a prompt one head per workgroup
        # gives more and shorter workgroups, which evens out the causal triangle
        rows = q.shape[0] - single
        keys = min([n for n in (window, chunk) if n] + [ctx.max_context])      # the most keys a row can see
        together = 4 if max(head_dim, v_dim) <= 64 and num_heads // num_kv_heads >= 4 and keys >= 4 * rows else 0
        if single == 0:
            return attention_prefill(q, num_heads, num_kv_heads, head_dim, k_pages, v_pages, block_table, tile_seg,
                                     tile_row0, ctx.seg_row0, ctx.row_pos, scale, window, heads_together=together, v_dim=v_dim,
                                     chunk=chunk, softcap=softcap, keep_first=keep_first, sinks=sinks, slopes=slopes)
        out = torch.empty((q.shape[0], num_heads * v_dim), dtype=q.dtype, device=q.device)
        attention_decode(q[:single], num_heads, num_kv_heads, head_dim, k_pages, v_pages, block_table, ctx.row_seg,
                         ctx.row_pos, scale, ctx.max_context, window, out=out[:single], decode_work=decode_work, v_dim=v_dim,
                         chunk=chunk, softcap=softcap, keep_first=keep_first, sinks=sinks, slopes=slopes)
        return attention_prefill(q, num_heads, num_kv_heads, head_dim, k_pages, v_pages, block_table,
                                 tile_seg[single:], tile_row0[single:], ctx.seg_row0, ctx.row_pos, scale, window,
                                 heads_together=together, out=out, v_dim=v_dim, chunk=chunk, softcap=softcap,
                                 keep_first=keep_first, sinks=sinks, slopes=slopes)
    return attention_generic(q, num_heads, num_kv_heads, head_dim, k_pages, v_pages, block_table, ctx.row_seg,
                             ctx.row_pos, scale, window, v_dim=v_dim, chunk=chunk, softcap=softcap, keep_first=keep_first, sinks=sinks, slopes=slopes)


# ---- attention whose weights are sigmoids and whose heads mix them ------------------------------------------
SIGMOID_MAX_HEADS = 256         # of the plain kernel (the matrix-core kernels: see sigmoid_attention_is_tiled)
SIGMOID_DECODE_WORKGROUPS = 256     # one per compute unit: up to here every page of a row gets a workgroup of its own


def sigmoid_attention_is_tiled(num_heads: int, head_dim: int, v_dim: int) -> bool:
    """Whether bfloat16 runs on the matrix-core kernels: up to 16 heads, sizes in steps of 16, all heads of 16 rows in LDS."""
    return bool(library().fw_sigmoid_attention_fits(int(num_heads), int(head_dim), int(v_dim)))


def _sigmoid_checks(num_heads: int, num_kv_heads: int, head_dim: int, v_dim: int, k_pages: torch.Tensor, v_pages: torch.Tensor,
                    block_table: torch.Tensor, row_seg: Optional[torch.Tensor], row_pos: torch.Tensor, rows: int, bias: torch.Tensor,
                    mix: torch.Tensor, gate: Optional[torch.Tensor]):
    _dev(k_pages, v_pages, block_table, row_seg, row_pos, bias, mix)
    pages = _check_pages(k_pages, v_pages, num_kv_heads, head_dim, k_pages.dtype, v_dim)
    for name, t in (("block_table", block_table), ("row_seg", row_seg), ("row_pos", row_pos)):
        if t is not None:
            _want(t, torch.int32, name)
    if block_table.dim() != 2 or (row_seg is not None and row_seg.numel() < rows) or row_pos.numel() < rows:
        raise KernelError("sigmoid_attention: batch index arrays are too short")
    for name, t, shape in (("bias", bias, (num_heads,)), ("mix", mix, (num_heads, num_heads))):
        _want(t, torch.float32, name)
        if t.shape != shape:
            raise KernelError(f"sigmoid_attention: {name} is {tuple(t.shape)}, expected {shape}")
    if gate is not None:
        _dev_rows(gate, "gate")
        if gate.dtype != torch.float32 or gate.shape != (rows, num_heads * v_dim):
            raise KernelError(f"sigmoid_attention: the gate is {tuple(gate.shape)} {gate.dtype}, expected {(rows, num_heads * v_dim)} float32")
    return pages


def sigmoid_attention_generic(q: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int, v_dim: int, k_pages: torch.Tensor,
                              v_pages: torch.Tensor, block_table: torch.Tensor, row_seg: torch.Tensor, row_pos: torch.Tensor,
                              scale: float, window: int, bias: torch.Tensor, mix: torch.Tensor,
                              gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """a_g = sigmoid(q_g . k * scale + bias[g]) over the visible keys, heads mixed by ``mix`` [heads, heads], the weighted
    sums of the values times sigmoid(``gate``) (float32 [rows, heads * v_dim], rows may lie apart; None: no gate)."""
    rows = q.shape[0]
    _dev(q)
    if q.shape != (rows, num_heads * head_dim) or q.dtype != k_pages.dtype:
        raise KernelError(f"sigmoid_attention: q is {tuple(q.shape)} {q.dtype}, expected {(rows, num_heads * head_dim)} {k_pages.dtype}")
    pages = _sigmoid_checks(num_heads, num_kv_heads, head_dim, v_dim, k_pages, v_pages, block_table, row_seg, row_pos, rows, bias, mix, gate)
    out = torch.empty((rows, num_heads * v_dim), dtype=q.dtype, device=q.device)
    _check(library().fw_sigmoid_attention_generic(
        _p(q), _p(out), _code(q.dtype), _p(k_pages), _p(v_pages), _p(block_table), block_table.shape[1], _p(row_seg), _p(row_pos), rows,
        num_heads, num_kv_heads, head_dim, v_dim, ctypes.c_float(scale), int(window), _p(bias), _p(mix), _p(gate),
        _stride(gate) if gate is not None else 0, PAGE_SIZE, pages, _stream()))
    return out


def sigmoid_attention_prefill(q: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int, v_dim: int, k_pages: torch.Tensor,
                              v_pages: torch.Tensor, block_table: torch.Tensor, tile_seg: torch.Tensor, tile_row0: torch.Tensor,
                              seg_row0: torch.Tensor, row_pos: torch.Tensor, scale: float, window: int, bias: torch.Tensor,
                              mix: torch.Tensor, gate: Optional[torch.Tensor] = None, out: Optional[torch.Tensor] = None,
                              max_context: int = 0, parts: int = 0) -> torch.Tensor:
    """The same on the matrix cores for the rows of the given tiles (of up to 64 rows; ``attention_prefill``).
    ``max_context`` bounds position + 1 of every row (0: what the block table holds). ``parts``: workgroups that share the keys of
    16 rows (0: as many as fill the chip)."""
    rows = q.shape[0]
    _dev(q, tile_seg, tile_row0, seg_row0)
    _want(q, torch.bfloat16, "q")
    for name, t in (("tile_seg", tile_seg), ("tile_row0", tile_row0), ("seg_row0", seg_row0)):
        _want(t, torch.int32, name)
    if q.shape != (rows, num_heads * head_dim) or k_pages.dtype != torch.bfloat16 or tile_seg.numel() != tile_row0.numel():
        raise KernelError(f"sigmoid_attention: q is {tuple(q.shape)}, pages {k_pages.dtype}, {tile_seg.numel()} / {tile_row0.numel()} tiles")
    pages = _sigmoid_checks(num_heads, num_kv_heads, head_dim, v_dim, k_pages, v_pages, block_table, None, row_pos, rows, bias, mix, gate)
    if out is None:
        out = torch.empty((rows, num_heads * v_dim), dtype=q.dtype, device=q.device)
    elif out.shape != (rows, num_heads * v_dim) or out.dtype != q.dtype or not out.is_contiguous():
        raise KernelError("sigmoid_attention: out must be bfloat16 [rows, heads * v_dim]")
    floats, counters = ctypes.c_longlong(0), ctypes.c_int(0)
    parts = library().fw_sigmoid_attention_prefill_plan(tile_seg.numel(), num_heads, head_dim, v_dim, int(window),
                                                        int(max_context) or block_table.shape[1] * PAGE_SIZE, int(parts),
                                                        ctypes.byref(floats), ctypes.byref(counters))
    partial = torch.empty((floats.value,), dtype=torch.float32, device=q.device) if parts > 1 else None
    tickets = _medium_counters(q.device, counters.value)
    _check(library().fw_sigmoid_attention_prefill(
        _p(q), _p(out), _p(partial), ctypes.c_longlong(floats.value), _p(tickets), tickets.numel(), parts, _p(k_pages), _p(v_pages), _p(block_table), block_table.shape[1], _p(tile_seg), _p(tile_row0), tile_seg.numel(),
        _p(seg_row0), _p(row_pos), rows, num_heads, num_kv_heads, head_dim, v_dim, ctypes.c_float(scale), int(window), _p(bias), _p(mix),
        _p(gate), _stride(gate) if gate is not None else 0, PAGE_SIZE, pages, _stream()))
    return out


def sigmoid_decode_splits(rows: int, max_context: int, window: int):
    """(workgroups a row's visible pages are cut into at most, pages each of them takes)."""
    blocks = (max_context + PAGE_SIZE - 1) // PAGE_SIZE
    if window > 0:
        blocks = min(blocks, (window + PAGE_SIZE - 2) // PAGE_SIZE + 1)
    each = max(1, rows * blocks // SIGMOID_DECODE_WORKGROUPS)
    return (blocks + each - 1) // each, each


def sigmoid_attention_decode(num_heads: int, num_kv_heads: int, head_dim: int, v_dim: int, k_pages: torch.Tensor, v_pages: torch.Tensor,
                             block_table: torch.Tensor, row_seg: torch.Tensor, row_pos: torch.Tensor, scale: float, window: int,
                             bias: torch.Tensor, mix: torch.Tensor, max_context: int, gate: Optional[torch.Tensor] = None,
                             q: Optional[torch.Tensor] = None, qkv: Optional[torch.Tensor] = None, qk_norm: bool = True, eps: float = 0.0,
                             write_kv: bool = True, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """One row per request on the matrix cores; ``max_context`` bounds position + 1 of every row. From finished queries
    ``q`` (bfloat16), or from the raw projections ``qkv`` (float32 [rows, q | k | v], rows may lie apart): queries and keys of a
    head divided by their root mean square (``qk_norm``, ``eps``) and the new keys and values stored (``write_kv``) in the same
    kernel."""
    if (q is None) == (qkv is None):
        raise KernelError("sigmoid_attention: finished queries or raw projections, one of the two")
    rows = (q if q is not None else qkv).shape[0]
    if q is not None:
        _dev(q)
        _want(q, torch.bfloat16, "q")
        if q.shape != (rows, num_heads * head_dim):
            raise KernelError(f"sigmoid_attention: q is {tuple(q.shape)}, expected {(rows, num_heads * head_dim)}")
    else:
        _dev_rows(qkv, "qkv")
        _want(qkv, torch.float32, "qkv")
        expected = (num_heads + num_kv_heads) * head_dim + num_kv_heads * v_dim
        if qkv.shape != (rows, expected):
            raise KernelError(f"sigmoid_attention: qkv is {tuple(qkv.shape)}, expected {(rows, expected)}")
    if k_pages.dtype != torch.bfloat16:
        raise KernelError("sigmoid_attention: the matrix-core kernels work on a bfloat16 cache")
    pages = _sigmoid_checks(num_heads, num_kv_heads, head_dim, v_dim, k_pages, v_pages, block_table, row_seg, row_pos, rows, bias, mix, gate)
    splits, each = sigmoid_decode_splits(rows, max_context, window)
    partial = torch.empty((rows, splits, num_heads * v_dim), dtype=torch.float32, device=k_pages.device) if splits > 1 else None
    tickets = _medium_counters(k_pages.device, rows)
    if out is None:
        out = torch.empty((rows, num_heads * v_dim), dtype=torch.bfloat16, device=k_pages.device)
    elif out.shape != (rows, num_heads * v_dim) or out.dtype != torch.bfloat16 or not out.is_contiguous():
        raise KernelError("sigmoid_attention: out must be bfloat16 [rows, heads * v_dim]")
    _check(library().fw_sigmoid_attention_decode(
        _p(q), _p(qkv), _stride(qkv) if qkv is not None else 0, int(qk_norm), ctypes.c_float(eps), int(write_kv), _p(out), _p(partial), splits,
        each, int(max_context), _p(tickets), tickets.numel(), _p(k_pages), _p(v_pages), _p(block_table), block_table.shape[1], _p(row_seg),
        _p(row_pos), rows, num_heads, num_kv_heads, head_dim, v_dim, ctypes.c_float(scale), int(window), _p(bias), _p(mix), _p(gate),
        _stride(gate) if gate is not None else 0, PAGE_SIZE, pages, _stream()))
    return out


def sigmoid_attention(q: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int, v_dim: int, k_pages: torch.Tensor,
                      v_pages: torch.Tensor, block_table: torch.Tensor, ctx, scale: float, window: int, bias: torch.Tensor,
                      mix: torch.Tensor, gate: Optional[torch.Tensor] = None, tile_seg: Optional[torch.Tensor] = None,
                      tile_row0: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The step's rows: bfloat16 in sizes the matrix-core kernels take goes to the decode kernel for segments of one row
    (all of them, or those a mixed step begins with) and to the tiled kernel for the rest; everything else to the plain one."""
    if q.dtype != torch.bfloat16 or not sigmoid_attention_is_tiled(num_heads, head_dim, v_dim):
        return sigmoid_attention_generic(q, num_heads, num_kv_heads, head_dim, v_dim, k_pages, v_pages, block_table, ctx.row_seg, ctx.row_pos,
                                         scale, window, bias, mix, gate)
    rows = q.shape[0]
    single = rows if ctx.all_decode else getattr(ctx, "decode_prefix", 0)
    out = torch.empty((rows, num_heads * v_dim), dtype=q.dtype, device=q.device)
    if single:
        sigmoid_attention_decode(num_heads, num_kv_heads, head_dim, v_dim, k_pages, v_pages, block_table, ctx.row_seg, ctx.row_pos, scale,
                                 window, bias, mix, ctx.max_context, gate=gate[:single] if gate is not None else None, q=q[:single],
                                 out=out[:single])
    if single < rows:
        if tile_seg is None or tile_row0 is None:
            raise KernelError("sigmoid_attention: the tiled kernel needs the step's query tiles")
        sigmoid_attention_prefill(q, num_heads, num_kv_heads, head_dim, v_dim, k_pages, v_pages, block_table, tile_seg[single:],
                                  tile_row0[single:], ctx.seg_row0, ctx.row_pos, scale, window, bias, mix, gate, out=out,
                                  max_context=ctx.max_context)
    return out


# ---- the gated delta rule -----------------------------------------------------------------------------
def delta_prepare(proj: torch.Tensor, beta_col: int, a: torch.Tensor, taps: torch.Tensor, conv_state: torch.Tensor,
                  A_log: torch.Tensor, dt_bias: torch.Tensor, row_seg: torch.Tensor, seg_row0: torch.Tensor,
                  seg_slot: torch.Tensor, segments: int, heads: int, kv_heads: int, dim: int, vdim: int,
                  decay_per_head: bool = False):
    """From a step's projections to what the recurrence reads. ``proj`` [rows, >= channels + ...]:
    its first ``channels`` = 2 kv_heads dim + heads vdim columns are q | k | v before their short
    convolutions, columns ``beta_col`` .. + heads the write strengths before the sigmoid; ``a``
    [rows, heads dim] the decays' arguments. ``conv_state`` [slots, channels, taps - 1] is read and
    moved on. ``decay_per_head``: one decay for all key channels of a head (``a`` [rows, heads],
    ``dt_bias`` [heads]). Returns float32 records [rows, heads, delta_record_floats(dim, vdim)]: per row and head
    q | k | g | beta | v as the recurrence reads them (q and k of the head's group)."""
    _dev(proj, taps, conv_state, A_log, dt_bias, row_seg, seg_row0, seg_slot)
    _dev_rows(a, "a")
    rows, stride = proj.shape
    channels = 2 * kv_heads * dim + heads * vdim
    count = taps.shape[1]
    if proj.dtype != a.dtype or not proj.is_contiguous() or a.dim() != 2 or a.stride(1) != 1:
        raise KernelError("delta_prepare: the projections and the decays' arguments come in one dtype, rows contiguous")
    decays = heads if decay_per_head else heads * dim
    if a.shape != (rows, decays):
        raise KernelError(f"delta_prepare: a is {tuple(a.shape)}, expected {(rows, decays)} (a view of wider rows will do)")
    for name, t, shape in (("taps", taps, (channels, count)), ("A_log", A_log, (heads,)), ("dt_bias", dt_bias, (decays,))):
        _want(t, torch.float32, name)
        if t.shape != shape or not t.is_contiguous():
            raise KernelError(f"delta_prepare: {name} is {tuple(t.shape)}, expected {shape}")
    _want(conv_state, torch.float32, "conv_state")
    if conv_state.dim() != 3 or conv_state.shape[1:] != (channels, count - 1) or not conv_state.is_contiguous():
        raise KernelError(f"delta_prepare: the convolutions' state is {tuple(conv_state.shape)}, expected [slots, {channels}, {count - 1}]")
    for name, t, n in (("row_seg", row_seg, rows), ("seg_row0", seg_row0, segments + 1), ("seg_slot", seg_slot, segments)):
        _want(t, torch.int32, name)
        if t.numel() < n:
            raise KernelError(f"delta_prepare: {name} holds {t.numel()} entries, needs {n}")
    records = torch.empty((rows, heads, delta_record_floats(dim, vdim)), dtype=torch.float32, device=proj.device)
    _check(library().fw_delta_prepare(_p(proj), _code(proj.dtype), stride, int(beta_col), _p(a), a.stride(0) if rows > 1 else max(decays, a.stride(0)),
                                      _p(taps), _p(conv_state), _p(A_log), _p(dt_bias), _p(row_seg), _p(seg_row0), _p(seg_slot),
                                      _p(records), rows, int(segments), heads, kv_heads, dim, vdim, count, conv_state.shape[0],
                                      int(decay_per_head), _stream()))
    return records


def delta_record_floats(dim: int, vdim: int) -> int:
    """Floats of what one token brings to one head of the recurrence: q | k | g (dim rounded up to a
    multiple of 4 each) | beta and three unused | v (vdim rounded up likewise)."""
    return 3 * ((dim + 3) // 4 * 4) + 4 + (vdim + 3) // 4 * 4


def gated_delta_rule(records: torch.Tensor, state: torch.Tensor, seg_row0: torch.Tensor, seg_slot: torch.Tensor,
                     segments: int, heads: int, dim: int, vdim: int) -> torch.Tensor:
    """The recurrence over each segment's rows. ``records`` [rows, heads, delta_record_floats]: what
    ``delta_prepare`` made. ``state`` [slots, heads, vdim, dim] float32 (the matrix transposed) is read
    at a segment's start and written at its end. Returns [rows, heads vdim]."""
    _dev(records, state, seg_row0, seg_slot)
    rows = records.shape[0]
    _want(records, torch.float32, "records")
    if records.shape != (rows, heads, delta_record_floats(dim, vdim)) or not records.is_contiguous():
        raise KernelError(f"gated_delta_rule: records are {tuple(records.shape)}, expected {(rows, heads, delta_record_floats(dim, vdim))}")
    _want(state, torch.float32, "state")
    if state.dim() != 4 or state.shape[1:] != (heads, vdim, dim) or not state.is_contiguous():
        raise KernelError(f"gated_delta_rule: the state is {tuple(state.shape)}, expected [slots, {heads}, {vdim}, {dim}]")
    for name, t, n in (("seg_row0", seg_row0, segments + 1), ("seg_slot", seg_slot, segments)):
        _want(t, torch.int32, name)
        if t.numel() < n:
            raise KernelError(f"gated_delta_rule: {name} holds {t.numel()} entries, needs {n}")
    out = torch.empty((rows, heads * vdim), dtype=torch.float32, device=records.device)
    _check(library().fw_gated_delta_rule(_p(records), _p(state), _p(out), _p(seg_row0), _p(seg_slot), rows, int(segments), heads,
                                         dim, vdim, state.shape[0], _stream()))
    return out


def gated_head_norm(o: torch.Tensor, gate: torch.Tensor, weight: torch.Tensor, heads: int, vdim: int, eps: float,
                    out_dtype: torch.dtype, gate_silu: bool = False) -> torch.Tensor:
    # ``weight`` [vdim] serves every head; [heads * vdim] gives each head its own
    """Per head: o / rms(o) * weight * sigmoid(gate) (``gate_silu``: times gate * sigmoid(gate)); ``o`` float32 [rows, heads vdim], ``gate``
    [rows, heads vdim] (float32, or bfloat16 beside a bfloat16 output; a view of wider rows will do)."""
    _dev(o, weight)
    _dev_rows(gate, "gate")
    _want(o, torch.float32, "o")
    _want(weight, torch.float32, "weight")
    rows = o.shape[0]
    per_head = weight.shape == (heads * vdim,) and heads > 1
    if o.shape != (rows, heads * vdim) or gate.shape != o.shape or (weight.shape != (vdim,) and not per_head) or not o.is_contiguous() or gate.stride(1) != 1:
        raise KernelError(f"gated_head_norm: o {tuple(o.shape)}, gate {tuple(gate.shape)}, weight {tuple(weight.shape)} do not fit {heads} x {vdim}")
    out = torch.empty((rows, heads * vdim), dtype=out_dtype, device=o.device)
    _check(library().fw_gated_head_norm(_p(o), _p(gate), _code(gate.dtype), gate.stride(0) if rows > 1 else max(heads * vdim, gate.stride(0)), _p(weight), int(per_head), _p(out), _code(out_dtype), rows,
                                        heads, vdim, ctypes.c_float(eps), int(gate_silu), _stream()))
    return out


# ---- sublayers whose output is normed --------------------------------------------------------------------
def norm_scale_add_(x: torch.Tensor, a: torch.Tensor, weight: torch.Tensor, eps: float, mult: float, *,
                    b: Optional[torch.Tensor] = None, scale_a: float = 1.0, scale_b: float = 1.0,
                    one_centered: bool = False, rounded_dtype: Optional[torch.dtype] = None) -> Optional[torch.Tensor]:
    """x += mult * rmsnorm(scale_a a + scale_b b) * w in place (float32 rows; ``b`` optional). With
    ``rounded_dtype`` the new x is also returned in that dtype (what the next products read)."""
    _dev(x, a, b, weight)
    rows, hidden = x.shape
    for name, t in (("x", x), ("a", a), ("b", b)):
        if t is not None:
            _want(t, torch.float32, name)
            if t.shape != (rows, hidden) or not t.is_contiguous():
                raise KernelError(f"norm_scale_add: {name} is {tuple(t.shape)}, expected {(rows, hidden)}")
    _want(weight, torch.float32, "weight")
    if weight.shape != (hidden,):
        raise KernelError(f"norm_scale_add: weight is {tuple(weight.shape)}, row width is {hidden}")
    rounded = torch.empty((rows, hidden), dtype=rounded_dtype, device=x.device) if rounded_dtype is not None else None
    _check(library().fw_norm_scale_add(_p(x), _p(a), _p(b), ctypes.c_float(scale_a), ctypes.c_float(scale_b), _p(weight),
                                       int(one_centered), ctypes.c_float(eps), ctypes.c_float(mult), _p(rounded),
                                       _code(rounded_dtype) if rounded_dtype is not None else F32, rows, hidden, _stream()))
    return rounded


def round_rows(x: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """float32 rows in the activation dtype (float32: the rows themselves)."""
    _want(x, torch.float32, "x")
    if dtype == torch.float32:
        return x
    _dev(x)
    out = torch.empty(x.shape, dtype=torch.bfloat16, device=x.device)
    _check(library().fw_round_rows(_p(x), _p(out), ctypes.c_longlong(x.numel()), _stream()))
    return out


def clamped_glu(gate_up: torch.Tensor, limit: float, alpha: float, shift: float, out_dtype: torch.dtype) -> torch.Tensor:
    """[rows, gate | up] -> min(gate, limit) * sigmoid(alpha * that) * (clamp(up, +-limit) + shift)."""
    _dev(gate_up)
    rows, width = gate_up.shape
    if width % 2 or not gate_up.is_contiguous():
        raise KernelError("clamped_glu: the input holds gate and up halves, contiguous")
    out = torch.empty((rows, width // 2), dtype=out_dtype, device=gate_up.device)
    _check(library().fw_clamped_glu(_p(gate_up), _code(gate_up.dtype), _p(out), _code(out_dtype), rows, width // 2,
                                    ctypes.c_float(limit), ctypes.c_float(alpha), ctypes.c_float(shift), _stream()))
    return out


# ---- a sublayer between two norms, layer norm, the gate on a second token table ------------------------------
NEXT_NOTHING, NEXT_ROUNDED, NEXT_RMS, NEXT_CENTERED = 0, 1, 2, 3


def layernorm_rows(x: torch.Tensor, weight: torch.Tensor, eps: float, out_dtype: torch.dtype,
                   row_index: Optional[torch.Tensor] = None, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """(x - mean) / sqrt(mean((x - mean)^2) + eps) * weight (+ bias) over float32 rows (gathered through
    ``row_index`` if given), in ``out_dtype``."""
    _dev(x, weight, row_index, bias)
    _want(x, torch.float32, "x")
    hidden = x.shape[-1]
    for name, t in (("weight", weight), ("bias", bias)):
        if t is not None:
            _want(t, torch.float32, name)
            if t.shape != (hidden,):
                raise KernelError(f"layernorm: {name} is {tuple(t.shape)}, row width is {hidden}")
    rows = x.numel() // hidden if row_index is None else row_index.numel()
    if row_index is not None:
        _want(row_index, torch.int32, "row_index")
    out = torch.empty((rows, hidden), dtype=out_dtype, device=x.device)
    _check(library().fw_layernorm_rows(_p(x), _p(weight), _p(bias), _p(out), _code(out_dtype), _p(row_index), rows, hidden,
                                       ctypes.c_float(eps), _stream()))
    return out


def norm_add_norm_(x: torch.Tensor, a: torch.Tensor, weight: torch.Tensor, centered: bool, eps: float, *,
                   bias: Optional[torch.Tensor] = None, mult: float = 1.0, next_kind: int = NEXT_NOTHING,
                   next_weight: Optional[torch.Tensor] = None, next_bias: Optional[torch.Tensor] = None, next_eps: float = 0.0,
                   next_dtype: Optional[torch.dtype] = None, next_out: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """x += mult * (norm(a) * weight + bias) in place (float32 rows; ``bias`` optional; ``centered``: the row's mean is
    taken off before its root mean square). What reads x next is formed from the new rows in the same kernel and
    returned: ``NEXT_ROUNDED`` the rows in ``next_dtype``, ``NEXT_RMS`` / ``NEXT_CENTERED`` their norm with ``next_weight``,
    ``next_bias`` (optional) and ``next_eps``, into ``next_out`` if given (rows may lie apart); ``NEXT_NOTHING`` returns None."""
    _dev(x, a, weight, bias, next_weight, next_bias)
    rows, hidden = x.shape
    for name, t in (("x", x), ("a", a)):
        _want(t, torch.float32, name)
        if t.shape != (rows, hidden):
            raise KernelError(f"norm_add_norm: {name} is {tuple(t.shape)}, expected {(rows, hidden)}")
    for name, t in (("weight", weight), ("bias", bias), ("next_weight", next_weight), ("next_bias", next_bias)):
        if t is not None:
            _want(t, torch.float32, name)
            if t.shape != (hidden,):
                raise KernelError(f"norm_add_norm: {name} is {tuple(t.shape)}, row width is {hidden}")
    if next_kind not in (NEXT_NOTHING, NEXT_ROUNDED, NEXT_RMS, NEXT_CENTERED):
        raise KernelError(f"norm_add_norm: unknown kind {next_kind} of what follows")
    if next_kind >= NEXT_RMS and next_weight is None:
        raise KernelError("norm_add_norm: the norm that follows needs its weight")
    out = None
    if next_kind != NEXT_NOTHING:
        out = next_out
        if out is None:
            out = torch.empty((rows, hidden), dtype=next_dtype or torch.float32, device=x.device)
        _dev_rows(out, "next_out")
        if out.shape != (rows, hidden) or (next_dtype is not None and out.dtype != next_dtype):
            raise KernelError(f"norm_add_norm: next_out is {tuple(out.shape)} {out.dtype}, expected {(rows, hidden)} {next_dtype}")
    _check(library().fw_norm_add_norm(_p(x), _p(a), _p(weight), _p(bias), ctypes.c_float(mult), int(centered), ctypes.c_float(eps),
                                      int(next_kind), _p(next_weight), _p(next_bias), ctypes.c_float(next_eps), _p(out),
                                      _code(out.dtype) if out is not None else F32, _stride(out) if out is not None else 0, rows, hidden,
                                      _stream()))
    return out


def place_rows(x: torch.Tensor, out: torch.Tensor, col0: int = 0, twice: bool = False) -> torch.Tensor:
    """float32 rows (which may lie apart) into columns ``col0`` .. of the wider rows ``out``, in its dtype; ``twice``: once
    more behind them."""
    _dev(out)
    _dev_rows(x, "x")
    _want(x, torch.float32, "x")
    if x.dim() != 2 or out.dim() != 2 or out.shape[0] != x.shape[0]:
        raise KernelError(f"place_rows: {tuple(x.shape)} into {tuple(out.shape)}")
    _check(library().fw_place_rows(_p(x), _stride(x), _p(out), _code(out.dtype), x.shape[0], x.shape[1], out.shape[1], int(col0), int(twice), _stream()))
    return out


def gelu_rows(z: torch.Tensor, out_dtype: torch.dtype) -> torch.Tensor:
    """z Phi(z) (the error-function gelu) of float32 values, in ``out_dtype``."""
    _dev(z)
    _want(z, torch.float32, "z")
    out = torch.empty(z.shape, dtype=out_dtype, device=z.device)
    _check(library().fw_gelu_rows(_p(z), _p(out), _code(out_dtype), ctypes.c_longlong(z.numel()), _stream()))
    return out


def gelu_gate_rows(z: torch.Tensor, table: torch.Tensor, ids: torch.Tensor, col0: int, out_dtype: torch.dtype) -> torch.Tensor:
    """gelu_tanh(z) * table[ids][:, col0 : col0 + width]: ``z`` float32 [rows, width], ``table`` [entries,
    columns], ``ids`` int32 [rows] (checked against the table by the caller)."""
    _dev(z, table, ids)
    _want(z, torch.float32, "z")
    _want(ids, torch.int32, "ids")
    rows, width = z.shape
    if table.dim() != 2 or col0 < 0 or col0 + width > table.shape[1] or ids.numel() < rows:
        raise KernelError(f"gelu_gate_rows: columns {col0}..{col0 + width} of a table {tuple(table.shape)}, {ids.numel()} ids for {rows} rows")
    out = torch.empty((rows, width), dtype=out_dtype, device=z.device)
    _check(library().fw_gelu_gate_rows(_p(z), width, _p(table), _code(table.dtype), table.shape[0], table.shape[1], int(col0), _p(ids),
                                       _p(out), _code(out_dtype), rows, width, _stream()))
    return out


# ---- attention over a cached latent ------------------------------------------------------------------------
def latent_norm_write(raw: torch.Tensor, weight: torch.Tensor, eps: float, k_pages: torch.Tensor, v_pages: torch.Tensor,
                      block_table: torch.Tensor, row_seg: torch.Tensor, row_pos: torch.Tensor, rot: int = 0,
                      cos: Optional[torch.Tensor] = None, sin: Optional[torch.Tensor] = None, turn: Optional[int] = None,
                      interleaved: bool = True) -> None:
    """The step's latents ``raw`` (float32 [rows, rank + rot]; a view of some columns of wider rows will do): the first
    rank columns RMS-normed times ``weight`` and stored at each row's position in a cache of one key/value head; the last
    ``rot`` columns (a key part all heads share) turned by the row's angles (``interleaved``: neighbouring channels paired,
    else channel i with channel i + turn / 2; ``cos``, ``sin`` float32 [rows, turn / 2]) and stored behind the latent in the keys' layout, whose head then has rank + rot channels."""
    _dev(weight, k_pages, v_pages, block_table, row_seg, row_pos, cos, sin)
    _dev_rows(raw, "raw")
    _want(raw, torch.float32, "raw")
    _want(weight, torch.float32, "weight")
    rows, rank = raw.shape[0], raw.shape[1] - int(rot)
    if weight.shape != (rank,):
        raise KernelError(f"latent_norm_write: weight is {tuple(weight.shape)}, the latent has {rank} channels")
    turn = int(rot) if turn is None else int(turn)      # the first so many channels of the part are turned, the rest pass
    if turn:
        for t in (cos, sin):
            if t is None or t.dtype != torch.float32 or t.shape != (rows, turn // 2):
                raise KernelError(f"latent_norm_write: {turn} turned channels need float32 tables {(rows, turn // 2)}")
    pages = _check_pages(k_pages, v_pages, 1, rank + int(rot), k_pages.dtype, rank)
    for name, t in (("block_table", block_table), ("row_seg", row_seg), ("row_pos", row_pos)):
        _want(t, torch.int32, name)
    if block_table.dim() != 2 or row_seg.numel() < rows or row_pos.numel() < rows:
        raise KernelError("latent_norm_write: batch index arrays are too short")
    _check(library().fw_latent_norm_write(_p(raw), raw.stride(0) if rows > 1 else max(rank + int(rot), raw.stride(0)), 0, _p(weight),
                                          ctypes.c_float(eps), _p(k_pages), _p(v_pages), _code(k_pages.dtype), _p(block_table),
                                          block_table.shape[1], _p(row_seg), _p(row_pos), rows, rank, int(rot), turn, int(interleaved), _p(cos), _p(sin),
                                          PAGE_SIZE, pages, _stream()))


def head_linear(x: torch.Tensor, w: torch.Tensor, out_dtype: torch.dtype, gate: Optional[torch.Tensor] = None,
                in_head: Optional[int] = None, out: Optional[torch.Tensor] = None, out_head: Optional[int] = None) -> torch.Tensor:
    """A map per head: ``x`` [rows, heads K] (rows may lie apart), ``w`` [heads, N, K] -> [rows, heads N], with
    ``gate`` (float32 [rows, heads N], or [rows, heads]: one number a head; rows may lie apart) times its sigmoid. ``in_head``: a head's vector in ``x`` holds
    that many channels of which the map reads the first K; ``out`` with ``out_head``: the results go to the first N
    channels of each head's vector of ``out_head`` channels in the rows of ``out``."""
    _dev(w)
    _dev_rows(x, "x")
    heads, N, K = w.shape
    rows = x.shape[0]
    in_head = K if in_head is None else int(in_head)
    if x.shape[1] != heads * in_head or in_head < K:
        raise KernelError(f"head_linear: x is {tuple(x.shape)}, the weight {tuple(w.shape)}, a head's vector {in_head}")
    if gate is not None:
        _dev_rows(gate, "gate")
        if gate.shape not in ((rows, heads * N), (rows, heads)) or gate.dtype != torch.float32:
            raise KernelError(f"head_linear: the gate is {tuple(gate.shape)} {gate.dtype}, expected {(rows, heads * N)} or {(rows, heads)} float32")
    out_head = N if out_head is None else int(out_head)
    if out is None:
        out = torch.empty((rows, heads * out_head), dtype=out_dtype, device=x.device)
    elif out.shape != (rows, heads * out_head) or out.dtype != out_dtype or not out.is_contiguous() or not out.is_cuda:
        raise KernelError(f"head_linear: out is {tuple(out.shape)} {out.dtype}, expected {(rows, heads * out_head)} {out_dtype}")
    if out_head < N or (gate is not None and out_head != N):
        raise KernelError("head_linear: a head's outputs do not fit its vector (a gate goes with outputs side by side)")

    def stride(t: torch.Tensor, width: int) -> int:
        return t.stride(0) if rows > 1 else max(width, t.stride(0))

    _check(library().fw_head_linear(_p(x), _code(x.dtype), stride(x, heads * in_head), _p(w), _code(w.dtype), _p(gate),
                                    stride(gate, gate.shape[1]) if gate is not None else 0,
                                    int(gate is not None and gate.shape[1] == heads and N > 1), _p(out), _code(out_dtype), rows, heads, N, K,
                                    in_head, out_head, heads * out_head, _stream()))
    return out


def rotate_place(x: torch.Tensor, heads: int, col0: int, rot: int, cos: torch.Tensor, sin: torch.Tensor, out: torch.Tensor,
                 out_col0: int, turn: Optional[int] = None, interleaved: bool = True) -> torch.Tensor:
    """Channels col0 .. col0 + rot - 1 of every head's vector in ``x`` [rows, heads * in_head], neighbouring channels
    (``interleaved``; else channels i and i + turn / 2) turned by the row's angles (``cos``, ``sin`` float32 [rows, rot / 2]), stored from channel ``out_col0`` of the head's
    vector in ``out`` [rows, heads * out_head]."""
    _dev(x, cos, sin, out)
    rows = x.shape[0]
    if x.dim() != 2 or out.dim() != 2 or x.shape[1] % heads or out.shape[1] % heads or out.shape[0] != rows:
        raise KernelError(f"rotate_place: {tuple(x.shape)} -> {tuple(out.shape)} with {heads} heads")
    turn = int(rot) if turn is None else int(turn)      # the first so many channels are turned, the rest pass
    for t in ((cos, sin) if turn else ()):
        if t is None or t.dtype != torch.float32 or t.shape != (rows, turn // 2):
            raise KernelError(f"rotate_place: {turn} turned channels need float32 tables {(rows, turn // 2)}")
    _check(library().fw_rotate_place(_p(x), _code(x.dtype), x.shape[1], x.shape[1] // heads, int(col0), _p(cos), _p(sin), _p(out),
                                     _code(out.dtype), out.shape[1], out.shape[1] // heads, int(out_col0), rows, heads, int(rot), turn,
                                     int(interleaved), _stream()))
    return out


# ---- a recurrence with a decay per key channel formed by the token ("wkv") --------------------------------------
def token_shift_mix(x: torch.Tensor, norm_weight: Optional[torch.Tensor], eps: float, one_centered: bool, mu: torch.Tensor,
                    last: torch.Tensor, row_seg: torch.Tensor, seg_row0: torch.Tensor, seg_slot: torch.Tensor, segments: int,
                    out_dtype: torch.dtype) -> torch.Tensor:
    """h = rmsnorm(x) * weight (``norm_weight`` None: h = x); returns [mixes, rows, hidden] = h + (h of the row before - h)
    * mu[s]. ``last`` float32 [slots, hidden]: the h of each request's last row so far, read for a segment's first
    row and moved on."""
    _dev(x, norm_weight, mu, last, row_seg, seg_row0, seg_slot)
    _want(x, torch.float32, "x")
    _want(mu, torch.float32, "mu")
    _want(last, torch.float32, "last")
    rows, hidden = x.shape
    if mu.dim() != 2 or mu.shape[1] != hidden or last.dim() != 2 or last.shape[1] != hidden:
        raise KernelError(f"token_shift_mix: mu {tuple(mu.shape)} / last {tuple(last.shape)} beside rows of {hidden}")
    if norm_weight is not None and (norm_weight.dtype != torch.float32 or norm_weight.shape != (hidden,)):
        raise KernelError("token_shift_mix: the norm's weight is float32 [hidden]")
    for name, t, n in (("row_seg", row_seg, rows), ("seg_row0", seg_row0, segments + 1), ("seg_slot", seg_slot, segments)):
        _want(t, torch.int32, name)
        if t.numel() < n:
            raise KernelError(f"token_shift_mix: {name} holds {t.numel()} entries, needs {n}")
    out = torch.empty((mu.shape[0], rows, hidden), dtype=out_dtype, device=x.device)
    _check(library().fw_token_shift_mix(_p(x), _p(norm_weight), ctypes.c_float(eps), int(one_centered), _p(mu), mu.shape[0], _p(last),
                                        last.shape[0], _p(row_seg), _p(seg_row0), _p(seg_slot), _p(out), _code(out_dtype), rows,
                                        int(segments), hidden, _stream()))
    return out


def tanh_rows(x: torch.Tensor, out_dtype: torch.dtype) -> torch.Tensor:
    _dev(x)
    _want(x, torch.float32, "x")
    out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
    _check(library().fw_tanh_rows(_p(x), _p(out), _code(out_dtype), ctypes.c_longlong(x.numel()), _stream()))
    return out


def wkv_recurrence(r: torch.Tensor, k: torch.Tensor, v: torch.Tensor, a: torch.Tensor, w0: torch.Tensor, u: torch.Tensor,
                   state: torch.Tensor, seg_row0: torch.Tensor, seg_slot: torch.Tensor, segments: int, heads: int, dim: int) -> torch.Tensor:
    """Per head o_t = S^T r_t + (r_t . (u k_t)) v_t, then S <- diag(exp(-exp(a_t + w0))) S + k_t v_t^T, over each segment's rows
    in order. ``r``, ``k``, ``v`` float32 [rows, heads dim] with one row stride (views of wider rows will do), ``a``
    likewise; ``state`` float32 [slots, heads, dim, dim] is read and moved on. Returns float32 [rows, heads dim]."""
    _dev(w0, u, state, seg_row0, seg_slot)
    rows = r.shape[0]
    width = heads * dim
    for name, t in (("r", r), ("k", k), ("v", v), ("a", a)):
        _dev_rows(t, name)
        _want(t, torch.float32, name)
        if t.shape != (rows, width):
            raise KernelError(f"wkv_recurrence: {name} is {tuple(t.shape)}, expected {(rows, width)}")

    def stride(t):
        return t.stride(0) if rows > 1 else max(width, t.stride(0))

    if not (stride(r) == stride(k) == stride(v)):
        raise KernelError("wkv_recurrence: r, k and v have one row stride")
    for name, t in (("w0", w0), ("u", u)):
        _want(t, torch.float32, name)
        if t.numel() != width:
            raise KernelError(f"wkv_recurrence: {name} holds {t.numel()} values, expected {width}")
    _want(state, torch.float32, "state")
    if state.dim() != 4 or state.shape[1:] != (heads, dim, dim):
        raise KernelError(f"wkv_recurrence: the state is {tuple(state.shape)}, expected [slots, {heads}, {dim}, {dim}]")
    for name, t, n in (("seg_row0", seg_row0, segments + 1), ("seg_slot", seg_slot, segments)):
        _want(t, torch.int32, name)
        if t.numel() < n:
            raise KernelError(f"wkv_recurrence: {name} holds {t.numel()} entries, needs {n}")
    out = torch.empty((rows, width), dtype=torch.float32, device=r.device)
    _check(library().fw_wkv_recurrence(_p(r), _p(k), _p(v), stride(r), _p(a), stride(a), _p(w0), _p(u), _p(state), state.shape[0], _p(out),
                                       _p(seg_row0), _p(seg_slot), rows, int(segments), heads, dim, _stream()))
    return out


# ---- a mixture of feed-forward units chosen per token ------------------------------------------------------------
MOE_SCORES = ("softmax_chosen", "softmax_all", "sigmoid")


def moe_route(logits: torch.Tensor, bias: Optional[torch.Tensor], top: int, groups: int = 1, keep: int = 1,
              score_all: bool = False, scores: Optional[str] = None, group_pair: bool = False, correction: Optional[torch.Tensor] = None,
              weight_scale: float = 1.0, normalize: bool = True):
    """(chosen int32 [rows, top], weight float32 [rows, top]): the ``top`` largest of logits + bias per row, largest
    first (ties: the lowest id), and the softmax over those alone. ``groups`` > 1: only experts of the ``keep`` groups
    (of neighbours, equal in size) whose best expert scores highest can be chosen. ``score_all``: the weights are the
    softmax over all experts at the chosen ones, divided by their sum + 1e-20. ``scores`` names the same choice
    ("softmax_chosen", "softmax_all") or "sigmoid": each expert's own sigmoid at the chosen ones, divided by their sum + 1e-20.
    ``group_pair``: groups are ranked by what their two best experts score together (not with "softmax_chosen").
    ``correction`` (float32 [experts], with "sigmoid"): the choice is by score + correction, the weights are the scores
    without it. ``weight_scale`` multiplies the weights; ``normalize`` False (with "softmax_all" and "sigmoid"): they are not
    divided by their sum. Rows of ``logits`` may lie apart."""
    scores = scores or ("softmax_all" if score_all else "softmax_chosen")
    if scores not in MOE_SCORES or (group_pair and scores == "softmax_chosen"):
        raise KernelError(f"moe_route: scores {scores!r} (known: {', '.join(MOE_SCORES)}; groups by pairs: {group_pair})")
    _dev(bias, correction)
    _dev_rows(logits, "logits")
    _want(logits, torch.float32, "logits")
    rows, experts = logits.shape
    if correction is not None and (correction.dtype != torch.float32 or correction.shape != (experts,) or scores != "sigmoid"):
        raise KernelError("moe_route: a correction is float32 [experts] and goes with sigmoid scores")
    if not normalize and scores == "softmax_chosen":
        raise KernelError("moe_route: the softmax over the chosen is a distribution over them")
    if bias is not None and (bias.dtype != torch.float32 or bias.shape != (experts,)):
        raise KernelError("moe_route: the bias is float32 [experts]")
    chosen = torch.empty((rows, top), dtype=torch.int32, device=logits.device)
    weight = torch.empty((rows, top), dtype=torch.float32, device=logits.device)
    _check(library().fw_moe_route(_p(logits), _stride(logits), _p(bias), _p(correction), _p(chosen), _p(weight), rows, experts, int(top),
                                  int(groups), int(keep), int(group_pair), MOE_SCORES.index(scores), ctypes.c_float(weight_scale),
                                  int(normalize), _stream()))
    return chosen, weight


def moe_arrange(chosen: torch.Tensor, experts: int):
    """The pairs (row, choice) sorted by expert, an expert's pairs in their order: (expert_begin int32 [experts + 1],
    place_row int32 [pairs], pair_place int32 [rows, top])."""
    _dev(chosen)
    _want(chosen, torch.int32, "chosen")
    rows, top = chosen.shape
    expert_begin = torch.empty((experts + 1,), dtype=torch.int32, device=chosen.device)
    place_row = torch.empty((rows * top,), dtype=torch.int32, device=chosen.device)
    pair_place = torch.empty((rows, top), dtype=torch.int32, device=chosen.device)
    _check(library().fw_moe_arrange(_p(chosen), _p(expert_begin), _p(place_row), _p(pair_place), rows, int(experts), top, _stream()))
    return expert_begin, place_row, pair_place


def grouped_gemm(a: torch.Tensor, place_row: Optional[torch.Tensor], w: torch.Tensor, expert_begin: torch.Tensor, places: int,
                 gated: bool, out_dtype: torch.dtype, glu: Optional[tuple] = None) -> torch.Tensor:
    """out[place] = a[place_row[place]] . w[expert of place]^T (``place_row`` None: a[place]); ``w`` [experts, N, K], or
    with ``gated`` [experts, 2 N, K] (gate rows, then up rows) and out = silu(gate) * up, or with ``glu`` = (limit, alpha,
    shift) the unit with clamped halves. Returns [places, N]."""
    _dev(a, place_row, w, expert_begin)
    experts, n_rows, K = w.shape
    N = n_rows // 2 if gated else n_rows
    if a.dim() != 2 or a.shape[1] != K or (gated and n_rows % 2) or expert_begin.numel() != experts + 1:
        raise KernelError(f"grouped_gemm: a is {tuple(a.shape)}, w {tuple(w.shape)}, {expert_begin.numel()} expert bounds")
    _want(expert_begin, torch.int32, "expert_begin")
    if place_row is not None:
        _want(place_row, torch.int32, "place_row")
        if place_row.numel() < places:
            raise KernelError("grouped_gemm: fewer rows named than places")
    elif a.shape[0] < places:
        raise KernelError("grouped_gemm: fewer rows than places")
    out = torch.empty((places, N), dtype=out_dtype, device=a.device)
    _check(library().fw_grouped_gemm(_p(a), _code(a.dtype), _p(place_row), _p(w), _code(w.dtype), _p(expert_begin), _p(out),
                                     _code(out_dtype), int(gated), int(places), experts, N, K, *_glu(glu if gated else None), _stream()))
    return out


def moe_combine_(x: torch.Tensor, y: torch.Tensor, weight: torch.Tensor, pair_place: torch.Tensor, shared: Optional[torch.Tensor] = None,
                 gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x[row] += sum over the row's choices, in their order, of weight[row, j] * y[pair_place[row, j]], plus with ``shared``
    [rows, hidden] and ``gate`` [rows, 1] (rows may lie apart) sigmoid(gate) * shared; float32."""
    _dev(x, y, weight, pair_place, shared)
    for name, t in (("x", x), ("y", y), ("weight", weight)):
        _want(t, torch.float32, name)
    _want(pair_place, torch.int32, "pair_place")
    rows, hidden = x.shape
    top = weight.shape[1]
    if weight.shape != (rows, top) or pair_place.shape != (rows, top) or y.shape != (rows * top, hidden):
        raise KernelError(f"moe_combine: x {tuple(x.shape)}, y {tuple(y.shape)}, weight {tuple(weight.shape)}, places {tuple(pair_place.shape)}")
    if (shared is None) != (gate is None):
        raise KernelError("moe_combine: rows to be gated and their gate come together")
    if shared is not None:
        _dev_rows(gate, "gate")
        if shared.dtype != torch.float32 or shared.shape != (rows, hidden) or gate.dtype != torch.float32 or gate.shape != (rows, 1):
            raise KernelError(f"moe_combine: shared rows {tuple(shared.shape)} and gate {tuple(gate.shape)} beside x {tuple(x.shape)}")
    _check(library().fw_moe_combine(_p(x), _p(y), _p(weight), _p(pair_place), _p(shared), _p(gate), _stride(gate) if gate is not None else 0,
                                    rows, top, hidden, _stream()))
    return x


# ---- a short causal convolution per channel, and a gated linear recurrence per channel ---------------------------------
def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: Optional[torch.Tensor], state: torch.Tensor, row_seg: torch.Tensor,
                seg_row0: torch.Tensor, seg_slot: torch.Tensor, segments: int, single_rows: bool = False,
                echo: Optional[tuple] = None, silu: bool = False, rounded: bool = False):
    """y[t, c] = sum_j taps[c, j] * x[t - L + 1 + j, c] (+ bias[c]) over the step's segments, float32. ``x`` float32
    [rows, channels] (rows may lie apart), ``taps`` [channels, L] with the last column the current token's, ``state``
    float32 [slots, channels, L - 1]: the inputs before each segment's first row, read and moved on. ``echo`` = (first
    channel, count): those channels are written once more behind the others (the output is then that much wider).
    ``single_rows``: every segment is one row. ``silu``: y passes silu. ``rounded``: y is returned twice, (float32, bfloat16)."""
    _dev(taps, bias, state, row_seg, seg_row0, seg_slot)
    _dev_rows(x, "x")
    for name, t in (("x", x), ("taps", taps), ("state", state)):
        _want(t, torch.float32, name)
    rows, channels = x.shape
    L = taps.shape[1]
    if taps.shape != (channels, L) or state.dim() != 3 or state.shape[1:] != (channels, L - 1):
        raise KernelError(f"causal_conv: x {tuple(x.shape)}, taps {tuple(taps.shape)}, state {tuple(state.shape)}")
    if bias is not None and (bias.dtype != torch.float32 or bias.shape != (channels,)):
        raise KernelError("causal_conv: the bias is float32 [channels]")
    for name, t, n in (("row_seg", row_seg, rows), ("seg_row0", seg_row0, segments + 1), ("seg_slot", seg_slot, segments)):
        _want(t, torch.int32, name)
        if t.numel() < n:
            raise KernelError(f"causal_conv: {name} holds {t.numel()} entries, needs {n}")
    first, count = echo if echo is not None else (0, 0)
    if count and not (0 <= first and first + count <= channels):
        raise KernelError(f"causal_conv: channels {first}..{first + count} of {channels}")
    out = torch.empty((rows, channels + count), dtype=torch.float32, device=x.device)
    short = torch.empty((rows, channels), dtype=torch.bfloat16, device=x.device) if rounded else None
    stride = x.stride(0) if rows > 1 else max(channels, x.stride(0))
    _check(library().fw_causal_conv(_p(x), stride, _p(taps), _p(bias), _p(state), _p(row_seg), _p(seg_row0), _p(seg_slot), _p(out),
                                    channels + count, int(first), int(count), channels, int(silu), _p(short), rows, int(segments), channels, L,
                                    state.shape[0], int(bool(single_rows)), _stream()))
    return (out, short) if rounded else out


SCAN_LONG = 256     # rows of a segment beyond which the recurrence walks it in chunks side by side


def rglru_scan(u: torch.Tensor, gates: torch.Tensor, y: torch.Tensor, r_bias: torch.Tensor, i_bias: torch.Tensor, lam: torch.Tensor,
               rate: float, state: torch.Tensor, seg_row0: torch.Tensor, seg_slot: torch.Tensor, segments: int, block_width: int,
               out_dtype: torch.dtype) -> torch.Tensor:
    """The gated linear recurrence per channel over the step's segments: r = sigmoid(g_r + r_bias), i = sigmoid(g_i +
    i_bias), a = exp(-rate r softplus(lam)), S <- a S + sqrt(1 - a^2) i u, out = S * gelu_tanh(y). ``u``, ``y`` float32
    [rows, channels] (rows may lie apart); ``gates`` float32 [rows, 2 channels], block after block [g_r of the block | g_i
    of the block]; ``state`` float32 [slots, channels], read and moved on."""
    _dev(gates, r_bias, i_bias, lam, state, seg_row0, seg_slot)
    _dev_rows(u, "u")
    _dev_rows(y, "y")
    rows, channels = u.shape
    for name, t in (("u", u), ("gates", gates), ("y", y), ("r_bias", r_bias), ("i_bias", i_bias), ("lam", lam), ("state", state)):
        _want(t, torch.float32, name)
    if y.shape != (rows, channels) or gates.shape != (rows, 2 * channels) or channels % block_width or state.dim() != 2 \
            or state.shape[1] != channels or any(t.numel() != channels for t in (r_bias, i_bias, lam)):
        raise KernelError(f"rglru_scan: u {tuple(u.shape)}, gates {tuple(gates.shape)}, y {tuple(y.shape)}, state {tuple(state.shape)}, "
                          f"blocks of {block_width}")
    for name, t, n in (("seg_row0", seg_row0, segments + 1), ("seg_slot", seg_slot, segments)):
        _want(t, torch.int32, name)
        if t.numel() < n:
            raise KernelError(f"rglru_scan: {name} holds {t.numel()} entries, needs {n}")
    out = torch.empty((rows, channels), dtype=out_dtype, device=u.device)
    # a step that may hold a long segment: the kernels walk such a one in chunks side by side and need room for it
    workspace = torch.empty((2, rows, channels), dtype=torch.float32, device=u.device) if rows > SCAN_LONG else None

    def stride(t: torch.Tensor) -> int:
        return t.stride(0) if rows > 1 else max(channels, t.stride(0))

    _check(library().fw_rglru_scan(_p(u), stride(u), _p(gates), 2 * channels, _p(y), stride(y), _p(r_bias), _p(i_bias), _p(lam),
                                   ctypes.c_float(rate), _p(state), _p(seg_row0), _p(seg_slot), _p(out), _code(out_dtype), rows,
                                   int(segments), channels, int(block_width), state.shape[0], _p(workspace), _stream()))
    return out


# ---- a residual stream of several rows side by side ----------------------------------------------------------------
NEXT_SUM, NEXT_TANH = 1, 2
SOURCE_ROWS, SOURCE_BRANCHES, SOURCE_CHOSEN = 0, 1, 2
MAX_STREAMS = 32


def _reader(kind: int, streams: int, hidden: int, reader_in: Optional[torch.Tensor], weight: Optional[torch.Tensor],
            bias: Optional[torch.Tensor], alpha: Optional[torch.Tensor]) -> tuple:
    for name, t, shape in (("reader_in", reader_in, (streams,)), ("weight", weight, (hidden,)), ("bias", bias, (hidden,))):
        if t is not None:
            _want(t, torch.float32, name)
            if t.shape != shape:
                raise KernelError(f"streams: {name} is {tuple(t.shape)}, expected {shape}")
    if kind == NEXT_TANH and (weight is None or bias is None or alpha is None or alpha.dtype != torch.float32 or alpha.numel() != 1):
        raise KernelError("streams: the tanh norm has a weight, a bias and one float32 alpha")
    return int(kind), _p(reader_in), _p(weight), _p(bias), _p(alpha)


def stream_read(x: torch.Tensor, reader_in: Optional[torch.Tensor], out_dtype: torch.dtype, *, kind: int = NEXT_SUM,
                weight: Optional[torch.Tensor] = None, bias: Optional[torch.Tensor] = None, alpha: Optional[torch.Tensor] = None,
                row_index: Optional[torch.Tensor] = None) -> torch.Tensor:
    """u = sum_s reader_in[s] x_s of the streams ``x`` float32 [rows, streams, hidden] (``reader_in`` None: their plain sum),
    as it is (``NEXT_SUM``) or through the norm tanh(alpha u) weight + bias (``NEXT_TANH``); rows gathered through
    ``row_index`` if given."""
    _dev(x, reader_in, weight, bias, alpha, row_index)
    _want(x, torch.float32, "x")
    if x.dim() != 3 or kind not in (NEXT_SUM, NEXT_TANH):
        raise KernelError(f"stream_read: the streams are {tuple(x.shape)}, kind {kind}")
    rows, streams, hidden = x.shape
    if row_index is not None:
        _want(row_index, torch.int32, "row_index")
        rows = row_index.numel()
    out = torch.empty((rows, hidden), dtype=out_dtype, device=x.device)
    _check(library().fw_stream_read(_p(x), streams, *_reader(kind, streams, hidden, reader_in, weight, bias, alpha), _p(row_index), _p(out),
                                    _code(out_dtype), rows, hidden, _stream()))
    return out


def stream_join_(x: torch.Tensor, ls: torch.Tensor, mix: torch.Tensor, out_weight: torch.Tensor, a: torch.Tensor, *,
                 branches: Optional[tuple] = None, chosen: Optional[tuple] = None, next_kind: int = NEXT_NOTHING,
                 next_in: Optional[torch.Tensor] = None, next_weight: Optional[torch.Tensor] = None,
                 next_bias: Optional[torch.Tensor] = None, next_alpha: Optional[torch.Tensor] = None,
                 next_dtype: Optional[torch.dtype] = None) -> Optional[torch.Tensor]:
    """In place on the streams ``x`` float32 [rows, streams, hidden]: x_t <- sum_s mix[s, t] x_s + out_weight[t] * (ls * y).
    y is ``a`` [rows, hidden]; with ``branches`` = (b, weight_a, weight_b, scale_a, scale_b, eps) it is scale_a rms(a) weight_a +
    scale_b rms(b) weight_b; with ``chosen`` = (choice_weight, pair_place, b or None, gate or None) it is the sum of the rows of
    ``a`` [places, hidden] that each row chose, in order, plus sigmoid(gate) b (``gate`` float32, one number a row, rows may lie
    apart; b [rows, hidden]). ``next_kind`` NEXT_SUM or NEXT_TANH: what reads the streams next (see ``stream_read``) is formed in
    the same kernel and returned in ``next_dtype``."""
    _dev(x, ls, mix, out_weight, a, next_in, next_weight, next_bias, next_alpha)
    for name, t in (("x", x), ("ls", ls), ("mix", mix), ("out_weight", out_weight), ("a", a)):
        _want(t, torch.float32, name)
    if x.dim() != 3:
        raise KernelError(f"stream_join: the streams are {tuple(x.shape)}, expected [rows, streams, hidden]")
    rows, streams, hidden = x.shape
    if ls.shape != (hidden,) or mix.shape != (streams, streams) or out_weight.shape != (streams,) or next_kind not in (NEXT_NOTHING, NEXT_SUM, NEXT_TANH):
        raise KernelError(f"stream_join: streams {tuple(x.shape)}, scales {tuple(ls.shape)}, mix {tuple(mix.shape)}, kind {next_kind}")
    source, b, weight_a, weight_b, scale_a, scale_b, eps = SOURCE_ROWS, None, None, None, 1.0, 1.0, 0.0
    choice_weight, pair_place, top, gate = None, None, 0, None
    places = rows
    if branches is not None:
        source = SOURCE_BRANCHES
        b, weight_a, weight_b, scale_a, scale_b, eps = branches
        for name, t, shape in (("b", b, (rows, hidden)), ("weight_a", weight_a, (hidden,)), ("weight_b", weight_b, (hidden,))):
            _dev(t)
            if t is None or t.dtype != torch.float32 or t.shape != shape:
                raise KernelError(f"stream_join: {name} must be float32 {shape}")
    elif chosen is not None:
        source = SOURCE_CHOSEN
        choice_weight, pair_place, b, gate = chosen
        _dev(choice_weight, pair_place, b)
        _want(choice_weight, torch.float32, "choice_weight")
        _want(pair_place, torch.int32, "pair_place")
        top = choice_weight.shape[1]
        places = rows * top
        if choice_weight.shape != (rows, top) or pair_place.shape != (rows, top):
            raise KernelError(f"stream_join: weights {tuple(choice_weight.shape)} and places {tuple(pair_place.shape)} of {rows} rows")
        if b is not None and (b.dtype != torch.float32 or b.shape != (rows, hidden)):
            raise KernelError(f"stream_join: b is {tuple(b.shape)}, expected float32 {(rows, hidden)}")
        if gate is not None:
            _dev_rows(gate, "gate")
            if b is None or gate.dtype != torch.float32 or gate.shape != (rows, 1):
                raise KernelError(f"stream_join: a gate is one float32 number a row beside rows to gate, found {tuple(gate.shape)}")
    if a.shape != (places, hidden):
        raise KernelError(f"stream_join: a is {tuple(a.shape)}, expected {(places, hidden)}")
    out = torch.empty((rows, hidden), dtype=next_dtype or torch.float32, device=x.device) if next_kind != NEXT_NOTHING else None
    _check(library().fw_stream_join(
        _p(x), streams, _p(ls), _p(mix), _p(out_weight), source, _p(a), _p(b), _p(weight_a), _p(weight_b), ctypes.c_float(scale_a),
        ctypes.c_float(scale_b), ctypes.c_float(eps), _p(choice_weight), _p(pair_place), int(top), _p(gate),
        _stride(gate) if gate is not None else 0, *_reader(next_kind, streams, hidden, next_in, next_weight, next_bias, next_alpha), _p(out),
        _code(out.dtype) if out is not None else F32, rows, hidden, _stream()))
    return out


# ---- a linear recurrence over a matrix state per head with a fixed decay -------------------------------------------------
def _segments(name: str, segments: int, seg_row0: torch.Tensor, seg_slot: torch.Tensor) -> None:
    _dev(seg_row0, seg_slot)
    for which, t, n in (("seg_row0", seg_row0, segments + 1), ("seg_slot", seg_slot, segments)):
        _want(t, torch.int32, which)
        if t.numel() < n:
            raise KernelError(f"{name}: {which} holds {t.numel()} entries, needs {n}")


MAX_DECAY_DIM = 256      # key channels of a head


def _chunks(name: str, chunks: Optional[tuple], segments: int):
    """(chunk_seg, chunk_row0, seg_chunk0, rows beyond which a segment is walked in chunks, whether every segment of the step is
    that long) -> a launch's arguments: the arrays, their number, the rows, the flag."""
    if chunks is None:
        return (None, None, None), 0, 0, 0
    chunk_seg, chunk_row0, seg_chunk0, long_rows, all_long = chunks
    _dev(chunk_seg, chunk_row0, seg_chunk0)
    count = chunk_seg.numel()
    for which, t, n in (("chunk_seg", chunk_seg, count), ("chunk_row0", chunk_row0, count), ("seg_chunk0", seg_chunk0, segments + 1)):
        _want(t, torch.int32, which)
        if t.numel() < n:
            raise KernelError(f"{name}: {which} holds {t.numel()} entries, needs {n}")
    return (chunk_seg, chunk_row0, seg_chunk0), count, int(long_rows), int(all_long)


DECAY_CHUNK = 64        # rows of a chunk, as the kernels have them


def decay_powers(decays, device) -> torch.Tensor:
    """decay^0 .. decay^chunk of every head, formed in float64: float32 [heads, chunk + 1]."""
    if library().fw_decay_chunk_rows() != DECAY_CHUNK or library().fw_scan_chunk_rows() != DECAY_CHUNK:
        raise KernelError("the kernel library's chunks are of another length")
    exponents = torch.arange(DECAY_CHUNK + 1, dtype=torch.float64)
    return torch.pow(torch.as_tensor(decays, dtype=torch.float64)[:, None], exponents[None, :]).to(dtype=torch.float32, device=device)


def decay_recurrence(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, powers: torch.Tensor, state: torch.Tensor, seg_row0: torch.Tensor,
                     seg_slot: torch.Tensor, segments: int, heads: int, dim: int, vdim: int, chunks: Optional[tuple] = None) -> torch.Tensor:
    """Per head S <- decay S + silu(k) silu(v)^T, o = S^T silu(q) over each segment's rows in order. ``q``, ``k`` float32
    [rows, heads dim] and ``v`` [rows, heads vdim] with one row stride (views of wider rows will do); ``powers``: see
    ``decay_powers``; ``state`` float32 [slots, heads, dim, vdim] is read and moved on. ``chunks`` (chunk_seg, chunk_row0, seg_chunk0,
    long_rows, whether every segment is longer than that): segments of more than long_rows rows are walked in these chunks side by side. Returns float32 [rows, heads vdim]."""
    _dev(powers, state)
    _segments("decay_recurrence", segments, seg_row0, seg_slot)
    rows = q.shape[0]
    for name, t, width in (("q", q, heads * dim), ("k", k, heads * dim), ("v", v, heads * vdim)):
        _dev_rows(t, name)
        _want(t, torch.float32, name)
        if t.shape != (rows, width):
            raise KernelError(f"decay_recurrence: {name} is {tuple(t.shape)}, expected {(rows, width)}")
    if rows > 1 and not (q.stride(0) == k.stride(0) == v.stride(0)):
        raise KernelError("decay_recurrence: q, k and v have one row stride")
    stride = max(_stride(q), _stride(k), _stride(v))
    for name, t, shape in (("powers", powers, (heads, DECAY_CHUNK + 1)), ("state", state[0], (heads, dim, vdim))):
        _want(t, torch.float32, name)
        if t.shape != shape:
            raise KernelError(f"decay_recurrence: {name} is {tuple(t.shape)}, expected {shape}")
    out = torch.empty((rows, heads * vdim), dtype=torch.float32, device=q.device)
    places, count, *how = _chunks("decay_recurrence", chunks, segments)
    workspace = torch.empty((count, heads, dim, vdim), dtype=torch.float32, device=q.device) if count else None
    _check(library().fw_decay_recurrence(_p(q), _p(k), _p(v), stride, _p(powers), _p(state), state.shape[0], _p(out), _p(seg_row0),
                                         _p(seg_slot), rows, int(segments), heads, dim, vdim, *(_p(t) for t in places), count, *how,
                                         _p(workspace), _stream()))
    return out


# ---- the selective scan ---------------------------------------------------------------------------------------------
MAX_SCAN_STATES = 128


def selective_scan(x: torch.Tensor, z: torch.Tensor, bc: torch.Tensor, gate: torch.Tensor, A2: torch.Tensor, D: torch.Tensor,
                   state: torch.Tensor, seg_row0: torch.Tensor, seg_slot: torch.Tensor, segments: int, out_dtype: torch.dtype,
                   chunks: Optional[tuple] = None) -> torch.Tensor:
    """Per channel c and state n, with dt = softplus(z): S <- 2^(dt A2[n, c]) S + dt x B[n], y = sum_n S C[n] + D x, out = y *
    silu(gate), over each segment's rows in order. ``x``, ``z``, ``gate`` float32 [rows, channels], ``bc`` float32 [rows, 2 states]
    (B, then C); rows may lie apart. ``A2`` [states, channels] and ``D`` [channels] float32; ``state`` float32 [slots, states,
    channels] is read and moved on. ``chunks``: as for ``decay_recurrence``. Returns [rows, channels] of ``out_dtype``."""
    _dev(A2, D, state)
    _segments("selective_scan", segments, seg_row0, seg_slot)
    rows, channels = x.shape
    states = A2.shape[0]
    for name, t, shape in (("x", x, (rows, channels)), ("z", z, (rows, channels)), ("bc", bc, (rows, 2 * states)), ("gate", gate, (rows, channels))):
        _dev_rows(t, name)
        _want(t, torch.float32, name)
        if t.shape != shape:
            raise KernelError(f"selective_scan: {name} is {tuple(t.shape)}, expected {shape}")
    for name, t, shape in (("A2", A2, (states, channels)), ("D", D, (channels,)), ("state", state[0], (states, channels))):
        _want(t, torch.float32, name)
        if t.shape != shape:
            raise KernelError(f"selective_scan: {name} is {tuple(t.shape)}, expected {shape}")
    out = torch.empty((rows, channels), dtype=out_dtype, device=x.device)
    places, count, *how = _chunks("selective_scan", chunks, segments)
    workspace = torch.empty((count, states + 1, channels), dtype=torch.float32, device=x.device) if count else None
    _check(library().fw_selective_scan(_p(x), _stride(x), _p(z), _stride(z), _p(bc), _stride(bc), _p(gate), _stride(gate), _p(A2), _p(D), _p(state),
                                       state.shape[0], _p(out), _code(out_dtype), _p(seg_row0), _p(seg_slot), rows, int(segments), channels,
                                       states, *(_p(t) for t in places), count, *how, _p(workspace), _stream()))
    return out


def low_rank_weights(w: torch.Tensor) -> torch.Tensor:
    """A map [channels, rank] as ``selective_scan_low_rank`` reads it: [rank, channels], or of bfloat16 [rank / 2, channels, 2]."""
    channels, rank = w.shape
    if w.dtype == torch.bfloat16 and rank % 2 == 0:
        return w.view(channels, rank // 2, 2).permute(1, 0, 2).contiguous()
    return w.to(torch.float32).t().contiguous()


def selective_scan_low_rank(x: torch.Tensor, low: torch.Tensor, w: torch.Tensor, bias: torch.Tensor, gate: torch.Tensor, A2: torch.Tensor,
                            D: torch.Tensor, state: torch.Tensor, seg_slot: torch.Tensor, out_dtype: torch.dtype) -> torch.Tensor:
    """``selective_scan`` over segments of one row each (row r is segment r), with the map in front of the step sizes: z = low[:,
    :rank] . W^T + bias. ``low`` float32 [rows, rank + 2 states] (the low part, B, C; rows may lie apart); ``w`` from
    ``low_rank_weights``."""
    _dev(A2, D, state, w, bias, seg_slot)
    _want(seg_slot, torch.int32, "seg_slot")
    rows, channels = x.shape
    states = A2.shape[0]
    rank = w.shape[0] * (2 if w.dim() == 3 else 1)
    for name, t, shape in (("x", x, (rows, channels)), ("low", low, (rows, rank + 2 * states)), ("gate", gate, (rows, channels))):
        _dev_rows(t, name)
        _want(t, torch.float32, name)
        if t.shape != shape:
            raise KernelError(f"selective_scan_low_rank: {name} is {tuple(t.shape)}, expected {shape}")
    for name, t, shape in (("A2", A2, (states, channels)), ("D", D, (channels,)), ("bias", bias, (channels,)), ("state", state[0], (states, channels))):
        _want(t, torch.float32, name)
        if t.shape != shape:
            raise KernelError(f"selective_scan_low_rank: {name} is {tuple(t.shape)}, expected {shape}")
    if w.shape != ((rank // 2, channels, 2) if w.dim() == 3 else (rank, channels)) or w.dtype != (torch.bfloat16 if w.dim() == 3 else torch.float32) \
            or seg_slot.numel() < rows:
        raise KernelError(f"selective_scan_low_rank: w is {tuple(w.shape)} {w.dtype}, {seg_slot.numel()} slots for {rows} rows")
    out = torch.empty((rows, channels), dtype=out_dtype, device=x.device)
    _check(library().fw_selective_scan_low_rank(_p(x), _stride(x), _p(low), _stride(low), rank, _p(w), _code(w.dtype), _p(bias), _p(gate),
                                                _stride(gate), _p(A2), _p(D), _p(state), state.shape[0], _p(out), _code(out_dtype),
                                                _p(seg_slot), rows, channels, states, _stream()))
    return out
