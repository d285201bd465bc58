"""Tensor-level entry points of the HIP kernels.

Each function checks on the host that shapes, dtypes, devices and layouts are what the kernel
and its grid assume, then launches on torch's current HIP stream.  There is no other code path:
a tensor that is not on the GPU, or a missing kernel library, is an error.
"""
from __future__ import annotations

import ctypes
from typing import Optional

import torch

from .library import KernelError, check, hip_lib

F32, BF16 = 0, 1
_DTYPE_CODE = {torch.float32: F32, torch.bfloat16: BF16}


def dtype_code(dt: torch.dtype) -> int:
    try:
        return _DTYPE_CODE[dt]
    except KeyError:
        raise KernelError(f"unsupported dtype {dt}; kernels take float32 and bfloat16") from None


_RAW_STREAM = getattr(torch._C, "_cuda_getCurrentRawStream", None)
_RAW_DEVICE = getattr(torch._C, "_cuda_getDevice", None) or torch.cuda.current_device


def _stream() -> int:
    """Handle of torch's current stream on the current device (also while a graph is captured).
    The raw accessor costs a fraction of a microsecond; ``torch.cuda.current_stream()`` some ten,
    once per launch."""
    if _RAW_STREAM is not None:
        return _RAW_STREAM(_RAW_DEVICE())
    return torch.cuda.current_stream().cuda_stream


def _dev(t: torch.Tensor, name: str, dtype: Optional[torch.dtype] = None, contiguous: bool = True):
    if not isinstance(t, torch.Tensor):
        raise KernelError(f"{name}: expected a tensor, got {type(t).__name__}")
    if not t.is_cuda:
        raise KernelError(f"{name}: tensor is on {t.device}; the kernels run on the GPU only")
    if dtype is not None and t.dtype != dtype:
        raise KernelError(f"{name}: dtype {t.dtype}, expected {dtype}")
    if contiguous and not t.is_contiguous():
        raise KernelError(f"{name}: tensor must be contiguous")
    return t.data_ptr()


def _opt(t: Optional[torch.Tensor], name: str, dtype: Optional[torch.dtype] = None):
    return None if t is None else _dev(t, name, dtype)


def k_chunk(head_dim: int) -> int:
    """Elements of a key that lie next to each other inside a K page (``csrc/kv_layout.h``)."""
    return 4 if head_dim % 8 else 8


def k_page_shape(num_kv_heads: int, head_dim: int) -> tuple:
    """Per-token shape of the K cache array: a key as ``head_dim / C`` chunks of ``C`` elements; the
    page's token axis lies between the two (``[kv_heads, head_dim / C, page_size, C]``)."""
    c = k_chunk(head_dim)
    return (num_kv_heads, head_dim // c, c)


def keys_to_pages(k: torch.Tensor) -> torch.Tensor:
    """Keys ``[..., page_size, head_dim]`` (row by row) in the cache's layout
    ``[..., head_dim / C, page_size, C]``."""
    *lead, page, d = k.shape
    c = k_chunk(d)
    return k.reshape(*lead, page, d // c, c).transpose(-3, -2).contiguous()


def pages_to_keys(k: torch.Tensor) -> torch.Tensor:
    """The inverse of :func:`keys_to_pages`: ``[..., head_dim / C, page_size, C]`` to ``[..., page_size, head_dim]``."""
    *lead, chunks, page, c = k.shape
    return k.transpose(-3, -2).reshape(*lead, page, chunks * c)


def check_cache_shapes(what: str, k_cache: torch.Tensor, v_cache: torch.Tensor, num_kv_heads: int,
                       head_dim: int) -> int:
    """K pages are [kv_heads, head_dim / C, page_size, C] (a key in chunks of C = 8 elements, the chunks
    of a page's keys next to each other: ``csrc/kv_layout.h``); V pages are transposed, [kv_heads,
    head_dim, page_size].  Returns the page size."""
    if k_cache.dim() != 5 or v_cache.dim() != 4:
        raise KernelError(f"{what}: the K cache must be 5-D and the V cache 4-D")
    pages, nkv, chunks, ps, c = k_cache.shape
    if (nkv, chunks, c) != k_page_shape(num_kv_heads, head_dim) or tuple(v_cache.shape) != (pages, nkv, head_dim, ps):
        raise KernelError(f"{what}: K cache {tuple(k_cache.shape)} / V cache {tuple(v_cache.shape)} are "
                          f"not [pages, {num_kv_heads}, {head_dim} / C, page, C] / [pages, {num_kv_heads}, "
                          f"{head_dim}, page] with C = {k_chunk(head_dim)}")
    return int(ps)


# --------------------------------------------------------------------------------------
def embed_gather(table: torch.Tensor, ids: torch.Tensor, out: torch.Tensor,
                 feedback: Optional[torch.Tensor] = None, scale: float = 1.0,
                 copy: Optional[torch.Tensor] = None) -> torch.Tensor:
    """out[t, :] = table[ids[t], :] * scale, converted to out's dtype; ``copy`` (out's shape and dtype)
    receives the rows a second time.  A negative id ``-1 - r`` stands
    for ``feedback[r]`` (a token still on the device); the caller guarantees ``r`` is inside
    ``feedback`` and that no id is negative when there is none.  An id outside the table (only
    what a kernel left in ``feedback`` can be: the host checks the ids it uploads) reads the
    nearest row of it."""
    rows, width = out.shape
    if table.dim() != 2 or table.shape[1] != width or ids.shape != (rows,):
        raise KernelError(f"embed_gather: shapes table {tuple(table.shape)} ids {tuple(ids.shape)} "
                          f"out {tuple(out.shape)} do not fit")
    if copy is not None and (copy.shape != out.shape or copy.dtype != out.dtype):
        raise KernelError("embed_gather: the second copy has out's shape and dtype")
    check(hip_lib().kva_embed_gather(_dev(out, "out"), _opt(copy, "copy"), _dev(table, "table"),
                                     _dev(ids, "ids", torch.int32),
                                     _opt(feedback, "feedback", torch.int32), rows, width, table.shape[0],
                                     dtype_code(table.dtype), dtype_code(out.dtype), float(scale), _stream()),
          "embed_gather")
    return out


def embed_gather_prep(table: torch.Tensor, ids: torch.Tensor, hidden: torch.Tensor, scaled: torch.Tensor,
                      sumsq: torch.Tensor, norm_weight: torch.Tensor,
                      feedback: Optional[torch.Tensor] = None) -> torch.Tensor:
    """:func:`embed_gather` for a bf16 table and stream that prepares the first norm in the same
    pass: ``scaled = round(hidden * norm_weight)`` and ``sumsq[t, 0] = sum(hidden[t]^2)``."""
    rows, width = hidden.shape
    if table.dim() != 2 or table.shape[1] != width or ids.shape != (rows,) or scaled.shape != (rows, width) \
            or sumsq.shape != (rows, 1) or norm_weight.shape != (width,):
        raise KernelError(f"embed_gather_prep: shapes table {tuple(table.shape)} ids {tuple(ids.shape)} hidden "
                          f"{tuple(hidden.shape)} scaled {tuple(scaled.shape)} sumsq {tuple(sumsq.shape)} do not fit")
    if not (table.dtype == hidden.dtype == scaled.dtype == torch.bfloat16) or width % 8 \
            or norm_weight.dtype not in (torch.bfloat16, torch.float32):
        raise KernelError("embed_gather_prep: bf16 table and outputs, a width that is a multiple of 8")
    check(hip_lib().kva_embed_gather_prep(
        _dev(hidden, "hidden"), _dev(scaled, "scaled"), _dev(sumsq, "sumsq", torch.float32), _dev(table, "table"),
        _dev(ids, "ids", torch.int32), _opt(feedback, "feedback", torch.int32), _dev(norm_weight, "norm_weight"),
        1 if norm_weight.dtype == torch.float32 else 0, rows, width, table.shape[0], _stream()), "embed_gather_prep")
    return hidden


class PartialSums:
    """A branch output that has not been added up yet: ``parts`` fp32 ``[ranges, rows, width]``, the
    products of :func:`gemm_skinny_partials` over ranges of K.  It stands where a bf16 ``[rows,
    width]`` delta stands; the norm kernel that adds the delta to the stream adds the ranges first
    (and rounds their sum to bf16, as the whole product would have been).  ``materialize()`` gives
    the plain delta."""

    def __init__(self, parts: torch.Tensor):
        if parts.dim() != 3 or parts.dtype != torch.float32:
            raise KernelError("PartialSums: fp32 [ranges, rows, width] needed")
        self.parts = parts

    @property
    def shape(self):
        return self.parts.shape[1:]

    @property
    def dtype(self):
        return torch.bfloat16

    @property
    def device(self):
        return self.parts.device

    def materialize(self) -> torch.Tensor:
        total = self.parts[0].clone()           # the ranges in order, by element-wise kernels only
        for r in range(1, self.parts.shape[0]):
            total += self.parts[r]
        return total.to(torch.bfloat16)


class AttentionPartials:
    """An attention output that has not been added up yet: what :func:`attention_mfma` leaves per
    key range when it is told to (``leave_partials``): ``part_o`` fp32 ``[tokens * heads, parts,
    head_dim]`` and ``part_ml`` fp32 ``[tokens * heads, parts, 2]`` (maximum in the base-2 domain,
    sum of exponentials).  It stands where the bf16 ``[tokens, heads * head_dim]`` output stands,
    for a consumer that adds the ranges up itself (:func:`gemv_merged`)."""

    def __init__(self, part_o: torch.Tensor, part_ml: torch.Tensor, tokens: int, heads: int):
        if part_o.dim() != 3 or part_o.dtype != torch.float32 or part_o.shape[0] != tokens * heads \
                or part_ml.shape != (tokens * heads, part_o.shape[1], 2) or part_ml.dtype != torch.float32:
            raise KernelError("AttentionPartials: fp32 [tokens * heads, parts, head_dim] and [tokens * heads, parts, 2] needed")
        self.part_o, self.part_ml, self.tokens, self.heads = part_o, part_ml, tokens, heads

    @property
    def parts(self) -> int:
        return self.part_o.shape[1]

    @property
    def head_dim(self) -> int:
        return self.part_o.shape[2]

    @property
    def shape(self):
        return (self.tokens, self.heads * self.head_dim)

    @property
    def dtype(self):
        return torch.bfloat16

    @property
    def device(self):
        return self.part_o.device


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float, out: torch.Tensor,
            delta=None, row_idx: Optional[torch.Tensor] = None) -> torch.Tensor:
    """out = rmsnorm(x) * weight.  With ``delta`` (a tensor like x, or :class:`PartialSums`): x +=
    delta first (in place, fp32 add).  With ``row_idx``: out[i] = rmsnorm(x[row_idx[i]])."""
    width = x.shape[-1]
    out_rows = out.shape[0]
    if x.dim() != 2 or out.dim() != 2 or out.shape[1] != width or weight.shape != (width,):
        raise KernelError(f"rmsnorm: shapes x {tuple(x.shape)} weight {tuple(weight.shape)} out "
                          f"{tuple(out.shape)} do not fit")
    if out.dtype != x.dtype:
        raise KernelError("rmsnorm: out must have x's dtype")
    if row_idx is None:
        if out_rows != x.shape[0]:
            raise KernelError("rmsnorm: out needs as many rows as x")
    elif row_idx.shape != (out_rows,):
        raise KernelError("rmsnorm: one row index per output row")
    parts = None
    if isinstance(delta, PartialSums):
        if tuple(delta.shape) != tuple(x.shape) or x.dtype != torch.bfloat16 or width % 8:
            raise KernelError("rmsnorm: partial sums stand in for a bf16 delta of x's shape, width a multiple of 8")
        parts, delta = delta.parts, None
    if delta is not None and (delta.shape != x.shape or delta.dtype != x.dtype):
        raise KernelError("rmsnorm: delta must match x")
    check(hip_lib().kva_rmsnorm(_dev(out, "out"), _dev(x, "x"), _opt(delta, "delta"),
                                _dev(weight, "weight"), _opt(row_idx, "row_idx", torch.int32),
                                out_rows, width, float(eps), dtype_code(x.dtype),
                                dtype_code(weight.dtype), _opt(parts, "partial sums", torch.float32),
                                parts.shape[0] if parts is not None else 0,
                                parts.shape[1] if parts is not None else 0, _stream()), "rmsnorm")
    return out


def residual_add(hidden: torch.Tensor, delta: torch.Tensor) -> torch.Tensor:
    if hidden.shape != delta.shape or hidden.dtype != delta.dtype:
        raise KernelError("residual_add: operands must match")
    check(hip_lib().kva_residual_add(_dev(hidden, "hidden"), _dev(delta, "delta"), hidden.numel(),
                                     dtype_code(hidden.dtype), _stream()), "residual_add")
    return hidden


def stream_read(x: torch.Tensor, workgroups: int, sink: torch.Tensor) -> None:
    """A probe: reads ``x`` once and stores nothing (``sink``: any int32 device tensor, practically
    never written).  Its time is the floor of any kernel that reads as many bytes."""
    check(hip_lib().kva_stream_read(_dev(x, "x"), x.numel() * x.element_size(), int(workgroups),
                                    _dev(sink, "sink", torch.int32), _stream()), "stream_read")


def stream_reread(x: torch.Tensor, workgroups: int, repeats: int, sink: torch.Tensor) -> None:
    """A probe: every one of ``workgroups`` workgroups reads all of ``x``, ``repeats`` times over,
    through the caches.  With an ``x`` that fits a die's L2: what a compute unit takes in from there."""
    check(hip_lib().kva_stream_reread(_dev(x, "x"), x.numel() * x.element_size(), int(workgroups), int(repeats),
                                      _dev(sink, "sink", torch.int32), _stream()), "stream_reread")


def stream_mixed(own: Optional[torch.Tensor], shared: Optional[torch.Tensor], workgroups: int,
                 sink: torch.Tensor) -> None:
    """A probe: half of each workgroup's wavefronts stream the workgroup's own 1/``workgroups`` of
    ``own`` from memory while the other half read all of ``shared`` (from L2); either may be None."""
    if int(workgroups) < 1:
        raise KernelError("stream_mixed: at least one workgroup")
    own_bytes = 0 if own is None else own.numel() * own.element_size() // int(workgroups) // 16 * 16
    shared_bytes = 0 if shared is None else shared.numel() * shared.element_size() // 16 * 16
    check(hip_lib().kva_stream_mixed(None if own is None else _dev(own, "own"), own_bytes,
                                     None if shared is None else _dev(shared, "shared"), shared_bytes,
                                     int(workgroups), _dev(sink, "sink", torch.int32), _stream()), "stream_mixed")


def probe_read_bandwidth(device, megabytes: int = 2048, workgroups: int = 2048, reps: int = 5) -> float:
    """GB/s of a plain read stream over a buffer far larger than every cache, best of ``reps``."""
    x = torch.empty(megabytes << 20, dtype=torch.uint8, device=device)
    x.zero_()
    sink = torch.zeros(4, dtype=torch.int32, device=device)
    stream_read(x, workgroups, sink)
    best = 0.0
    for _ in range(reps):
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        stream_read(x, workgroups, sink)
        b.record()
        b.synchronize()
        best = max(best, x.numel() / (a.elapsed_time(b) * 1e-3) / 1e9)
    return best


def scale_softcap(x: torch.Tensor, scale: float, cap: float = 0.0) -> torch.Tensor:
    """In place: ``x *= scale``, then with ``cap > 0`` ``x = cap * tanh(x / cap)``."""
    if cap < 0:
        raise KernelError("scale_softcap: the cap must not be negative")
    check(hip_lib().kva_scale_softcap(_dev(x, "x"), x.numel(), float(scale), float(cap), dtype_code(x.dtype),
                                      _stream()), "scale_softcap")
    return x


def silu_mul(gate_up: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
    """out[t, i] = silu(gate_up[t, i]) * gate_up[t, I + i]."""
    rows, inter = out.shape
    if gate_up.shape != (rows, 2 * inter) or gate_up.dtype != out.dtype:
        raise KernelError(f"silu_mul: gate_up {tuple(gate_up.shape)} does not fit out {tuple(out.shape)}")
    check(hip_lib().kva_silu_mul(_dev(out, "out"), _dev(gate_up, "gate_up"), rows, inter,
                                 dtype_code(out.dtype), _stream()), "silu_mul")
    return out


def cast(src: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
    if src.shape != out.shape:
        raise KernelError("cast: shapes differ")
    if src.dtype == out.dtype:
        raise KernelError("cast: same dtype on both sides")
    check(hip_lib().kva_cast(_dev(out, "out"), _dev(src, "src"), src.numel(), dtype_code(src.dtype),
                             dtype_code(out.dtype), _stream()), "cast")
    return out


def rope_kv_write(qkv: torch.Tensor, positions: torch.Tensor, num_q_heads: int, num_kv_heads: int,
                  head_dim: int, cos: Optional[torch.Tensor], sin: Optional[torch.Tensor],
                  k_cache: Optional[torch.Tensor], v_cache: Optional[torch.Tensor],
                  slot_mapping: Optional[torch.Tensor], page_size: int) -> None:
    """Rotates the Q and K heads of ``qkv`` [T, (nq + 2 nkv) d] by the tokens' positions; Q in
    place, rotated K and plain V into the cache [pages, nkv, page_size, d] at ``slot_mapping``."""
    tokens = qkv.shape[0]
    if qkv.dim() != 2 or qkv.shape[1] != (num_q_heads + 2 * num_kv_heads) * head_dim:
        raise KernelError(f"rope_kv_write: qkv {tuple(qkv.shape)} is not [T, (nq + 2 nkv) * d]")
    if positions.shape != (tokens,):
        raise KernelError("rope_kv_write: one position per token")
    rot = 0
    if cos is not None:
        if sin is None or cos.shape != sin.shape or cos.dim() != 2:
            raise KernelError("rope_kv_write: cos and sin tables must be [positions, rot/2]")
        rot = 2 * cos.shape[1]
    write = k_cache is not None
    if write:
        if v_cache is None or slot_mapping is None:
            raise KernelError("rope_kv_write: K and V cache and a slot mapping are all needed")
        check_cache_shapes("rope_kv_write", k_cache, v_cache, num_kv_heads, head_dim)
        if k_cache.shape[3] != page_size:
            raise KernelError(f"rope_kv_write: cache pages hold {k_cache.shape[3]} tokens, not {page_size}")
        if k_cache.dtype != qkv.dtype or slot_mapping.shape != (tokens,):
            raise KernelError("rope_kv_write: cache dtype or slot mapping shape does not fit")
    check(hip_lib().kva_rope_kv_write(
        _dev(qkv, "qkv"), _opt(k_cache, "k_cache"), _opt(v_cache, "v_cache"),
        _opt(cos, "cos", torch.float32), _opt(sin, "sin", torch.float32),
        _dev(positions, "positions", torch.int32), _opt(slot_mapping, "slot_mapping", torch.int32),
        tokens, num_q_heads, num_kv_heads, head_dim, rot, page_size, 1 if write else 0,
        dtype_code(qkv.dtype), _stream()), "rope_kv_write")


def check_kv_cache_shapes(what: str, k_cache: torch.Tensor, v_cache: torch.Tensor, num_kv_heads: int,
                          head_dim: int, value_dim: int) -> int:
    """:func:`check_cache_shapes` for values of another size than the keys: V pages are
    ``[kv_heads, value_dim, page_size]``.  Returns the page size."""
    if value_dim == head_dim:
        return check_cache_shapes(what, k_cache, v_cache, num_kv_heads, head_dim)
    if k_cache.dim() != 5 or v_cache.dim() != 4:
        raise KernelError(f"{what}: the K cache must be 5-D and the V cache 4-D")
    pages, nkv, chunks, ps, c = k_cache.shape
    if (nkv, chunks, c) != k_page_shape(num_kv_heads, head_dim) or tuple(v_cache.shape) != (pages, nkv, value_dim, ps):
        raise KernelError(f"{what}: K cache {tuple(k_cache.shape)} / V cache {tuple(v_cache.shape)} are not "
                          f"[pages, {num_kv_heads}, {head_dim} / C, page, C] / [pages, {num_kv_heads}, {value_dim}, page]")
    return int(ps)


def attention_rowwise(q: torch.Tensor, q_row_stride: int, out: torch.Tensor, k_cache: torch.Tensor,
                      v_cache: torch.Tensor, block_table: torch.Tensor, tok_seat: torch.Tensor,
                      tok_pos: torch.Tensor, num_q_heads: int, num_kv_heads: int, head_dim: int,
                      scale: float, window: int = 0, keep_first: int = 0, sinks: Optional[torch.Tensor] = None,
                      value_dim: Optional[int] = None, chunk: int = 0) -> torch.Tensor:
    """Causal GQA attention of every token over its request's cached keys; ``q`` is a view whose
    rows are ``q_row_stride`` elements apart (the Q part of a fused QKV buffer).  With a
    ``window`` a query at position i sees key j when ``i - j < window`` or ``j < keep_first``; with a
    ``chunk`` when both lie in the same run of ``chunk`` positions counted from 0;
    ``sinks`` (fp32, one per query head) adds ``exp(sink)`` to every softmax denominator;
    ``value_dim`` is the size of a value where it differs from a key's."""
    tokens = out.shape[0]
    value_dim = head_dim if value_dim is None else int(value_dim)
    if out.shape != (tokens, num_q_heads * value_dim):
        raise KernelError("attention: out must be [T, nq * value size]")
    check_kv_cache_shapes("attention", k_cache, v_cache, num_kv_heads, head_dim, value_dim)
    if block_table.dim() != 2 or tok_seat.shape != (tokens,) or tok_pos.shape != (tokens,):
        raise KernelError("attention: block table [seats, blocks], one seat and position per token")
    if q.dtype != out.dtype or k_cache.dtype != out.dtype or v_cache.dtype != out.dtype:
        raise KernelError("attention: q, cache and out must share a dtype")
    if q.data_ptr() % 16 or q_row_stride < num_q_heads * head_dim:
        raise KernelError("attention: q view is misaligned or its stride is too small")
    if sinks is not None and (sinks.shape != (num_q_heads,) or sinks.dtype != torch.float32):
        raise KernelError("attention: sinks are fp32, one per query head")
    page_size = k_cache.shape[3]
    check(hip_lib().kva_attention_rowwise(
        _dev(out, "out"), _dev(q, "q", contiguous=False), q_row_stride, _dev(k_cache, "k_cache"),
        _dev(v_cache, "v_cache"), _dev(block_table, "block_table", torch.int32), block_table.shape[1],
        _dev(tok_seat, "tok_seat", torch.int32), _dev(tok_pos, "tok_pos", torch.int32), tokens,
        num_q_heads, num_kv_heads, head_dim, value_dim, page_size, float(scale), int(window), int(keep_first),
        int(chunk), _opt(sinks, "sinks"), dtype_code(out.dtype), _stream()), "attention_rowwise")
    return out


def latent_attention_rowwise(q: torch.Tensor, out: torch.Tensor, cache: torch.Tensor, block_table: torch.Tensor,
                             tok_seat: torch.Tensor, tok_pos: torch.Tensor, scale: float, window: int = 0,
                             keep_first: int = 0, sinks: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Causal attention over low-rank entries: ``cache`` ``[pages, page_size, key_dim]`` holds one
    row per token for all heads, ``q`` ``[T, heads, key_dim]`` rows of the same layout, ``out``
    ``[T, heads, rank]`` the weighted sums of the rows' first ``rank`` elements."""
    if q.dim() != 3 or out.dim() != 3 or cache.dim() != 3 or q.shape[:2] != out.shape[:2]:
        raise KernelError("latent attention: q [T, heads, key_dim], out [T, heads, rank], cache [pages, page, key_dim]")
    tokens, heads, key_dim = q.shape
    rank = out.shape[2]
    if cache.shape[2] != key_dim or rank > key_dim:
        raise KernelError(f"latent attention: rows of {cache.shape[2]} in the cache, queries of {key_dim}, rank {rank}")
    if block_table.dim() != 2 or tok_seat.shape != (tokens,) or tok_pos.shape != (tokens,):
        raise KernelError("latent attention: block table [seats, blocks], one seat and position per token")
    if q.dtype != out.dtype or cache.dtype != out.dtype:
        raise KernelError("latent attention: q, cache and out must share a dtype")
    if sinks is not None and (sinks.shape != (heads,) or sinks.dtype != torch.float32):
        raise KernelError("latent attention: sinks are fp32, one per head")
    check(hip_lib().kva_latent_attention_rowwise(
        _dev(out, "out"), _dev(q, "q"), _dev(cache, "cache"), _dev(block_table, "block_table", torch.int32),
        block_table.shape[1], _dev(tok_seat, "tok_seat", torch.int32), _dev(tok_pos, "tok_pos", torch.int32),
        tokens, heads, rank, key_dim, cache.shape[1], float(scale), int(window), int(keep_first),
        _opt(sinks, "sinks"), dtype_code(out.dtype), _stream()), "latent_attention_rowwise")
    return out


def latent_attention_mfma_supported(rank: int, key_dim: int, page_size: int) -> bool:
    return bool(hip_lib().kva_latent_attention_mfma_supported(int(rank), int(key_dim), int(page_size)))


def latent_attention_mfma(q: torch.Tensor, out: torch.Tensor, cache: torch.Tensor,
                          block_table: torch.Tensor, item_entry: torch.Tensor, item_row0: torch.Tensor,
                          entry_seat: torch.Tensor, entry_q_start: torch.Tensor, entry_start_pos: torch.Tensor,
                          scale: float, window: int = 0, keep_first: int = 0, sinks: Optional[torch.Tensor] = None,
                          splits: int = 1, per_split: int = 0, rows_per_item: int = 16, more=()) -> torch.Tensor:
    """:func:`latent_attention_rowwise` on the matrix cores (bf16); a work item is ``rows_per_item`` rows
    ``token_in_entry * heads + head`` of entry ``item_entry[i]`` from ``item_row0[i]`` on: 16 (the wavefronts
    of its workgroup share the keys: decoded tokens) or 64 (they share the loads: prompt portions).  ``more``:
    further ``(item_entry, item_row0, rows_per_item)`` of the same step.  With ``splits`` > 1 the keys are cut
    into ranges of ``per_split`` (a multiple of 32), one workgroup each, and a second kernel adds their
    results up: the items then name every row of the step."""
    if q.dim() != 3 or out.dim() != 3 or cache.dim() != 3 or q.shape[:2] != out.shape[:2]:
        raise KernelError("latent_attention_mfma: q [T, heads, key_dim], out [T, heads, rank], cache [pages, page, key_dim]")
    tokens, heads, key_dim = q.shape
    rank, page_size = out.shape[2], cache.shape[1]
    if cache.shape[2] != key_dim:
        raise KernelError(f"latent_attention_mfma: cache {tuple(cache.shape)} does not fit rows of {key_dim}")
    if not (q.dtype == out.dtype == cache.dtype == torch.bfloat16):
        raise KernelError("latent_attention_mfma: bfloat16 only")
    if not latent_attention_mfma_supported(rank, key_dim, page_size):
        raise KernelError(f"latent_attention_mfma: no instance for rank {rank}, rows of {key_dim}, pages of {page_size}")
    entries = entry_seat.shape[0]
    launches = [(item_entry, item_row0, int(rows_per_item)), *more]
    if any(row0.shape != ent.shape or ent.dim() != 1 for ent, row0, _ in launches) or entry_q_start.shape != (entries + 1,) \
            or entry_start_pos.shape != (entries,):
        raise KernelError("latent_attention_mfma: one row0 per item, entries + 1 starts, one start position per entry")
    if sinks is not None and (sinks.shape != (heads,) or sinks.dtype != torch.float32):
        raise KernelError("latent_attention_mfma: sinks are fp32, one per head")
    part_o = part_ml = None
    if splits > 1:
        if per_split <= 0 or per_split % 32:
            raise KernelError("latent_attention_mfma: key ranges are multiples of 32 keys")
        part_o = torch.empty((tokens * heads, splits, rank), dtype=torch.float32, device=q.device)
        part_ml = torch.empty((tokens * heads, splits, 2), dtype=torch.float32, device=q.device)
    for ent, row0, rows in launches:
        check(hip_lib().kva_latent_attention_mfma(
            _dev(out, "out"), _opt(part_o, "part_o"), _opt(part_ml, "part_ml"), _dev(q, "q"), _dev(cache, "cache"),
            _dev(block_table, "block_table", torch.int32), block_table.shape[1],
            _dev(ent, "item_entry", torch.int32), _dev(row0, "item_row0", torch.int32),
            _dev(entry_seat, "entry_seat", torch.int32), _dev(entry_q_start, "entry_q_start", torch.int32),
            _dev(entry_start_pos, "entry_start_pos", torch.int32), ent.shape[0], int(rows), heads, rank, key_dim, page_size,
            float(scale), int(window), int(keep_first), _opt(sinks, "sinks"), int(splits), int(per_split), _stream()),
            "latent_attention_mfma")
    if splits > 1:
        check(hip_lib().kva_latent_attention_merge(_dev(out, "out"), _dev(part_o, "part_o"), _dev(part_ml, "part_ml"),
                                                   _opt(sinks, "sinks"), tokens * heads, heads, rank, int(splits), _stream()),
              "latent_attention_merge")
    return out


def attention_rows_mfma_supported(head_dim: int, value_dim: int, page_size: int) -> bool:
    return bool(hip_lib().kva_attention_rows_mfma_supported(int(head_dim), int(value_dim), int(page_size)))


def attention_rows_mfma(q: torch.Tensor, q_row_stride: int, out: torch.Tensor, k_cache: torch.Tensor,
                        v_cache: torch.Tensor, block_table: torch.Tensor, item_entry: torch.Tensor,
                        item_row0: torch.Tensor, entry_seat: torch.Tensor, entry_q_start: torch.Tensor,
                        entry_start_pos: torch.Tensor, num_q_heads: int, num_kv_heads: int, head_dim: int,
                        scale: float, window: int = 0, keep_first: int = 0, sinks: Optional[torch.Tensor] = None,
                        value_dim: Optional[int] = None, splits: int = 1, per_split: int = 0,
                        row_tiles: int = 1, chunk: int = 0) -> torch.Tensor:
    """:func:`attention_rowwise` with all its options on the matrix cores (bf16): a work item is
    ``16 * row_tiles`` rows ``token_in_entry * group + head_in_group`` of entry ``item_entry[i]`` from
    ``item_row0[i]`` on, for every kv head (two row tiles, for heads up to 128, share what a
    wavefront loads); with ``splits`` > 1 the keys are cut into ranges of ``per_split`` and a
    second kernel adds the ranges' results up."""
    tokens = out.shape[0]
    value_dim = head_dim if value_dim is None else int(value_dim)
    if out.shape != (tokens, num_q_heads * value_dim):
        raise KernelError("attention_rows_mfma: out must be [T, nq * value size]")
    page_size = check_kv_cache_shapes("attention_rows_mfma", k_cache, v_cache, num_kv_heads, head_dim, value_dim)
    if not (q.dtype == out.dtype == k_cache.dtype == v_cache.dtype == torch.bfloat16):
        raise KernelError("attention_rows_mfma: bfloat16 only")
    if not attention_rows_mfma_supported(head_dim, value_dim, page_size):
        raise KernelError(f"attention_rows_mfma: no instance for keys of {head_dim}, values of {value_dim}, pages of {page_size}")
    if q.data_ptr() % 16 or q_row_stride < num_q_heads * head_dim or q_row_stride % 8:
        raise KernelError("attention_rows_mfma: q view is misaligned or its stride does not fit")
    n, entries = item_entry.shape[0], entry_seat.shape[0]
    if item_row0.shape != (n,) or entry_q_start.shape != (entries + 1,) or entry_start_pos.shape != (entries,):
        raise KernelError("attention_rows_mfma: one row0 per item, entries + 1 starts, one start position per entry")
    if sinks is not None and (sinks.shape != (num_q_heads,) or sinks.dtype != torch.float32):
        raise KernelError("attention_rows_mfma: sinks are fp32, one per query head")
    part_o = part_ml = None
    if splits > 1:
        if per_split <= 0 or per_split % 32:
            raise KernelError("attention_rows_mfma: key ranges are multiples of 32 keys")
        part_o = torch.empty((tokens * num_q_heads, splits, value_dim), dtype=torch.float32, device=q.device)
        part_ml = torch.empty((tokens * num_q_heads, splits, 2), dtype=torch.float32, device=q.device)
    check(hip_lib().kva_attention_rows_mfma(
        _dev(out, "out"), _opt(part_o, "part_o"), _opt(part_ml, "part_ml"), _dev(q, "q", contiguous=False), q_row_stride,
        _dev(k_cache, "k_cache"), _dev(v_cache, "v_cache"), _dev(block_table, "block_table", torch.int32),
        block_table.shape[1], _dev(item_entry, "item_entry", torch.int32), _dev(item_row0, "item_row0", torch.int32),
        _dev(entry_seat, "entry_seat", torch.int32), _dev(entry_q_start, "entry_q_start", torch.int32),
        _dev(entry_start_pos, "entry_start_pos", torch.int32), n, tokens * num_q_heads, num_q_heads, num_kv_heads,
        head_dim, value_dim, page_size, float(scale), int(window), int(keep_first), int(chunk), _opt(sinks, "sinks"),
        int(splits), int(per_split), int(row_tiles), _stream()), "attention_rows_mfma")
    return out


def layernorm(x: torch.Tensor, weight: torch.Tensor, eps: float, out: torch.Tensor, deltas=(),
              row_idx: Optional[torch.Tensor] = None, weight2: Optional[torch.Tensor] = None,
              out2: Optional[torch.Tensor] = None, rms: bool = False, delta_scale: float = 1.0) -> torch.Tensor:
    """``out = (x - mean) / sqrt(var + eps) * weight`` per row (``rms``: without taking the mean
    off).  ``deltas`` (up to two tensors of x's shape, any of the two storage types) are added to
    ``x`` first, in place (not written back when ``row_idx`` gathers rows); with a ``delta_scale``
    other than 1 their sum is multiplied by it before it enters ``x``.  ``weight2`` / ``out2``:
    a second normalised copy with another weight from the same statistics.  ``x`` may be fp32
    while ``out`` is bf16."""
    width = x.shape[-1]
    rows = out.shape[0]
    deltas = [d for d in deltas if d is not None]
    if x.dim() != 2 or out.dim() != 2 or out.shape[1] != width or weight.shape != (width,) or len(deltas) > 2:
        raise KernelError(f"layernorm: shapes x {tuple(x.shape)} weight {tuple(weight.shape)} out {tuple(out.shape)} do not fit")
    if (row_idx is None and rows != x.shape[0]) or (row_idx is not None and row_idx.shape != (rows,)):
        raise KernelError("layernorm: one output row per row of x, or per row index")
    if (weight2 is None) != (out2 is None) or (out2 is not None and (out2.shape != out.shape or out2.dtype != out.dtype
                                                                      or weight2.shape != (width,) or weight2.dtype != weight.dtype)):
        raise KernelError("layernorm: the second output needs a weight and out's shape and dtype")
    for d in deltas:
        if d.shape != x.shape:
            raise KernelError("layernorm: a delta must have x's shape")
    d1 = deltas[0] if deltas else None
    d2 = deltas[1] if len(deltas) > 1 else None
    check(hip_lib().kva_layernorm(
        _dev(out, "out"), _opt(out2, "out2"), dtype_code(out.dtype), _dev(x, "x"), dtype_code(x.dtype),
        _opt(d1, "delta"), dtype_code(d1.dtype) if d1 is not None else 0,
        _opt(d2, "delta"), dtype_code(d2.dtype) if d2 is not None else 0,
        _dev(weight, "weight"), _opt(weight2, "weight2"), dtype_code(weight.dtype),
        _opt(row_idx, "row_idx", torch.int32), rows, width, float(eps), 1 if rms else 0, float(delta_scale),
        _stream()), "layernorm")
    return out


def stream_join(x: torch.Tensor, other: torch.Tensor, out: torch.Tensor, deltas=()) -> torch.Tensor:
    """``out[t] = [x[t] + deltas ; other[t]]`` in out's type; ``x`` takes the sum in place."""
    deltas = [d for d in deltas if d is not None]
    rows, wx = x.shape
    if other.dim() != 2 or other.shape[0] != rows or out.shape != (rows, wx + other.shape[1]) or len(deltas) > 2 \
            or any(d.shape != x.shape for d in deltas):
        raise KernelError(f"stream_join: x {tuple(x.shape)}, other {tuple(other.shape)}, out {tuple(out.shape)} do not fit")
    d1 = deltas[0] if deltas else None
    d2 = deltas[1] if len(deltas) > 1 else None
    check(hip_lib().kva_stream_join(
        _dev(out, "out"), dtype_code(out.dtype), _dev(x, "x"), dtype_code(x.dtype),
        _opt(d1, "delta"), dtype_code(d1.dtype) if d1 is not None else 0,
        _opt(d2, "delta"), dtype_code(d2.dtype) if d2 is not None else 0,
        _dev(other, "other"), dtype_code(other.dtype), rows, wx, other.shape[1], _stream()), "stream_join")
    return out


def norm_into_stream(x: torch.Tensor, y: torch.Tensor, weight: torch.Tensor, eps: float,
                     copy: Optional[torch.Tensor] = None) -> torch.Tensor:
    """In place: ``x += y / sqrt(mean(y^2) + eps) * weight`` per row - a branch's output normed on its
    way into the stream.  ``x`` (the stream) and ``y`` may be of different storage types; ``copy``
    (x's shape, any storage type) receives the new rows of the stream as well."""
    if x.dim() != 2 or y.shape != x.shape or weight.shape != (x.shape[1],) or (copy is not None and copy.shape != x.shape):
        raise KernelError(f"norm_into_stream: x {tuple(x.shape)}, y {tuple(y.shape)}, weight {tuple(weight.shape)} do not fit")
    check(hip_lib().kva_norm_into_stream(
        _dev(x, "x"), dtype_code(x.dtype), _dev(y, "y"), dtype_code(y.dtype), _dev(weight, "weight"), dtype_code(weight.dtype),
        _opt(copy, "copy"), dtype_code(copy.dtype) if copy is not None else 0, x.shape[0], x.shape[1], float(eps),
        _stream()), "norm_into_stream")
    return x


ACTIVATIONS = {"silu": 0, "relu": 1, "gelu_tanh": 2, "relu2": 4}        # relu2: the square of relu
# gated forms only: act(gate) * up with "swish_clamped" = g sigmoid(1.702 g) (u + 1), g = min(gate, limit),
# u = clamp(up, -limit, limit)
GATED_ACTIVATIONS = dict(ACTIVATIONS, swish_clamped=3)
BIAS_ACTIVATIONS = dict(ACTIVATIONS, none=5)            # bias_act alone: a bias without an activation


def table_gate(z: torch.Tensor, table: torch.Tensor, ids: torch.Tensor, col0: int, out: torch.Tensor, activation: str,
               feedback: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``out[t, j] = act(z[t, j]) * table[ids[t], col0 + j]``: a gate times the columns ``col0 ..`` of the
    table row the token picks.  A negative id ``-1 - r`` stands for ``feedback[r]`` as in
    :func:`embed_gather`."""
    rows, dim = z.shape
    if activation not in ACTIVATIONS:
        raise KernelError(f"table_gate: activation {activation!r} is not one of {sorted(ACTIVATIONS)}")
    if out.shape != z.shape or out.dtype != z.dtype or table.dim() != 2 or ids.shape != (rows,) \
            or not 0 <= col0 <= table.shape[1] - dim:
        raise KernelError(f"table_gate: z {tuple(z.shape)}, table {tuple(table.shape)}, columns from {col0} do not fit")
    check(hip_lib().kva_table_gate(
        _dev(out, "out"), _dev(z, "z"), dtype_code(z.dtype), _dev(table, "table"), dtype_code(table.dtype), table.shape[1],
        table.shape[0], int(col0), _dev(ids, "ids", torch.int32), _opt(feedback, "feedback", torch.int32), rows, dim,
        ACTIVATIONS[activation], _stream()), "table_gate")
    return out


def act_mul(gate_up: torch.Tensor, out: torch.Tensor, activation: str, limit: float = 0.0) -> torch.Tensor:
    """out[t, i] = act(gate_up[t, i]) * gate_up[t, I + i] with ``activation`` one of silu, relu,
    gelu_tanh (0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))), or the gated form swish_clamped
    with its ``limit``."""
    rows, inter = out.shape
    if activation not in GATED_ACTIVATIONS:
        raise KernelError(f"act_mul: activation {activation!r} is not one of {sorted(GATED_ACTIVATIONS)}")
    if gate_up.shape != (rows, 2 * inter) or gate_up.dtype != out.dtype:
        raise KernelError(f"act_mul: gate_up {tuple(gate_up.shape)} does not fit out {tuple(out.shape)}")
    check(hip_lib().kva_act_mul(_dev(out, "out"), _dev(gate_up, "gate_up"), rows, inter, GATED_ACTIVATIONS[activation],
                                float(limit), dtype_code(out.dtype), _stream()), "act_mul")
    return out


def bias_act(x: torch.Tensor, out: torch.Tensor, activation: str, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``out = act(x + bias)`` element by element (``bias`` fp32, one value per column, optional); ``out``
    may be ``x``.  ``activation="none"``: the bias alone."""
    if activation not in BIAS_ACTIVATIONS:
        raise KernelError(f"bias_act: activation {activation!r} is not one of {sorted(BIAS_ACTIVATIONS)}")
    if x.dim() != 2 or out.shape != x.shape or out.dtype != x.dtype \
            or (bias is not None and (bias.shape != (x.shape[1],) or bias.dtype != torch.float32)):
        raise KernelError(f"bias_act: x {tuple(x.shape)} and out {tuple(out.shape)} do not fit")
    check(hip_lib().kva_bias_act(_dev(out, "out"), _dev(x, "x"), dtype_code(x.dtype), _opt(bias, "bias"), x.shape[0],
                                 x.shape[1], BIAS_ACTIVATIONS[activation], _stream()), "bias_act")
    return out


def hyper_step(x: torch.Tensor, streams: int, *, y: Optional[torch.Tensor] = None, mix: Optional[torch.Tensor] = None,
               out_w: Optional[torch.Tensor] = None, mult: float = 1.0, in_w: Optional[torch.Tensor] = None,
               norm_weight: Optional[torch.Tensor] = None, norm_bias: Optional[torch.Tensor] = None, eps: float = 0.0,
               out: Optional[torch.Tensor] = None, row_idx: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """One step between two branches over ``streams`` copies of the residual stream, ``x`` fp32 ``[T, streams *
    width]`` (a row's copies side by side).  With ``y`` ``[T, width]`` every copy is replaced, all at once from
    the old ones: ``x_t <- sum_s mix[s, t] x_s + mult * out_w[t] * y``.  With ``out`` the new copies are read out,
    ``u = sum_s in_w[s] x_s``, and normed: ``out = (u - mean) / sqrt(var + eps) * norm_weight + norm_bias``.
    ``row_idx``: only these rows are read out, and nothing is written back.  ``mix`` ``[streams, streams]``,
    ``out_w`` and ``in_w`` ``[streams]`` are fp32."""
    S = int(streams)
    if x.dim() != 2 or x.dtype != torch.float32 or x.shape[1] % S:
        raise KernelError(f"hyper_step: x {tuple(x.shape)} is not fp32 [T, {S} copies * width]")
    T, width = x.shape[0], x.shape[1] // S
    if y is not None and (y.shape != (T, width) or mix is None or out_w is None or mix.shape != (S, S)
                          or out_w.shape != (S,) or mix.dtype != torch.float32 or out_w.dtype != torch.float32):
        raise KernelError("hyper_step: a branch output [T, width] enters through fp32 mix [S, S] and out_w [S]")
    rows = T
    if out is not None:
        rows = T if row_idx is None else row_idx.shape[0]
        if out.shape != (rows, width) or in_w is None or in_w.shape != (S,) or in_w.dtype != torch.float32 \
                or norm_weight is None or norm_weight.shape != (width,) \
                or (norm_bias is not None and (norm_bias.shape != (width,) or norm_bias.dtype != norm_weight.dtype)):
            raise KernelError("hyper_step: the read-out needs out [rows, width], fp32 in_w [S] and a norm weight (and bias) [width]")
    elif row_idx is not None:
        raise KernelError("hyper_step: rows are gathered for the read-out only")
    check(hip_lib().kva_hyper_step(
        _dev(x, "x"), S, _opt(y, "y"), dtype_code(y.dtype) if y is not None else 0, _opt(mix, "mix"), _opt(out_w, "out_w"),
        float(mult), _opt(in_w, "in_w"), _opt(norm_weight, "norm_weight"), _opt(norm_bias, "norm_bias"),
        dtype_code(norm_weight.dtype) if norm_weight is not None else 0, float(eps), _opt(out, "out"),
        dtype_code(out.dtype) if out is not None else 0, _opt(row_idx, "row_idx", torch.int32), rows, width, _stream()),
        "hyper_step")
    return out


def hyper_fill(x: torch.Tensor, first: torch.Tensor, streams: int) -> torch.Tensor:
    """Every row of ``first`` ``[T, width]`` into all ``streams`` copies of ``x`` fp32 ``[T, streams * width]``."""
    T, width = first.shape
    if x.shape != (T, int(streams) * width) or x.dtype != torch.float32:
        raise KernelError(f"hyper_fill: x {tuple(x.shape)} does not hold {streams} copies of {tuple(first.shape)}")
    check(hip_lib().kva_hyper_fill(_dev(x, "x"), _dev(first, "first"), dtype_code(first.dtype), int(streams), T, width,
                                   _stream()), "hyper_fill")
    return x


def sandwich_step(x: torch.Tensor, *, y: Optional[torch.Tensor] = None, post=None, addend: Optional[torch.Tensor] = None,
                  pre=None, out: Optional[torch.Tensor] = None, row_idx: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """What lies between two branches that have norms on both sides, over a residual stream ``x`` fp32 ``[T,
    width]``: ``x += n_post(y) (+ addend)``, then ``out = n_pre(x)``.  ``post`` and ``pre`` are ``(weight, bias or
    None, eps, center)``: ``(v - mean) / sqrt(var + eps) * weight + bias``, without ``center`` the mean is not taken
    off.  Without ``post`` the branch output enters as it is; ``addend`` (fp32) always does.  ``row_idx``: only
    these rows are read out, and nothing is written back."""
    T, width = x.shape
    if x.dim() != 2 or x.dtype != torch.float32:
        raise KernelError(f"sandwich_step: x {tuple(x.shape)} is not an fp32 [T, width] stream")
    if (y is not None and y.shape != x.shape) or (addend is not None and (addend.shape != x.shape or addend.dtype != torch.float32)):
        raise KernelError("sandwich_step: the branch output and the addend (fp32) have the stream's shape")
    for norm in (post, pre):
        if norm is not None and (norm[0].shape != (width,) or (norm[1] is not None and (
                norm[1].shape != (width,) or norm[1].dtype != norm[0].dtype))):
            raise KernelError("sandwich_step: a norm has a weight [width] and a bias of its shape and type, or none")
    if (post is not None and y is None) or (out is None) != (pre is None):
        raise KernelError("sandwich_step: the first norm goes with a branch output, the second with an output")
    rows = T
    if out is not None:
        rows = T if row_idx is None else row_idx.shape[0]
        if out.shape != (rows, width):
            raise KernelError(f"sandwich_step: out {tuple(out.shape)} is not [{rows}, {width}]")
    elif row_idx is not None:
        raise KernelError("sandwich_step: rows are gathered for the read-out only")

    def args(norm, name):
        if norm is None:
            return None, None, 0, 0, 0.0
        w, b, eps, center = norm
        return _dev(w, name), _opt(b, name), dtype_code(w.dtype), 1 if center else 0, float(eps)
    check(hip_lib().kva_sandwich_step(
        _dev(x, "x"), _opt(y, "y"), dtype_code(y.dtype) if y is not None else 0, *args(post, "post norm"), _opt(addend, "addend"),
        *args(pre, "pre norm"), _opt(out, "out"), dtype_code(out.dtype) if out is not None else 0,
        _opt(row_idx, "row_idx", torch.int32), rows, width, _stream()), "sandwich_step")
    return out


def tanh_step(x: torch.Tensor, *, y: Optional[torch.Tensor] = None, y_bias: Optional[torch.Tensor] = None, post=None,
              pre=None, out: Optional[torch.Tensor] = None, row_idx: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """What lies between two branches that have tanh norms on both sides, over a residual stream ``x`` fp32 ``[T,
    width]``: ``x += n_post(y + y_bias)``, then ``out = n_pre(x)``.  ``post`` and ``pre`` are ``(weight, bias, alpha)``:
    ``tanh(alpha v) * weight + bias``.  Without ``post`` the branch output enters as it is (with its bias, fp32).
    ``y`` may be :class:`ExpertRows`: the sum is formed on the way.  ``row_idx``: only these rows are read out, and
    nothing is written back."""
    T, width = x.shape
    if x.dim() != 2 or x.dtype != torch.float32:
        raise KernelError(f"tanh_step: x {tuple(x.shape)} is not an fp32 [T, width] stream")
    if y is not None and y.shape != x.shape:
        raise KernelError("tanh_step: the branch output has the stream's shape")
    rows_of, gate, top, gate_stride = None, None, 0, 0
    if isinstance(y, ExpertRows):
        if y.rows.shape != (T * y.top, width) or y.rows.dtype != torch.float32:
            raise KernelError(f"tanh_step: experts' rows {tuple(y.rows.shape)} are not fp32 [T * top, width]")
        rows_of, top = y.rows, y.top
        gate, gate_stride = y.gate_column()
        y = y.extra
    if y_bias is not None and ((y is None and rows_of is None) or y_bias.shape != (width,) or y_bias.dtype != torch.float32):
        raise KernelError("tanh_step: a product's bias is fp32 [width] and goes with the product")
    for norm in (post, pre):
        if norm is not None and (norm[0].shape != (width,) or norm[1].shape != (width,) or norm[1].dtype != norm[0].dtype):
            raise KernelError("tanh_step: a norm has a weight [width] and a bias of its shape and type")
    if (post is not None and y is None and rows_of is None) or (out is None) != (pre is None):
        raise KernelError("tanh_step: the first norm goes with a branch output, the second with an output")
    rows = T
    if out is not None:
        rows = T if row_idx is None else row_idx.shape[0]
        if out.shape != (rows, width):
            raise KernelError(f"tanh_step: out {tuple(out.shape)} is not [{rows}, {width}]")
    elif row_idx is not None:
        raise KernelError("tanh_step: rows are gathered for the read-out only")

    def args(norm, name):
        if norm is None:
            return None, None, 0, 0.0
        w, b, alpha = norm
        return _dev(w, name), _dev(b, name), dtype_code(w.dtype), float(alpha)
    check(hip_lib().kva_tanh_step(
        _dev(x, "x"), _opt(y, "y"), dtype_code(y.dtype) if y is not None else 0, _opt(y_bias, "y_bias"), *args(post, "post norm"),
        *args(pre, "pre norm"), _opt(out, "out"), dtype_code(out.dtype) if out is not None else 0,
        _opt(row_idx, "row_idx", torch.int32), rows, width, _opt(rows_of, "rows"),
        None if gate is None else _dev(gate, "gate", torch.float32, contiguous=False), top, int(gate_stride), _stream()), "tanh_step")
    return out


def pair_embed(x: torch.Tensor, table: torch.Tensor, scale: float, pairs: Optional[torch.Tensor], mul_prev: int, mul_cur: int,
               norm, ids: torch.Tensor, state: torch.Tensor, entry_q_start: torch.Tensor, entry_seat: torch.Tensor,
               feedback: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``x[t] = n(table[id] * scale + pairs[row])`` fp32, ``row = (previous id * mul_prev + id * mul_cur) mod (len(pairs)
    - 1)`` or the last one for a sequence's first token.  ``norm``: ``(weight, bias, alpha)`` as :func:`tanh_step`
    takes it, or None; ``pairs`` may be None.  ``state`` int32 ``[seats, 1]``: the last id of every seat's sequence plus
    one (0: none yet); it is left at the entries' last ids.  A negative id ``-1 - r`` stands for ``feedback[r]``."""
    rows, width = x.shape
    if x.dtype != torch.float32 or table.dim() != 2 or table.shape[1] != width or ids.shape != (rows,):
        raise KernelError(f"pair_embed: x {tuple(x.shape)} (fp32), table {tuple(table.shape)}, ids {tuple(ids.shape)} do not fit")
    if pairs is not None and (pairs.dim() != 2 or pairs.shape[1] != width or pairs.shape[0] < 2):
        raise KernelError(f"pair_embed: the pairs' table {tuple(pairs.shape)} needs rows of {width}, two at least")
    if norm is not None and (norm[0].shape != (width,) or norm[1].shape != (width,) or norm[1].dtype != norm[0].dtype):
        raise KernelError("pair_embed: the norm has a weight [width] and a bias of its shape and type")
    if state.dim() != 2 or state.dtype != torch.int32:
        raise KernelError("pair_embed: the state is int32 [seats, n]")
    qs, seat, entries = _entries((entry_q_start, entry_seat), "pair_embed")
    w, b, alpha = norm if norm is not None else (None, None, 0.0)
    check(hip_lib().kva_pair_embed(
        _dev(x, "x"), _dev(table, "table"), dtype_code(table.dtype), table.shape[0], float(scale), _opt(pairs, "pairs"),
        dtype_code(pairs.dtype) if pairs is not None else 0, pairs.shape[0] - 1 if pairs is not None else 1, int(mul_prev),
        int(mul_cur), _opt(w, "norm weight"), _opt(b, "norm bias"), dtype_code(w.dtype) if w is not None else 0, float(alpha),
        _dev(ids, "ids", torch.int32), _opt(feedback, "feedback", torch.int32), _dev(state, "state"), state.shape[1], qs, seat,
        entries, rows, width, _stream()), "pair_embed")
    return x


def head_gate(x: torch.Tensor, gates: torch.Tensor, heads: int) -> torch.Tensor:
    """In place: head h of row t of ``x`` ``[T, heads * d]`` times ``sigmoid(gates[t, h])``; ``gates``
    is a ``[T, heads]`` view whose rows may be columns of a wider buffer."""
    rows = x.shape[0]
    if x.dim() != 2 or x.shape[1] % heads or gates.shape != (rows, heads) or gates.dtype != x.dtype \
            or gates.stride(1) != 1:
        raise KernelError(f"head_gate: x {tuple(x.shape)} and gates {tuple(gates.shape)} do not fit {heads} heads")
    check(hip_lib().kva_head_gate(_dev(x, "x"), _dev(gates, "gates", contiguous=False), rows, heads,
                                  x.shape[1] // heads, gates.stride(0) if rows > 1 else heads,
                                  dtype_code(x.dtype), _stream()), "head_gate")
    return x


def qk_encode_cache(qkv: torch.Tensor, positions: torch.Tensor, num_q_heads: int, num_kv_heads: int, head_dim: int,
                    value_dim: int, cos: Optional[torch.Tensor], sin: Optional[torch.Tensor], interleaved: bool,
                    unit_eps: Optional[float], k_cache: Optional[torch.Tensor], v_cache: Optional[torch.Tensor],
                    slot_mapping: Optional[torch.Tensor], bias: Optional[torch.Tensor] = None,
                    q_weight: Optional[torch.Tensor] = None, k_weight: Optional[torch.Tensor] = None,
                    norm_first: bool = False) -> None:
    """Rotates the first ``2 * cos.shape[1]`` elements of every Q and K head of ``qkv``
    ``[T, nq d + nkv d + nkv value_dim]`` (pair i = elements (2i, 2i + 1) when ``interleaved``, else
    (i, i + rot / 2)), then - with ``unit_eps`` - divides every head by its root mean square; Q in
    place, K and the plain V into the paged cache at ``slot_mapping``.  ``qkv`` may be the first
    columns of a wider buffer (rows ``qkv.stride(0)`` apart).  ``bias`` (qkv's type, one value per
    column) is added to Q, K and V first: the projection's bias, applied here.  ``q_weight`` /
    ``k_weight`` (fp32 ``[head_dim]``, with ``unit_eps``): every query / key head is multiplied by it
    after the division - an RMS norm of the head with a weight shared by the heads.
    ``norm_first``: the division and the weights come before the rotation instead (the normed head is
    what is rotated).
    ``num_kv_heads = 0``: ``qkv`` holds queries alone (a layer that reads another layer's keys and
    values); nothing is written to a cache."""
    tokens = qkv.shape[0]
    for w in (q_weight, k_weight):
        if w is not None and (unit_eps is None or w.shape != (head_dim,) or w.dtype != torch.float32):
            raise KernelError("qk_encode_cache: a head's norm weight is fp32 [head_dim] and goes with unit_eps")
    if num_kv_heads == 0 and k_cache is not None:
        raise KernelError("qk_encode_cache: rows of queries alone write no cache")
    k_off = num_q_heads * head_dim
    v_off = k_off + num_kv_heads * head_dim
    if qkv.dim() != 2 or qkv.shape[1] != v_off + num_kv_heads * value_dim or positions.shape != (tokens,) \
            or qkv.stride(1) != 1:
        raise KernelError(f"qk_encode_cache: qkv {tuple(qkv.shape)} is not [T, nq d + nkv d + nkv dv]")
    if bias is not None and (bias.shape != (qkv.shape[1],) or bias.dtype != qkv.dtype):
        raise KernelError("qk_encode_cache: the bias has one value of qkv's type per column")
    row_stride = qkv.stride(0) if tokens > 1 else qkv.shape[1]
    rot = 0
    if cos is not None:
        if sin is None or cos.shape != sin.shape or cos.dim() != 2:
            raise KernelError("qk_encode_cache: cos and sin tables must be [positions, rot / 2]")
        rot = 2 * cos.shape[1]
    write = k_cache is not None
    page_size = 0
    if write:
        if v_cache is None or slot_mapping is None or slot_mapping.shape != (tokens,) or k_cache.dtype != qkv.dtype \
                or v_cache.dtype != qkv.dtype:
            raise KernelError("qk_encode_cache: K and V cache of qkv's dtype and one slot per token are needed")
        page_size = check_kv_cache_shapes("qk_encode_cache", k_cache, v_cache, num_kv_heads, head_dim, value_dim)
    check(hip_lib().kva_qk_encode_cache(
        _dev(qkv, "qkv", contiguous=False), row_stride, k_off, v_off, _opt(k_cache, "k_cache"), _opt(v_cache, "v_cache"),
        _opt(cos, "cos", torch.float32), _opt(sin, "sin", torch.float32), _dev(positions, "positions", torch.int32),
        _opt(slot_mapping if write else None, "slot_mapping", torch.int32), tokens, num_q_heads, num_kv_heads,
        head_dim, value_dim, rot, 1 if interleaved else 0, -1.0 if unit_eps is None else float(unit_eps),
        page_size, dtype_code(qkv.dtype), _opt(bias, "bias"), _opt(q_weight, "q_weight"), _opt(k_weight, "k_weight"),
        1 if norm_first else 0, _stream()), "qk_encode_cache")


def maps_encode_cache(qkv: torch.Tensor, q_rows: torch.Tensor, positions: torch.Tensor, heads: int, kv_heads: int, dim: int,
                      value_dim: int, cos: Optional[torch.Tensor], sin: Optional[torch.Tensor], interleaved: bool,
                      k_cache: Optional[torch.Tensor], v_cache: Optional[torch.Tensor], slot_mapping: Optional[torch.Tensor],
                      bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Queries and keys of heads with two maps of ``dim`` elements each, ``qkv`` ``[T, (heads 2 + kv_heads 2) dim +
    kv_heads value_dim]`` (possibly the first columns of a wider buffer): the biases (fp32, one per column) are
    added, the first ``2 * cos.shape[1]`` elements of every map are rotated; a query head becomes two rows of ``2
    dim`` elements, each zero where the other map lies, in ``q_rows`` ``[T, 2 heads * 2 dim]``; keys of ``2 dim``
    elements (both maps side by side) and values go to the paged cache.  Attention over ``2 heads`` query rows
    and ``kv_heads`` key heads of ``2 dim`` then gives every head's two outputs side by side.  ``kv_heads = 0``:
    queries alone, and nothing is written to a cache."""
    tokens = qkv.shape[0]
    width = 2 * (heads + kv_heads) * dim + kv_heads * value_dim
    if qkv.dim() != 2 or qkv.shape[1] != width or qkv.stride(1) != 1 or positions.shape != (tokens,) \
            or q_rows.shape != (tokens, 4 * heads * dim) or q_rows.dtype != qkv.dtype:
        raise KernelError(f"maps_encode_cache: qkv {tuple(qkv.shape)}, q_rows {tuple(q_rows.shape)} do not fit {heads} / {kv_heads} heads of 2 x {dim}")
    if bias is not None and (bias.shape != (width,) or bias.dtype != torch.float32):
        raise KernelError("maps_encode_cache: the biases are fp32, one per column")
    rot = 0
    if cos is not None:
        if sin is None or cos.shape != sin.shape or cos.dim() != 2:
            raise KernelError("maps_encode_cache: cos and sin tables must be [positions, rot / 2]")
        rot = 2 * cos.shape[1]
    write = k_cache is not None
    page_size = 0
    if write:
        if kv_heads == 0 or v_cache is None or slot_mapping is None or slot_mapping.shape != (tokens,) \
                or k_cache.dtype != qkv.dtype or v_cache.dtype != qkv.dtype:
            raise KernelError("maps_encode_cache: key heads, K and V cache of qkv's dtype and one slot per token are needed")
        page_size = check_kv_cache_shapes("maps_encode_cache", k_cache, v_cache, kv_heads, 2 * dim, value_dim)
    check(hip_lib().kva_maps_encode_cache(
        _dev(qkv, "qkv", contiguous=False), qkv.stride(0) if tokens > 1 else width, _dev(q_rows, "q_rows"),
        _opt(k_cache, "k_cache"), _opt(v_cache, "v_cache"), _opt(cos, "cos", torch.float32), _opt(sin, "sin", torch.float32),
        _dev(positions, "positions", torch.int32), _opt(slot_mapping if write else None, "slot_mapping", torch.int32), tokens,
        int(heads), int(kv_heads), int(dim), int(value_dim), rot, 1 if interleaved else 0, page_size, _opt(bias, "bias"),
        dtype_code(qkv.dtype), _stream()), "maps_encode_cache")
    return q_rows


def maps_combine(x: torch.Tensor, heads: int, value_dim: int, weight: float, eps: float, out: torch.Tensor, out_off: int = 0,
                 mul: float = 1.0) -> torch.Tensor:
    """``o = a1 - weight * a2`` of every head's two outputs (``x`` ``[T, heads * 2 * value_dim]``), then ``o /
    sqrt(mean(o^2) + eps) * mul`` into columns ``out_off ..`` of ``out``."""
    rows = x.shape[0]
    if x.shape != (rows, 2 * heads * value_dim) or out.dim() != 2 or out.shape[0] != rows or out.dtype != x.dtype \
            or not 0 <= out_off <= out.shape[1] - heads * value_dim:
        raise KernelError(f"maps_combine: x {tuple(x.shape)} and out {tuple(out.shape)} do not fit {heads} heads of {value_dim}")
    check(hip_lib().kva_maps_combine(_dev(out, "out"), out.shape[1], int(out_off), _dev(x, "x"), float(weight), float(eps),
                                     float(mul), rows, int(heads), int(value_dim), dtype_code(x.dtype), _stream()), "maps_combine")
    return out


def latent_encode_cache(y: torch.Tensor, kv_off: int, q_lat: Optional[torch.Tensor], cache: Optional[torch.Tensor],
                        norm_weight: torch.Tensor, eps: float, cos: torch.Tensor, sin: torch.Tensor,
                        positions: torch.Tensor, slot_mapping: Optional[torch.Tensor], heads: int, plain_dim: int,
                        rank: int, interleaved: bool = False,
                        c_q: Optional[torch.Tensor] = None, q_norm_weight: Optional[torch.Tensor] = None) -> None:
    """From a projection row ``y[t] = [heads x (plain_dim + rot) | ... rank + rot at kv_off ...]``:
    the rotated part of every query head goes to ``q_lat[t, h, rank:]``; the entry's first ``rank``
    elements, RMS-normed with ``norm_weight``, and its rotated last ``rot`` go to row
    ``slot_mapping[t]`` of ``cache`` ``[pages, page_size, rank + rot]``.

    With ``c_q`` ``[T, q_rank]`` (and without ``q_lat``) the rows start with a query latent instead of the
    query heads, ``y[t] = [q_rank | ... rank + rot at kv_off ...]``: it is RMS-normed with ``q_norm_weight`` (and
    the same eps) into ``c_q``, and the query heads are somebody else's to rotate."""
    tokens = y.shape[0]
    rot = 2 * cos.shape[1]
    if (q_lat is None) == (c_q is None):
        raise KernelError("latent_encode_cache: rows start with the query heads or with a query latent")
    if c_q is not None:
        heads = 0
        if c_q.dim() != 2 or c_q.shape[0] != tokens or c_q.dtype != y.dtype or q_norm_weight is None \
                or q_norm_weight.shape != (c_q.shape[1],) or q_norm_weight.dtype != norm_weight.dtype:
            raise KernelError("latent_encode_cache: the query latent [T, q_rank] of y's dtype has a norm weight [q_rank]")
    if y.dim() != 2 or positions.shape != (tokens,):
        raise KernelError(f"latent_encode_cache: y {tuple(y.shape)} does not fit one position per token")
    if q_lat is not None and (q_lat.shape != (tokens, heads, rank + rot) or q_lat.dtype != y.dtype):
        raise KernelError(f"latent_encode_cache: y {tuple(y.shape)} and q_lat {tuple(q_lat.shape)} do not fit")
    if cos.shape != sin.shape or norm_weight.shape != (rank,):
        raise KernelError("latent_encode_cache: tables [positions, rot / 2] and a norm weight [rank] are needed")
    write = cache is not None and slot_mapping is not None
    if write and (cache.dim() != 3 or cache.shape[2] != rank + rot or cache.dtype != y.dtype
                  or slot_mapping.shape != (tokens,)):
        raise KernelError("latent_encode_cache: cache [pages, page_size, rank + rot] of y's dtype, one slot per token")
    check(hip_lib().kva_latent_encode_cache(
        _dev(y, "y"), y.shape[1], int(kv_off), _opt(q_lat, "q_lat"), _opt(c_q, "c_q"), _opt(q_norm_weight, "q_norm_weight"),
        c_q.shape[1] if c_q is not None else 0, _opt(cache if write else None, "cache"),
        _dev(norm_weight, "norm_weight"), dtype_code(norm_weight.dtype), float(eps),
        _dev(cos, "cos", torch.float32), _dev(sin, "sin", torch.float32), _dev(positions, "positions", torch.int32),
        _opt(slot_mapping if write else None, "slot_mapping", torch.int32), tokens, heads, plain_dim, rank, rot,
        1 if interleaved else 0, dtype_code(y.dtype), _stream()), "latent_encode_cache")


def heads_matmul(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor, gates: Optional[torch.Tensor] = None,
                 rotate: Optional[tuple] = None) -> torch.Tensor:
    """``out[t, h, :] = w[h] @ x[t, h, :]`` for ``w`` ``[heads, N, K]``.  ``x`` ``[T, heads, K]`` and
    ``out`` ``[T, heads, N]`` may be views into wider buffers (unit stride along the last axis).
    With ``gates`` (``[T, heads]``, a column range of another buffer) head h of row t is multiplied
    by ``sigmoid(gates[t, h])``; gates ``[T, heads, N]`` multiply every output element by its own.

    ``rotate = (src, dst, cos, sin, positions, interleaved)``: in the same launch the rows ``src`` ``[T, heads,
    rot]`` are rotated by their positions into ``dst`` (views like ``x`` and ``out``; pair i is ``(2i, 2i + 1)`` when
    ``interleaved``, else ``(i, i + rot / 2)``; fp32 tables ``[positions, rot / 2]``)."""
    heads, n, k = w.shape
    rows = x.shape[0]

    def strides(t, last):
        """(row, head) strides of a [T, heads, last] view, also where T or heads is 1 and they are arbitrary"""
        head = t.stride(1) if heads > 1 else max(t.stride(1), last)
        row = t.stride(0) if rows > 1 else max(t.stride(0), (heads - 1) * head + last)
        return row, head
    options = [None, 0, 0, 0]
    if gates is not None:
        elementwise = gates.dim() == 3
        if gates.shape != ((rows, heads, n) if elementwise else (rows, heads)) or gates.dtype != x.dtype or gates.stride(-1) != 1:
            raise KernelError(f"heads_matmul: gates {tuple(gates.shape)} do not fit {rows} rows of {heads} heads")
        g_row, g_head = strides(gates, n) if elementwise else (gates.stride(0) if rows > 1 else heads, 1)
        options = [_dev(gates, "gates", contiguous=False), g_row, g_head, 1 if elementwise else 0]
    if rotate is None:
        options += [None, 0, 0, None, 0, 0, None, None, None, 0, 0]
    else:
        src, dst, cos, sin, positions, interleaved = rotate
        rot = src.shape[2]
        if src.shape != (rows, heads, rot) or dst.shape != src.shape or src.stride(2) != 1 or dst.stride(2) != 1 \
                or src.dtype != x.dtype or dst.dtype != x.dtype or cos.shape != sin.shape or cos.dim() != 2 \
                or 2 * cos.shape[1] != rot or positions.shape != (rows,):
            raise KernelError(f"heads_matmul: the rotated rows {tuple(src.shape)} -> {tuple(dst.shape)} do not fit")
        options += [_dev(src, "rotate source", contiguous=False), *strides(src, rot), _dev(dst, "rotate target", contiguous=False),
                    *strides(dst, rot), _dev(cos, "cos", torch.float32), _dev(sin, "sin", torch.float32),
                    _dev(positions, "positions", torch.int32), rot, 1 if interleaved else 0]
    if x.shape != (rows, heads, k) or out.shape != (rows, heads, n) or x.stride(2) != 1 or out.stride(2) != 1 \
            or not (x.dtype == w.dtype == out.dtype):
        raise KernelError(f"heads_matmul: x {tuple(x.shape)}, w {tuple(w.shape)}, out {tuple(out.shape)} do not fit")
    (xr, xh), (orr, oh) = strides(x, k), strides(out, n)
    if x.dtype == torch.bfloat16 and x.data_ptr() % 16 == 0 and out.data_ptr() % 8 == 0 \
            and hip_lib().kva_heads_matmul_mfma_supported(k, xr, xh):
        # bf16 with a K that has an instance: the matrix cores
        check(hip_lib().kva_heads_matmul_mfma(_dev(out, "out", contiguous=False), orr, oh, _dev(x, "x", contiguous=False),
                                              xr, xh, _dev(w, "w"), rows, heads, n, k, *options, _stream()),
              "heads_matmul_mfma")
        return out
    check(hip_lib().kva_heads_matmul(_dev(out, "out", contiguous=False), orr, oh, _dev(x, "x", contiguous=False), xr, xh,
                                     _dev(w, "w"), rows, heads, n, k, *options, dtype_code(x.dtype), _stream()), "heads_matmul")
    return out


def gemm_nt_f32(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
    """out[M, N] = a[M, K] @ w[N, K]^T in true fp32."""
    m, k = a.shape
    n = w.shape[0]
    if w.shape != (n, k) or out.shape != (m, n):
        raise KernelError(f"gemm_f32: a {tuple(a.shape)} w {tuple(w.shape)} out {tuple(out.shape)} do not fit")
    check(hip_lib().kva_gemm_nt_f32(_dev(out, "out", torch.float32), _dev(a, "a", torch.float32),
                                    _dev(w, "w", torch.float32), m, n, k, k, k, n, _stream()),
          "gemm_nt_f32")
    return out


def host_memory_is_mapped(t: torch.Tensor) -> bool:
    """Whether a kernel may write into this host tensor (pinned memory mapped for the device)."""
    if t.is_cuda or not t.is_pinned():
        return False
    return bool(hip_lib().kva_host_memory_is_mapped(ctypes.c_void_p(t.data_ptr())))


def sample(logits: torch.Tensor, out_tokens: torch.Tensor, *, chunks: int = 128,
           inv_temperature: Optional[torch.Tensor] = None, seed: int = 0,
           rng_key: Optional[torch.Tensor] = None, rng_step: Optional[torch.Tensor] = None,
           penalty_mask: Optional[torch.Tensor] = None, row_seat: Optional[torch.Tensor] = None,
           penalty: float = 1.0, mark_mask: Optional[torch.Tensor] = None,
           mark_seat: Optional[torch.Tensor] = None, host_tokens: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Greedy (rows whose inv_temperature is 0 or absent) or temperature sampling per row.
    ``penalty_mask`` ``[seats, vocab]`` with ``row_seat`` (-1: none) names the logits that are
    penalised; ``mark_mask`` with ``mark_seat`` (-1: none) gets ``mark_mask[seat, token] = 1`` for
    every chosen token, in the same launch.  ``host_tokens``: a pinned host int32 tensor with a
    place per row that takes the tokens too, written by the kernel itself (valid once the stream
    has passed the launch)."""
    rows, vocab = logits.shape
    if out_tokens.shape != (rows,):
        raise KernelError("sample: one output token per row")
    any_sampled = inv_temperature is not None
    if any_sampled and (rng_key is None or rng_step is None or inv_temperature.shape != (rows,)
                        or rng_key.shape != (rows,) or rng_step.shape != (rows,)):
        raise KernelError("sample: inv_temperature, rng_key and rng_step are needed per row")
    if penalty_mask is not None:
        if row_seat is None or row_seat.shape != (rows,) or penalty_mask.dim() != 2 \
                or penalty_mask.shape[1] != vocab:
            raise KernelError("sample: penalty mask [seats, vocab] needs a seat per row")
    if (mark_mask is None) != (mark_seat is None) or (mark_mask is not None and (
            mark_seat.shape != (rows,) or mark_mask.dim() != 2 or mark_mask.shape[1] != vocab)):
        raise KernelError("sample: marking needs a mask [seats, vocab] and a seat per row")
    if host_tokens is not None and (host_tokens.is_cuda or not host_tokens.is_pinned() or host_tokens.dtype != torch.int32
                                    or host_tokens.dim() != 1 or host_tokens.shape[0] < rows
                                    or not host_tokens.is_contiguous()):
        raise KernelError("sample: host_tokens must be a pinned host int32 vector with a place per row")
    lib = hip_lib()
    ws = torch.empty(max(1, lib.kva_sample_workspace_bytes(rows, chunks) // 4), dtype=torch.float32,
                     device=logits.device)
    check(lib.kva_sample(
        _dev(out_tokens, "out_tokens", torch.int32), _dev(logits, "logits", torch.float32), rows, vocab,
        chunks, _opt(penalty_mask, "penalty_mask", torch.uint8), _opt(row_seat, "row_seat", torch.int32),
        float(penalty), _opt(inv_temperature, "inv_temperature", torch.float32), int(seed) & 0xFFFFFFFF,
        _opt(rng_key, "rng_key", torch.int32), _opt(rng_step, "rng_step", torch.int32),
        1 if any_sampled else 0, _dev(ws, "workspace"), _opt(mark_mask, "mark_mask", torch.uint8),
        _opt(mark_seat, "mark_seat", torch.int32),
        ctypes.c_void_p(host_tokens.data_ptr()) if host_tokens is not None else None, _stream()), "sample")
    return out_tokens


def mark_tokens(mask: torch.Tensor, seats: torch.Tensor, tokens: torch.Tensor) -> None:
    n = seats.shape[0]
    if tokens.shape != (n,) or mask.dim() != 2:
        raise KernelError("mark_tokens: one seat per token, mask [seats, vocab]")
    check(hip_lib().kva_mark_tokens(_dev(mask, "mask", torch.uint8), _dev(seats, "seats", torch.int32),
                                    _dev(tokens, "tokens", torch.int32), n, mask.shape[1], _stream()),
          "mark_tokens")


_MAX_SPLITS = None


def attention_max_splits() -> int:
    """Most key splits the matrix-core attention kernels and their merge take."""
    global _MAX_SPLITS
    if _MAX_SPLITS is None:
        _MAX_SPLITS = int(hip_lib().kva_attention_max_splits())
    return _MAX_SPLITS


def attention_mfma_supported(head_dim: int, page_size: int) -> bool:
    return bool(hip_lib().kva_attention_mfma_supported(int(head_dim), int(page_size)))


def attention_mfma_row_tiles(head_dim: int, wide: bool) -> int:
    """Row tiles (of 16 query rows) per work item the kernel offers for this head size."""
    return int(hip_lib().kva_attention_mfma_row_tiles(int(head_dim), 1 if wide else 0))


def attention_mfma(q: torch.Tensor, q_row_stride: int, out: torch.Tensor, k_cache: torch.Tensor,
                   v_cache: torch.Tensor, block_table: torch.Tensor, item_entry: torch.Tensor,
                   item_row0: torch.Tensor, entry_seat: torch.Tensor, entry_q_start: torch.Tensor,
                   entry_start_pos: torch.Tensor, num_q_heads: int, num_kv_heads: int, head_dim: int,
                   scale: float, window: int = 0, splits: int = 1, keys_per_split: int = 0,
                   row_tiles: int = 1, pair: bool = False,
                   item_meta: Optional[torch.Tensor] = None, covers_all_rows: bool = True,
                   keep_cached: bool = False, waves: int = 1, leave_partials: bool = False):
    """bf16 matrix-core attention over the paged cache.  Items are (entry, first query row) pairs
    of ``16 * row_tiles`` query rows each, row = token_in_step * (nq / nkv) + head_in_group.
    With ``pair`` one wavefront takes item i and item n-1-i of the list (give the list ordered by
    keys visited, most first, and every wavefront has about the same work).  ``item_meta``
    ``[items, 8]`` int32 (q_start, q_len, start_pos, seat, row0, 0, 0, 0 per item) saves the
    kernel the chain of lookups item -> entry -> entry arrays; it must say the same as they do.
    ``covers_all_rows=False``: the items are only some of the step's rows (the others belong to
    another launch) and a split merge must leave those alone.  ``keep_cached`` (items of one row
    tile): keys and values are loaded through the caches instead of past them - for the few
    short contexts that are still in the memory-side cache when the next step reads them.
    ``waves`` (1, 2 or 4; items of one row tile, head sizes up to 128): so many of the ``splits``
    key ranges go to the wavefronts of one workgroup, which adds their results up itself; only
    ``splits // waves`` partial results per row are left for the merge (none: no merge launch).
    ``leave_partials`` (the items cover every row of the step): where more than one partial result
    a row is left they are not merged into ``out`` but returned as :class:`AttentionPartials`."""
    tokens = out.shape[0]
    if out.dtype != torch.bfloat16 or q.dtype != torch.bfloat16 or k_cache.dtype != torch.bfloat16:
        raise KernelError("attention_mfma: bfloat16 only")
    if leave_partials and not covers_all_rows:
        raise KernelError("attention_mfma: partial results can only be left for a launch that covers every row")
    if waves < 1 or splits % waves:
        raise KernelError(f"attention_mfma: {waves} wavefronts per item do not divide {splits} key ranges")
    if out.shape != (tokens, num_q_heads * head_dim):
        raise KernelError("attention_mfma: out must be [T, nq * d]")
    check_cache_shapes("attention_mfma", k_cache, v_cache, num_kv_heads, head_dim)
    n_items = item_entry.shape[0]
    n_entries = entry_seat.shape[0]
    if item_row0.shape != (n_items,) or entry_q_start.shape != (n_entries + 1,) \
            or entry_start_pos.shape != (n_entries,) or block_table.dim() != 2:
        raise KernelError("attention_mfma: index arrays do not fit each other")
    if q.data_ptr() % 16 or q_row_stride < num_q_heads * head_dim:
        raise KernelError("attention_mfma: q view is misaligned or its stride is too small")
    if item_meta is not None and item_meta.shape != (n_items, 8):
        raise KernelError("attention_mfma: item_meta must be [items, 8]")
    part_o = part_ml = None
    if splits // waves > 1:
        part_o = torch.empty((tokens * num_q_heads, splits // waves, head_dim), dtype=torch.float32, device=out.device)
        part_ml = torch.empty((tokens * num_q_heads, splits // waves, 2), dtype=torch.float32, device=out.device)
    left = leave_partials and part_o is not None
    check(hip_lib().kva_attention_mfma(
        None if left else _dev(out, "out"), _opt(part_o, "part_o"), _opt(part_ml, "part_ml"),
        _dev(q, "q", contiguous=False), q_row_stride, _dev(k_cache, "k_cache"), _dev(v_cache, "v_cache"),
        _dev(block_table, "block_table", torch.int32), block_table.shape[1],
        _opt(item_meta, "item_meta", torch.int32),
        _dev(item_entry, "item_entry", torch.int32), _dev(item_row0, "item_row0", torch.int32), n_items,
        int(row_tiles), _dev(entry_seat, "entry_seat", torch.int32), _dev(entry_q_start, "entry_q_start", torch.int32),
        _dev(entry_start_pos, "entry_start_pos", torch.int32), tokens * num_q_heads, num_q_heads,
        num_kv_heads, head_dim, k_cache.shape[3], float(scale), int(window), int(splits),
        int(keys_per_split), 1 if pair else 0, 1 if covers_all_rows else 0, 1 if keep_cached else 0,
        int(waves), _stream()), "attention_mfma")
    return AttentionPartials(part_o, part_ml, tokens, num_q_heads) if left else out


def attention_mfma_rope_supported(head_dim: int, page_size: int, group: int) -> bool:
    """Whether the decode attention kernel that rotates and caches inside takes this geometry
    (``group``: query heads per kv head)."""
    return bool(hip_lib().kva_attention_mfma_rope_supported(int(head_dim), int(page_size), int(group)))


def attention_mfma_rope(qkv: torch.Tensor, out: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
                        block_table: torch.Tensor, item_meta: torch.Tensor, num_q_heads: int, num_kv_heads: int,
                        head_dim: int, scale: float, cos: Optional[torch.Tensor], sin: Optional[torch.Tensor],
                        slot_mapping: Optional[torch.Tensor], window: int = 0, splits: int = 1,
                        keys_per_split: int = 0, keep_cached: bool = False, waves: int = 1) -> torch.Tensor:
    """bf16 matrix-core attention of decoded tokens (one token per item) straight from the joined
    Q/K/V projection ``qkv`` ``[T, (nq + 2 nkv) d]``, not yet rotated: the kernel rotates Q and the
    token's K by its position (``cos`` / ``sin`` ``[positions, d / 2]`` fp32, both None: no
    rotation), stores the rotated K and the V at ``slot_mapping[token]`` (None: the cache is only
    read) and attends, the token's own key and value taken from registers.  ``item_meta``
    ``[items, 8]`` int32: (token row, 1, position, seat, 0, 0, 0, 0).  ``waves``: as for
    :func:`attention_mfma`."""
    tokens = out.shape[0]
    if out.dtype != torch.bfloat16 or qkv.dtype != torch.bfloat16 or k_cache.dtype != torch.bfloat16:
        raise KernelError("attention_mfma_rope: bfloat16 only")
    if waves < 1 or splits % waves:
        raise KernelError(f"attention_mfma_rope: {waves} wavefronts per item do not divide {splits} key ranges")
    if out.shape != (tokens, num_q_heads * head_dim) or qkv.dim() != 2 or qkv.shape[0] != tokens \
            or qkv.shape[1] != (num_q_heads + 2 * num_kv_heads) * head_dim or not qkv.is_contiguous():
        raise KernelError("attention_mfma_rope: qkv must be [T, (nq + 2 nkv) d] and out [T, nq * d]")
    check_cache_shapes("attention_mfma_rope", k_cache, v_cache, num_kv_heads, head_dim)
    if item_meta.dim() != 2 or item_meta.shape[1] != 8 or block_table.dim() != 2:
        raise KernelError("attention_mfma_rope: item_meta must be [items, 8] and the block table [seats, blocks]")
    if (cos is None) != (sin is None) or (cos is not None and (cos.shape != sin.shape or cos.dim() != 2
                                                               or cos.shape[1] != head_dim // 2)):
        raise KernelError("attention_mfma_rope: cos and sin tables must both be [positions, d / 2]")
    if slot_mapping is not None and slot_mapping.shape != (tokens,):
        raise KernelError("attention_mfma_rope: one cache slot per token")
    part_o = part_ml = None
    if splits // waves > 1:
        part_o = torch.empty((tokens * num_q_heads, splits // waves, head_dim), dtype=torch.float32, device=out.device)
        part_ml = torch.empty((tokens * num_q_heads, splits // waves, 2), dtype=torch.float32, device=out.device)
    check(hip_lib().kva_attention_mfma_rope(
        _dev(out, "out"), _opt(part_o, "part_o"), _opt(part_ml, "part_ml"), _dev(qkv, "qkv"), qkv.shape[1],
        _dev(k_cache, "k_cache"), _dev(v_cache, "v_cache"), _dev(block_table, "block_table", torch.int32),
        block_table.shape[1], _dev(item_meta, "item_meta", torch.int32), item_meta.shape[0], tokens * num_q_heads,
        num_q_heads, num_kv_heads, head_dim, k_cache.shape[3], float(scale), int(window), int(splits),
        int(keys_per_split), 1 if keep_cached else 0, _opt(cos, "cos", torch.float32), _opt(sin, "sin", torch.float32),
        _opt(slot_mapping, "slot_mapping", torch.int32), int(waves), _stream()), "attention_mfma_rope")
    return out


def attention_lds_supported(head_dim: int, page_size: int) -> bool:
    return bool(hip_lib().kva_attention_lds_supported(int(head_dim), int(page_size)))


def attention_lds(q: torch.Tensor, q_row_stride: int, out: torch.Tensor, k_cache: torch.Tensor,
                  v_cache: torch.Tensor, block_table: torch.Tensor, item_meta: torch.Tensor,
                  num_q_heads: int, num_kv_heads: int, head_dim: int, scale: float, window: int = 0,
                  pair: bool = False, splits: int = 1, keys_per_split: int = 0,
                  covers_all_rows: bool = True) -> torch.Tensor:
    """bf16 matrix-core attention for prompt portions: a workgroup of four wavefronts per 128
    query rows (row = token_in_step * (nq / nkv) + head_in_group) shares every key and value
    block through LDS.  ``item_meta`` ``[items, 8]`` int32: (q_start, q_len, start_pos, seat,
    row0, 0, 0, 0) with ``row0`` a multiple of 128.  With ``pair`` a workgroup takes item i and
    item n-1-i of the list.  With ``splits`` > 1 the keys are cut into ranges of
    ``keys_per_split`` (a multiple of 32), one workgroup each, and merged afterwards
    (``covers_all_rows=False``: only over the items' rows, the others belong to another launch)."""
    tokens = out.shape[0]
    if out.dtype != torch.bfloat16 or q.dtype != torch.bfloat16 or k_cache.dtype != torch.bfloat16:
        raise KernelError("attention_lds: bfloat16 only")
    if out.shape != (tokens, num_q_heads * head_dim):
        raise KernelError("attention_lds: out must be [T, nq * d]")
    check_cache_shapes("attention_lds", k_cache, v_cache, num_kv_heads, head_dim)
    if item_meta.dim() != 2 or item_meta.shape[1] != 8 or block_table.dim() != 2:
        raise KernelError("attention_lds: item_meta must be [items, 8] and the block table [seats, blocks]")
    if q.data_ptr() % 16 or q_row_stride < num_q_heads * head_dim:
        raise KernelError("attention_lds: q view is misaligned or its stride is too small")
    part_o = part_ml = None
    if splits > 1:
        part_o = torch.empty((tokens * num_q_heads, splits, head_dim), dtype=torch.float32, device=out.device)
        part_ml = torch.empty((tokens * num_q_heads, splits, 2), dtype=torch.float32, device=out.device)
    check(hip_lib().kva_attention_lds(
        _dev(out, "out"), _opt(part_o, "part_o"), _opt(part_ml, "part_ml"),
        _dev(q, "q", contiguous=False), q_row_stride, _dev(k_cache, "k_cache"),
        _dev(v_cache, "v_cache"), _dev(block_table, "block_table", torch.int32), block_table.shape[1],
        _dev(item_meta, "item_meta", torch.int32), item_meta.shape[0], 1 if pair else 0, num_q_heads,
        num_kv_heads, head_dim, k_cache.shape[3], float(scale), int(window), int(splits), int(keys_per_split),
        tokens * num_q_heads, 1 if covers_all_rows else 0, _stream()), "attention_lds")
    return out


def gemm_vendor_init() -> None:
    """Makes the vendor GEMM library's handle and workspace on the current device; called when a
    weight is loaded, so that no product makes them in the middle of a graph capture."""
    check(hip_lib().kva_gemm_vendor_init(), "gemm_vendor_init")


def gemm_vendor(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor) -> bool:
    """out = x @ w^T by the vendor GEMM library (bf16 operands, fp32 accumulation, bf16 or fp32
    result).  False when the library has no algorithm for the shape: nothing was launched."""
    m, k = x.shape
    n = w.shape[0]
    if w.shape[1] != k or out.shape != (m, n) or x.dtype != torch.bfloat16 or w.dtype != torch.bfloat16 \
            or out.dtype not in (torch.bfloat16, torch.float32):
        raise KernelError(f"gemm_vendor: x {tuple(x.shape)} {x.dtype}, w {tuple(w.shape)} {w.dtype}, out "
                          f"{tuple(out.shape)} {out.dtype} do not fit")
    code = hip_lib().kva_gemm_vendor(_dev(out, "out"), _dev(x, "x"), _dev(w, "w"), m, n, k, k, n,
                                     1 if out.dtype == torch.float32 else 0, _stream())
    if code == 1:
        return False
    check(code, "gemm_vendor")
    return True


def gemm_vendor_tune(rows: int, weights, out_dtype: torch.dtype = torch.bfloat16) -> tuple:
    """Finds the vendor library's fastest algorithm for products of ``rows`` rows with weights of
    the shape of ``weights`` (bf16 matrices of one shape, e.g. the same projection of every
    layer; they are used in turn so that each comes from memory) and keeps it for later
    :func:`gemm_vendor` calls of that shape.  Runs every algorithm the library has for the shape:
    seconds, at start-up, never inside a graph capture.  A winner whose product differs from the
    heuristic's choice by more than rounding is dropped again.  Returns (microseconds of the
    heuristic's choice, microseconds of the one kept, algorithms run)."""
    import ctypes
    weights = list(weights)
    if not weights or rows < 1:
        raise KernelError("gemm_vendor_tune: needs at least one weight and one row")
    n, k = weights[0].shape
    for w in weights:
        if w.shape != (n, k) or w.dtype != torch.bfloat16 or not w.is_cuda or not w.is_contiguous():
            raise KernelError("gemm_vendor_tune: weights must be contiguous bf16 matrices of one shape on the GPU")
    dev = weights[0].device
    x = (torch.randn((rows, k), device=dev, dtype=torch.float32) * 0.5).to(torch.bfloat16)
    out = torch.empty((rows, n), dtype=out_dtype, device=dev)
    if not gemm_vendor(x, weights[0], out):
        return (-1.0, -1.0, 0)
    before = out.float()
    ptrs = (ctypes.c_void_p * len(weights))(*[w.data_ptr() for w in weights])
    first, best, tried = ctypes.c_float(), ctypes.c_float(), ctypes.c_int()
    check(hip_lib().kva_gemm_vendor_tune(_dev(out, "out"), _dev(x, "x"), ptrs, len(weights), rows, n, k, k, n,
                                         1 if out_dtype == torch.float32 else 0, _stream(),
                                         ctypes.byref(first), ctypes.byref(best), ctypes.byref(tried)),
          "gemm_vendor_tune")
    gemm_vendor(x, weights[0], out)
    scale = float(before.abs().max())
    if not float((out.float() - before).abs().max()) <= 0.02 * scale:
        check(hip_lib().kva_gemm_vendor_forget(rows, n, k, k, n, 1 if out_dtype == torch.float32 else 0),
              "gemm_vendor_forget")
        return (first.value, first.value, tried.value)
    return (first.value, best.value, tried.value)


def gemm_skinny_supported(m: int, n: int, k: int) -> bool:
    return bool(hip_lib().kva_gemm_skinny_supported(int(m), int(n), int(k)))


class TiledWeight:
    """A bf16 ``[N, K]`` weight re-laid for the few-rows product: ``[n-tile][K/32][4][16][8]``
    (tile of 16 rows, step of 32 of K, quarter of the step, row, 8 of K), rows padded with zeros
    to a multiple of 16, so that the 1 KiB a wavefront needs per step is contiguous and in the
    order of its lanes.  With ``halves=2`` (a joined ``[gate; up]`` matrix) each half is tiled on its own
    and the gate tiles come first."""

    def __init__(self, weight: torch.Tensor, halves: int = 1):
        n, k = weight.shape
        if weight.dtype != torch.bfloat16 or k % 32 or n % halves:
            raise KernelError(f"TiledWeight: bf16 [N, K] with K % 32 == 0 needed, got {tuple(weight.shape)} {weight.dtype}")
        self.n, self.k, self.halves = n, k, halves
        parts = []
        for h in weight.view(halves, n // halves, k):
            rows = h.shape[0]
            pad = (-rows) % 16
            if pad:
                h = torch.cat([h, torch.zeros((pad, k), dtype=h.dtype, device=h.device)])
            # [tile][row 16][step][g 4][8] -> [tile][step][g][row][8]: the 16 bytes of lane r + 16 g
            # of a wavefront lie at byte 16 (r + 16 g) of the step's 1 KiB, so neighbouring lanes
            # read neighbouring memory (four lanes per 64-byte access instead of one)
            parts.append(h.view((rows + pad) // 16, 16, k // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous())
        self.data = torch.cat(parts).contiguous()


class TiledRows:
    """At most 64 rows of ``width`` bf16 columns laid out ``[width / 8, R, 8]`` with ``R`` the row
    count rounded up to a multiple of 16, or 8 for up to 8 rows (the library says which:
    ``kva_tiled_rows``): element (m, c) at ``[c // 8, m, c % 8]``, rows past ``rows`` unwritten.  It is the order in which the lanes of a few-rows product read X (sixteen
    neighbouring lanes take the same 8 columns of sixteen neighbouring rows: 256 contiguous bytes
    instead of sixteen pieces a row apart), so a product that feeds another can leave its result
    like this.  ``to_rows()`` gives the plain ``[rows, width]``."""

    MAX_ROWS = 64

    def __init__(self, rows: int, width: int, device):
        if not (1 <= rows <= self.MAX_ROWS) or width % 8:
            raise KernelError(f"TiledRows: 1..{self.MAX_ROWS} rows and a multiple of 8 columns, not {rows} x {width}")
        self.rows, self.width = rows, width
        self.padded = int(hip_lib().kva_tiled_rows(int(rows)))
        self.data = torch.empty((width // 8, self.padded, 8), dtype=torch.bfloat16, device=device)

    @classmethod
    def from_rows(cls, x: torch.Tensor) -> "TiledRows":
        t = cls(x.shape[0], x.shape[1], x.device)
        t.data[:, :t.rows, :] = x.view(t.rows, t.width // 8, 8).permute(1, 0, 2)
        return t

    @property
    def shape(self):
        return (self.rows, self.width)

    @property
    def dtype(self):
        return self.data.dtype

    @property
    def device(self):
        return self.data.device

    def to_rows(self) -> torch.Tensor:
        return self.data.permute(1, 0, 2).reshape(self.padded, self.width)[:self.rows].contiguous()


def gemm_skinny(x: torch.Tensor, w: TiledWeight, out: Optional[torch.Tensor], swiglu: bool = False, *,
                sumsq: Optional[torch.Tensor] = None, norm_width: int = 0, eps: float = 0.0,
                hidden: Optional[torch.Tensor] = None, next_weight: Optional[torch.Tensor] = None,
                scaled_out: Optional[torch.Tensor] = None, sumsq_out: Optional[torch.Tensor] = None,
                x_tiled: bool = False, out_tiled: bool = False, activation: str = "silu"):
    """out = x @ W^T for at most 64 rows of x (bf16 operands, fp32 accumulation); ``w`` is the
    :class:`TiledWeight` of W.

    * ``out`` bf16 or fp32 ``[M, N]``; with ``swiglu`` the weight is a joined ``[gate; up]``
      matrix (tiled with ``halves=2``) and ``out`` is bf16 ``[M, N / 2]`` = silu(x gate^T) * (x up^T).
    * ``sumsq`` ``[M, parts]`` fp32: the rows of ``x`` are un-normalised norm inputs
      (``round(h * w_norm)``) and the product is scaled per token by
      ``rsqrt(sum(sumsq[m]) / norm_width + eps)``.
    * ``hidden`` (instead of ``out``): ``hidden += x @ W^T`` in place (fp32 add, rounded), plus
      ``scaled_out = round(hidden * next_weight)`` and ``sumsq_out[M, ceil(N / 16)]``.
    * ``out_tiled`` (gated product): ``out`` is ``[N / 2 / 8, R, 8]`` (``R``: see :class:`TiledRows`), element
      (m, c) at ``[c // 8, m, c % 8]`` - the order in which the lanes of a following few-rows
      product read it (a :class:`TiledRows`); such a result is given to that product as ``x``
      with ``x_tiled``."""
    if not isinstance(w, TiledWeight):
        raise KernelError("gemm_skinny: the weight must be a TiledWeight")
    if x_tiled:
        if not isinstance(x, TiledRows):
            raise KernelError("gemm_skinny: x_tiled needs a TiledRows")
        m, k, x = x.rows, x.width, x.data
    else:
        m, k = x.shape
    n = w.n
    if x.dtype != torch.bfloat16 or k != w.k or (swiglu != (w.halves == 2)):
        raise KernelError(f"gemm_skinny: bf16 x {tuple(x.shape)} does not fit weight [{w.n}, {w.k}] "
                          f"(halves {w.halves})")
    lib = hip_lib()
    if sumsq is not None and (sumsq.dim() != 2 or sumsq.shape[0] != m or norm_width <= 0):
        raise KernelError("gemm_skinny: sumsq must be [M, parts] and norm_width positive")
    parts = sumsq.shape[1] if sumsq is not None else 0
    if hidden is not None:
        if swiglu or out is not None:
            raise KernelError("gemm_skinny: the residual epilogue has no other output")
        p_out = lib.kva_gemm_skinny_sumsq_parts(n)
        if hidden.shape != (m, n) or hidden.dtype != torch.bfloat16 or scaled_out is None \
                or scaled_out.shape != (m, n) or scaled_out.dtype != torch.bfloat16 \
                or sumsq_out is None or sumsq_out.shape != (m, p_out):
            raise KernelError("gemm_skinny: hidden / scaled_out [M, N] bf16 and sumsq_out [M, ceil(N/16)] needed")
        if next_weight is not None and next_weight.shape != (n,):
            raise KernelError("gemm_skinny: the next norm's weight must be [N]")
        check(lib.kva_gemm_skinny(
            None, _dev(x, "x"), _dev(w.data, "w"), m, n, k, k, n, 3, _opt(sumsq, "sumsq", torch.float32), parts,
            int(norm_width), float(eps), _dev(hidden, "hidden"), _opt(next_weight, "next_weight"),
            1 if next_weight is not None and next_weight.dtype == torch.float32 else 0,
            _dev(scaled_out, "scaled_out"), _dev(sumsq_out, "sumsq_out", torch.float32),
            1 if x_tiled else 0, 0, _stream()),
            "gemm_skinny")
        return hidden
    cols = n // 2 if swiglu else n
    out_t = out
    if out_tiled:
        if not (isinstance(out, TiledRows) and swiglu and out.rows == m and out.width == cols):
            raise KernelError("gemm_skinny: out_tiled needs the gated product and a TiledRows of its size")
        out_t = out.data
    elif out.shape != (m, cols) or (swiglu and out.dtype != torch.bfloat16) \
            or out.dtype not in (torch.bfloat16, torch.float32):
        raise KernelError(f"gemm_skinny: out {tuple(out.shape)} {out.dtype} does not fit")
    mode = (2 | ACTIVATIONS[activation] << 4) if swiglu else (1 if out_t.dtype == torch.float32 else 0)     # (the gate's activation rides on mode 2)
    check(lib.kva_gemm_skinny(_dev(out_t, "out"), _dev(x, "x"), _dev(w.data, "w"), m, n, k, k, cols, mode,
                              _opt(sumsq, "sumsq", torch.float32), parts, int(norm_width), float(eps),
                              None, None, 0, None, None, 1 if x_tiled else 0, 1 if out_tiled else 0, _stream()),
          "gemm_skinny")
    return out


def gemm_skinny_partial_ranges(m: int, n: int, k: int) -> int:
    """Into how many ranges of K :func:`gemm_skinny_partials` cuts an [n, k] product of ``m`` rows;
    0: it does not take the shape (it takes 17 to 64 rows, K a multiple of 128)."""
    return int(hip_lib().kva_gemm_skinny_partial_slices(int(m), int(n), int(k)))


def gemm_skinny_partials(x: torch.Tensor, w: "TiledWeight") -> PartialSums:
    """x @ W^T for 17 to 64 rows as fp32 partial products over ranges of K, one per group of
    workgroups, so that a matrix with few rows of tiles still fills the chip while the rows of x go
    through LDS; whoever takes the :class:`PartialSums` adds them up."""
    if not isinstance(w, TiledWeight) or w.halves != 1:
        raise KernelError("gemm_skinny_partials: the weight must be a plain TiledWeight")
    m, k = x.shape
    if x.dtype != torch.bfloat16 or k != w.k:
        raise KernelError(f"gemm_skinny_partials: bf16 x {tuple(x.shape)} does not fit weight [{w.n}, {w.k}]")
    ranges = gemm_skinny_partial_ranges(m, w.n, k)
    if ranges < 1:
        raise KernelError(f"gemm_skinny_partials: {m} rows of a [{w.n}, {k}] product are not taken (17..64 rows, K % 128 == 0)")
    parts = torch.empty((ranges, m, w.n), dtype=torch.float32, device=x.device)
    check(hip_lib().kva_gemm_skinny_partials(_dev(parts, "parts"), _dev(x, "x"), _dev(w.data, "w"), m, w.n, k, k,
                                             ranges, _stream()), "gemm_skinny_partials")
    return PartialSums(parts)


def gemm_skinny_qkv_rope_supported(m: int, k: int, head_dim: int) -> bool:
    return bool(hip_lib().kva_gemm_skinny_qkv_rope_supported(int(m), int(k), int(head_dim)))


def gemm_skinny_qkv_rope(x: torch.Tensor, w: TiledWeight, q_out: torch.Tensor, num_q_heads: int,
                         num_kv_heads: int, head_dim: int, positions: torch.Tensor,
                         cos: Optional[torch.Tensor], sin: Optional[torch.Tensor],
                         k_cache: Optional[torch.Tensor], v_cache: Optional[torch.Tensor],
                         slot_mapping: Optional[torch.Tensor], page_size: int, *,
                         sumsq: Optional[torch.Tensor] = None, norm_width: int = 0, eps: float = 0.0):
    """The joined Q/K/V projection of at most 64 rows with rotation and cache write in its
    epilogue: ``q_out`` [M, nq*d] takes the rotated Q heads, the cache takes rotated K and plain V
    at ``slot_mapping`` (``k_cache`` None: nothing is cached).  ``cos``/``sin`` are the full
    tables [positions, d/2], or both None for no rotation.  ``sumsq`` as in :func:`gemm_skinny`."""
    if not isinstance(w, TiledWeight) or w.halves != 1:
        raise KernelError("gemm_skinny_qkv_rope: the weight must be a plain TiledWeight")
    m, k = x.shape
    if x.dtype != torch.bfloat16 or k != w.k or w.n != (num_q_heads + 2 * num_kv_heads) * head_dim:
        raise KernelError(f"gemm_skinny_qkv_rope: bf16 x {tuple(x.shape)} does not fit weight [{w.n}, {w.k}] "
                          f"for {num_q_heads}+2*{num_kv_heads} heads of {head_dim}")
    if q_out.shape != (m, num_q_heads * head_dim) or q_out.dtype != torch.bfloat16:
        raise KernelError("gemm_skinny_qkv_rope: q_out must be bf16 [M, nq * d]")
    if positions.shape != (m,):
        raise KernelError("gemm_skinny_qkv_rope: one position per row")
    if (cos is None) != (sin is None) or (cos is not None and (
            cos.shape != sin.shape or cos.dim() != 2 or cos.shape[1] * 2 != head_dim)):
        raise KernelError("gemm_skinny_qkv_rope: cos and sin tables must both be [positions, d/2]")
    if sumsq is not None and (sumsq.dim() != 2 or sumsq.shape[0] != m or norm_width <= 0):
        raise KernelError("gemm_skinny_qkv_rope: sumsq must be [M, parts] and norm_width positive")
    write = k_cache is not None
    if write:
        if v_cache is None or slot_mapping is None or slot_mapping.shape != (m,):
            raise KernelError("gemm_skinny_qkv_rope: K and V cache and one slot per row are all needed")
        check_cache_shapes("gemm_skinny_qkv_rope", k_cache, v_cache, num_kv_heads, head_dim)
        if k_cache.shape[3] != page_size or k_cache.dtype != torch.bfloat16:
            raise KernelError("gemm_skinny_qkv_rope: cache page size or dtype does not fit")
    check(hip_lib().kva_gemm_skinny_qkv_rope(
        _dev(q_out, "q_out"), q_out.shape[1], _dev(x, "x"), _dev(w.data, "w"), m, k, k, num_q_heads,
        num_kv_heads, head_dim, _opt(sumsq, "sumsq", torch.float32), sumsq.shape[1] if sumsq is not None else 0,
        int(norm_width), float(eps), _opt(cos, "cos", torch.float32), _opt(sin, "sin", torch.float32),
        _dev(positions, "positions", torch.int32),
        _dev(slot_mapping, "slot_mapping", torch.int32) if write else None,
        _opt(k_cache, "k_cache") if write else None, _opt(v_cache, "v_cache") if write else None,
        int(page_size), _stream()), "gemm_skinny_qkv_rope")
    return q_out


def gemm_skinny_sumsq_parts(n: int) -> int:
    return int(hip_lib().kva_gemm_skinny_sumsq_parts(int(n)))


def gemv_supported(m: int, n: int, k: int) -> bool:
    return bool(hip_lib().kva_gemv_supported(int(m), int(n), int(k)))


def gemv_sumsq_parts(n: int, k: int) -> int:
    """Partial sums of squares per token that :func:`gemv` writes with its residual epilogue."""
    return int(hip_lib().kva_gemv_sumsq_parts(int(n), int(k)))


def gemv(x: torch.Tensor, w: torch.Tensor, out: Optional[torch.Tensor], swiglu: bool = False, *,
         sumsq: Optional[torch.Tensor] = None, norm_width: int = 0, eps: float = 0.0,
         hidden: Optional[torch.Tensor] = None, next_weight: Optional[torch.Tensor] = None,
         scaled_out: Optional[torch.Tensor] = None, sumsq_out: Optional[torch.Tensor] = None,
         activation: str = "silu"):
    """out = x @ W^T for one or two rows of x over the plain row-major bf16 weight ``w`` [N, K]
    (fp32 accumulation).  The options are :func:`gemm_skinny`'s: ``swiglu`` for a joined
    ``[gate; up]`` matrix, ``sumsq`` to finish the input's norm, ``hidden`` / ``next_weight`` /
    ``scaled_out`` / ``sumsq_out`` [M, :func:`gemv_sumsq_parts`] for the residual epilogue."""
    if x.dim() != 2 or w.dim() != 2 or x.dtype != torch.bfloat16 or w.dtype != torch.bfloat16 \
            or x.shape[1] != w.shape[1] or not w.is_contiguous() or x.stride(1) != 1:
        raise KernelError(f"gemv: bf16 x {tuple(x.shape)} does not fit a row-major bf16 weight {tuple(w.shape)}")
    m, k = x.shape
    n = w.shape[0]
    lib = hip_lib()
    if sumsq is not None and (sumsq.dim() != 2 or sumsq.shape[0] != m or norm_width <= 0):
        raise KernelError("gemv: sumsq must be [M, parts] and norm_width positive")
    parts = sumsq.shape[1] if sumsq is not None else 0
    norm = (_opt(sumsq, "sumsq", torch.float32), parts, int(norm_width), float(eps))
    if hidden is not None:
        if swiglu or out is not None:
            raise KernelError("gemv: the residual epilogue has no other output")
        p_out = gemv_sumsq_parts(n, k)
        if hidden.shape != (m, n) or hidden.dtype != torch.bfloat16 or scaled_out is None \
                or scaled_out.shape != (m, n) or scaled_out.dtype != torch.bfloat16 \
                or sumsq_out is None or sumsq_out.shape != (m, p_out):
            raise KernelError(f"gemv: hidden / scaled_out [M, N] bf16 and sumsq_out [M, {p_out}] needed")
        if next_weight is not None and next_weight.shape != (n,):
            raise KernelError("gemv: the next norm's weight must be [N]")
        check(lib.kva_gemv(None, _dev(x, "x", contiguous=False), _dev(w, "w"), m, n, k, x.stride(0), n, 3, *norm,
                           _dev(hidden, "hidden"), _opt(next_weight, "next_weight"),
                           1 if next_weight is not None and next_weight.dtype == torch.float32 else 0,
                           _dev(scaled_out, "scaled_out"), _dev(sumsq_out, "sumsq_out", torch.float32), _stream()),
              "gemv")
        return hidden
    cols = n // 2 if swiglu else n
    if out.shape != (m, cols) or (swiglu and out.dtype != torch.bfloat16) \
            or out.dtype not in (torch.bfloat16, torch.float32) or not out.is_contiguous():
        raise KernelError(f"gemv: out {tuple(out.shape)} {out.dtype} does not fit")
    mode = (2 | ACTIVATIONS[activation] << 4) if swiglu else (1 if out.dtype == torch.float32 else 0)
    check(lib.kva_gemv(_dev(out, "out"), _dev(x, "x", contiguous=False), _dev(w, "w"), m, n, k, x.stride(0), cols, mode, *norm,
                       None, None, 0, None, None, _stream()), "gemv")
    return out


def gemv_merged_supported(m: int, n: int, k: int, head_dim: int, parts: int) -> bool:
    """Whether :func:`gemv_merged` takes ``m`` tokens of ``k / head_dim`` heads with ``parts``
    partial results each."""
    return bool(hip_lib().kva_gemv_merged_supported(int(m), int(n), int(k), int(head_dim), int(parts)))


def gemv_merge_max_parts(m: int = 2) -> int:
    """Partial results a row that :func:`gemv_merged` adds up for ``m`` tokens."""
    return int(hip_lib().kva_gemv_merge_max_parts(int(m)))


def gemv_merged(x: AttentionPartials, w: torch.Tensor, hidden: torch.Tensor, next_weight: Optional[torch.Tensor],
                scaled_out: torch.Tensor, sumsq_out: torch.Tensor) -> torch.Tensor:
    """:func:`gemv` with its residual epilogue over an attention output that is still in partial
    results per key range: the kernel adds them up (as the merge kernel would, rounded to bf16)
    where it would have read the tokens."""
    m, k = x.shape
    n = w.shape[0]
    if w.dim() != 2 or w.dtype != torch.bfloat16 or w.shape[1] != k or not w.is_contiguous():
        raise KernelError(f"gemv_merged: partial results of {tuple(x.shape)} do not fit a row-major bf16 weight {tuple(w.shape)}")
    if not gemv_merged_supported(m, n, k, x.head_dim, x.parts):
        raise KernelError(f"gemv_merged: {m} tokens, weight {tuple(w.shape)}, heads of {x.head_dim}, {x.parts} partial results: not supported")
    p_out = gemv_sumsq_parts(n, k)
    if hidden.shape != (m, n) or hidden.dtype != torch.bfloat16 or scaled_out.shape != (m, n) \
            or scaled_out.dtype != torch.bfloat16 or sumsq_out.shape != (m, p_out):
        raise KernelError(f"gemv_merged: hidden / scaled_out [M, N] bf16 and sumsq_out [M, {p_out}] needed")
    if next_weight is not None and next_weight.shape != (n,):
        raise KernelError("gemv_merged: the next norm's weight must be [N]")
    check(hip_lib().kva_gemv_merged(
        _dev(x.part_o, "part_o", torch.float32), _dev(x.part_ml, "part_ml", torch.float32), x.parts, x.head_dim,
        _dev(w, "w"), m, n, k, _dev(hidden, "hidden"), _opt(next_weight, "next_weight"),
        1 if next_weight is not None and next_weight.dtype == torch.float32 else 0,
        _dev(scaled_out, "scaled_out"), _dev(sumsq_out, "sumsq_out", torch.float32), _stream()), "gemv_merged")
    return hidden


def gemv_qkv_rope_supported(m: int, k: int, head_dim: int) -> bool:
    return bool(hip_lib().kva_gemv_qkv_rope_supported(int(m), int(k), int(head_dim)))


def gemv_qkv_rope(x: torch.Tensor, w: torch.Tensor, q_out: torch.Tensor, num_q_heads: int,
                  num_kv_heads: int, head_dim: int, positions: torch.Tensor,
                  cos: Optional[torch.Tensor], sin: Optional[torch.Tensor],
                  k_cache: Optional[torch.Tensor], v_cache: Optional[torch.Tensor],
                  slot_mapping: Optional[torch.Tensor], page_size: int, *,
                  sumsq: Optional[torch.Tensor] = None, norm_width: int = 0, eps: float = 0.0):
    """:func:`gemm_skinny_qkv_rope` for one or two rows, over the plain row-major weight."""
    m, k = x.shape
    if x.dtype != torch.bfloat16 or w.dtype != torch.bfloat16 or not w.is_contiguous() \
            or w.shape != ((num_q_heads + 2 * num_kv_heads) * head_dim, k):
        raise KernelError(f"gemv_qkv_rope: bf16 x {tuple(x.shape)} does not fit weight {tuple(w.shape)} "
                          f"for {num_q_heads}+2*{num_kv_heads} heads of {head_dim}")
    if q_out.shape != (m, num_q_heads * head_dim) or q_out.dtype != torch.bfloat16 or not q_out.is_contiguous():
        raise KernelError("gemv_qkv_rope: q_out must be bf16 [M, nq * d]")
    if positions.shape != (m,):
        raise KernelError("gemv_qkv_rope: one position per row")
    if (cos is None) != (sin is None) or (cos is not None and (
            cos.shape != sin.shape or cos.dim() != 2 or cos.shape[1] * 2 != head_dim)):
        raise KernelError("gemv_qkv_rope: cos and sin tables must both be [positions, d/2]")
    if sumsq is not None and (sumsq.dim() != 2 or sumsq.shape[0] != m or norm_width <= 0):
        raise KernelError("gemv_qkv_rope: sumsq must be [M, parts] and norm_width positive")
    write = k_cache is not None
    if write:
        if v_cache is None or slot_mapping is None or slot_mapping.shape != (m,):
            raise KernelError("gemv_qkv_rope: K and V cache and one slot per row are all needed")
        check_cache_shapes("gemv_qkv_rope", k_cache, v_cache, num_kv_heads, head_dim)
        if k_cache.shape[3] != page_size or k_cache.dtype != torch.bfloat16:
            raise KernelError("gemv_qkv_rope: cache page size or dtype does not fit")
    check(hip_lib().kva_gemv_qkv_rope(
        _dev(q_out, "q_out"), q_out.shape[1], _dev(x, "x"), _dev(w, "w"), m, k, x.stride(0), num_q_heads,
        num_kv_heads, head_dim, _opt(sumsq, "sumsq", torch.float32), sumsq.shape[1] if sumsq is not None else 0,
        int(norm_width), float(eps), _opt(cos, "cos", torch.float32), _opt(sin, "sin", torch.float32),
        _dev(positions, "positions", torch.int32),
        _dev(slot_mapping, "slot_mapping", torch.int32) if write else None,
        _opt(k_cache, "k_cache") if write else None, _opt(v_cache, "v_cache") if write else None,
        int(page_size), _stream()), "gemv_qkv_rope")
    return q_out


def normed_rows_finish(scaled: torch.Tensor, sumsq: torch.Tensor, norm_width: int, eps: float,
                       out: torch.Tensor, row_idx: Optional[torch.Tensor] = None) -> torch.Tensor:
    """out[i] = scaled[row] * rsqrt(sum(sumsq[row]) / norm_width + eps), row = row_idx[i] or i."""
    rows, width = out.shape
    if scaled.dim() != 2 or scaled.shape[1] != width or sumsq.shape[0] != scaled.shape[0] \
            or scaled.dtype != torch.bfloat16 or out.dtype != torch.bfloat16:
        raise KernelError("normed_rows_finish: bf16 scaled [T, H], sumsq [T, parts], out [rows, H]")
    if row_idx is None and rows != scaled.shape[0]:
        raise KernelError("normed_rows_finish: out needs as many rows as scaled")
    check(hip_lib().kva_normed_rows_finish(
        _dev(out, "out"), _dev(scaled, "scaled"), _dev(sumsq, "sumsq", torch.float32), sumsq.shape[1],
        rows, _opt(row_idx, "row_idx", torch.int32), width, float(eps), _stream()), "normed_rows_finish")
    return out


# --------------------------------------------------------------------------------------
# Mixers with a fixed-size state per request, and what goes with them.
def _entries(batch_arrays, what: str):
    q_start, seat = batch_arrays
    entries = seat.shape[0]
    if q_start.shape != (entries + 1,):
        raise KernelError(f"{what}: entries + 1 starts, one seat per entry")
    return _dev(q_start, "entry_q_start", torch.int32), _dev(seat, "entry_seat", torch.int32), entries


def _state_row(state: torch.Tensor, offset: int, elements: int, what: str) -> int:
    if state.dim() != 2 or state.dtype != torch.float32 or not state.is_contiguous() \
            or offset < 0 or offset + elements > state.shape[1]:
        raise KernelError(f"{what}: the state is fp32 [seats, n] and holds {elements} elements from {offset} on")
    return state.shape[1]


def causal_conv_act(y: torch.Tensor, col_off: int, weight: torch.Tensor, out: torch.Tensor, state: torch.Tensor,
                    state_off: int, entry_q_start: torch.Tensor, entry_seat: torch.Tensor, max_q_len: int,
                    in_bias: Optional[torch.Tensor] = None, out_bias: Optional[torch.Tensor] = None,
                    activation: Optional[str] = "silu") -> torch.Tensor:
    """A short causal convolution over time per channel, then silu: ``out[t, c] = silu(sum_j
    weight[c, j] * in[t - taps + 1 + j, c])`` with ``in`` the columns ``col_off ..`` of ``y``; the inputs
    before an entry's first token come from the seat's state (``taps - 1`` values per channel at
    ``state_off``, oldest first; zero for a fresh seat), which afterwards holds the entry's last ones.
    ``out`` is ``[T, channels]``, fp32 or bf16.  ``in_bias`` (fp32 per channel) is added to every input (the state
    holds inputs with it), ``out_bias`` to every sum; ``activation`` is ``"silu"`` or ``None``."""
    tokens, channels = out.shape
    for bias in (in_bias, out_bias):
        if bias is not None and (bias.shape != (channels,) or bias.dtype != torch.float32):
            raise KernelError("causal_conv_act: a bias is fp32, one value per channel")
    if activation not in (None, "silu"):
        raise KernelError(f"causal_conv_act: activation {activation!r} is neither None nor 'silu'")
    if weight.dim() != 2 or weight.shape[0] != channels or y.dim() != 2 \
            or y.shape[0] != tokens or col_off < 0 or col_off + channels > y.shape[1]:
        raise KernelError(f"causal_conv_act: y {tuple(y.shape)}, weight {tuple(weight.shape)}, out {tuple(out.shape)} do not fit")
    taps = weight.shape[1]
    seat_stride = _state_row(state, state_off, channels * (taps - 1), "causal_conv_act")
    qs, seat, entries = _entries((entry_q_start, entry_seat), "causal_conv_act")
    check(hip_lib().kva_causal_conv_act(
        _dev(out, "out"), dtype_code(out.dtype), channels, _dev(y, "y"), dtype_code(y.dtype), y.shape[1], int(col_off), _dev(weight, "weight"),
        dtype_code(weight.dtype), _dev(state, "state"), seat_stride, int(state_off), qs, seat, entries, int(max_q_len),
        channels, taps, _opt(in_bias, "in_bias"), _opt(out_bias, "out_bias"), 1 if activation == "silu" else 0,
        _stream()), "causal_conv_act")
    return out


def gated_delta_rule(qkv: torch.Tensor, y: torch.Tensor, beta_off: int, decay_off: int, a_log: Optional[torch.Tensor],
                     dt_bias: Optional[torch.Tensor], out: torch.Tensor, state: torch.Tensor, state_off: int,
                     entry_q_start: torch.Tensor, entry_seat: torch.Tensor, heads: int, kv_heads: int, dim: int,
                     vdim: int, unit_eps: float = 1e-6, channel_decay: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Per head and token, in order: ``S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q`` with
    q and k made unit vectors (``x / sqrt(sum x^2 + unit_eps)``, q also times ``dim^-1/2``),
    ``beta = sigmoid(y[t, beta_off + h])`` and ``g = exp(-exp(a_log[h]) softplus(y[t, decay_off + h] +
    dt_bias[h]))``.  ``qkv`` fp32 ``[T, 2 kv_heads dim + heads vdim]`` holds q, k (``kv_heads`` heads) and v;
    head h uses q/k head ``h // (heads / kv_heads)``.  ``S`` ``[heads, dim, vdim]`` lives at ``state_off`` of
    the seat's fp32 state row.  ``out`` fp32 ``[T, heads * vdim]``.

    ``channel_decay`` (fp32 ``[T, heads * dim]``, e.g. from :func:`small_product_f32` with ``rate_log``):
    the decay has one value per head and key channel and multiplies the rows of ``S`` one by one,
    ``S <- diag(g) S``; ``decay_off``, ``a_log`` and ``dt_bias`` are then not used."""
    tokens = out.shape[0]
    if qkv.shape != (tokens, 2 * kv_heads * dim + heads * vdim) or qkv.dtype != torch.float32 \
            or out.shape != (tokens, heads * vdim) or out.dtype != torch.float32 or y.dim() != 2 or y.shape[0] != tokens:
        raise KernelError(f"gated_delta_rule: qkv {tuple(qkv.shape)}, y {tuple(y.shape)}, out {tuple(out.shape)} do not fit")
    if not 0 <= beta_off <= y.shape[1] - heads:
        raise KernelError("gated_delta_rule: beta columns lie outside y")
    if channel_decay is not None:
        if channel_decay.shape != (tokens, heads * dim) or channel_decay.dtype != torch.float32:
            raise KernelError(f"gated_delta_rule: decays per channel are fp32 [T, heads * dim], got {tuple(channel_decay.shape)}")
        decay_off = 0
    elif not 0 <= decay_off <= y.shape[1] - heads or a_log is None or dt_bias is None \
            or a_log.shape != (heads,) or dt_bias.shape != (heads,):
        raise KernelError("gated_delta_rule: decay columns inside y, one rate and one bias per head")
    seat_stride = _state_row(state, state_off, heads * dim * vdim, "gated_delta_rule")
    qs, seat, entries = _entries((entry_q_start, entry_seat), "gated_delta_rule")
    check(hip_lib().kva_gated_delta_rule(
        _dev(out, "out"), _dev(state, "state"), seat_stride, int(state_off), _dev(qkv, "qkv"), qkv.shape[1],
        _dev(y, "y"), dtype_code(y.dtype), y.shape[1], int(beta_off), int(decay_off),
        _opt(a_log, "a_log", torch.float32), _opt(dt_bias, "dt_bias", torch.float32), float(unit_eps),
        _opt(channel_decay, "channel_decay"), channel_decay.shape[1] if channel_decay is not None else 0, qs, seat,
        entries, heads, kv_heads, dim, vdim, _stream()), "gated_delta_rule")
    return out


def gated_linear_attention(y: torch.Tensor, q_off: int, k_off: int, v_off: int, alpha: Optional[torch.Tensor], q_mul: float,
                           out: torch.Tensor, state: torch.Tensor, state_off: int, entry_q_start: torch.Tensor,
                           entry_seat: torch.Tensor, heads: int, dim: int, vdim: int,
                           head_decay: Optional[torch.Tensor] = None, activation: Optional[str] = None) -> torch.Tensor:
    """Per head and token, in order: ``S <- diag(alpha) S + k v^T; o = S^T (q_mul q)`` with a decay per
    key channel ``alpha`` (fp32 ``[T, heads * dim]``; :func:`small_product_f32` makes it from a low-rank
    projection).  q, k (``heads x dim``) and v (``heads x vdim``) are columns of ``y`` from ``q_off``,
    ``k_off``, ``v_off`` on.  ``out`` fp32 ``[T, heads * vdim]``.

    ``alpha=None`` with ``head_decay`` (fp32 ``[heads]``): one fixed decay a head for all its channels
    and every token, ``S <- decay_h S + k v^T``.  ``activation="silu"``: q, k and v pass a silu (in
    fp32) on their way in."""
    tokens = out.shape[0]
    if y.dim() != 2 or y.shape[0] != tokens or out.shape != (tokens, heads * vdim) or out.dtype != torch.float32:
        raise KernelError(f"gated_linear_attention: y {tuple(y.shape)}, out {tuple(out.shape)} do not fit")
    if alpha is not None:
        if alpha.shape != (tokens, heads * dim) or alpha.dtype != torch.float32 or head_decay is not None:
            raise KernelError(f"gated_linear_attention: alpha {tuple(alpha.shape)} is fp32 [T, heads * dim], without fixed decays")
    elif head_decay is None or head_decay.shape != (heads,) or head_decay.dtype != torch.float32:
        raise KernelError("gated_linear_attention: decays per token and channel, or one fp32 value a head")
    if activation not in (None, "silu"):
        raise KernelError(f"gated_linear_attention: activation {activation!r} is neither None nor 'silu'")
    for off, n in ((q_off, heads * dim), (k_off, heads * dim), (v_off, heads * vdim)):
        if not 0 <= off <= y.shape[1] - n:
            raise KernelError("gated_linear_attention: q, k or v columns lie outside y")
    seat_stride = _state_row(state, state_off, heads * dim * vdim, "gated_linear_attention")
    qs, seat, entries = _entries((entry_q_start, entry_seat), "gated_linear_attention")
    check(hip_lib().kva_gated_linear_attention(
        _dev(out, "out"), _dev(state, "state"), seat_stride, int(state_off), _dev(y, "y"), dtype_code(y.dtype),
        y.shape[1], int(q_off), int(k_off), int(v_off), _opt(alpha, "alpha"), alpha.shape[1] if alpha is not None else 0,
        float(q_mul), _opt(head_decay, "head_decay"), 1 if activation == "silu" else 0, qs, seat,
        entries, heads, dim, vdim, _stream()), "gated_linear_attention")
    return out


STATE_SPACE_MAX_STATE = 512
STATE_SPACE_KERNELS = {"scan": 0, "token": 1, "chunks": 2}
STATE_SPACE_CHUNK_FROM = 24         # entries of so many tokens and more go in chunks on the matrix cores


def state_space_plan(lengths, heads: int, groups: int, state_size: int, vdim: int, dtype: torch.dtype) -> list:
    """The launches of :func:`state_space` for entries of ``lengths`` tokens (host numbers): ``(kernel, shortest,
    longest)``.  Which kernel takes an entry depends on its own length and the sizes alone."""
    def takes(kernel):
        return bool(hip_lib().kva_state_space_supported(STATE_SPACE_KERNELS[kernel], int(heads), int(groups), int(state_size),
                                                        int(vdim), dtype_code(dtype)))
    token = 1 if takes("token") else 0
    chunk = STATE_SPACE_CHUNK_FROM if takes("chunks") else 1 << 30
    ranges = [("token", 1, token), ("scan", token + 1, chunk - 1), ("chunks", chunk, 1 << 30)]
    return [(k, lo, hi) for k, lo, hi in ranges if any(lo <= int(n) <= hi for n in lengths)]


def state_space_workspace(tokens: int, entries: int, heads: int, state_size: int, vdim: int) -> int:
    """Bytes of workspace :func:`state_space` takes for a step whose entries go in chunks: the state in front of each."""
    return int(hip_lib().kva_state_space_workspace(int(tokens), int(entries), int(heads), int(state_size), int(vdim)))


def state_space(xbc: torch.Tensor, y: torch.Tensor, dt_off: int, a_log: torch.Tensor, dt_bias: torch.Tensor,
                skip: torch.Tensor, out: torch.Tensor, state: torch.Tensor, state_off: int, entry_q_start: torch.Tensor,
                entry_seat: torch.Tensor, heads: int, groups: int, state_size: int, vdim: int, lengths,
                plan: Optional[list] = None) -> torch.Tensor:
    """Per head and token, in order: ``dt = softplus(y[t, dt_off + h] + dt_bias[h])``, ``S <- exp(-exp(a_log[h]) dt) S
    + dt B x^T``, ``out = S^T C + skip[h] x``.  ``xbc`` (fp32 or bf16) ``[T, heads vdim + 2 groups state_size]`` holds x,
    then B and C of every group; head h uses group ``h // (heads / groups)``.  ``S`` ``[heads, state_size, vdim]`` lives
    at ``state_off`` of the seat's fp32 state row; ``out`` is fp32 ``[T, heads * vdim]``.  ``lengths``: the entries'
    numbers of tokens on the host, from which the launches are chosen (``plan``: other ones)."""
    tokens = out.shape[0]
    if heads % groups or xbc.shape != (tokens, heads * vdim + 2 * groups * state_size) \
            or out.shape != (tokens, heads * vdim) or out.dtype != torch.float32 or y.dim() != 2 or y.shape[0] != tokens:
        raise KernelError(f"state_space: xbc {tuple(xbc.shape)}, y {tuple(y.shape)}, out {tuple(out.shape)} do not fit")
    if not 0 <= dt_off <= y.shape[1] - heads:
        raise KernelError("state_space: the step sizes' columns lie outside y")
    for v in (a_log, dt_bias, skip):
        if v.shape != (heads,) or v.dtype != torch.float32:
            raise KernelError("state_space: rates, step biases and skips are fp32, one a head")
    seat_stride = _state_row(state, state_off, heads * state_size * vdim, "state_space")
    qs, seat, entries = _entries((entry_q_start, entry_seat), "state_space")
    if plan is None:
        # (the walk over the tokens takes any state; the other kernels want it at multiples of 16 bytes)
        plan = [("scan", 1, 1 << 30)] if state_off % 4 or seat_stride % 4 else \
            state_space_plan(lengths, heads, groups, state_size, vdim, xbc.dtype)
    lengths = [int(m) for m in lengths]
    if len(lengths) != entries or sum(lengths) != tokens:
        raise KernelError("state_space: one length per entry, of all the rows together")
    work = None
    if any(kernel == "chunks" for kernel, _, _ in plan):
        work = torch.empty(state_space_workspace(tokens, entries, heads, state_size, vdim), dtype=torch.uint8, device=out.device)
    for kernel, lo, hi in plan:
        check(hip_lib().kva_state_space(
            STATE_SPACE_KERNELS[kernel], int(lo), int(hi), _dev(out, "out"), _dev(state, "state"), seat_stride, int(state_off),
            _dev(xbc, "xbc"), dtype_code(xbc.dtype), xbc.shape[1], _dev(y, "y"), dtype_code(y.dtype), y.shape[1], int(dt_off),
            _dev(a_log, "a_log"), _dev(dt_bias, "dt_bias"), _dev(skip, "skip"), qs, seat, entries, int(heads), int(groups),
            int(state_size), int(vdim), _opt(work, "work"), 0 if work is None else work.numel(), tokens, max(lengths, default=0),
            _stream()), "state_space")
    return out


def block_gates(u: torch.Tensor, w_a: torch.Tensor, w_i: torch.Tensor, bias_a: torch.Tensor, bias_i: torch.Tensor,
                rate: torch.Tensor, a_out: torch.Tensor, b_out: torch.Tensor) -> None:
    """The decays and inputs of a real-gated linear recurrent unit for all tokens: with the channels of ``u``
    fp32 ``[T, width]`` in ``blocks`` equal runs and the square matrices ``w_a``, ``w_i`` ``[blocks, bs, bs]``
    (``[out, in]``, bf16 or fp32) of every run, ``r = sigmoid(w_a u_b + bias_a)``, ``i = sigmoid(w_i u_b + bias_i)``,
    ``a_out = exp(-rate r)`` and ``b_out = sqrt(1 - a^2) i u``; everything fp32."""
    T, width = u.shape
    if w_a.dim() != 3 or w_a.shape != w_i.shape or w_a.shape[1] != w_a.shape[2] or w_a.shape[0] * w_a.shape[1] != width \
            or w_a.dtype != w_i.dtype:
        raise KernelError(f"block_gates: matrices {tuple(w_a.shape)} / {tuple(w_i.shape)} do not cut {width} channels into equal runs")
    for t in (u, bias_a, bias_i, rate, a_out, b_out):
        if t.dtype != torch.float32:
            raise KernelError("block_gates: inputs, biases, rates and results are fp32")
    if bias_a.numel() != width or bias_i.numel() != width or rate.shape != (width,) or a_out.shape != u.shape or b_out.shape != u.shape:
        raise KernelError("block_gates: one bias and one rate per channel, results of u's shape")
    check(hip_lib().kva_block_gates(_dev(a_out, "a_out"), _dev(b_out, "b_out"), _dev(u, "u"), T, width, w_a.shape[0],
                                    _dev(w_a, "w_a"), _dev(w_i, "w_i"), dtype_code(w_a.dtype), _dev(bias_a, "bias_a"),
                                    _dev(bias_i, "bias_i"), _dev(rate, "rate"), _stream()), "block_gates")


def linear_scan_gate(a: torch.Tensor, b: torch.Tensor, gate: torch.Tensor, gate_off: int, gate_bias: Optional[torch.Tensor],
                     out: torch.Tensor, out_off: int, state: torch.Tensor, state_off: int, entry_q_start: torch.Tensor,
                     entry_seat: torch.Tensor, mul: float = 1.0) -> torch.Tensor:
    """``S_t = a_t S_(t-1) + b_t`` per channel over every entry's tokens in order, from the seat's ``S`` fp32
    ``[width]`` at ``state_off`` (which takes the last one); ``out[t, out_off + c] = S_t * gelu_tanh(gate[t,
    gate_off + c] + gate_bias[c]) * mul``.  ``a``, ``b`` fp32 ``[T, width]``; ``gate`` and ``out`` may be wider."""
    T, width = a.shape
    if b.shape != a.shape or a.dtype != torch.float32 or b.dtype != torch.float32 or gate.dim() != 2 or gate.shape[0] != T \
            or out.dim() != 2 or out.shape[0] != T or not 0 <= gate_off <= gate.shape[1] - width \
            or not 0 <= out_off <= out.shape[1] - width:
        raise KernelError(f"linear_scan_gate: a {tuple(a.shape)}, gate {tuple(gate.shape)}, out {tuple(out.shape)} do not fit")
    if gate_bias is not None and (gate_bias.shape != (width,) or gate_bias.dtype != torch.float32):
        raise KernelError("linear_scan_gate: the gate's bias is fp32, one value per channel")
    seat_stride = _state_row(state, state_off, width, "linear_scan_gate")
    qs, seat, entries = _entries((entry_q_start, entry_seat), "linear_scan_gate")
    check(hip_lib().kva_linear_scan_gate(
        _dev(out, "out"), dtype_code(out.dtype), out.shape[1], int(out_off), _dev(a, "a"), _dev(b, "b"), width,
        _dev(gate, "gate"), dtype_code(gate.dtype), gate.shape[1], int(gate_off), _opt(gate_bias, "gate_bias"),
        _dev(state, "state"), seat_stride, int(state_off), qs, seat, entries, float(mul), _stream()), "linear_scan_gate")
    return out


def matrix_memory_state(heads: int, dim: int, vdim: int) -> int:
    """fp32 values of state :func:`matrix_memory` keeps per request."""
    return int(hip_lib().kva_matrix_memory_state(int(heads), int(dim), int(vdim)))


def matrix_memory(y: torch.Tensor, q_off: int, k_off: int, v_off: int, gates: torch.Tensor, cap: float, q_mul: float,
                  out: torch.Tensor, state: torch.Tensor, state_off: int, entry_q_start: torch.Tensor,
                  entry_seat: torch.Tensor, heads: int, dim: int, vdim: int) -> torch.Tensor:
    """A matrix memory with exponential gates per head: with ``i = cap tanh(zi / cap)``, ``f = logsigmoid(cap
    tanh(zf / cap))`` from ``gates`` fp32 ``[T, 2 heads]`` (``zi`` of all heads, then ``zf``) and a running maximum
    ``m' = max(f + m, i)``: ``S <- e^(f + m - m') S + e^(i - m') k v^T``, ``n`` likewise with ``k`` alone, ``o =
    S^T q / (max(|n . q|, e^(-m')) + 1e-6)`` with ``q`` times ``q_mul``.  q, k (``heads x dim``) and v (``heads x
    vdim``) are columns of ``y``; ``out`` is fp32 ``[T, heads * vdim]``; S, n and m live in the seat's state row."""
    T = out.shape[0]
    if out.shape != (T, heads * vdim) or out.dtype != torch.float32 or y.dim() != 2 or y.shape[0] != T \
            or gates.shape != (T, 2 * heads) or gates.dtype != torch.float32:
        raise KernelError(f"matrix_memory: y {tuple(y.shape)}, gates {tuple(gates.shape)}, out {tuple(out.shape)} do not fit")
    for off, n in ((q_off, heads * dim), (k_off, heads * dim), (v_off, heads * vdim)):
        if not 0 <= off <= y.shape[1] - n:
            raise KernelError("matrix_memory: q, k or v lies outside the projection's columns")
    seat_stride = _state_row(state, state_off, matrix_memory_state(heads, dim, vdim), "matrix_memory")
    qs, seat, entries = _entries((entry_q_start, entry_seat), "matrix_memory")
    check(hip_lib().kva_matrix_memory(
        _dev(out, "out"), _dev(state, "state"), seat_stride, int(state_off), _dev(y, "y"), dtype_code(y.dtype), y.shape[1],
        int(q_off), int(k_off), int(v_off), _dev(gates, "gates"), float(cap), float(q_mul), qs, seat, entries, int(heads),
        int(dim), int(vdim), _stream()), "matrix_memory")
    return out


HEAD_GATES = {"silu": 0, "sigmoid": 1}


def head_norm_gate(x: torch.Tensor, weight: Optional[torch.Tensor], eps: float, gate: Optional[torch.Tensor], gate_off: int,
                   out: torch.Tensor, out_off: int, heads: int, vdim: int, activation: Optional[str], mul: float = 1.0,
                   gate_first: bool = False) -> torch.Tensor:
    """``out[t, out_off + h vdim + j] = n(x)[t, h, j] * act(gate[t, gate_off + h vdim + j]) * mul`` where
    ``n`` divides every head by its root mean square (``sqrt(mean_j x^2 + eps)``) and multiplies by
    ``weight[j]`` (fp32 ``[vdim]``, shared by the heads) or ``weight[h vdim + j]`` (fp32 ``[heads * vdim]``),
    or leaves x as it is without a weight.  ``gate`` and ``out`` may be wider buffers; ``act`` is silu or
    sigmoid; without a ``gate`` the rows are only normed and multiplied.  ``gate_first``: the gate multiplies what is
    normed, ``n(x * act(gate))``."""
    rows = x.shape[0]
    if gate_first and gate is None:
        raise KernelError("head_norm_gate: a gate in front of the norm needs the gate")
    if x.shape != (rows, heads * vdim) or out.dim() != 2 \
            or out.shape[0] != rows or not 0 <= out_off <= out.shape[1] - heads * vdim:
        raise KernelError(f"head_norm_gate: x {tuple(x.shape)} and out {tuple(out.shape)} do not fit")
    if gate is not None and (gate.dim() != 2 or gate.shape[0] != rows or not 0 <= gate_off <= gate.shape[1] - heads * vdim):
        raise KernelError(f"head_norm_gate: x {tuple(x.shape)} and gate {tuple(gate.shape)} do not fit")
    if weight is not None and (weight.shape not in ((vdim,), (heads * vdim,)) or weight.dtype != torch.float32):
        raise KernelError("head_norm_gate: the weight is fp32, one value per element of a head (shared or not)")
    if gate is not None and activation not in HEAD_GATES:
        raise KernelError(f"head_norm_gate: activation {activation!r} is not one of {sorted(HEAD_GATES)}")
    w_stride = vdim if weight is not None and heads > 1 and weight.shape == (heads * vdim,) else 0
    check(hip_lib().kva_head_norm_gate(
        _dev(out, "out"), dtype_code(out.dtype), out.shape[1], int(out_off), _dev(x, "x"), dtype_code(x.dtype),
        _opt(weight, "weight"), float(eps), _opt(gate, "gate"), dtype_code(gate.dtype) if gate is not None else 0,
        gate.shape[1] if gate is not None else 0, int(gate_off),
        rows, heads, vdim, HEAD_GATES.get(activation, 0), 1 if gate_first else 0, float(mul), w_stride, _stream()), "head_norm_gate")
    return out


# --------------------------------------------------------------------------------------
# Routed experts.
MOE_TILE = 16
EXPERT_ACTIVATIONS = {"silu": 0, "relu": 1, "gelu_tanh": 2, "gelu": 3, "swish_clamped": 4, "relu2": 5}     # swish_clamped: gated only, with a limit


def moe_route(logits: torch.Tensor, correction: Optional[torch.Tensor], top: int, idx: torch.Tensor,
              wgt: torch.Tensor, renormalise: bool = False, over_chosen: bool = False, *, scores: str = "softmax",
              groups: int = 1, keep_groups: int = 1, group_top: int = 2, weight_scale: float = 1.0,
              sum_eps: float = 0.0) -> None:
    """``scores = softmax(logits)`` over all router outputs; the ``top`` largest of ``scores +
    correction`` are chosen (of equal ones the lowest index) into ``idx`` ``[T, top]``; ``wgt`` gets their
    plain scores, divided by their sum with ``renormalise``.  ``over_chosen``: the ``top`` largest
    logits (plus correction) are chosen and the weights are the softmax over the chosen logits alone.
    ``scores="sigmoid"``: every output's score is its own ``sigmoid(logit)``.  ``groups`` > 1: the outputs form
    that many equal runs of neighbours; a run's score is the sum of its ``group_top`` largest ``scores +
    correction``, and only outputs of the ``keep_groups`` best runs can be chosen.  With ``renormalise`` the
    weights are ``score / (sum + sum_eps) * weight_scale``, without it ``score * weight_scale``."""
    tokens, outputs = logits.shape
    if scores not in ("softmax", "sigmoid"):
        raise KernelError(f"moe_route: scores {scores!r} is neither 'softmax' nor 'sigmoid'")
    if logits.dim() != 2 or logits.stride(1) != 1:
        raise KernelError("moe_route: the logits are rows with unit stride (possibly the first columns of a wider array)")
    if logits.dtype != torch.float32 or idx.shape != (tokens, top) or wgt.shape != (tokens, top) \
            or (correction is not None and correction.shape != (outputs,)):
        raise KernelError(f"moe_route: logits {tuple(logits.shape)}, idx {tuple(idx.shape)}, wgt {tuple(wgt.shape)} do not fit")
    check(hip_lib().kva_moe_route(_dev(idx, "idx", torch.int32), _dev(wgt, "wgt", torch.float32), _dev(logits, "logits", contiguous=False),
                                  _opt(correction, "correction", torch.float32), tokens, outputs, int(top),
                                  1 if renormalise else 0, 1 if over_chosen else 0, 1 if scores == "sigmoid" else 0,
                                  int(groups), int(keep_groups), int(group_top), float(weight_scale), float(sum_eps),
                                  logits.stride(0) if tokens > 1 else outputs, _stream()), "moe_route")


MOE_ROUTER_LIST_TOKENS = 16         # a step of up to so many tokens has its slots sorted by the router's launch


def moe_router_supported(x: torch.Tensor, w: torch.Tensor) -> bool:
    """Whether :func:`moe_router` takes rows like ``x`` and the router's matrix ``w``."""
    return bool(hip_lib().kva_moe_router_supported(dtype_code(x.dtype), dtype_code(w.dtype), w.shape[0], w.shape[1]))


def moe_router(x: torch.Tensor, w: torch.Tensor, bias: Optional[torch.Tensor], correction: Optional[torch.Tensor], outputs: int,
               top: int, idx: torch.Tensor, wgt: torch.Tensor, rest: Optional[torch.Tensor], renormalise: bool = False,
               over_chosen: bool = False, *, scores: str = "softmax", groups: int = 1, keep_groups: int = 1, group_top: int = 2,
               weight_scale: float = 1.0, sum_eps: float = 0.0, experts: int = 0, sorted_slot: Optional[torch.Tensor] = None,
               tile_expert: Optional[torch.Tensor] = None, group: int = 1) -> None:
    """The product ``logits = x @ w^T + bias`` of bf16 operands with fp32 sums and :func:`moe_route` over its first
    ``outputs`` columns in one launch; the columns behind them go to ``rest`` fp32 ``[T, N - outputs]``.  With
    ``sorted_slot`` and ``tile_expert`` (at most ``MOE_ROUTER_LIST_TOKENS`` tokens) the chosen slots are sorted as
    :func:`moe_align` does, in the same launch."""
    tokens, k = x.shape
    n = w.shape[0]
    if scores not in ("softmax", "sigmoid"):
        raise KernelError(f"moe_router: scores {scores!r} is neither 'softmax' nor 'sigmoid'")
    if w.dim() != 2 or w.shape[1] != k or not moe_router_supported(x, w) or idx.shape != (tokens, top) or wgt.shape != (tokens, top) \
            or not 0 < outputs <= n or (rest is None) != (outputs == n) or (rest is not None and rest.shape != (tokens, n - outputs)) \
            or (correction is not None and correction.shape != (outputs,)) or (bias is not None and bias.shape != (n,)):
        raise KernelError(f"moe_router: x {tuple(x.shape)}, w {tuple(w.shape)}, idx {tuple(idx.shape)} do not fit {outputs} outputs")
    tiles = 0
    if sorted_slot is not None:
        tiles = tile_expert.shape[0]
        if tokens > MOE_ROUTER_LIST_TOKENS or sorted_slot.shape != (tiles * MOE_TILE,) or tiles < moe_tiles(tokens * top, experts, group):
            raise KernelError(f"moe_router: {tiles} tiles cannot hold {tokens * top} slots of {experts} experts, or too many tokens")
    check(hip_lib().kva_moe_router(
        _dev(idx, "idx", torch.int32), _dev(wgt, "wgt", torch.float32), _opt(rest, "rest", torch.float32), _dev(x, "x"), k,
        _dev(w, "w"), _opt(bias, "bias", torch.float32), _opt(correction, "correction", torch.float32), tokens, n, k, int(outputs),
        int(top), 1 if renormalise else 0, 1 if over_chosen else 0, 1 if scores == "sigmoid" else 0, int(groups), int(keep_groups),
        int(group_top), float(weight_scale), float(sum_eps), _opt(sorted_slot, "sorted_slot", torch.int32),
        _opt(tile_expert, "tile_expert", torch.int32), int(experts), tiles * MOE_TILE, tiles, int(group), _stream()), "moe_router")


def moe_tiles(slots: int, experts: int, group: int = 1) -> int:
    """Tiles of 16 rows that hold ``slots`` (token, choice) pairs sorted by expert, whatever the split, every
    expert's run a multiple of ``group`` tiles."""
    rows = MOE_TILE * int(group)
    return (int(slots) + int(experts) * (rows - 1) + rows - 1) // rows * int(group)


# (token, choice) pairs an expert gets on average from which on its products go through LDS in groups of tiles
MOE_GROUPS = ((160, 8), (56, 4))


def moe_group(slots: int, experts: int, dtype: torch.dtype, *inner: int) -> int:
    """How many tiles of 16 rows the experts' products take at once (``group`` below) for products over
    ``inner`` elements: decided by sizes alone."""
    if dtype == torch.bfloat16:
        for least, group in MOE_GROUPS:
            if slots >= least * experts and all(hip_lib().kva_moe_group_supported(group, int(k)) for k in inner):
                return group
    return 1


def moe_align(idx: torch.Tensor, experts: int, sorted_slot: torch.Tensor, tile_expert: torch.Tensor, group: int = 1) -> None:
    """The slots ``idx.view(-1)`` that name one of the first ``experts`` router outputs, sorted by
    expert into ``sorted_slot`` (every tile of 16 places belongs to one expert, -1 pads) with the
    tiles' experts in ``tile_expert`` (-1: unused).  ``group``: an expert's run starts at a multiple of so many tiles."""
    slots, tiles = idx.numel(), tile_expert.shape[0]
    if sorted_slot.shape != (tiles * MOE_TILE,) or tiles < moe_tiles(slots, experts, group):
        raise KernelError(f"moe_align: {tiles} tiles cannot hold {slots} slots of {experts} experts")
    check(hip_lib().kva_moe_align(_dev(sorted_slot, "sorted_slot", torch.int32), _dev(tile_expert, "tile_expert", torch.int32),
                                  _dev(idx, "idx", torch.int32), slots, int(experts), tiles * MOE_TILE, tiles,
                                  int(group), _stream()), "moe_align")


def moe_table_align(table: torch.Tensor, ids: torch.Tensor, idx: torch.Tensor, wgt: torch.Tensor, experts: int,
                    sorted_slot: torch.Tensor, tile_expert: torch.Tensor, feedback: Optional[torch.Tensor] = None,
                    group: int = 1) -> None:
    """Experts by token id, without a router: ``idx[t] = table[ids[t]]`` (int32 ``[rows, top]``) with equal
    weights ``wgt[t, k] = 1 / top``, and the slots sorted by expert as :func:`moe_align` does, in one launch.  A
    negative id ``-1 - r`` stands for ``feedback[r]`` as in :func:`embed_gather`."""
    tokens, top = idx.shape
    tiles = tile_expert.shape[0]
    if table.dim() != 2 or table.shape[1] != top or ids.shape != (tokens,) or wgt.shape != (tokens, top):
        raise KernelError(f"moe_table_align: table {tuple(table.shape)}, ids {tuple(ids.shape)}, idx {tuple(idx.shape)} do not fit")
    if sorted_slot.shape != (tiles * MOE_TILE,) or tiles < moe_tiles(tokens * top, experts, group):
        raise KernelError(f"moe_table_align: {tiles} tiles cannot hold {tokens * top} slots of {experts} experts")
    check(hip_lib().kva_moe_table_align(
        _dev(sorted_slot, "sorted_slot", torch.int32), _dev(tile_expert, "tile_expert", torch.int32), _dev(idx, "idx", torch.int32),
        _dev(wgt, "wgt", torch.float32), _dev(table, "table", torch.int32), table.shape[0], _dev(ids, "ids", torch.int32),
        _opt(feedback, "feedback", torch.int32), tokens, top, 1.0 / top, int(experts), tiles * MOE_TILE, tiles,
        int(group), _stream()), "moe_table_align")


def moe_can_tile(w: torch.Tensor) -> bool:
    """Whether experts' matrices ``[experts, N, K]`` can be stored in operand order."""
    return w.is_cuda and w.dtype == torch.bfloat16 and w.shape[1] % 16 == 0 and w.shape[2] % 32 == 0


def moe_tiled_weight(w: torch.Tensor) -> torch.Tensor:
    """Experts' matrices ``[experts, N, K]`` in operand order: every tile of 16 x 32 elements, which a
    wavefront loads at once, is 1 KiB of neighbouring bytes (``[experts, N / 16, K / 32, k % 32 / 8, n % 16,
    8]``); the shape is left as it was."""
    e, n, k = w.shape
    return w.view(e, n // 16, 16, k // 32, 4, 8).permute(0, 1, 3, 4, 2, 5).contiguous().view(e, n, k)


def moe_expert_rows(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor, sorted_slot: torch.Tensor,
                    tile_expert: torch.Tensor, top: int, *, activation: Optional[str] = None,
                    slot_weight: Optional[torch.Tensor] = None, gated: bool = False, limit: float = 0.0,
                    group: int = 1, tiled: bool = False) -> torch.Tensor:
    """One product per tile against its expert's matrix ``w[e]`` ``[N, K]``.  With an ``activation``
    (the first product): row ``slot // top`` of ``x`` ``[T, K]`` - times the slot's ``slot_weight`` if given: a
    weight on the expert's input - goes through the product and the activation to the slot's sorted place of
    ``out`` ``[places, N]`` (x's type).  Without one (the second): the row at the sorted place of ``x`` ``[places,
    K]`` goes, times the slot's ``slot_weight`` if given, to row ``slot`` of ``out`` fp32 ``[slots, N]``.  ``gated`` (first product): rows ``2 j`` and ``2 j + 1`` of an expert's matrix are
    output j's gate and up rows, and ``out`` ``[places, N / 2]`` gets ``act(gate) * up``.  ``group`` (as the list
    was sorted, :func:`moe_group`): so many tiles at a time, through LDS.  ``tiled``: the matrices are
    stored in operand order (:func:`moe_tiled_weight`)."""
    tiles = tile_expert.shape[0]
    n_out = w.shape[1] // 2 if gated else w.shape[1]
    if gated and (activation is None or w.shape[1] % 2):
        raise KernelError("moe_expert_rows: gate and up rows come in pairs, in the first product")
    if slot_weight is not None and slot_weight.dtype != torch.float32:
        raise KernelError("moe_expert_rows: the slots' weights are fp32")
    if w.dim() != 3 or w.dtype != x.dtype or x.dim() != 2 or x.shape[1] != w.shape[2] or out.dim() != 2 \
            or out.shape[1] != n_out or sorted_slot.shape != (tiles * MOE_TILE,):
        raise KernelError(f"moe_expert_rows: x {tuple(x.shape)}, w {tuple(w.shape)}, out {tuple(out.shape)} do not fit")
    if activation is not None:
        if activation not in EXPERT_ACTIVATIONS:
            raise KernelError(f"moe_expert_rows: activation {activation!r} is not one of {sorted(EXPERT_ACTIVATIONS)}")
        if out.shape[0] != tiles * MOE_TILE or out.dtype != x.dtype:
            raise KernelError("moe_expert_rows: the first product writes one row of x's type per sorted place")
        if slot_weight is not None and slot_weight.numel() != x.shape[0] * int(top):
            raise KernelError("moe_expert_rows: one weight per (token, choice) slot")
    else:
        if x.shape[0] != tiles * MOE_TILE or out.dtype != torch.float32 \
                or (slot_weight is not None and slot_weight.numel() != out.shape[0]):
            raise KernelError("moe_expert_rows: the second product reads sorted places and writes fp32 rows per slot")
    check(hip_lib().kva_moe_expert_rows(
        _dev(out, "out"), dtype_code(out.dtype), _dev(x, "x"), _dev(w, "w"), dtype_code(x.dtype),
        _dev(sorted_slot, "sorted_slot", torch.int32), _dev(tile_expert, "tile_expert", torch.int32),
        _opt(slot_weight, "slot_weight"), tiles, int(top), w.shape[1], w.shape[2], 0 if activation is not None else 1,
        EXPERT_ACTIVATIONS.get(activation, 0), 1 if gated else 0, float(limit), int(group), 1 if tiled else 0, _stream()),
        "moe_expert_rows")
    return out


SMALL_PRODUCT_MAX_K = 8192


def small_product_f32(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor, bias: Optional[torch.Tensor] = None,
                      decay_tau: float = 0.0, rate_log: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``out = x @ w^T (+ bias)`` with fp32 products, sums and results, for small matrices whose results must
    not be rounded to 16 bits (a router's logits, the second half of a low-rank projection that makes
    decays).  With ``decay_tau`` > 0 the result is turned into a decay, ``sigmoid(.)^(1 / decay_tau)``.
    With ``rate_log`` (fp32 ``[G]``, G dividing N) it is turned into ``exp(-exp(rate_log[n // (N / G)]) *
    softplus(.))``: a decay per output whose rate is shared by runs of neighbouring outputs.
    ``x`` ``[T, K]`` may be columns of a wider buffer; ``x`` and ``w`` ``[N, K]`` are bf16 or fp32."""
    tokens, k = x.shape
    if rate_log is not None and (rate_log.dim() != 1 or rate_log.dtype != torch.float32 or w.shape[0] % rate_log.shape[0]
                                 or decay_tau > 0):
        raise KernelError("small_product_f32: rates are fp32, one per run of outputs, and exclude decay_tau")
    if bias is not None and (bias.shape != (w.shape[0],) or bias.dtype != torch.float32):
        raise KernelError("small_product_f32: the bias is fp32, one value per output")
    if w.dim() != 2 or w.shape[1] != k or out.shape != (tokens, w.shape[0]) or out.dtype != torch.float32 \
            or x.stride(1) != 1 or not 0 < k <= SMALL_PRODUCT_MAX_K:
        raise KernelError(f"small_product_f32: x {tuple(x.shape)}, w {tuple(w.shape)}, out {tuple(out.shape)} do not fit")
    check(hip_lib().kva_small_product_f32(
        _dev(out, "out"), _dev(x, "x", contiguous=False), dtype_code(x.dtype), x.stride(0) if tokens > 1 else k,
        _dev(w, "w"), dtype_code(w.dtype), tokens, w.shape[0], k, _opt(bias, "bias"),
        1.0 / float(decay_tau) if decay_tau > 0 else 0.0, _opt(rate_log, "rate_log"),
        w.shape[0] // rate_log.shape[0] if rate_log is not None else 0, _stream()), "small_product_f32")
    return out


class ExpertRows:
    """What routed experts returned, not added up yet: ``rows`` (fp32 ``[T * top, width]``, weighted) and, optionally, the
    output ``extra`` of an expert every token uses, times ``sigmoid(extra_gate[t])`` (fp32, a column) if that is there.
    Whoever reads the sum next may form it in its own pass (:func:`tanh_step`); :meth:`sum` forms it with
    :func:`moe_combine`."""

    def __init__(self, x, rows, idx, wgt, experts: int, extra=None, extra_gate=None):
        self.x, self.rows, self.idx, self.wgt, self.experts, self.extra, self.extra_gate = x, rows, idx, wgt, experts, extra, extra_gate
        self.top = idx.shape[1]

    @property
    def shape(self):
        return self.x.shape

    @property
    def dtype(self):
        return self.x.dtype

    def gate_column(self):
        """(the gate's numbers as a one-dimensional view or None, elements from one to the next)"""
        g = self.extra_gate
        if g is None:
            return None, 0
        g = g[:, 0] if g.dim() == 2 else g
        return g, g.stride(0) if g.shape[0] > 1 else 1

    def sum(self) -> torch.Tensor:
        return moe_combine(self.x, self.rows, self.idx, self.wgt, self.experts, torch.empty_like(self.x), extra=self.extra,
                           extra_gate=self.extra_gate)


def moe_combine(x: torch.Tensor, rows: torch.Tensor, idx: torch.Tensor, wgt: torch.Tensor, experts: int,
                out: torch.Tensor, extra: Optional[torch.Tensor] = None,
                extra_gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``out[t] = sum over the token's choices`` of the slot's row of ``rows`` (fp32 ``[T * top, width]``,
    already weighted) or, for a choice past the real ``experts`` (an identity expert), ``wgt * x[t]``;
    ``extra`` (x's shape and type: what an expert that every token uses returned) is added last - times
    ``sigmoid(extra_gate[t])`` with ``extra_gate`` (fp32, one number a token; it may be a column of a wider array)."""
    if extra_gate is not None and (extra is None or extra_gate.numel() != x.shape[0] or extra_gate.dtype != torch.float32):
        raise KernelError("moe_combine: the addend's gate is fp32, one number a token")
    gate_stride = 1
    if extra_gate is not None:
        if extra_gate.dim() == 2:
            extra_gate = extra_gate[:, 0]
        if extra_gate.dim() != 1:
            raise KernelError("moe_combine: the addend's gate is one column")
        gate_stride = extra_gate.stride(0) if extra_gate.shape[0] > 1 else 1
    tokens, width = x.shape
    top = idx.shape[1]
    if out.shape != x.shape or out.dtype != x.dtype or rows.shape != (tokens * top, width) or rows.dtype != torch.float32 \
            or idx.shape != (tokens, top) or wgt.shape != (tokens, top) \
            or (extra is not None and (extra.shape != x.shape or extra.dtype != x.dtype)):
        raise KernelError(f"moe_combine: x {tuple(x.shape)}, rows {tuple(rows.shape)}, idx {tuple(idx.shape)} do not fit")
    check(hip_lib().kva_moe_combine(_dev(out, "out"), _dev(x, "x"), dtype_code(x.dtype), _dev(rows, "rows"),
                                    _dev(idx, "idx", torch.int32), _dev(wgt, "wgt", torch.float32), _opt(extra, "extra"),
                                    None if extra_gate is None else _dev(extra_gate, "extra_gate", contiguous=False),
                                    int(gate_stride), tokens, width, top, int(experts), _stream()), "moe_combine")
    return out


# --------------------------------------------------------------------------------------
# Measurement: device time per class of kernel, from events around every launch.
KERNEL_CLASSES = {
    "embed_gather": "embedding", "embed_gather_prep": "embedding", "rmsnorm": "norm", "normed_rows_finish": "norm",
    "residual_add": "elementwise", "scale_softcap": "elementwise", "cast": "elementwise",
    "silu_mul": "activation", "rope_kv_write": "rope + cache write",
    "attention_rowwise": "attention", "attention_mfma": "attention", "attention_lds": "attention",
    "attention_rows_mfma": "attention", "latent_attention_rowwise": "attention", "latent_attention_mfma": "attention",
    "layernorm": "norm", "stream_join": "elementwise", "head_gate": "elementwise", "act_mul": "activation",
    "qk_encode_cache": "rope + cache write", "latent_encode_cache": "rope + cache write",
    "heads_matmul": "per-head products",
    "attention_mfma_rope": "attention",
    "gemm_nt_f32": "gemm fp32", "gemm_vendor": "gemm (vendor library)",
    "gemm_skinny": "gemm (few rows)", "gemm_skinny_qkv_rope": "gemm (few rows)",
    "gemv": "gemm (few rows)", "gemv_qkv_rope": "gemm (few rows)", "gemv_merged": "gemm (few rows)",
    "sample": "sampling", "mark_tokens": "sampling",
    "causal_conv_act": "recurrent mixers", "gated_delta_rule": "recurrent mixers",
    "gated_linear_attention": "recurrent mixers", "head_norm_gate": "elementwise",
    "moe_route": "routed experts", "moe_router": "routed experts", "moe_align": "routed experts", "moe_table_align": "routed experts", "moe_expert_rows": "routed experts",
    "moe_combine": "routed experts", "small_product_f32": "small fp32 products",
    "norm_into_stream": "norm", "table_gate": "elementwise",
    "hyper_step": "norm", "sandwich_step": "norm", "hyper_fill": "embedding", "bias_act": "activation",
    "tanh_step": "norm", "pair_embed": "embedding", "maps_encode_cache": "rope + cache write", "maps_combine": "elementwise",
    "state_space": "recurrent mixers",
    "block_gates": "recurrent mixers", "linear_scan_gate": "recurrent mixers", "matrix_memory": "recurrent mixers",
}


class KernelClassTimer:
    """``with KernelClassTimer() as t: ...`` brackets every kernel entry point of this module
    with a pair of events on the current stream; ``t.milliseconds()`` then gives the device time
    per class of kernel (the reference times its attention micro-benchmark the same way,
    ``micro/main_paged.cu:102-114``).  Launches one by one - a step replayed from a graph shows
    nothing here - so a class's time includes the gaps between its launches and their
    predecessors; it tells where a step's time goes, not how fast a kernel can be."""

    def __init__(self):
        self._marks = []
        self._saved = {}

    def __enter__(self):
        module = globals()
        for name, cls in KERNEL_CLASSES.items():
            fn = module[name]
            self._saved[name] = fn
            module[name] = self._wrap(fn, cls)
        return self

    def _wrap(self, fn, cls):
        marks = self._marks

        def timed(*args, **kwargs):
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            try:
                return fn(*args, **kwargs)
            finally:
                b.record()
                marks.append((cls, a, b))
        return timed

    def __exit__(self, *exc):
        globals().update(self._saved)
        self._saved = {}
        return False

    def milliseconds(self) -> dict:
        torch.cuda.synchronize()
        out: dict = {}
        for cls, a, b in self._marks:
            out[cls] = out.get(cls, 0.0) + a.elapsed_time(b)
        return {k: round(v, 4) for k, v in sorted(out.items(), key=lambda kv: -kv[1])}
