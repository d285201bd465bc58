"""Kernel choice for attention over low-rank entries and for the per-head products around it."""
from __future__ import annotations

import torch

from . import kernels as K


def heads_product(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor, gates=None, rotate=None) -> torch.Tensor:
    """``out[t, h] = w[h] @ x[t, h]`` for ``w`` ``[heads, N, K]``; ``x`` and ``out`` may be views into
    wider buffers.  ``gates`` ``[T, heads]``: head h of row t times ``sigmoid(gates[t, h])``;
    gates ``[T, heads, N]``: every element times its own.  ``rotate``: rows rotated in the same launch
    (``kernels.heads_matmul``)."""
    return K.heads_matmul(x, w, out, gates, rotate)


# Workgroups (of four wavefronts) a launch should have before keys stop being cut into ranges: one a compute
# unit; two where two fit one (small ranks).
_TARGET_WORKGROUPS = 256
_SMALL_RANK = 128
_MIN_KEYS_PER_RANGE = 128       # a block of 32 keys for each wavefront of an item of few rows
FEW_ROWS, MANY_ROWS = 16, 64    # rows of a work item of the two kernels


def mfma_supported(rank: int, key_dim: int, page_size: int = 16) -> bool:
    """Whether the matrix-core kernels have an instance for these sizes."""
    return K.latent_attention_mfma_supported(rank, key_dim, page_size)


def choose_ranges(items: int, max_context: int, visible: int = 0, workgroups: int = _TARGET_WORKGROUPS) -> tuple:
    """(ranges, keys per range) for ``items`` work items over at most ``max_context`` keys: ranges
    of at least 128 keys until the launch has ``workgroups`` workgroups.  ``visible``
    > 0: a row sees at most so many keys (a window and the kept first positions), wherever they
    lie: the ranges are sized as if the context were that long, and most of them stay empty."""
    want = max(1, workgroups // max(1, items))
    span = min(max_context, visible) if visible > 0 else max_context
    ranges = max(1, min(want, span // _MIN_KEYS_PER_RANGE))
    if ranges == 1:
        return 1, 0
    per = (-(-span // ranges) + 31) // 32 * 32
    return -(-max_context // per), per


def latent_attention(q_lat: torch.Tensor, out: torch.Tensor, kv, batch, scale: float, window: int = 0,
                     keep_first: int = 0, sinks=None) -> torch.Tensor:
    """Causal attention of the step's tokens over the rows of ``kv.arrays["latent"]``
    (``[pages, page_size, key_dim]``): ``q_lat`` ``[T, heads, key_dim]``, ``out`` ``[T, heads, rank]``."""
    if window <= 0:
        keep_first = 0
    cache = kv.arrays["latent"]
    if q_lat.dtype == torch.bfloat16 and mfma_supported(out.shape[2], q_lat.shape[2], cache.shape[1]):
        # entries of at most 16 rows (decoded tokens) and longer ones (prompt portions) have a kernel each
        heads = q_lat.shape[1]
        if batch.max_q_len * heads <= FEW_ROWS:
            launches = [(*batch.attention_items(heads, 1, "all")[:2], FEW_ROWS)]
        elif batch.min_q_len * heads > FEW_ROWS:
            launches = [(*batch.attention_items(heads, MANY_ROWS // 16, "all")[:2], MANY_ROWS)]
        else:
            launches = [(*batch.attention_items(heads, MANY_ROWS // 16, "long")[:2], MANY_ROWS),
                        (*batch.attention_items(heads, 1, "short")[:2], FEW_ROWS)]
        ranges, per = choose_ranges(sum(l[0].shape[0] for l in launches), batch.max_context,
                                    window + keep_first if window > 0 else 0,
                                    _TARGET_WORKGROUPS * (2 if out.shape[2] <= _SMALL_RANK else 1))
        (item_entry, item_row0, rows), *more = launches
        return K.latent_attention_mfma(q_lat, out, cache, kv.block_table, item_entry, item_row0,
                                       batch.entry_seat, batch.entry_q_start, batch.entry_start_pos, scale, window,
                                       keep_first, sinks, ranges, per, rows, more)
    return K.latent_attention_rowwise(q_lat, out, kv.arrays["latent"], kv.block_table, batch.tok_seat,
                                      batch.positions, scale, window, keep_first, sinks)
