"""Attention of runs of prompt tokens, and the gather of the cached rows they look back on."""
from __future__ import annotations

import torch

from zipage_amd import _lib


def gather_rows(src: torch.Tensor, rows: torch.Tensor) -> torch.Tensor:
    """src viewed as (slots, width): its rows `rows` (int32)."""
    width = src.shape[-1]
    assert src.is_contiguous() and rows.dtype == torch.int32 and rows.is_contiguous()
    out = torch.empty((rows.numel(), width), dtype=src.dtype, device=src.device)
    _lib.call_models("zp_gather_rows", _lib.dev_ptr(src), _lib.dev_ptr(rows), _lib.dev_ptr(out),
                     rows.numel(), width * src.element_size(), src.numel() // width, _lib.stream_ptr(src))
    return out


def run_attention(q: torch.Tensor, kv: torch.Tensor, heads: int, kv_heads: int, dim: int, vdim: int,
                  tiles: torch.Tensor, scale: float, out: torch.Tensor, window: int | None = None,
                  chunk: int | None = None, sinks: torch.Tensor | None = None, out_scale: float = 1.0):
    """q (N, heads * dim); kv (Nk, kv_heads * dim + kv_heads * vdim); tiles (T, 4) int32 as
    `inputs.plan_runs` makes them; out (N, heads * vdim), rows may be part of wider ones.  A query sees
    the last `window` positions, its own block of `chunk` positions, or all of its run; sinks (heads,)
    fp32 join the softmax's denominator."""
    assert q.stride(1) == 1 and kv.is_contiguous() and out.stride(1) == 1
    assert kv.shape[1] == kv_heads * (dim + vdim) and out.shape == (q.shape[0], heads * vdim)
    assert tiles.dtype == torch.int32 and tiles.is_contiguous() and tiles.shape[1] == 4
    assert sinks is None or (sinks.dtype == torch.float32 and sinks.numel() == heads)
    v = kv[:, kv_heads * dim:]
    _lib.call_models("zp_run_attention", _lib.dev_ptr(q), _lib.dev_ptr(kv), v.data_ptr(), _lib.dev_ptr(out),
                     _lib.dev_ptr(tiles), _lib.dev_ptr(sinks), tiles.shape[0], heads, kv_heads, dim, vdim,
                     window or 0, chunk or 0, q.shape[0], kv.shape[0], q.stride(0), kv.stride(0), out.stride(0),
                     float(scale), float(out_scale), _lib.dtype_tag(q), _lib.stream_ptr(q))
    return out
