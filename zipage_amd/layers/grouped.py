"""Grouped-query attention with rotary positions over paged rows of keys and values.

A mixer that shares its input with others does not own its projections' launch: it names the rows it
wants (`project`), is handed the columns of the common product, and writes its part of the common
output rows."""
from __future__ import annotations

import torch

from zipage_amd import _lib
from zipage_amd.sight import Chunk

from .linear import fit, pad_to_multiple
from .runs import gather_rows, run_attention


def rotary_store(proj: torch.Tensor, positions: torch.Tensor, freqs: torch.Tensor, heads: int, kv_heads: int,
                 dim: int, vdim: int, cache: torch.Tensor, slot_mapping: torch.Tensor, return_kv: bool = False):
    """proj (N, >= heads * dim + kv_heads * (dim + vdim)), rows may be part of wider ones: q, k, v.
    Rotates the first 2 * len(freqs) dimensions of q's and k's heads (i with i + len(freqs)); [k | v] goes
    to the flat cache slots (-1 skips) and is returned too with `return_kv`.  Returns q (N, heads * dim)."""
    N, row = proj.shape[0], kv_heads * (dim + vdim)
    assert proj.stride(1) == 1 and proj.shape[1] >= heads * dim + row
    assert positions.dtype == slot_mapping.dtype == torch.int32 and positions.is_contiguous() and slot_mapping.is_contiguous()
    assert positions.numel() == slot_mapping.numel() == N and freqs.dtype == torch.float32
    assert cache.is_contiguous() and cache.dtype == proj.dtype and cache.shape[-1] == row
    q = torch.empty((N, heads * dim), dtype=proj.dtype, device=proj.device)
    kv = torch.empty((N, row), dtype=proj.dtype, device=proj.device) if return_kv else None
    _lib.call_models("zp_rotary_store", _lib.dev_ptr(proj), _lib.dev_ptr(positions), _lib.dev_ptr(freqs),
                     _lib.dev_ptr(q), _lib.dev_ptr(kv), _lib.dev_ptr(cache), _lib.dev_ptr(slot_mapping), N, heads,
                     kv_heads, dim, vdim, 2 * freqs.numel(), proj.stride(0), cache.numel() // row,
                     _lib.dtype_tag(proj), _lib.stream_ptr(proj))
    return (q, kv) if return_kv else q


def grouped_rows_attention(q: torch.Tensor, cache: torch.Tensor, heads: int, kv_heads: int, dim: int, vdim: int,
                           block_tables: torch.Tensor, context_lens: torch.Tensor, scale: float, out: torch.Tensor,
                           window: int | None = None, chunk: int | None = None, sinks: torch.Tensor | None = None,
                           table_rows: torch.Tensor | None = None, out_scale: float = 1.0):
    """Single tokens over paged rows [k | v].  q (N, heads * dim); cache (pages, BS, kv_heads * (dim + vdim));
    token i is the last of context_lens[i] tokens in row table_rows[i] (default i) of block_tables and sees
    what `run_attention` says.  out (N, heads * vdim), rows may be part of wider ones."""
    N = q.shape[0]
    assert q.is_contiguous() and q.shape[1] == heads * dim and out.stride(1) == 1 and out.shape == (N, heads * vdim)
    assert cache.is_contiguous() and cache.dtype == q.dtype == out.dtype and cache.shape[2] == kv_heads * (dim + vdim)
    for t in (block_tables, context_lens) + (() if table_rows is None else (table_rows,)):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert context_lens.numel() == N and (table_rows is None or table_rows.numel() == N)
    assert sinks is None or (sinks.dtype == torch.float32 and sinks.numel() == heads)
    B, NB = block_tables.shape
    pages, BS, _ = cache.shape
    w, c, tag = window or 0, chunk or 0, _lib.dtype_tag(q)
    size = _lib.load_models("hybrid").zp_grouped_rows_workspace(N, heads, kv_heads, dim, vdim, w, c, NB, BS, tag)
    ws = torch.empty(size, dtype=torch.uint8, device=q.device) if size > 0 else None
    _lib.call_models("zp_grouped_rows_attention", _lib.dev_ptr(q), _lib.dev_ptr(cache), _lib.dev_ptr(block_tables),
                     _lib.dev_ptr(context_lens), _lib.dev_ptr(table_rows), _lib.dev_ptr(sinks), _lib.dev_ptr(out), N,
                     heads, kv_heads, dim, vdim, BS, B, NB, pages, w, c, out.stride(0), float(scale),
                     float(out_scale), tag, _lib.dev_ptr(ws), max(size, 0), _lib.stream_ptr(q))
    return out


class GroupedAttention:
    """Queries of `heads` heads over keys and values of `kv_heads`; rotary positions on the first
    `rot_dims` dimensions (half-split pairs); the softmax may share its denominator with a learned sink
    per head.  `sight`: a Chunk, a window, or None (see zipage_amd/sight.py).

    Sizes are padded once, at load: dim to 32, vdim to 16, zero weights in between."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, sight,
                 rot_base: float, rot_dims: int, sinks: bool, out_scale: float = 1.0):
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads over {kv_heads} key heads")
        if rot_dims % 2 or rot_dims > dim:
            raise ValueError(f"{rot_dims} rotated dimensions of {dim}")
        self.width, self.heads, self.kv_heads, self.dim, self.vdim = width, heads, kv_heads, dim, vdim
        self.scale, self.sight, self.rot_base, self.rot_dims = scale, sight, rot_base, rot_dims
        self.has_sinks, self.out_scale, self.sinks = sinks, out_scale, None
        self.dim_p, self.vdim_p = pad_to_multiple(dim, 32), pad_to_multiple(vdim, 16)
        self.row = kv_heads * (self.dim_p + self.vdim_p)           # of a cached token
        self.columns = heads * self.dim_p + self.row               # of its projections
        self.out_columns = heads * self.vdim_p
        self._see = dict(chunk=sight.size) if isinstance(sight, Chunk) else dict(window=sight)

    @property
    def can_run(self) -> bool:
        """Sizes the run form's kernel covers; others run token by token."""
        return self.dim_p <= 256 and self.vdim_p <= 256

    def shapes(self) -> dict:
        H, G, D, V = self.heads, self.kv_heads, self.dim, self.vdim
        return {"q": (H * D, self.width), "k": (G * D, self.width), "v": (G * V, self.width),
                "o": (self.width, H * V), **({"sink": (H,)} if self.has_sinks else {})}

    def load(self, w: dict, dtype, device, padded_width: int):
        """Returns the rows of the common input product and the columns of the output product."""
        H, G, D, V, W = self.heads, self.kv_heads, self.dim, self.vdim, self.width
        rows = lambda t, n, d, dp: fit(t.view(n, d, W), n, dp, padded_width).flatten(0, 1)
        f = [self.rot_base ** (-2.0 * i / self.rot_dims) for i in range(self.rot_dims // 2)]
        self.freqs = torch.tensor(f, dtype=torch.float64).to(device=device, dtype=torch.float32)
        if self.has_sinks:
            self.sinks = w["sink"].to(device=device, dtype=torch.float32).contiguous()
        into = torch.cat([rows(w["q"], H, D, self.dim_p), rows(w["k"], G, D, self.dim_p),
                          rows(w["v"], G, V, self.vdim_p)])
        out = fit(w["o"].view(W, H, V), padded_width, H, self.vdim_p).flatten(1, 2)
        return into, out

    def allocate(self, num_pages: int, page_size: int, dtype, device) -> torch.Tensor:
        return torch.zeros(num_pages, page_size, self.row, dtype=dtype, device=device)

    def attend(self, proj: torch.Tensor, positions: torch.Tensor, cache: torch.Tensor, ctx, out: torch.Tensor):
        """proj: this mixer's columns of the projections, out: of the output rows.  The first
        ctx.context_lens.numel() tokens are attended singly, the rest in the runs of ctx.runs[sight]."""
        N = proj.shape[0]
        singles = ctx.context_lens.numel()
        runs = ctx.runs[self.sight] if singles < N else None
        direct = runs is not None and runs.key_slots is None      # the runs' keys are this step's own tokens
        sizes = (self.heads, self.kv_heads, self.dim_p, self.vdim_p)
        q = rotary_store(proj, positions, self.freqs, *sizes, cache, ctx.slot_mapping, return_kv=direct)
        q, kv = q if direct else (q, None)
        if runs is not None:
            kv = kv[singles:] if direct else gather_rows(cache, runs.key_slots)
            run_attention(q[singles:], kv, *sizes, runs.tiles, self.scale, out[singles:], sinks=self.sinks,
                          out_scale=self.out_scale, **self._see)
        if singles:
            grouped_rows_attention(q[:singles], cache, *sizes, ctx.block_tables, ctx.context_lens, self.scale,
                                   out[:singles], sinks=self.sinks, table_rows=ctx.table_rows,
                                   out_scale=self.out_scale, **self._see)
