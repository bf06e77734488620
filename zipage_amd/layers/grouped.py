"""Grouped-query attention with rotary positions over paged rows of keys and values.

A mixer that shares its input with others does not own its projections' launch: it names the rows it
wants (`project`), is handed the columns of the common product, and writes its part of the common
output rows."""
from __future__ import annotations

import ctypes as C
import math

import torch

from zipage_amd import _lib
from zipage_amd.sight import Chunk

from .linear import fit, pad_to_multiple
from .rotary import Rotary
from .runs import attention_form, gather_rows, run_attention


def rotary_store(proj: torch.Tensor, positions: torch.Tensor, freqs: torch.Tensor, heads: int, kv_heads: int,
                 dim: int, vdim: int, cache: torch.Tensor, slot_mapping: torch.Tensor, return_kv: bool = False,
                 maps: int = 1, bias: torch.Tensor | None = None):
    """proj (N, >= maps * (heads + kv_heads) * dim + kv_heads * vdim), rows may be part of wider ones: q, k, v, to
    which `bias` (fp32, one row) is added.  Rotates the first 2 * len(freqs) dimensions of every map of q's and
    k's heads (i with i + len(freqs)); [k | v] goes to the flat cache slots (-1 skips) and is returned too with
    `return_kv`.  Returns q (N, heads * maps * dim)."""
    values, heads, kv_heads = kv_heads * vdim, heads * maps, kv_heads * maps
    N, row = proj.shape[0], kv_heads * dim + values
    assert proj.stride(1) == 1 and proj.shape[1] >= heads * dim + row
    assert bias is None or (bias.dtype == torch.float32 and bias.is_contiguous() and bias.numel() == heads * dim + row)
    assert positions.dtype == slot_mapping.dtype == torch.int32 and positions.is_contiguous() and slot_mapping.is_contiguous()
    assert positions.numel() == slot_mapping.numel() == N and freqs.dtype == torch.float32
    assert cache.is_contiguous() and cache.dtype == proj.dtype and cache.shape[-1] == row
    q = torch.empty((N, heads * dim), dtype=proj.dtype, device=proj.device)
    kv = torch.empty((N, row), dtype=proj.dtype, device=proj.device) if return_kv else None
    _lib.call_models("zp_rotary_store", _lib.dev_ptr(proj), _lib.dev_ptr(bias), _lib.dev_ptr(positions),
                     _lib.dev_ptr(freqs), _lib.dev_ptr(q), _lib.dev_ptr(kv), _lib.dev_ptr(cache),
                     _lib.dev_ptr(slot_mapping), N, heads, kv_heads, dim, values, 2 * freqs.numel(), proj.stride(0), cache.numel() // row,
                     _lib.dtype_tag(proj), _lib.stream_ptr(proj))
    return (q, kv) if return_kv else q


def grouped_rows_attention(q: torch.Tensor, cache: torch.Tensor, heads: int, kv_heads: int, dim: int, vdim: int,
                           block_tables: torch.Tensor, context_lens: torch.Tensor, scale: float, out: torch.Tensor,
                           window: int | None = None, chunk: int | None = None, sinks: torch.Tensor | None = None,
                           table_rows: torch.Tensor | None = None, out_scale: float = 1.0, form=None):
    """Single tokens over paged rows [k | v].  q (N, heads * maps * dim); cache (pages, BS, kv_heads * (maps * dim
    + vdim)); token i is the last of context_lens[i] tokens in row table_rows[i] (default i) of block_tables and
    sees what `run_attention` says.  out (N, heads * vdim), rows may be part of wider ones."""
    N, maps = q.shape[0], form.maps if form is not None else 1
    assert q.is_contiguous() and q.shape[1] == heads * maps * dim and out.stride(1) == 1 and out.shape == (N, heads * vdim)
    assert cache.is_contiguous() and cache.dtype == q.dtype == out.dtype
    assert cache.shape[2] == kv_heads * (maps * dim + vdim)
    for t in (block_tables, context_lens) + (() if table_rows is None else (table_rows,)):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert context_lens.numel() == N and (table_rows is None or table_rows.numel() == N)
    assert sinks is None or (sinks.dtype == torch.float32 and sinks.numel() == heads)
    B, NB = block_tables.shape
    pages, BS, _ = cache.shape
    w, c, tag = window or 0, chunk or 0, _lib.dtype_tag(q)
    size = _lib.load_models("grouped").zp_grouped_rows_workspace(N, heads, kv_heads, dim, vdim, maps, w, c, NB, BS, tag)
    ws = torch.empty(size, dtype=torch.uint8, device=q.device) if size > 0 else None
    _lib.call_models("zp_grouped_rows_attention", _lib.dev_ptr(q), _lib.dev_ptr(cache), _lib.dev_ptr(block_tables),
                     _lib.dev_ptr(context_lens), _lib.dev_ptr(table_rows), _lib.dev_ptr(sinks), form and C.byref(form),
                     _lib.dev_ptr(out), N, heads, kv_heads, dim, vdim, BS, B, NB, pages, w, c, out.stride(0), float(scale),
                     float(out_scale), tag, _lib.dev_ptr(ws), max(size, 0), _lib.stream_ptr(q))
    return out


class GroupedAttention:
    """Queries of `heads` heads over keys and values of `kv_heads`; rotary positions on the first dimensions of
    every head (half-split pairs); the softmax may share its denominator with a learned sink per head, and
    scores may be soft-capped.  `sight`: a Chunk, a window, or None (see zipage_amd/sight.py).

    With `diff` it is differential: a head has two queries and two keys, each pair with a softmax of its own
    over the same values; the second result, times one learned number per layer, is taken off the first, and
    what is left is normed over the head and scaled by 1 - diff.  `bias`: q, k and v have one; `gated`: the
    output is multiplied with the sigmoid of a projection of the same input.

    Sizes are padded once, at load: dim to 8, vdim to 16, zero weights in between."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, sight,
                 rotary: Rotary, sinks: bool = False, out_scale: float = 1.0, softcap: float = 0.0,
                 diff: float | None = None, eps: float = 0.0, bias: bool = False, gated: bool = False):
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads over {kv_heads} key heads")
        if rotary.dims % 2 or rotary.dims > dim:
            raise ValueError(f"{rotary.dims} rotated dimensions of {dim}")
        if diff is not None and sinks or gated and diff is None:
            raise ValueError("sinks go with one map, the output gate with two")
        self.width, self.heads, self.kv_heads, self.dim, self.vdim = width, heads, kv_heads, dim, vdim
        self.scale, self.sight, self.rotary, self.softcap = scale, sight, rotary, softcap
        self.has_sinks, self.out_scale, self.sinks = sinks, out_scale, None
        self.diff, self.eps, self.has_bias, self.gated = diff, eps, bias, gated
        self.maps = 1 if diff is None else 2
        if diff is not None:
            self.out_scale *= 1.0 - diff
        self.balance, self.bias = 0.0, None
        self.dim_p, self.vdim_p = pad_to_multiple(dim, 8), pad_to_multiple(vdim, 16)
        self.row = kv_heads * (self.maps * self.dim_p + self.vdim_p)          # of a cached token
        self.gate_at = heads * self.maps * self.dim_p + self.row               # behind q, k and v
        self.out_columns = heads * self.vdim_p
        self.columns = self.gate_at + (self.out_columns if gated else 0)       # of its projections
        self._see = dict(chunk=sight.size) if isinstance(sight, Chunk) else dict(window=sight)

    @property
    def can_run(self) -> bool:
        """Sizes the run form's kernel covers; others run token by token."""
        return self.maps * self.dim_p <= 256 and self.vdim_p <= 256

    def shapes(self) -> dict:
        H, G, D, V = self.heads, self.kv_heads, self.dim, self.vdim
        rows = {"q": H * self.maps * D, "k": G * self.maps * D, "v": G * V}
        return {**{k: (n, self.width) for k, n in rows.items()},
                **({k + ".b": (n,) for k, n in rows.items()} if self.has_bias else {}),
                **({k: (D,) for k in ("lq1", "lk1", "lq2", "lk2")} if self.maps == 2 else {}),
                **({"g": (H * V, self.width)} if self.gated else {}),
                "o": (self.width, H * V), **({"sink": (H,)} if self.has_sinks else {})}

    def load(self, w: dict, dtype, device, padded_width: int):
        """Returns the rows of the common input product and the columns of the output product."""
        H, G, D, V, W = self.heads, self.kv_heads, self.dim, self.vdim, self.width
        parts = {"q": (H * self.maps, D, self.dim_p), "k": (G * self.maps, D, self.dim_p), "v": (G, V, self.vdim_p)}
        rows = lambda t, n, d, dp: fit(t.view(n, d, W), n, dp, padded_width).flatten(0, 1)
        self.freqs = self.rotary.frequencies(device)
        if self.has_sinks:
            self.sinks = w["sink"].to(device=device, dtype=torch.float32).contiguous()
        if self.has_bias:
            bias = [fit(w[k + ".b"].view(n, d), n, dp).flatten() for k, (n, d, dp) in parts.items()]
            self.bias = torch.cat(bias).to(device=device, dtype=torch.float32).contiguous()
        if self.maps == 2:
            dot = lambda i: float((w[f"lq{i}"].double() * w[f"lk{i}"].double()).sum())
            self.balance = math.exp(dot(1)) - math.exp(dot(2)) + self.diff
        into = [rows(w[k], *p) for k, p in parts.items()]
        if self.gated:
            into.append(rows(w["g"], H, V, self.vdim_p))
        out = fit(w["o"].view(W, H, V), padded_width, H, self.vdim_p).flatten(1, 2)
        return torch.cat(into), out

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
        q = rotary_store(proj, positions, self.freqs, *sizes, cache, ctx.slot_mapping, return_kv=direct,
                         maps=self.maps, bias=self.bias)
        q, kv = q if direct else (q, None)
        form = lambda rows: attention_form(self.softcap, self.maps, self.balance, self.eps, self.vdim,
                                           proj[rows, self.gate_at:self.columns] if self.gated else None)
        if runs is not None:
            kv = kv[singles:] if direct else gather_rows(cache, runs.key_slots)
            run_attention(q[singles:], kv, *sizes, runs.tiles, self.scale, out[singles:], sinks=self.sinks,
                          out_scale=self.out_scale, form=form(slice(singles, N)), **self._see)
        if singles:
            grouped_rows_attention(q[:singles], cache, *sizes, ctx.block_tables, ctx.context_lens, self.scale,
                                   out[:singles], sinks=self.sinks, table_rows=ctx.table_rows,
                                   out_scale=self.out_scale, form=form(slice(0, singles)), **self._see)
