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
                 maps: int = 1, bias: torch.Tensor | None = None, form=None):
    """proj (N, >= maps * (heads + kv_heads) * dim + kv_heads * vdim), rows may be part of wider ones: q, k, v, to
    which `bias` (fp32, one row) is added.  Rotates the first 2 * len(freqs) dimensions of every map of q's and
    k's heads (i with i + len(freqs)); [k | v] goes to the flat cache slots (-1 skips) and is returned too with
    `return_kv`.  `form` see store_form.  Returns q (N, heads * maps * dim)."""
    values, heads, kv_heads = kv_heads * vdim, heads * maps, kv_heads * maps
    N, row = proj.shape[0], kv_heads * dim + values
    assert proj.stride(1) == 1 and proj.shape[1] >= heads * dim + (kv_heads * dim if form is not None and form.tied else row)
    assert bias is None or (bias.dtype == torch.float32 and bias.is_contiguous() and bias.numel() == heads * dim + row)
    assert positions.dtype == slot_mapping.dtype == torch.int32 and positions.is_contiguous() and slot_mapping.is_contiguous()
    assert positions.numel() == slot_mapping.numel() == N and freqs.dtype == torch.float32
    assert cache.is_contiguous() and cache.dtype == proj.dtype and cache.shape[-1] == row
    assert form is None or not form.V or form.V == vdim
    q = torch.empty((N, heads * dim), dtype=proj.dtype, device=proj.device)
    kv = torch.empty((N, row), dtype=proj.dtype, device=proj.device) if return_kv else None
    _lib.call_models("zp_rotary_store", _lib.dev_ptr(proj), _lib.dev_ptr(bias), _lib.dev_ptr(positions),
                     _lib.dev_ptr(freqs), form and C.byref(form), _lib.dev_ptr(q), _lib.dev_ptr(kv), _lib.dev_ptr(cache),
                     _lib.dev_ptr(slot_mapping), N, heads, kv_heads, dim, values, 2 * freqs.numel(), proj.stride(0), cache.numel() // row,
                     _lib.dtype_tag(proj), _lib.stream_ptr(proj))
    return (q, kv) if return_kv else q


def store_form(norm: torch.Tensor | None = None, q_norm: int = 0, k_norm: int = 0, eps: float = 0.0, tied: bool = False,
               value_freqs: torch.Tensor | None = None, turns: torch.Tensor | None = None):
    """What else a store does (zp_store_form), or None.  norm: fp32 weights of RMS norms over the whole of q and
    the whole of k, whose means run over q_norm and k_norm elements; tied: the values are the keys as projected;
    value_freqs (V / 2,) fp32: values turn too, adjacent elements a pair, and `turns` (N, V / 2, 2) fp32 receives
    cos and sin."""
    if norm is None and not tied and value_freqs is None:
        return None
    assert norm is None or (norm.dtype == torch.float32 and norm.is_contiguous())
    if value_freqs is not None:
        assert value_freqs.dtype == turns.dtype == torch.float32 and value_freqs.is_contiguous() and turns.is_contiguous()
        assert turns.shape[1:] == (value_freqs.numel(), 2)
    form = _lib.StoreForm(_lib.dev_ptr(norm) or None, q_norm, k_norm, float(eps), int(tied),
                          0 if value_freqs is None else 2 * value_freqs.numel(), _lib.dev_ptr(value_freqs) or None,
                          _lib.dev_ptr(turns) or None)
    form.held = (norm, value_freqs, turns)    # the form alone has their addresses
    return form


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
    every head; the softmax may share its denominator with a learned sink per head, and
    scores may be soft-capped.  `sight`: a Chunk, a window, or None (see zipage_amd/sight.py).

    With `diff` it is differential: a head has two queries and two keys, each pair with a softmax of its own
    over the same values; the second result, times one learned number per layer, is taken off the first, and
    what is left is normed over the head and scaled by 1 - diff.  `bias`: q, k and v have one; `gated`: the
    output is multiplied with the sigmoid of a projection of the same input.

    `qk_norm`: q and k are RMS-normed, each over all its heads at once, before they turn.  `tied`: the values are
    the keys as projected.  `turn_values`: values turn like keys, over their whole heads, and are cached so; the
    output turns back with its own position.

    Sizes are padded once, at load: dim to 8 (tied: 16), vdim to 16, zero weights in between; and rows of q, k and
    v are put in the order in which the kernels turn them."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, sight,
                 rotary: Rotary, sinks: bool = False, out_scale: float = 1.0, softcap: float = 0.0,
                 diff: float | None = None, eps: float = 0.0, bias: bool = False, gated: bool = False,
                 qk_norm: bool = False, tied: bool = False, turn_values: bool = False):
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads over {kv_heads} key heads")
        if rotary.dims % 2 or rotary.dims > dim:
            raise ValueError(f"{rotary.dims} rotated dimensions of {dim}")
        if diff is not None and sinks or gated and diff is None:
            raise ValueError("sinks go with one map, the output gate with two")
        if (qk_norm or tied or turn_values) and (diff is not None or bias) or tied and (turn_values or vdim != dim):
            raise ValueError("normed, tied and turning projections go with one map, without bias; tied values do not turn")
        if turn_values and vdim % 2:
            raise ValueError(f"values of {vdim} dimensions do not turn in pairs")
        self.width, self.heads, self.kv_heads, self.dim, self.vdim = width, heads, kv_heads, dim, vdim
        self.scale, self.sight, self.rotary, self.softcap = scale, sight, rotary, softcap
        self.has_sinks, self.out_scale, self.sinks = sinks, out_scale, None
        self.diff, self.eps, self.has_bias, self.gated = diff, eps, bias, gated
        self.maps = 1 if diff is None else 2
        if diff is not None:
            self.out_scale *= 1.0 - diff
        self.balance, self.bias = 0.0, None
        self.qk_norm, self.tied, self.turn_values, self.norm, self.value_freqs = qk_norm, tied, turn_values, None, None
        self.dim_p, self.vdim_p = pad_to_multiple(dim, 16 if tied else 8), pad_to_multiple(vdim, 16)
        self.row = kv_heads * (self.maps * self.dim_p + self.vdim_p)          # of a cached token
        # behind q, k and v
        self.gate_at = heads * self.maps * self.dim_p + self.row - (kv_heads * self.vdim_p if tied else 0)
        self.out_columns = heads * self.vdim_p
        self.columns = self.gate_at + (self.out_columns if gated else 0)       # of its projections
        self._see = dict(chunk=sight.size) if isinstance(sight, Chunk) else dict(window=sight)

    @property
    def can_run(self) -> bool:
        """Sizes the run form's kernel covers; others run token by token."""
        return self.maps * self.dim_p <= 256 and self.vdim_p <= 256

    def shapes(self) -> dict:
        H, G, D, V = self.heads, self.kv_heads, self.dim, self.vdim
        rows = {"q": H * self.maps * D, "k": G * self.maps * D, **({} if self.tied else {"v": G * V})}
        return {**{k: (n, self.width) for k, n in rows.items()},
                **({k + ".b": (n,) for k, n in rows.items()} if self.has_bias else {}),
                **({k: (D,) for k in ("lq1", "lk1", "lq2", "lk2")} if self.maps == 2 else {}),
                **({"g": (H * V, self.width)} if self.gated else {}),
                **({"q.norm": (H * D,), "k.norm": (G * D,)} if self.qk_norm else {}),
                "o": (self.width, H * V), **({"sink": (H,)} if self.has_sinks else {})}

    def load(self, w: dict, dtype, device, padded_width: int):
        """Returns the rows of the common input product and the columns of the output product."""
        H, G, D, V, W = self.heads, self.kv_heads, self.dim, self.vdim, self.width
        order = self.rotary.order(D)
        values = order if self.tied else self.rotary.adjacent_order(V) if self.turn_values else list(range(V))
        parts = {"q": (H * self.maps, D, self.dim_p, order), "k": (G * self.maps, D, self.dim_p, order),
                 "v": (G, V, self.vdim_p, values)}
        if self.tied:
            del parts["v"]
        rows = lambda t, n, d, dp, at: fit(t.view(n, d, W)[:, at], n, dp, padded_width).flatten(0, 1)
        flat = lambda t, n, d, dp, at: fit(t.view(n, d)[:, at], n, dp).flatten()
        f32 = lambda t: t.to(device=device, dtype=torch.float32).contiguous()
        self.freqs = self.rotary.frequencies(device)
        if self.has_sinks:
            self.sinks = f32(w["sink"])
        if self.has_bias:
            self.bias = f32(torch.cat([flat(w[k + ".b"], *p) for k, p in parts.items()]))
        if self.qk_norm:
            self.norm = f32(torch.cat([flat(w[k + ".norm"], *parts[k]) for k in ("q", "k")]))
        if self.turn_values:
            self.value_freqs = fit(Rotary(self.rotary.base, V).frequencies(device), self.vdim_p // 2)
        if self.maps == 2:
            dot = lambda i: float((w[f"lq{i}"].double() * w[f"lk{i}"].double()).sum())
            self.balance = math.exp(dot(1)) - math.exp(dot(2)) + self.diff
        into = [rows(w[k], *p) for k, p in parts.items()]
        if self.gated:
            into.append(rows(w["g"], H, V, self.vdim_p, values))
        out = fit(w["o"].view(W, H, V)[:, :, values], padded_width, H, self.vdim_p).flatten(1, 2)
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
        turns = torch.empty((N, self.vdim_p // 2, 2), dtype=torch.float32, device=proj.device) if self.turn_values else None
        store = store_form(self.norm, self.heads * self.dim, self.kv_heads * self.dim, self.eps, self.tied, self.value_freqs,
                           turns)
        q = rotary_store(proj, positions, self.freqs, *sizes, cache, ctx.slot_mapping, return_kv=direct,
                         maps=self.maps, bias=self.bias, form=store)
        q, kv = q if direct else (q, None)
        form = lambda rows: attention_form(self.softcap, self.maps, self.balance, self.eps, self.vdim,
                                           proj[rows, self.gate_at:self.columns] if self.gated else None,
                                           None if turns is None else turns[rows])
        if runs is not None:
            kv = kv[singles:] if direct else gather_rows(cache, runs.key_slots)
            run_attention(q[singles:], kv, *sizes, runs.tiles, self.scale, out[singles:], sinks=self.sinks,
                          out_scale=self.out_scale, form=form(slice(singles, N)), **self._see)
        if singles:
            grouped_rows_attention(q[:singles], cache, *sizes, ctx.block_tables, ctx.context_lens, self.scale,
                                   out[:singles], sinks=self.sinks, table_rows=ctx.table_rows,
                                   out_scale=self.out_scale, form=form(slice(0, singles)), **self._see)
