"""Attention of runs of prompt tokens, and the gather of the cached rows they look back on."""
from __future__ import annotations

import ctypes as C

import torch

from zipage_amd import _lib


def attention_form(softcap: float = 0.0, maps: int = 1, balance: float = 0.0, eps: float = 0.0, vdim: int = 0,
                   gate: torch.Tensor | None = None, turns: torch.Tensor | None = None):
    """What an attention does beyond the softmax of scaled products (zp_attention_form), or None.  maps 2: two
    softmaxes over the same values, o = rms(o1 - balance o2) (mean over `vdim`) times sigmoid(gate).  turns (N,
    V / 2, 2) fp32: cos and sin by which adjacent elements of every head's output turn back."""
    if not softcap and maps == 1 and turns is None:
        return None
    assert gate is None or gate.stride(1) == 1
    assert turns is None or (turns.dtype == torch.float32 and turns.is_contiguous() and turns.shape[2] == 2)
    form = _lib.AttentionForm(float(softcap), maps, float(balance), float(eps), vdim, _lib.dev_ptr(gate) or None,
                              0 if gate is None else gate.stride(0), _lib.dev_ptr(turns) or None)
    form.held = (gate, turns)                 # the form alone has their addresses
    return form


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
                  chunk: int | None = None, sinks: torch.Tensor | None = None, out_scale: float = 1.0, form=None,
                  shared: torch.Tensor | None = None):
    """q (N, heads * maps * (dim + shared dims)); kv (Nk, kv_heads * maps * dim + kv_heads * vdim); tiles (T,
    4) int32 as `inputs.plan_runs` makes them; out (N, heads * vdim), rows may be part of wider ones.  A query
    sees the last `window` positions, its own block of `chunk` positions, or all of its run; sinks (heads,)
    fp32 join the softmax's denominator; `form` see attention_form; `shared` (Nk, dims): the end of every
    head's key."""
    maps, extra = form.maps if form is not None else 1, 0 if shared is None else shared.shape[1]
    assert q.stride(1) == 1 and kv.is_contiguous() and out.stride(1) == 1 and q.shape[1] == heads * maps * (dim + extra)
    assert kv.shape[1] == kv_heads * (maps * dim + vdim) and out.shape == (q.shape[0], heads * vdim)
    assert shared is None or (shared.stride(1) == 1 and shared.shape[0] == kv.shape[0] and shared.dtype == kv.dtype)
    assert tiles.dtype == torch.int32 and tiles.is_contiguous() and tiles.shape[1] == 4
    assert sinks is None or (sinks.dtype == torch.float32 and sinks.numel() == heads)
    v = kv[:, kv_heads * maps * dim:]
    _lib.call_models("zp_run_attention", _lib.dev_ptr(q), _lib.dev_ptr(kv), v.data_ptr(), _lib.dev_ptr(shared),
                     _lib.dev_ptr(out), _lib.dev_ptr(tiles), _lib.dev_ptr(sinks), form and C.byref(form),
                     tiles.shape[0], heads, kv_heads, dim, extra, vdim, window or 0, chunk or 0, q.shape[0],
                     kv.shape[0], q.stride(0), kv.stride(0), 0 if shared is None else shared.stride(0), out.stride(0), float(scale), float(out_scale), _lib.dtype_tag(q), _lib.stream_ptr(q))
    return out
