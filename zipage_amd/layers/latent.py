"""Latent attention: one cached vector per token, from which every head's key and value follow.

The wrappers are one HIP launch each; `LatentAttention` is the mixer a model puts together from
them, with its sizes and constants as parameters."""
from __future__ import annotations

import torch
import torch.nn.functional as F

from zipage_amd import _lib

from .linear import ResidualLinear, fit, pad_to_multiple
from .runs import gather_rows, run_attention


def latent_norm_store(down: torch.Tensor, q_weight: torch.Tensor, c_weight: torch.Tensor, q_norm: int,
                      c_norm: int, eps: float, cache: torch.Tensor, slot_mapping: torch.Tensor,
                      return_c: bool = False):
    """down (N, q_width + c_width): RMS norms of both parts (means over q_norm and c_norm elements,
    plain fp32 weights).  Returns the first (N, q_width); the second goes to the flat cache slots
    (-1 skips) and is returned too with `return_c`."""
    N = down.shape[0]
    qw, cw = q_weight.numel(), c_weight.numel()
    assert down.is_contiguous() and down.shape[1] == qw + cw
    assert q_weight.dtype == c_weight.dtype == torch.float32
    assert cache.is_contiguous() and cache.dtype == down.dtype and cache.shape[-1] == cw
    assert slot_mapping.dtype == torch.int32 and slot_mapping.is_contiguous() and slot_mapping.numel() == N
    q = torch.empty((N, qw), dtype=down.dtype, device=down.device)
    c = torch.empty((N, cw), dtype=down.dtype, device=down.device) if return_c else None
    _lib.call_models("zp_latent_norm_store", _lib.dev_ptr(down), _lib.dev_ptr(q_weight),
                     _lib.dev_ptr(c_weight), _lib.dev_ptr(q), _lib.dev_ptr(c), _lib.dev_ptr(cache),
                     _lib.dev_ptr(slot_mapping), N, qw, cw, q_norm, c_norm, cache.numel() // cw, float(eps),
                     _lib.dtype_tag(down), _lib.stream_ptr(down))
    return (q, c) if return_c else q


def headwise_linear(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
    """x (N, H, K), w (H, M, K) -> (N, H, M): every head its own matrix."""
    N, H, K = x.shape
    assert x.is_contiguous() and w.is_contiguous() and w.dtype == x.dtype and w.shape[0] == H and w.shape[2] == K
    if out is None:
        out = torch.empty((N, H, w.shape[1]), dtype=x.dtype, device=x.device)
    assert out.is_contiguous() and out.numel() == N * H * w.shape[1] and out.dtype == x.dtype
    _lib.call_models("zp_headwise_linear", _lib.dev_ptr(x), _lib.dev_ptr(w), _lib.dev_ptr(out), N, H, K,
                     w.shape[1], _lib.dtype_tag(x), _lib.stream_ptr(x))
    return out


def latent_rows_attention(q: torch.Tensor, cache: torch.Tensor, block_tables: torch.Tensor,
                          context_lens: torch.Tensor, scale: float, window: int | None = None,
                          table_rows: torch.Tensor | None = None) -> torch.Tensor:
    """Single tokens over paged latents.  q (N, H, R); cache (pages, BS, R); token i sees the last
    `window` of the context_lens[i] tokens in row table_rows[i] (default i) of block_tables."""
    N, H, R = q.shape
    assert q.is_contiguous() and cache.is_contiguous() and cache.dtype == q.dtype and cache.shape[2] == R
    for t in (block_tables, context_lens) + (() if table_rows is None else (table_rows,)):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert context_lens.numel() == N and (table_rows is None or table_rows.numel() == N)
    B, NB = block_tables.shape
    pages, BS, _ = cache.shape
    w, tag = window or 0, _lib.dtype_tag(q)
    size = _lib.load_models("latent").zp_latent_rows_workspace(N, H, R, w, NB, BS, tag)
    ws = torch.empty(max(size, 0), dtype=torch.uint8, device=q.device) if size > 0 else None
    out = torch.empty_like(q)
    _lib.call_models("zp_latent_rows_attention", _lib.dev_ptr(q), _lib.dev_ptr(cache),
                     _lib.dev_ptr(block_tables), _lib.dev_ptr(context_lens), _lib.dev_ptr(table_rows),
                     _lib.dev_ptr(out), N, H, R, BS, B, NB, pages, w, float(scale), tag, _lib.dev_ptr(ws),
                     max(size, 0), _lib.stream_ptr(q))
    return out


def latent_tiles_attention(q: torch.Tensor, kv: torch.Tensor, heads: int, dim: int, vdim: int,
                           tiles: torch.Tensor, scale: float, window: int | None, out: torch.Tensor):
    """Runs of prompt tokens over expanded keys and values.  q (N, heads * dim); kv (Nk, heads * dim
    + heads * vdim); tiles (T, 4) int32 as `inputs.plan_runs` makes them; out (N, heads * vdim)."""
    return run_attention(q, kv, heads, heads, dim, vdim, tiles, scale, out, window=window)


class LatentAttention:
    """The mixer.  Queries pass a low-rank bottleneck, keys and values of all heads are images of one
    normed latent c; no rotation.  Only c is cached.

    Two forms of the same sum run side by side in one step: single tokens work on the latents
    themselves (W_uk^T q against c, W_uv after the sum), so a decode reads kv_rank elements per
    cached token for all heads together; runs of prompt tokens expand c to keys and values once per
    run and use the smaller per-head dimensions.  float32 always takes the first form.

    Sizes are padded once, at load: ranks and dim to 32, vdim to 16, zero weights in between; the
    means of the norms run over the true sizes."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, q_rank: int, kv_rank: int,
                 scale: float, window: int | None, eps: float):
        self.width, self.heads, self.dim, self.vdim = width, heads, dim, vdim
        self.q_rank, self.kv_rank, self.scale, self.window, self.eps = q_rank, kv_rank, scale, window, eps
        self.padded_width = pad_to_multiple(width, 8)
        self.dim_p, self.vdim_p = pad_to_multiple(dim, 32), pad_to_multiple(vdim, 16)
        self.q_rank_p, self.kv_rank_p = pad_to_multiple(q_rank, 32), pad_to_multiple(kv_rank, 32)

    @property
    def can_expand(self) -> bool:
        """Sizes the run form's kernel covers; others run token by token."""
        return self.dim_p <= 256 and self.vdim_p <= 256

    def load(self, w: dict, dtype, device):
        """w: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, o as stored ([out, in], heads in order)."""
        H, D, V, R, Q, W = self.heads, self.dim, self.vdim, self.kv_rank, self.q_rank, self.width
        put = lambda t, dt=dtype: t.to(device=device, dtype=dt).contiguous()

        self.down = put(torch.cat([fit(w["dq"], self.q_rank_p, self.padded_width),
                                   fit(w["dkv"], self.kv_rank_p, self.padded_width)]))
        self.q_norm = put(fit(w["dq.norm"], self.q_rank_p), torch.float32)
        self.c_norm = put(fit(w["dkv.norm"], self.kv_rank_p), torch.float32)
        self.uq = put(fit(w["uq"].view(H, D, Q), H, self.dim_p, self.q_rank_p).flatten(0, 1))
        uk = fit(w["uk"].view(H, D, R), H, self.dim_p, self.kv_rank_p)
        uv = fit(w["uv"].view(H, V, R), H, self.vdim_p, self.kv_rank_p)
        self.uk_t = put(uk.transpose(1, 2))              # (H, R, D): q -> latent space
        self.uv = put(uv)                                # (H, V, R): latent space -> values
        self.expand = None
        if dtype == torch.bfloat16 and self.can_expand:
            self.expand = put(torch.cat([uk.flatten(0, 1), uv.flatten(0, 1)]))
        self.o = ResidualLinear(put(fit(w["o"].view(W, H, V), self.padded_width, H, self.vdim_p).flatten(1, 2)))

    def random(self, dtype, device, generator, std: float = 0.02):
        r = lambda *s: torch.empty(*s, dtype=dtype, device=device).normal_(0.0, std, generator=generator)
        one = lambda n: torch.ones(n, dtype=dtype, device=device)
        H = self.heads
        self.load({"dq": r(self.q_rank, self.width), "dq.norm": one(self.q_rank),
                   "uq": r(H * self.dim, self.q_rank), "dkv": r(self.kv_rank, self.width),
                   "dkv.norm": one(self.kv_rank), "uk": r(H * self.dim, self.kv_rank),
                   "uv": r(H * self.vdim, self.kv_rank), "o": r(self.width, H * self.vdim)}, dtype, device)

    # ------------------------------------------------------------------ forward
    def forward(self, h: torch.Tensor, cache: torch.Tensor, ctx) -> torch.Tensor:
        """h (N, padded width); cache (pages, BS, kv_rank_p) of this layer.  The first
        ctx.context_lens.numel() tokens are attended singly, the rest in the runs of
        ctx.runs[window].  Returns planes of partial sums (see ResidualLinear)."""
        N, H = h.shape[0], self.heads
        singles = ctx.context_lens.numel()
        runs = ctx.runs[self.window] if singles < N else None
        direct = runs is not None and runs.key_slots is None    # the runs' keys are this step's own tokens
        down = F.linear(h, self.down)
        norms = latent_norm_store(down, self.q_norm, self.c_norm, self.q_rank, self.kv_rank, self.eps, cache,
                                  ctx.slot_mapping, return_c=direct)
        cq, c = norms if direct else (norms, None)
        q = F.linear(cq, self.uq)
        mixed = torch.empty((N, H * self.vdim_p), dtype=h.dtype, device=h.device)
        if runs is not None:
            c = c[singles:] if direct else gather_rows(cache, runs.key_slots)
            latent_tiles_attention(q[singles:], F.linear(c, self.expand), H, self.dim_p, self.vdim_p,
                                   runs.tiles, self.scale, self.window, mixed[singles:])
        if singles:
            ql = headwise_linear(q[:singles].view(singles, H, self.dim_p), self.uk_t)
            ol = latent_rows_attention(ql, cache, ctx.block_tables, ctx.context_lens, self.scale, self.window,
                                       ctx.table_rows)
            headwise_linear(ol, self.uv, mixed[:singles])
        return self.o.forward(mixed)
