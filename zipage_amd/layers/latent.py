"""Latent attention: one cached vector per token, from which every head's key and value follow.

The wrappers are one HIP launch each; `LatentAttention` is the mixer a model puts together from
them, with its sizes and constants as parameters."""
from __future__ import annotations

import torch
import torch.nn.functional as F

from zipage_amd import _lib

from .linear import ResidualLinear, fit, pad_to_multiple
from .rotary import Rotary
from .runs import gather_rows, run_attention


def latent_norm_store(down: torch.Tensor, q_weight: torch.Tensor, c_weight: torch.Tensor | None, q_norm: int,
                      c_norm: int, eps: float, cache: torch.Tensor | None, slot_mapping: torch.Tensor | None,
                      return_c: bool = False, positions: torch.Tensor | None = None,
                      freqs: torch.Tensor | None = None):
    """down (N, q_width + c_width + p_width): RMS norms of the first two parts (means over q_norm and c_norm
    elements, plain fp32 weights), the third's first 2 * len(freqs) elements turned by their positions.
    Returns the first (N, q_width); the others go to the flat cache slots (-1 skips) and are returned too with
    `return_c`.  Without c_weight there is only the first."""
    N = down.shape[0]
    qw, cw = q_weight.numel(), 0 if c_weight is None else c_weight.numel()
    row = down.shape[1] - qw
    assert down.is_contiguous() and q_weight.dtype == torch.float32
    rot = 0 if freqs is None else 2 * freqs.numel()
    if cw:
        assert c_weight.dtype == torch.float32 and row >= cw
        assert cache.is_contiguous() and cache.dtype == down.dtype and cache.shape[-1] == row
        assert slot_mapping.dtype == torch.int32 and slot_mapping.is_contiguous() and slot_mapping.numel() == N
    else:
        assert row == 0 and not return_c and not rot
    if rot:
        assert freqs.dtype == torch.float32 and positions.dtype == torch.int32 and positions.is_contiguous()
        assert positions.numel() == N
    q = torch.empty((N, qw), dtype=down.dtype, device=down.device)
    c = torch.empty((N, row), dtype=down.dtype, device=down.device) if return_c else None
    _lib.call_models("zp_latent_norm_store", _lib.dev_ptr(down), _lib.dev_ptr(q_weight),
                     _lib.dev_ptr(c_weight), _lib.dev_ptr(q), _lib.dev_ptr(c), _lib.dev_ptr(cache),
                     _lib.dev_ptr(slot_mapping), _lib.dev_ptr(positions), _lib.dev_ptr(freqs), N, qw, cw, row - cw,
                     q_norm, c_norm, rot, cache.numel() // row if cw else 0, float(eps),
                     _lib.dtype_tag(down), _lib.stream_ptr(down))
    return (q, c) if return_c else q


def rotate_heads(x: torch.Tensor, positions: torch.Tensor, freqs: torch.Tensor, heads: int, at: int):
    """x (N, heads * head), rows may be part of wider ones: elements at .. at + 2 * len(freqs) of every head
    turn in place (i with i + len(freqs))."""
    N, wide = x.shape
    assert x.stride(1) == 1 and wide % heads == 0 and freqs.dtype == torch.float32
    assert positions.dtype == torch.int32 and positions.is_contiguous() and positions.numel() == N
    _lib.call_models("zp_rotate_heads", _lib.dev_ptr(x), _lib.dev_ptr(positions), _lib.dev_ptr(freqs), N, heads,
                     wide // heads, at, 2 * freqs.numel(), x.stride(0), _lib.dtype_tag(x), _lib.stream_ptr(x))


def headwise_linear(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor | None = None,
                    positions: torch.Tensor | None = None, freqs: torch.Tensor | None = None) -> torch.Tensor:
    """x (N, H, K + tail), w (H, M, K) -> (N, H, M + tail): every head its own matrix; the tail passes, its first
    2 * len(freqs) elements turned by their token's position."""
    N, H, wide = x.shape
    K, M = w.shape[2], w.shape[1]
    tail, rot = wide - K, 0 if freqs is None else 2 * freqs.numel()
    assert x.is_contiguous() and w.is_contiguous() and w.dtype == x.dtype and w.shape[0] == H and tail >= rot
    if rot:
        assert freqs.dtype == torch.float32 and positions.dtype == torch.int32 and positions.is_contiguous()
        assert positions.numel() == N
    if out is None:
        out = torch.empty((N, H, M + tail), dtype=x.dtype, device=x.device)
    assert out.is_contiguous() and out.numel() == N * H * (M + tail) and out.dtype == x.dtype
    _lib.call_models("zp_headwise_linear", _lib.dev_ptr(x), _lib.dev_ptr(w), _lib.dev_ptr(out),
                     _lib.dev_ptr(positions), _lib.dev_ptr(freqs), N, H, K, M, tail, rot, _lib.dtype_tag(x),
                     _lib.stream_ptr(x))
    return out


def latent_rows_attention(q: torch.Tensor, cache: torch.Tensor, block_tables: torch.Tensor,
                          context_lens: torch.Tensor, scale: float, window: int | None = None,
                          table_rows: torch.Tensor | None = None, rank: int | None = None) -> torch.Tensor:
    """Single tokens over paged latents.  q (N, H, row); cache (pages, BS, row); token i sees the last
    `window` of the context_lens[i] tokens in row table_rows[i] (default i) of block_tables.  Scores are
    products of whole rows, values their first `rank` elements (default: all).  Returns (N, H, rank)."""
    N, H, row = q.shape
    R = row if rank is None else rank
    assert q.is_contiguous() and cache.is_contiguous() and cache.dtype == q.dtype and cache.shape[2] == row >= R
    for t in (block_tables, context_lens) + (() if table_rows is None else (table_rows,)):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert context_lens.numel() == N and (table_rows is None or table_rows.numel() == N)
    B, NB = block_tables.shape
    pages, BS, _ = cache.shape
    w, tag = window or 0, _lib.dtype_tag(q)
    size = _lib.load_models("latent").zp_latent_rows_workspace(N, H, R, w, NB, BS, tag)
    ws = torch.empty(max(size, 0), dtype=torch.uint8, device=q.device) if size > 0 else None
    out = torch.empty((N, H, R), dtype=q.dtype, device=q.device)
    _lib.call_models("zp_latent_rows_attention", _lib.dev_ptr(q), _lib.dev_ptr(cache),
                     _lib.dev_ptr(block_tables), _lib.dev_ptr(context_lens), _lib.dev_ptr(table_rows),
                     _lib.dev_ptr(out), N, H, R, row - R, BS, B, NB, pages, w, float(scale), tag, _lib.dev_ptr(ws),
                     max(size, 0), _lib.stream_ptr(q))
    return out


def latent_tiles_attention(q: torch.Tensor, kv: torch.Tensor, heads: int, dim: int, vdim: int,
                           tiles: torch.Tensor, scale: float, window: int | None, out: torch.Tensor,
                           shared: torch.Tensor | None = None):
    """Runs of prompt tokens over expanded keys and values.  q (N, heads * (dim + shared dims)); kv (Nk, heads
    * dim + heads * vdim); shared (Nk, dims): the key part of all heads; tiles (T, 4) int32 as
    `inputs.plan_runs` makes them; out (N, heads * vdim)."""
    return run_attention(q, kv, heads, heads, dim, vdim, tiles, scale, out, window=window, shared=shared)


class LatentAttention:
    """The mixer.  Queries pass a low-rank bottleneck, keys and values of all heads are images of one
    normed latent c.  With `rotary`, heads have a second, rotated query part, which meets one rotated key
    part per token that all heads share; its size is rotary.dims.  Only c and that key part are cached, and a
    mixer with `own_latent` False reads the cache of another one with the same latent and rotated sizes.

    Two forms of the same sum run side by side in one step: single tokens work on the latents
    themselves (W_uk^T q against c, W_uv after the sum), so a decode reads kv_rank elements per
    cached token for all heads together; runs of prompt tokens expand c to keys and values once per
    run and use the smaller per-head dimensions.  float32 always takes the first form.

    Sizes are padded once, at load: ranks and dim to 32, vdim to 16, the rotated part to 8, zero weights in
    between; the means of the norms run over the true sizes."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, q_rank: int, kv_rank: int,
                 scale: float, window: int | None, eps: float, rotary: Rotary | None = None,
                 own_latent: bool = True, padded_width: int | None = None):
        if rotary is not None and rotary.dims % 2:
            raise ValueError(f"{rotary.dims} rotated dimensions")
        self.width, self.heads, self.dim, self.vdim = width, heads, dim, vdim
        self.q_rank, self.kv_rank, self.scale, self.window, self.eps = q_rank, kv_rank, scale, window, eps
        self.rotary, self.rot = rotary, 0 if rotary is None else rotary.dims
        self.own_latent = own_latent
        self.padded_width = padded_width or pad_to_multiple(width, 8)
        self.dim_p, self.vdim_p = pad_to_multiple(dim, 32), pad_to_multiple(vdim, 16)
        self.q_rank_p, self.kv_rank_p = pad_to_multiple(q_rank, 32), pad_to_multiple(kv_rank, 32)
        self.rot_p = pad_to_multiple(self.rot, 8)
        self.head = self.dim_p + self.rot_p          # of a query row
        self.row = self.kv_rank_p + self.rot_p       # of a cached token
        self.freqs = None

    @property
    def can_expand(self) -> bool:
        """Sizes the run form's kernel covers; others run token by token."""
        return self.head <= 256 and self.vdim_p <= 256

    def shapes(self) -> dict:
        H, D, V, R, Q, W, P = self.heads, self.dim, self.vdim, self.kv_rank, self.q_rank, self.width, self.rot
        return {"dq": (Q, W), "dq.norm": (Q,), "uq": (H * (D + P), Q),
                **({"dkv": (R + P, W), "dkv.norm": (R,)} if self.own_latent else {}),
                "uk": (H * D, R), "uv": (H * V, R), "o": (W, H * V)}

    def load(self, w: dict, dtype, device):
        """w: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, o as stored ([out, in], heads in order)."""
        H, D, V, R, Q, W, P = self.heads, self.dim, self.vdim, self.kv_rank, self.q_rank, self.width, self.rot
        put = lambda t, dt=dtype: t.to(device=device, dtype=dt).contiguous()

        down = [fit(w["dq"], self.q_rank_p, self.padded_width)]
        if self.own_latent:
            down += [fit(w["dkv"][:R], self.kv_rank_p, self.padded_width)]
            if P:
                down += [fit(w["dkv"][R:], self.rot_p, self.padded_width)]
        self.down = put(torch.cat(down))
        self.q_norm = put(fit(w["dq.norm"], self.q_rank_p), torch.float32)
        self.c_norm = put(fit(w["dkv.norm"], self.kv_rank_p), torch.float32) if self.own_latent else None
        if self.rotary is not None:
            self.freqs = self.rotary.frequencies(device)
        uq = w["uq"].view(H, D + P, Q)
        uq = [fit(uq[:, :D], H, self.dim_p, self.q_rank_p)] + ([fit(uq[:, D:], H, self.rot_p, self.q_rank_p)] if P else [])
        self.uq = put(torch.cat(uq, dim=1).flatten(0, 1))
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
        self.load({k: torch.ones(s, dtype=dtype, device=device) if k.endswith("norm") else r(*s)
                   for k, s in self.shapes().items()}, dtype, device)

    def allocate(self, num_pages: int, page_size: int, dtype, device) -> torch.Tensor | None:
        """One page pool: a page holds page_size rows of latent and rotated key part."""
        if not self.own_latent:
            return None
        return torch.zeros(num_pages, page_size, self.row, dtype=dtype, device=device)

    # ------------------------------------------------------------------ forward
    def forward(self, h: torch.Tensor, cache: torch.Tensor, ctx, positions: torch.Tensor | None = None,
                held: dict | None = None) -> torch.Tensor:
        """h (N, padded width); cache (pages, BS, row): this layer's, or the one it reads.  The first
        ctx.context_lens.numel() tokens are attended singly, the rest in the runs of ctx.runs[window].
        positions (N,) int32 where something is rotated.  `held` carries the runs' rows of this cache from the
        mixer that wrote them to those that only read.  Returns planes of partial sums (see ResidualLinear)."""
        N, H = h.shape[0], self.heads
        held = {} if held is None else held
        singles = ctx.context_lens.numel()
        runs = ctx.runs[self.window] if singles < N else None
        direct = runs is not None and runs.key_slots is None    # the runs' keys are this step's own tokens
        down = F.linear(h, self.down)
        if self.own_latent:
            norms = latent_norm_store(down, self.q_norm, self.c_norm, self.q_rank, self.kv_rank, self.eps, cache,
                                      ctx.slot_mapping, direct, positions, self.freqs)
            cq = norms[0] if direct else norms
            if runs is not None:
                held["rows"] = norms[1][singles:] if direct else gather_rows(cache, runs.key_slots)
        else:
            cq = latent_norm_store(down, self.q_norm, None, self.q_rank, 0, self.eps, None, None)
        q = F.linear(cq, self.uq)
        mixed = torch.empty((N, H * self.vdim_p), dtype=h.dtype, device=h.device)
        if runs is not None:
            rows, qr, shared = held["rows"], q[singles:], None
            if self.rot:
                rotate_heads(qr, positions[singles:], self.freqs, H, self.dim_p)
                rows, shared = rows[:, :self.kv_rank_p], rows[:, self.kv_rank_p:]
            latent_tiles_attention(qr, F.linear(rows, self.expand), H, self.dim_p, self.vdim_p, runs.tiles, self.scale,
                                   self.window, mixed[singles:], shared)
        if singles:
            ql = headwise_linear(q[:singles].view(singles, H, self.head), self.uk_t,
                                 positions=None if positions is None else positions[:singles], freqs=self.freqs)
            ol = latent_rows_attention(ql, cache, ctx.block_tables, ctx.context_lens, self.scale, self.window,
                                       ctx.table_rows, self.kv_rank_p)
            headwise_linear(ol, self.uv, mixed[:singles])
        return self.o.forward(mixed)
