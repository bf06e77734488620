"""Recurrent mixers: a matrix memory with exponential gates, a gated delta rule with a decay per key channel, and
linear attention with decay.  All keep a float32 matrix per head and sequence slot; a step hands them its portions as
segments (`StepContext.segments`, and `.run_segments` where 16 tokens at a time pay)."""
from __future__ import annotations

import ctypes

import torch
import torch.nn.functional as F

from zipage_amd import _lib

from .linear import fit, pad_to_multiple
from .moe import small_linear
from .rotary import Rotary


def _key_size(n: int) -> int:
    """Key sizes the scan kernels have."""
    for size in (32, 64, 128, 256):
        if n <= size:
            return size
    raise ValueError(f"a recurrent head of {n} key dimensions (at most 256)")


def _value_size(n: int) -> int:
    if n > 256:
        raise ValueError(f"a recurrent head of {n} value dimensions (at most 256)")
    return pad_to_multiple(n, 32)


def _segments(seg, num_slots: int, num_rows: int) -> _lib.Segments:
    for t in (seg.counts, seg.slots, seg.starts) + (() if seg.rows is None else (seg.rows,)):
        assert t.dtype == torch.int32 and t.is_contiguous() and t.numel() == seg.counts.numel()
    return _lib.Segments(_lib.dev_ptr(seg.rows), _lib.dev_ptr(seg.counts), _lib.dev_ptr(seg.slots),
                         _lib.dev_ptr(seg.starts), seg.counts.numel(), seg.max_count, num_slots, num_rows)


class MatrixMemory:
    """Per head S <- e^{f + m - m'} S + e^{i - m'} k v^T with the running maximum m' = max(f + m, i), a
    normaliser n of the same recurrence, and the read-out S^T q / (max(|n . q|, e^{-m'}) + 1e-6); log gates
    capped at `gate_cap`; then a norm per head and a sigmoid gate."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, gate_cap: float, eps: float,
                 out_scale: float = 1.0):
        self.width, self.heads, self.dim, self.vdim = width, heads, dim, vdim
        self.gate_cap, self.eps, self.out_scale = gate_cap, eps, out_scale
        self.dim_p, self.vdim_p = _key_size(dim), _value_size(vdim)
        self.columns = 2 * heads * (self.dim_p + self.vdim_p)
        self.out_columns = heads * self.vdim_p

    def shapes(self) -> dict:
        H, D, V, W = self.heads, self.dim, self.vdim, self.width
        return {"q": (H * D, W), "k": (H * D, W), "v": (H * V, W), "g": (H * V, W), "o": (W, H * V), "norm": (H * V,),
                "i": (H, W), "i.b": (H,), "f": (H, W), "f.b": (H,)}

    def load(self, w: dict, dtype, device, padded_width: int):
        """Returns the rows of the common input product and the columns of the output product."""
        H, D, V, W = self.heads, self.dim, self.vdim, self.width
        rows = lambda t, d, dp: fit(t.view(H, d, W), H, dp, padded_width).flatten(0, 1)
        f32 = lambda t: t.to(device=device, dtype=torch.float32).contiguous()
        self.norm = f32(fit(w["norm"].view(H, V), H, self.vdim_p).flatten())
        self.i_bias, self.f_bias = f32(w["i.b"]), f32(w["f.b"])
        gates = torch.cat([w["i"], w["f"]])
        self.gates = fit(gates, pad_to_multiple(2 * H, 4), padded_width).to(device=device, dtype=dtype).contiguous()
        into = torch.cat([rows(w["q"], D, self.dim_p), rows(w["k"], D, self.dim_p), rows(w["v"], V, self.vdim_p),
                          rows(w["g"], V, self.vdim_p)])
        out = fit(w["o"].view(W, H, V), padded_width, H, self.vdim_p).flatten(1, 2)
        return into, out

    def allocate(self, num_slots: int, dtype, device) -> torch.Tensor:
        """Per slot and head: S (dim, vdim), n (dim), m and padding."""
        return torch.zeros(num_slots, self.heads, self.dim_p * self.vdim_p + self.dim_p + 4, dtype=torch.float32,
                           device=device)

    @property
    def can_run(self) -> bool:
        """Sizes the blocked kernel covers; others run token by token."""
        return self.dim_p <= 128 and self.vdim_p <= 128

    def scan(self, h: torch.Tensor, proj: torch.Tensor, state: torch.Tensor, ctx, out: torch.Tensor):
        """h: the mixer's input (for the gates, which stay in fp32), proj: this mixer's columns of the
        projections, out: of the output rows."""
        H, D, V = self.heads, self.dim_p, self.vdim_p
        gates = small_linear(h, self.gates)
        assert proj.stride(1) == out.stride(1) == 1 and proj.dtype == out.dtype and state.is_contiguous()
        tag, stream = _lib.dtype_tag(proj), _lib.stream_ptr(proj)
        for segments, runs in ((ctx.segments, False), (ctx.run_segments, self.can_run and proj.dtype == torch.bfloat16)):
            if segments is None:
                continue
            args = _lib.MlstmArgs(
                _segments(segments, state.shape[0], h.shape[0]), _lib.dev_ptr(proj), _lib.dev_ptr(gates),
                _lib.dev_ptr(self.i_bias), _lib.dev_ptr(self.f_bias), _lib.dev_ptr(self.norm), _lib.dev_ptr(state),
                _lib.dev_ptr(out), proj.stride(0), gates.stride(0), out.stride(0), H, D, V, self.vdim, 0, H * D,
                2 * H * D, 2 * H * D + H * V, self.gate_cap, self.dim ** -0.5, self.eps, self.out_scale)
            if not runs:
                _lib.call_models("zp_mlstm_scan", ctypes.byref(args), tag, stream)
                continue
            size = _lib.load_models("recurrent").zp_mlstm_runs_workspace(h.shape[0] - segments.first_row,
                                                                      segments.counts.numel(), H)
            ws = torch.empty(size, dtype=torch.uint8, device=proj.device)
            _lib.call_models("zp_mlstm_runs", ctypes.byref(args), segments.first_row, segments.longest, _lib.dev_ptr(ws),
                             size, tag, stream)


class ChannelDelta:
    """Gated delta rule: per head S <- g * S (a decay per key channel), u = beta (v - S^T k), S <- S + k u^T,
    o = S^T q.  q, k, v pass a short causal convolution and silu, q and k are unit vectors; decays and
    output gates come through low-rank products whose ranks the tensors give."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, eps: float,
                 out_scale: float = 1.0):
        if heads % kv_heads:
            raise ValueError(f"{heads} value heads over {kv_heads} key heads")
        self.width, self.heads, self.kv_heads, self.dim, self.vdim = width, heads, kv_heads, dim, vdim
        self.taps, self.eps, self.out_scale = taps, eps, out_scale
        self.dim_p, self.vdim_p = _key_size(dim), _value_size(vdim)
        self.channels = 2 * kv_heads * self.dim_p + heads * self.vdim_p
        self.out_columns = heads * self.vdim_p

    def shapes(self, a_rank: int, g_rank: int) -> dict:
        H, G, D, V, W = self.heads, self.kv_heads, self.dim, self.vdim, self.width
        return {"q": (G * D, W), "k": (G * D, W), "v": (H * V, W), "q.conv": (G * D, self.taps),
                "k.conv": (G * D, self.taps), "v.conv": (H * V, self.taps), "b": (H, W), "A_log": (H,), "norm": (V,),
                "a1": (a_rank, W), "a2": (H * D, a_rank), "dt_bias": (H * D,), "g1": (g_rank, W),
                "g2": (H * V, g_rank), "o": (W, H * V)}

    def load(self, w: dict, dtype, device, padded_width: int):
        """Returns the rows of the input product and the columns of the output product."""
        H, G, D, V, W = self.heads, self.kv_heads, self.dim, self.vdim, self.width
        Dp, Vp = self.dim_p, self.vdim_p
        f32 = lambda t: t.to(device=device, dtype=torch.float32).contiguous()
        rows = lambda t, n, d, dp: fit(t.view(n, d, W), n, dp, padded_width).flatten(0, 1)
        taps = lambda t, n, d, dp: fit(t.view(n, d, self.taps), n, dp, self.taps).flatten(0, 1)
        self.filters = f32(torch.cat([taps(w["q.conv"], G, D, Dp), taps(w["k.conv"], G, D, Dp),
                                      taps(w["v.conv"], H, V, Vp)]).t())
        self.a_log, self.norm = f32(w["A_log"]), f32(fit(w["norm"], Vp).repeat(H))
        self.dt_bias = f32(fit(w["dt_bias"].view(H, D), H, Dp).flatten())
        ra, rg = w["a1"].shape[0], w["g1"].shape[0]
        ra_p, rg_p = pad_to_multiple(ra, 8), pad_to_multiple(rg, 8)
        self.b_at = self.channels
        self.low_at = self.b_at + pad_to_multiple(H, 8)
        self.low_rank = ra_p + rg_p
        self.columns = self.low_at + self.low_rank
        low = torch.zeros(H * (Dp + Vp), self.low_rank, dtype=w["a2"].dtype)
        low[:H * Dp, :ra] = fit(w["a2"].view(H, D, ra), H, Dp, ra).flatten(0, 1)
        low[H * Dp:, ra_p:ra_p + rg] = fit(w["g2"].view(H, V, rg), H, Vp, rg).flatten(0, 1)
        self.low = low.to(device=device, dtype=dtype).contiguous()
        into = torch.cat([rows(w["q"], G, D, Dp), rows(w["k"], G, D, Dp), rows(w["v"], H, V, Vp),
                          fit(w["b"], pad_to_multiple(H, 8), padded_width), fit(w["a1"], ra_p, padded_width),
                          fit(w["g1"], rg_p, padded_width)])
        out = fit(w["o"].view(W, H, V), padded_width, H, Vp).flatten(1, 2)
        return into, out

    def allocate(self, num_slots: int, dtype, device):
        """Per slot and head: S (dim, vdim), and the last inputs of the head's convolutions."""
        return (torch.zeros(num_slots, self.heads, self.dim_p, self.vdim_p, dtype=torch.float32, device=device),
                torch.zeros(num_slots, self.heads, self.taps - 1, 2 * self.dim_p + self.vdim_p, dtype=dtype,
                            device=device))

    @property
    def can_run(self) -> bool:
        """Sizes the blocked kernels cover; others run token by token."""
        return self.dim_p <= 128 and self.vdim_p <= 128

    def scan(self, proj: torch.Tensor, state, ctx, out: torch.Tensor):
        """proj: this mixer's columns of the projections, out: of the output rows."""
        S, tail = state
        H, D = self.heads, self.dim_p
        assert proj.stride(1) == out.stride(1) == 1 and proj.dtype == out.dtype == tail.dtype and S.is_contiguous()
        low = F.linear(proj[:, self.low_at:self.low_at + self.low_rank], self.low)
        tag, stream = _lib.dtype_tag(proj), _lib.stream_ptr(proj)
        for segments, runs in ((ctx.segments, False), (ctx.run_segments, self.can_run and proj.dtype == torch.bfloat16)):
            if segments is None:
                continue
            args = _lib.DeltaArgs(
                _segments(segments, S.shape[0], proj.shape[0]), _lib.dev_ptr(proj), _lib.dev_ptr(low),
                _lib.dev_ptr(self.filters), _lib.dev_ptr(self.a_log), _lib.dev_ptr(self.dt_bias), _lib.dev_ptr(self.norm),
                _lib.dev_ptr(S), _lib.dev_ptr(tail), _lib.dev_ptr(out), proj.stride(0), low.stride(0), out.stride(0), H,
                self.kv_heads, D, self.vdim_p, self.vdim, self.taps, self.b_at, H * D, self.dim ** -0.5, self.eps,
                self.out_scale)
            if not runs:
                _lib.call_models("zp_delta_scan", ctypes.byref(args), tag, stream)
                continue
            size = _lib.load_models("recurrent").zp_delta_runs_workspace(proj.shape[0] - segments.first_row,
                                                                      segments.counts.numel(), H, D, self.vdim_p)
            ws = torch.empty(size, dtype=torch.uint8, device=proj.device)
            _lib.call_models("zp_delta_runs", ctypes.byref(args), segments.first_row, segments.longest,
                             _lib.dev_ptr(ws), size, tag, stream)


class LinearAttention:
    """Per head S <- g * S (rows) + k v^T, o = S^T q, a norm per head and a silu gate.  Decays: with `tau` one per key
    channel, sigmoid(a low-rank product + bias)^(1 / tau), whose rank the tensors give; else the numbers `decay`, one
    per head.  `rotary`: q and k turn with their position.  `weighted`: the norm has weights, shared by the heads."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, eps: float, q_scale: float = 1.0, k_scale: float = 1.0,
                 tau: float | None = None, decay: tuple[float, ...] | None = None, rotary: Rotary | None = None,
                 weighted: bool = False):
        if (tau is None) == (decay is None) or decay is not None and len(decay) != heads:
            raise ValueError(f"decays come from tau or are one per head: {tau}, {decay} for {heads} heads")
        if rotary is not None and (rotary.dims % 2 or rotary.dims > dim):
            raise ValueError(f"{rotary.dims} rotated dimensions of {dim}")
        self.width, self.heads, self.dim, self.vdim, self.eps = width, heads, dim, vdim, eps
        self.q_scale, self.k_scale, self.tau, self.decay, self.rotary, self.weighted = q_scale, k_scale, tau, decay, rotary, weighted
        self.dim_p, self.vdim_p = _key_size(dim), _value_size(vdim)
        self.low_at = 2 * heads * (self.dim_p + self.vdim_p)
        self.out_columns = heads * self.vdim_p

    def shapes(self, a_rank: int = 1) -> dict:
        H, D, V, W = self.heads, self.dim, self.vdim, self.width
        return {"q": (H * D, W), "k": (H * D, W), "v": (H * V, W), "g": (H * V, W), "o": (W, H * V),
                **({"norm": (V,)} if self.weighted else {}),
                **({"a1": (a_rank, W), "a2": (H * D, a_rank), "a2.b": (H * D,)} if self.tau is not None else {})}

    def load(self, w: dict, dtype, device, padded_width: int):
        """Returns the rows of the common input product and the columns of the output product."""
        H, D, V, W = self.heads, self.dim, self.vdim, self.width
        order = list(range(D)) if self.rotary is None else self.rotary.order(D)
        f32 = lambda t: t.to(device=device, dtype=torch.float32).contiguous()
        keys = lambda t: fit(t.view(H, D, W)[:, order], H, self.dim_p, padded_width).flatten(0, 1)
        values = lambda t: fit(t.view(H, V, W), H, self.vdim_p, padded_width).flatten(0, 1)
        norm = w["norm"] if self.weighted else torch.ones(V)
        self.norm = f32(fit(norm.to(device), self.vdim_p).repeat(H))
        self.freqs = None if self.rotary is None or not self.rotary.dims else self.rotary.frequencies(device)
        into = [keys(w["q"]), keys(w["k"]), values(w["v"]), values(w["g"])]
        self.low, self.low_rank = None, 0
        if self.tau is not None:
            rank = w["a1"].shape[0]
            self.low_rank = pad_to_multiple(rank, 8)
            into.append(fit(w["a1"], self.low_rank, padded_width))
            low = w["a2"].view(H, D, rank)[:, order]
            self.low = fit(low, H, self.dim_p, self.low_rank).flatten(0, 1).to(device=device, dtype=dtype).contiguous()
            self.decays = f32(fit(w["a2.b"].view(H, D)[:, order], H, self.dim_p).flatten())
        else:
            self.decays = torch.tensor(self.decay, dtype=torch.float32, device=device)
        out = fit(w["o"].view(W, H, V), padded_width, H, self.vdim_p).flatten(1, 2)
        self.columns = self.low_at + self.low_rank
        return torch.cat(into), out

    def allocate(self, num_slots: int, dtype, device) -> torch.Tensor:
        """Per slot and head: S (dim, vdim)."""
        return torch.zeros(num_slots, self.heads, self.dim_p, self.vdim_p, dtype=torch.float32, device=device)

    @property
    def can_run(self) -> bool:
        """Sizes the blocked kernels cover; others run token by token."""
        return self.dim_p <= 128 and self.vdim_p <= 128

    def scan(self, proj: torch.Tensor, state: torch.Tensor, ctx, out: torch.Tensor):
        """proj: this mixer's columns of the projections, out: of the output rows."""
        H, D, V = self.heads, self.dim_p, self.vdim_p
        assert proj.stride(1) == out.stride(1) == 1 and proj.dtype == out.dtype and state.is_contiguous()
        low = None if self.low is None else F.linear(proj[:, self.low_at:self.low_at + self.low_rank], self.low)
        tag, stream = _lib.dtype_tag(proj), _lib.stream_ptr(proj)
        for segments, runs in ((ctx.segments, False), (ctx.run_segments, self.can_run and proj.dtype == torch.bfloat16)):
            if segments is None:
                continue
            args = _lib.LinearArgs(
                _segments(segments, state.shape[0], proj.shape[0]), _lib.dev_ptr(proj), _lib.dev_ptr(low),
                _lib.dev_ptr(self.decays), _lib.dev_ptr(self.freqs), _lib.dev_ptr(self.norm), _lib.dev_ptr(state),
                _lib.dev_ptr(out), proj.stride(0), 0 if low is None else low.stride(0), out.stride(0), H, D, V, self.vdim,
                0 if self.freqs is None else 2 * self.freqs.numel(), 0, H * D, 2 * H * D, 2 * H * D + H * V, self.q_scale,
                self.k_scale, 0.0 if self.tau is None else 1.0 / self.tau, self.eps)
            if not runs:
                _lib.call_models("zp_linear_scan", ctypes.byref(args), tag, stream)
                continue
            size = _lib.load_models("linear").zp_linear_runs_workspace(proj.shape[0] - segments.first_row,
                                                                    segments.counts.numel(), H, D)
            ws = torch.empty(size, dtype=torch.uint8, device=proj.device)
            _lib.call_models("zp_linear_runs", ctypes.byref(args), segments.first_row, segments.longest, _lib.dev_ptr(ws),
                             size, tag, stream)
