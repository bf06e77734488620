"""Row steps of decoders with an fp32 residual stream (one HIP launch each).

`x` is the stream (N, width) fp32; what feeds a matrix product has the model's dtype.  Widths are
padded to a multiple of 8 with zeros, `norm_width` is the length the mean runs over.  With `norm_bias` the
norm is tanh(norm_alpha x) * (weight_offset + norm_weight) + norm_bias, without a mean."""
import torch

from zipage_amd import _lib


def _rows(t: torch.Tensor | None, width: int):
    if t is not None:
        assert t.is_contiguous() and t.shape[-1] == width
    return _lib.dev_ptr(t)


def embed_norm(tokens: torch.Tensor, positions: torch.Tensor, embed: torch.Tensor,
               pos: torch.Tensor | None, x: torch.Tensor, norm_weight: torch.Tensor, eps: float,
               norm_width: int, weight_offset: float = 0.0, embed_scale: float = 1.0,
               norm_bias: torch.Tensor | None = None, norm_alpha: float = 0.0,
               shift: torch.Tensor | None = None, result: torch.Tensor | None = None) -> torch.Tensor:
    """x = embed[tokens] * embed_scale (+ pos[positions]), kept in `result`, (+ the row `shift`) into `x`; returns
    its RMS norm times (weight_offset + norm_weight) in the table's dtype.  tokens (N,) int64, positions (N,) int32."""
    N, W = x.shape
    assert tokens.dtype == torch.int64 and positions.dtype == torch.int32
    assert tokens.is_contiguous() and positions.is_contiguous() and tokens.numel() == positions.numel() == N
    assert x.dtype == torch.float32 and norm_weight.dtype == torch.float32
    assert all(t is None or t.dtype == torch.float32 for t in (norm_bias, shift, result))
    assert result is None or result.shape == x.shape
    assert pos is None or pos.dtype == embed.dtype
    out = torch.empty((N, W), dtype=embed.dtype, device=x.device)
    _lib.call_models("zp_embed_norm", _lib.dev_ptr(tokens), _lib.dev_ptr(positions), _rows(embed, W), _rows(pos, W),
                     _rows(shift, W), _rows(result, W), _rows(x, W), _rows(norm_weight, W), _rows(norm_bias, W),
                     _lib.dev_ptr(out), N, W, norm_width, embed.shape[0], 0 if pos is None else pos.shape[0],
                     float(embed_scale), float(eps), float(weight_offset), float(norm_alpha), _lib.dtype_tag(embed),
                     _lib.stream_ptr(x))
    return out


def residual_norm(x: torch.Tensor, y: torch.Tensor, norm_weight: torch.Tensor | None, eps: float,
                  norm_width: int, weight_offset: float = 0.0, out_scale: float = 1.0,
                  x_out: torch.Tensor | None = None, result: torch.Tensor | None = None,
                  history: torch.Tensor | None = None, mix: torch.Tensor | None = None,
                  y_weight: torch.Tensor | None = None, norm_bias: torch.Tensor | None = None,
                  norm_alpha: float = 0.0, more: tuple = (), shift: torch.Tensor | None = None):
    """r = x + y (y also as planes (P, N, width), all of them added; with `y_weight` their sum is
    RMS-normed, times that weight, before it joins x) + the branches of `more`, pairs like (y, y_weight); kept in
    `result`; with `mix`, r <- mix[-1] r + sum_j mix[j] history[j]; plus the row `shift`; kept in `x_out`; returns
    rmsnorm(r) * (weight_offset + norm_weight) * out_scale in y's dtype (None without a norm).  history (planes, N,
    width) fp32, of which the first len(mix) - 1 are read."""
    N, W = x.shape
    branches = [(t if t.dim() == 3 else t.unsqueeze(0), w) for t, w in ((y, y_weight), *more)]
    assert x.dtype == torch.float32 and all(t.shape[1:] == x.shape and t.dtype == y.dtype for t, _ in branches)
    assert all(t is None or t.dtype == torch.float32 for t in (norm_bias, shift, *(w for _, w in branches)))
    n_hist, plane = 0, 0
    if mix is not None:
        assert mix.dtype == torch.float32 and mix.is_contiguous()
        n_hist = mix.numel() - 1
        if n_hist:
            assert history.dtype == torch.float32 and history.shape[0] >= n_hist and history[0].shape == x.shape
            plane = history.stride(0)
            assert history.stride(1) == W and history.stride(2) == 1
    out = torch.empty((N, W), dtype=y.dtype, device=x.device) if norm_weight is not None else None
    table = (_lib.Branch * len(branches))(*(_lib.Branch(_rows(t, W), _rows(w, W), t.shape[0]) for t, w in branches))
    _lib.call_models("zp_residual_norm", _rows(x, W), table, len(branches), _lib.dev_ptr(history if n_hist else None),
                     plane, _lib.dev_ptr(mix), n_hist, _rows(shift, W), _rows(result, W), _rows(x_out, W),
                     _rows(norm_weight, W), _rows(norm_bias, W), _lib.dev_ptr(out), N, W, norm_width, float(eps),
                     float(weight_offset), float(norm_alpha), float(out_scale), _lib.dtype_tag(y), _lib.stream_ptr(x))
    return out


def normed_powers(z: torch.Tensor, act: tuple[float, float, float, float], eps: float, norm_width: int,
                  out: torch.Tensor) -> torch.Tensor:
    """a N(z) + b N(z^2) + c N(z^3) + e into `out`, N dividing a row by its root mean square (of norm_width
    elements).  z and out (N, width), rows may be part of wider ones."""
    N, W = z.shape
    assert out.shape == z.shape and out.dtype == z.dtype and z.stride(1) == out.stride(1) == 1
    _lib.call_models("zp_normed_powers", _lib.dev_ptr(z), _lib.dev_ptr(out), N, W, norm_width, z.stride(0), out.stride(0),
                     *(float(v) for v in act), float(eps), _lib.dtype_tag(z), _lib.stream_ptr(z))
    return out


def xielu(z: torch.Tensor, alpha_p: float, alpha_n: float) -> torch.Tensor:
    """z > 0: alpha_p z^2 + z / 2; z <= 0: alpha_n (exp(z) - 1 - z) + z / 2."""
    assert z.is_contiguous()
    out = torch.empty_like(z)
    _lib.call_models("zp_xielu", _lib.dev_ptr(z), _lib.dev_ptr(out), z.numel(), float(alpha_p),
                     float(alpha_n), _lib.dtype_tag(z), _lib.stream_ptr(z))
    return out


def relu_square(z: torch.Tensor) -> torch.Tensor:
    """max(z, 0)^2."""
    assert z.is_contiguous()
    out = torch.empty_like(z)
    _lib.call_models("zp_relu_square", _lib.dev_ptr(z), _lib.dev_ptr(out), z.numel(), _lib.dtype_tag(z),
                     _lib.stream_ptr(z))
    return out


def softcap(z: torch.Tensor, cap: float) -> torch.Tensor:
    """cap * tanh(z / cap) in fp32."""
    assert z.is_contiguous()
    out = torch.empty(z.shape, dtype=torch.float32, device=z.device)
    _lib.call_models("zp_softcap", _lib.dev_ptr(z), _lib.dev_ptr(out), z.numel(), float(cap), _lib.dtype_tag(z),
                     _lib.stream_ptr(z))
    return out
