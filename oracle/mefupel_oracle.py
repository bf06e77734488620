"""Plain, slow restatement of the Mefupel decoder, one function per mechanism, on whole sequences.

One sequence at a time, recurrences as loops over its tokens, attention as dense matrices under an explicit
mask; in the floating type of the inputs (the tests pass float64).  It shares no code with the product path:
no padding, no cache, no reordered dimensions, no blocked forms.
"""
from __future__ import annotations

import math

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm(x, w, eps):
    """The model's norm: its weights are kept around zero."""
    return rms(x, eps) * (1 + w)


def silu(x):
    return x * torch.sigmoid(x)


def turn(x, positions, base, dims, layout, back=False):
    """x (n, heads, dim): pair number i of the first `dims` dimensions turns by position * base^(-2i/dims), or
    back by as much.  "halves": i and i + dims / 2 are a pair; "interleaved": 2i and 2i + 1."""
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    a = (positions.double()[:, None] * f).to(x.dtype)[:, None, :] * (-1 if back else 1)
    one = torch.arange(half) if layout == "halves" else 2 * torch.arange(half)
    two = one + half if layout == "halves" else one + 1
    u, v = x[..., one], x[..., two]
    out = x.clone()
    out[..., one] = u * a.cos() - v * a.sin()
    out[..., two] = v * a.cos() + u * a.sin()
    return out


def window_mask(n: int, size: int) -> torch.Tensor:
    """visible[i, j]: j is i or one of the size - 1 positions before it."""
    d = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (d >= 0) & (d < size)


def weights_of(score, seen, sink=None):
    """Softmax over the visible keys; a sink is one more logit that takes its share and weighs nothing."""
    score = score.masked_fill(~seen, -math.inf)
    if sink is None:
        return torch.softmax(score, dim=-1)
    column = sink.expand(score.shape[0], 1)
    return torch.softmax(torch.cat([score, column], dim=-1), dim=-1)[:, :-1]


def attend(q, k, v, seen, scale, sink=None):
    """q (n, H, D), k (n, G, D), v (n, G, V) -> (n, H, V)."""
    H, G = q.shape[1], k.shape[1]
    out = torch.empty(q.shape[0], H, v.shape[-1], dtype=q.dtype)
    for a in range(H):
        b = a // (H // G)
        out[:, a] = weights_of(q[:, a] @ k[:, b].T * scale, seen, None if sink is None else sink[a]) @ v[:, b]
    return out


def rotated_value_attention(h, w, m):
    """Attention whose values turn with their position, and whose results turn back with the query's."""
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos, base, dims = torch.arange(n), m["rot"]["base"], m["rot"]["dims"]
    q = turn((h @ w["q"].T).view(n, H, D), pos, base, dims, "interleaved")
    k = turn((h @ w["k"].T).view(n, G, D), pos, base, dims, "interleaved")
    v = turn((h @ w["v"].T).view(n, G, V), pos, base, V, "interleaved")
    o = attend(q, k, v, window_mask(n, m["mask"]["size"]), m["scale"])
    return turn(o, pos, base, V, "interleaved", back=True).reshape(n, H * V) @ w["o"].T


def key_value_attention(h, w, m, eps):
    """Attention over values that are the keys as projected; queries and keys normed over all heads at once;
    a sink per head."""
    n, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    pos, base, dims = torch.arange(n), m["rot"]["base"], m["rot"]["dims"]
    q, k = h @ w["q"].T, h @ w["k"].T
    v = k.view(n, G, D)
    q = turn((rms(q, eps) * w["q.norm"]).view(n, H, D), pos, base, dims, "halves")
    k = turn((rms(k, eps) * w["k.norm"]).view(n, G, D), pos, base, dims, "halves")
    o = attend(q, k, v, window_mask(n, m["mask"]["size"]), m["scale"], w["sink"])
    return o.reshape(n, H * D) @ w["o"].T


def linear_recurrence(q, k, v, decay):
    """S <- decay * S (rows) + k v^T, o = S^T q.  q, k, decay (n, H, D), v (n, H, V) -> (n, H, V)."""
    n, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = torch.empty_like(v)
    for t in range(n):
        S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def gated_linear_attention(h, w, m, eps):
    n, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(n, H, D) * D ** -0.5
    k, v = (h @ w["k"].T).view(n, H, D), (h @ w["v"].T).view(n, H, V)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    alpha = (torch.sigmoid(z) ** (1.0 / m["tau"])).view(n, H, D)
    o = rms(linear_recurrence(q, k, v, alpha), eps) * w["norm"]
    return (o.reshape(n, H * V) * silu(h @ w["g"].T)) @ w["o"].T


def retention(h, w, m, eps):
    n, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    pos, base, dims = torch.arange(n), m["rot"]["base"], m["rot"]["dims"]
    q = turn((h @ w["q"].T).view(n, H, D), pos, base, dims, "halves")
    k = turn((h @ w["k"].T).view(n, H, D), pos, base, dims, "halves") * D ** -0.5
    v = (h @ w["v"].T).view(n, H, V)
    decay = torch.tensor(m["decay"], dtype=torch.float64).to(h.dtype)[None, :, None].expand(n, H, D)
    o = rms(linear_recurrence(q, k, v, decay), eps)
    return (o.reshape(n, H * V) * silu(h @ w["g"].T)) @ w["o"].T


def side_by_side(h, w, m, eps):
    """Half the sum of the two mixers' normed results."""
    part = lambda s: {k[len(s) + 1:]: v for k, v in w.items() if k.startswith(s + ".")}
    left = rms(key_value_attention(h, part("left"), m["left"], eps), eps) * w["left.out"]
    right = rms(retention(h, part("right"), m["right"], eps), eps) * w["right.out"]
    return 0.5 * (left + right)


def poly_norm(z, act, eps):
    a, b, c, e = act
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def dense(h, w, eps):
    return poly_norm(h @ w["up"].T, w["act"], eps) @ w["down"].T


def mixer(layer, h, w, eps):
    m = layer["mixer"]
    if layer["type"] == "attention":
        return rotated_value_attention(h, w, m)
    if layer["type"] == "gla":
        return gated_linear_attention(h, w, m, eps)
    assert layer["type"] == "parallel"
    return side_by_side(h, w, m, eps)


def layer_runs(config):
    """(layer, pass) in the order they run; pass is None outside the loop."""
    n, loop = len(config["layers"]), config.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    body = [(i, t) for t in range(loop["times"]) for i in range(loop["start"], loop["stop"])]
    return [(i, None) for i in range(loop["start"])] + body + [(i, None) for i in range(loop["stop"], n)]


def forward(config: dict, tensors: dict, tokens, dtype=torch.float64):
    """(logits (n, vocab), streams: (n, width) after every layer run)."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = config["norm"]["eps"]
    embedded = t["embed"][tokens]
    x, streams = embedded, []
    for i, turn_no in layer_runs(config):
        if turn_no is not None and i == config["loop"]["start"]:
            x = (x + embedded if turn_no > 0 else x) + t["loop.step"][turn_no]
        layer, pre = config["layers"][i], f"l{i}."
        part = lambda s: {k[len(pre + s):]: v for k, v in t.items() if k.startswith(pre + s)}
        h = norm(x, t[pre + "norm1"], eps)
        y = mixer(layer, h, part("mix."), eps)
        if layer["mlp"] is not None:
            y = y + dense(h, part("mlp."), eps)
        x = x + y
        streams.append(x)
    return norm(x, t["final.norm"], eps) @ t["head"].T, streams


def greedy(config, tensors, prompt, count, dtype=torch.float64):
    """Greedy continuation by running the whole sequence again for every token."""
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(forward(config, tensors, tokens, dtype)[0][-1].argmax()))
    return tokens[len(prompt):]
