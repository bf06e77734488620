"""Plain, slow restatement of the Kapolorn decoder, one function per mechanism, on whole sequences.

One sequence at a time, recurrences as loops over its tokens, attention as dense matrices under an
explicit mask, experts one after the other; in the floating type of the inputs (the tests pass
float64).  It shares no code with the product path: no padding, no cache, no chunked forms.
"""
from __future__ import annotations

import math

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * w


def unit(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def rotate(x, positions, base, dims):
    """x (n, heads, dim): dimension i < dims / 2 turns with dimension i + dims / 2."""
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    a = (positions.double()[:, None] * f).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), x[..., dims:]], dim=-1)


def chunk_mask(n: int, size: int) -> torch.Tensor:
    """visible[i, j]: j <= i and both in the same block of `size` positions."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & (i // size == j // size)


def sink_softmax(score, sink):
    """Rows of weights that share their denominator with exp(sink)."""
    top = torch.maximum(score.max(dim=-1, keepdim=True).values, sink)
    e = torch.exp(score - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink - top))


def sink_attention(h, w, m):
    """Grouped-query attention inside chunks of positions, with a sink per head."""
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(n)
    q = rotate((h @ w["q"].T).view(n, H, D), pos, m["rot"]["base"], m["rot"]["dims"])
    k = rotate((h @ w["k"].T).view(n, G, D), pos, m["rot"]["base"], m["rot"]["dims"])
    v = (h @ w["v"].T).view(n, G, V)
    seen = chunk_mask(n, m["mask"]["size"])
    out = torch.empty(n, H, V, dtype=h.dtype)
    for a in range(H):
        b = a // (H // G)
        score = (q[:, a] @ k[:, b].T * m["scale"]).masked_fill(~seen, -math.inf)
        out[:, a] = sink_softmax(score, w["sink"][a]) @ v[:, b]
    return out.reshape(n, H * V) @ w["o"].T


def mlstm_recurrence(q, k, v, i, f):
    """q, k (n, H, D), v (n, H, V), log gates i, f (n, H) -> (n, H, V)."""
    n, H, D = q.shape
    V = v.shape[-1]
    S, z = torch.zeros(H, D, V, dtype=q.dtype), torch.zeros(H, D, dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    out = torch.empty(n, H, V, dtype=q.dtype)
    for t in range(n):
        new = torch.maximum(f[t] + m, i[t])
        keep, write = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        m = new
        S = keep[:, None, None] * S + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = keep[:, None] * z + write[:, None] * k[t]
        den = torch.maximum((z * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = torch.einsum("hdv,hd->hv", S, q[t]) / den[:, None]
    return out


def mlstm(h, w, m, eps):
    n, H, D, V, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ w["q"].T).view(n, H, D) * D ** -0.5
    k, v = (h @ w["k"].T).view(n, H, D), (h @ w["v"].T).view(n, H, V)
    i = cap * torch.tanh((h @ w["i"].T + w["i.b"]) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((h @ w["f"].T + w["f.b"]) / cap))
    o = rms(mlstm_recurrence(q, k, v, i, f), eps).reshape(n, H * V) * w["norm"]
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def short_conv(x, w):
    """x (n, channels), w (channels, taps): causal, the last tap is the current token's; then silu."""
    n, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for t in range(n):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += w[:, j] * x[s]
    return y * torch.sigmoid(y)


def delta_recurrence(q, k, v, g, beta):
    """q, k, g (n, H, D), v (n, H, V), beta (n, H) -> (n, H, V)."""
    n, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = torch.empty_like(v)
    for t in range(n):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def channel_delta(h, w, m, eps):
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit(short_conv(h @ w["q"].T, w["q.conv"]).view(n, G, D)) * D ** -0.5
    k = unit(short_conv(h @ w["k"].T, w["k.conv"]).view(n, G, D))
    v = short_conv(h @ w["v"].T, w["v.conv"]).view(n, H, V)
    beta = torch.sigmoid(h @ w["b"].T)
    a = torch.nn.functional.softplus((h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]).view(n, H, D)
    g = torch.exp(-torch.exp(w["A_log"])[None, :, None] * a)
    head = torch.arange(H) // (H // G)
    o = norm(delta_recurrence(q[:, head], k[:, head], v, g, beta), w["norm"], eps).reshape(n, H * V)
    return (o * torch.sigmoid((h @ w["g1"].T) @ w["g2"].T)) @ w["o"].T


def expert(h, w, limit):
    g = (h @ w["gate"].T).clamp(max=limit)
    u = (h @ w["up"].T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w["down"].T


def route(z, top, count, keep):
    """Router logits (n, E) -> weights (n, E), zero for the experts a token does not use."""
    n, E = z.shape
    s = torch.softmax(z, dim=-1)
    out = torch.zeros_like(s)
    size = E // count
    for t in range(n):
        best = sorted(range(count), key=lambda c: -float(s[t, c * size:(c + 1) * size].max()))[:keep]
        allowed = [e for c in sorted(best) for e in range(c * size, (c + 1) * size)]
        for e in sorted(allowed, key=lambda e: -float(s[t, e]))[:top]:
            out[t, e] = s[t, e]
    return out


def experts(h, w, c):
    """The weighted sum of the chosen experts, and the shared one."""
    part = lambda p: {k[len(p) + 1:]: v for k, v in w.items() if k.startswith(p + ".")}
    r = c["router"]
    a = route(h @ w["router"].T, r["top"], r["groups"]["count"], r["groups"]["keep"])
    y = expert(h, part("shared"), c["shared"]["limit"])
    for e in range(r["experts"]):
        y = y + a[:, e:e + 1] * expert(h, part(f"e{e}"), c["expert"]["limit"])
    return y


def layer_order(config):
    """Layer indices in the order they run."""
    n, loop = len(config["layers"]), config["loop"]
    body = list(range(loop["start"], loop["stop"]))
    return list(range(loop["start"])) + body * loop["times"] + list(range(loop["stop"], n))


def mixer(layer, h, w, eps):
    m = layer["mixer"]
    if layer["type"] == "channel_delta":
        return channel_delta(h, w, m, eps)
    assert layer["type"] == "parallel"
    side = lambda s: {k[len(s) + 1:]: v for k, v in w.items() if k.startswith(s + ".")}
    return m["left_scale"] * sink_attention(h, side("left"), m["left"]) \
        + m["right_scale"] * mlstm(h, side("right"), m["right"], eps)


def forward(config: dict, tensors: dict, tokens, dtype=torch.float64):
    """(logits (n, vocab), streams: (n, width) after every layer run)."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = config["norm"]["eps"]
    x = t["embed"][tokens] * config["embedding"]["scale"]
    streams = []
    for i in layer_order(config):
        layer, pre = config["layers"][i], f"l{i}."
        mix = {k[len(pre) + 4:]: v for k, v in t.items() if k.startswith(pre + "mix.")}
        x = x + norm(mixer(layer, norm(x, t[pre + "norm1"], eps), mix, eps), t[pre + "norm1b"], eps)
        if layer["mlp"] is not None:
            mlp = {k[len(pre) + 4:]: v for k, v in t.items() if k.startswith(pre + "mlp.")}
            x = x + norm(experts(norm(x, t[pre + "norm2"], eps), mlp, layer["mlp"]), t[pre + "norm2b"], eps)
        streams.append(x)
    logits = norm(x, t["final.norm"], eps) @ t["embed"].T
    cap = config["logit_softcap"]
    return cap * torch.tanh(logits / cap), streams


def greedy(config, tensors, prompt, count, dtype=torch.float64):
    """Greedy continuation by running the whole sequence again for every token."""
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(forward(config, tensors, tokens, dtype)[0][-1].argmax()))
    return tokens[len(prompt):]
