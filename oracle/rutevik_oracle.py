"""Plain, slow restatement of the Rutevik decoder, one function per mechanism, on whole sequences.

One sequence at a time, attention as dense matrices under an explicit mask, keys and values of every head
written out, experts one after the other; in the floating type of the inputs (the tests pass float64).  It
shares no code with the product path: no padding, no cache, no absorbed products.
"""
from __future__ import annotations

import math

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def dyt(x, w, b, alpha):
    """The norm without statistics."""
    return torch.tanh(alpha * x) * w + b


def frequencies(rot: dict) -> list[float]:
    """One per rotated pair.  With 'scaling', long wavelengths are stretched by its factor and those between
    two lengths partly."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        s = rot.get("scaling")
        if s is not None:
            length = 2.0 * math.pi / f
            if length > s["original"] / s["low"]:
                f = f / s["factor"]
            elif length >= s["original"] / s["high"]:
                t = (s["original"] / length - s["low"]) / (s["high"] - s["low"])
                f = (1.0 - t) * f / s["factor"] + t * f
        out.append(f)
    return out


def rotate(x, positions, rot):
    """x (n, heads, dim): dimension i < dims / 2 turns with dimension i + dims / 2."""
    dims, half = rot["dims"], rot["dims"] // 2
    f = torch.tensor(frequencies(rot), dtype=torch.float64)
    a = (positions.double()[:, None] * f).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), x[..., dims:]], dim=-1)


def causal_softmax(score):
    """score (n, n) -> weights over the keys up to the query's own."""
    n = score.shape[0]
    seen = torch.arange(n)[None, :] <= torch.arange(n)[:, None]
    return torch.softmax(score.masked_fill(~seen, -math.inf), dim=-1)


def shared_keys(h, w, m, eps):
    """(latent, rotated key part) of every token: what a cache of this layer holds."""
    both = h @ w["dkv"].T
    c = rms(both[:, :m["kv_rank"]], eps) * w["dkv.norm"]
    k = rotate(both[:, None, m["kv_rank"]:], torch.arange(h.shape[0]), m["rot"])[:, 0]
    return c, k


def latent_attention(h, w, m, eps, held):
    """`held`: the (latent, rotated key part) it attends to."""
    n, H, D, P, V = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, k_rot = held
    q = ((rms(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T).view(n, H, D + P)
    q_rot = rotate(q[..., D:], torch.arange(n), m["rot"])
    k = (c @ w["uk"].T).view(n, H, D)
    v = (c @ w["uv"].T).view(n, H, V)
    out = torch.empty(n, H, V, dtype=h.dtype)
    for a in range(H):
        score = (q[:, a, :D] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * m["scale"]
        out[:, a] = causal_softmax(score) @ v[:, a]
    return out.reshape(n, H * V) @ w["o"].T


def capped(score, cap):
    return cap * torch.tanh(score / cap)


def balance(w, diff):
    """The weight of the second map."""
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def differential_attention(h, w, m, eps):
    """Two softmax maps per head over the same values; their difference, normed, scaled and gated."""
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(n)
    q = rotate((h @ w["q"].T + w["q.b"]).view(n, H * 2, D), pos, m["rot"]).view(n, H, 2, D)
    k = rotate((h @ w["k"].T + w["k.b"]).view(n, G * 2, D), pos, m["rot"]).view(n, G, 2, D)
    v = (h @ w["v"].T + w["v.b"]).view(n, G, V)
    lam = balance(w, m["diff"])
    out = torch.empty(n, H, V, dtype=h.dtype)
    for a in range(H):
        b = a // (H // G)
        maps = [causal_softmax(capped(q[:, a, j] @ k[:, b, j].T * m["scale"], m["softcap"])) @ v[:, b] for j in (0, 1)]
        out[:, a] = rms(maps[0] - lam * maps[1], eps) * (1.0 - m["diff"])
    return (out.reshape(n, H * V) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def dense(h, w):
    u = torch.relu(h @ w["up"].T)
    return (u * u) @ w["down"].T


def expert(h, w):
    g = h @ w["gate"].T
    return (g * torch.sigmoid(g) * (h @ w["up"].T)) @ w["down"].T


def route(z, top):
    """Router logits (n, E) -> weights (n, E), zero for the experts a token does not use."""
    s = torch.sigmoid(z)
    out = torch.zeros_like(s)
    for t in range(z.shape[0]):
        for e in sorted(range(z.shape[1]), key=lambda e: -float(z[t, e]))[:top]:
            out[t, e] = s[t, e]
    return out


def experts(h, w, c):
    """The sum of the chosen experts, each on its own weighted copy of the input."""
    a = route(h @ w["router"].T, c["router"]["top"])
    y = torch.zeros_like(h)
    for e in range(c["router"]["experts"]):
        part = {k: w[f"e{e}.{k}"] for k in ("gate", "up", "down")}
        y = y + expert(a[:, e:e + 1] * h, part)
    return y


def forward(config: dict, tensors: dict, tokens, dtype=torch.float64):
    """(logits (n, vocab), streams: (n, width) after every layer)."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = config["norm"]["eps"]
    norm = lambda x, name: dyt(x, t[name], t[name + ".b"], t[name + ".alpha"])
    x = t["embed"][tokens]
    held, streams = {}, []
    for i, layer in enumerate(config["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        mix = {k[len(pre) + 4:]: v for k, v in t.items() if k.startswith(pre + "mix.")}
        h = norm(x, pre + "norm1")
        if layer["type"] == "latent_attention":
            source = m.get("kv_from")
            if source is None:
                held[i] = shared_keys(h, mix, m, eps)
                source = i
            y = latent_attention(h, mix, m, eps, held[source])
        else:
            assert layer["type"] == "attention"
            y = differential_attention(h, mix, m, eps)
        x = x + y
        if layer["mlp"] is not None:
            mlp = {k[len(pre) + 4:]: v for k, v in t.items() if k.startswith(pre + "mlp.")}
            h = norm(x, pre + "norm2")
            x = x + (dense(h, mlp) if layer["mlp"]["kind"] == "dense" else experts(h, mlp, layer["mlp"]))
        streams.append(x)
    return norm(x, "final.norm") @ t["head"].T * config["logit_scale"], streams


def greedy(config, tensors, prompt, count, dtype=torch.float64):
    """Greedy continuation by running the whole sequence again for every token."""
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(forward(config, tensors, tokens, dtype)[0][-1].argmax()))
    return tokens[len(prompt):]
