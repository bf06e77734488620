"""Plain, slow restatement of the Pedivik decoder, one function per mechanism, on whole sequences.

Everything is written for one sequence at a time with dense matrices and an explicit visibility
mask, in the floating type of its inputs (the tests pass float64).  It shares no code with the
product path: no padding, no cache, no absorbed projections.
"""
from __future__ import annotations

import math

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm_around_one(x, w, eps):
    """The stored weight is the distance from one."""
    return rms(x, eps) * (1 + w)


def norm_plain(x, w, eps):
    return rms(x, eps) * w


def embedding(tokens, positions, embed, pos):
    return embed[tokens] + pos[positions]


def window_mask(n: int, size: int) -> torch.Tensor:
    """visible[i, j]: 0 <= i - j < size."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    return (i - j >= 0) & (i - j < size)


def latent_attention(h, w, heads, dim, vdim, scale, size, eps):
    """h (n, width); w: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, o."""
    n = h.shape[0]
    c_q = norm_plain(h @ w["dq"].T, w["dq.norm"], eps)
    q = (c_q @ w["uq"].T).view(n, heads, dim)
    c = norm_plain(h @ w["dkv"].T, w["dkv.norm"], eps)
    k = (c @ w["uk"].T).view(n, heads, dim)
    v = (c @ w["uv"].T).view(n, heads, vdim)
    seen = window_mask(n, size)
    out = torch.empty(n, heads, vdim, dtype=h.dtype)
    for a in range(heads):
        score = (q[:, a] @ k[:, a].T) * scale
        score = score.masked_fill(~seen, -math.inf)
        out[:, a] = torch.softmax(score, dim=-1) @ v[:, a]
    return out.reshape(n, heads * vdim) @ w["o"].T


def xielu(z, p, q):
    sp = lambda t: math.log1p(math.exp(float(t)))
    pos = sp(p) * z * z + z / 2
    neg = (0.5 + sp(q)) * (torch.expm1(z) - z) + z / 2
    return torch.where(z > 0, pos, neg)


def dense_ff(h, w):
    return xielu(h @ w["up"].T, w["act"][0], w["act"][1]) @ w["down"].T


def depth_average(history, weights):
    """Sum of the embedding output and every layer result so far, one weight each."""
    out = torch.zeros_like(history[0])
    for a, x in zip(weights, history, strict=True):
        out = out + a * x
    return out


def forward(config: dict, tensors: dict, tokens, dtype=torch.float64):
    """(logits (n, vocab), streams: one (n, width) per layer, after its depth average)."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = config["norm"]["eps"]
    x = embedding(tokens, torch.arange(len(tokens)), t["embed"], t["pos"])
    history, streams = [x], []
    for i, layer in enumerate(config["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        assert layer["type"] == "latent_attention"
        mix = {k[len(pre) + 4:]: v for k, v in t.items() if k.startswith(pre + "mix.")}
        x = x + latent_attention(norm_around_one(x, t[pre + "norm1"], eps), mix, m["heads"], m["dim"],
                                 m["vdim"], m["scale"], m["mask"]["size"], eps)
        if layer["mlp"] is not None:
            mlp = {k[len(pre) + 4:]: v for k, v in t.items() if k.startswith(pre + "mlp.")}
            x = x + dense_ff(norm_around_one(x, t[pre + "norm2"], eps), mlp)
        history.append(x)
        x = depth_average(history, t[pre + "dwa"].tolist())
        streams.append(x)
    return norm_around_one(x, t["final.norm"], eps) @ t["embed"].T * config["logit_scale"], streams


def greedy(config, tensors, prompt, count, dtype=torch.float64):
    """Greedy continuation by running the whole sequence again for every token."""
    tokens = list(prompt)
    margins = []
    for _ in range(count):
        logits = forward(config, tensors, tokens, dtype)[0][-1]
        top = logits.topk(2).values
        margins.append(float(top[0] - top[1]))
        tokens.append(int(logits.argmax()))
    return tokens[len(prompt):], margins
