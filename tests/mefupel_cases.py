"""Small Mefupel configurations with seeded weights that make every mechanism show in the logits."""
import math

import torch

from oracle import mefupel_oracle as O


def attention(heads, kv_heads, dim, vdim, window, rot, base=1000.0, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
            "rot": {"base": base, "dims": rot}, "scale": scale if scale is not None else dim ** -0.5}


def gla(heads, dim, vdim, tau):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def pair(left, memory, rot, decay, base=300.0):
    """left: heads, kv_heads, dim, window, rot and what else attention() takes; memory: heads, dim, vdim."""
    heads, kv_heads, dim, window, lrot, *more = left
    h, d, v = memory
    assert len(decay) == h
    return {"left": attention(heads, kv_heads, dim, dim, window, lrot, *more),
            "right": {"heads": h, "dim": d, "vdim": v, "rot": {"base": base, "dims": rot}, "decay": list(decay)}}


def layer(mixer, ff):
    kind = "parallel" if "left" in mixer else "gla" if "tau" in mixer else "attention"
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, loop=None, eps=1e-5):
    return {"architecture": "Mefupel", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps},
            **({} if loop is None else {"loop": dict(zip(("start", "stop", "times"), loop))})}


CONFIGS = {
    # nothing is a multiple of anything; every layer its own sizes; parts of heads turn; three passes of three
    # layers, one of them without feed-forward
    "odd": config(76, 131, [
        layer(gla(2, 12, 20, 5.0), 36),
        layer(attention(6, 3, 20, 14, 7, 10), 44),
        layer(gla(3, 20, 24, 2.5), None),
        layer(pair((4, 2, 24, 33, 10, 50.0), (3, 20, 12), 6, (0.5, 0.93, 0.999)), 52),
        layer(attention(5, 1, 36, 22, 18, 36, 40.0, 0.31), 100),
    ], (1, 4, 3), eps=1e-3),
    # more query heads per key head than an MFMA tile has rows, heads beyond one column block and beyond the blocked
    # recurrences, no loop
    "wide": config(160, 203, [
        layer(attention(34, 2, 136, 144, 50, 64, 500.0), 240),
        layer(pair((20, 1, 72, 21, 72), (2, 136, 144), 136, (0.9, 0.99)), 96),
        layer(gla(4, 72, 136, 16.0), 64),
        layer(attention(4, 4, 64, 64, 64, 2), 520),
    ], eps=1e-6),
    # a token that sees itself alone, a window longer than any sequence, the smallest heads, sizes that the matrix-core
    # kernels do not cover, decays at both ends; the whole model twice, from its first layer on
    "ends": config(96, 97, [
        layer(attention(1, 1, 264, 2, 5, 264), 8),
        layer(attention(2, 2, 8, 260, 1, 2), None),
        layer(pair((3, 3, 8, 4096, 2), (4, 8, 8), 2, (0.0, 1.0, 0.25, 0.75)), 33),
        layer(gla(1, 200, 250, 1.0), 16),
        layer(pair((18, 9, 40, 2, 8), (1, 32, 32), 32, (0.97,)), None),
    ], (0, 5, 2), eps=1e-2),
    # a loop of one pass up to the last layer; one head of each kind
    "once": config(64, 89, [
        layer(gla(1, 16, 16, 4.0), 48),
        layer(attention(3, 1, 16, 32, 9, 16), 24),
        layer(pair((2, 1, 32, 12, 16), (1, 64, 16), 30, (0.9,)), 40),
    ], (1, 3, 1)),
    # bfloat16 on the kernels of serving sizes
    "calm": config(128, 113, [
        layer(attention(8, 2, 32, 48, 37, 16), 160),
        layer(gla(4, 32, 64, 8.0), 96),
        layer(pair((4, 2, 64, 70, 64), (2, 64, 32), 64, (0.95, 0.995)), 128),
        layer(attention(4, 4, 64, 32, 16, 64), None),
    ], (1, 3, 2)),
}


def weights(cfg, seed):
    """bf16 tensors under the names a model folder uses."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s, std=1.0: torch.randn(*s, generator=g) * std
    W = cfg["width"]
    lin = lambda o, i, gain=1.0: r(o, i, std=gain * i ** -0.5)
    t = {"embed": r(cfg["vocab"], W), "head": lin(cfg["vocab"], W, 2.0), "final.norm": r(W, std=0.3)}
    if "loop" in cfg:
        t["loop.step"] = r(cfg["loop"]["times"], W, std=0.7)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        t[p + "norm1"] = r(W, std=0.3)

        def linear(q, m, rank=None):
            H, D, V = m["heads"], m["dim"], m["vdim"]
            t[q + "q"], t[q + "k"] = lin(H * D, W), lin(H * D, W)
            t[q + "v"], t[q + "g"], t[q + "o"] = lin(H * V, W), lin(H * V, W, 1.5), lin(W, H * V, 2.0)
        if l["type"] == "attention":
            H, G, D, V, q = m["heads"], m["kv_heads"], m["dim"], m["vdim"], p + "mix."
            # scores of a few units: single keys carry visible weight
            gain = math.sqrt(2.5 / (m["scale"] * math.sqrt(D)))
            t[q + "q"], t[q + "k"] = lin(H * D, W, gain), lin(G * D, W, gain)
            t[q + "v"], t[q + "o"] = lin(G * V, W), lin(W, H * V, 2.0)
        elif l["type"] == "gla":
            H, D, V, q, rank = m["heads"], m["dim"], m["vdim"], p + "mix.", 3 + m["dim"] // 4
            linear(q, m)
            t[q + "norm"], t[q + "a1"], t[q + "a2"] = 1 + r(V, std=0.3), lin(rank, W), lin(H * D, rank)
            t[q + "a2.b"] = 1 + 2 * r(H * D)
        else:
            a, q = m["left"], p + "mix.left."
            H, G, D = a["heads"], a["kv_heads"], a["dim"]
            t[q + "q"], t[q + "k"] = lin(H * D, W), lin(G * D, W)
            gain = math.sqrt(2.5 / (a["scale"] * math.sqrt(D)))
            t[q + "q.norm"], t[q + "k.norm"] = gain * (1 + r(H * D, std=0.3)), gain * (1 + r(G * D, std=0.3))
            t[q + "sink"], t[q + "o"], t[q + "out"] = 1 + r(H), lin(W, H * D, 2.0), 1 + r(W, std=0.3)
            linear(p + "mix.right.", m["right"])
            t[p + "mix.right.out"] = 1 + r(W, std=0.3)
        if l["mlp"] is not None:
            ff, q = l["mlp"]["ff"], p + "mlp."
            t[q + "up"], t[q + "down"] = lin(ff, W), lin(W, ff)
            t[q + "act"] = torch.tensor([0.7, -0.5, 0.4, 0.3]) + r(4, std=0.1)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


_cache: dict = {}


def case(name):
    """(config, weights) of a named configuration."""
    if name not in _cache:
        _cache[name] = (CONFIGS[name], weights(CONFIGS[name], 400 + len(name)))
    return _cache[name]


def expected(name, toks):
    """Oracle logits of a whole sequence (float64), kept per sequence."""
    key = (name, tuple(toks))
    if key not in _cache:
        cfg, w = case(name)
        _cache[key] = O.forward(cfg, w, toks)[0]
    return _cache[key]


def row_errors(got, want, whole=None):
    """Root mean square difference of the logits (their mean taken off) per row, in units of the spread of
    `whole` (default: `want`)."""
    whole = want if whole is None else whole
    d = got.double().cpu() - want
    d = d - d.mean(dim=-1, keepdim=True)
    spread = (whole - whole.mean(dim=-1, keepdim=True)).square().mean().sqrt()
    return d.square().mean(dim=-1).sqrt() / spread


def close(name, got, want, dtype, whole=None):
    """Every row, in both dtypes.  A read-out near zero (a first token whose query and key are nearly at right
    angles), normed, amplifies rounding: nine rows in ten are held to less than the worst."""
    e = row_errors(got, want, whole)
    worst, most = (5e-4, 1e-4) if dtype == torch.float32 else (0.5, 0.08)
    assert float(e.max()) < worst, float(e.max())
    assert len(e) < 20 or float(e.quantile(0.9)) < most, float(e.quantile(0.9))
