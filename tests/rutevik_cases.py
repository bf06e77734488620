"""Small Rutevik configurations with seeded weights that make every mechanism show in the logits."""
import math

import torch

from oracle import rutevik_oracle as O

STRETCH = {"factor": 3.0, "low": 1.5, "high": 6.0, "original": 96}


def attention(heads, kv_heads, dim, vdim, rot, base=1000.0, scale=None, softcap=5.0, diff=0.25, scaling=STRETCH):
    turn = {"base": base, "dims": rot, **({"scaling": scaling} if scaling else {})}
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": turn, "softcap": softcap, "diff": diff,
            "scale": scale if scale is not None else dim ** -0.5}


def latent(heads, dim, vdim, rot_dim, q_rank, kv_rank, base=300.0, scale=None, kv_from=None, scaling=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "rot_dim": rot_dim, "q_rank": q_rank, "kv_rank": kv_rank,
            "rot": {"base": base, "dims": rot_dim, **({"scaling": scaling} if scaling else {})},
            "scale": scale if scale is not None else (dim + rot_dim) ** -0.5, **({} if kv_from is None else {"kv_from": kv_from})}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def layer(mixer, mlp):
    return {"type": "latent_attention" if "kv_rank" in mixer else "attention", "mixer": mixer, "mlp": mlp}


def config(width, vocab, layers, eps=1e-5, logit_scale=0.7):
    return {"architecture": "Rutevik", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps},
            "logit_scale": logit_scale}


CONFIGS = {
    # nothing is a multiple of anything; every layer its own sizes; two layers read one cache, one of them behind
    # a layer with its own
    "odd": config(76, 131, [
        layer(attention(6, 3, 20, 40, 10), moe(10, 3, 44)),
        layer(latent(5, 24, 40, 10, 50, 44), dense(52)),
        layer(latent(3, 40, 24, 10, 37, 44, scale=0.2, kv_from=1), None),
        layer(latent(7, 12, 20, 26, 30, 70, base=50.0, scaling={**STRETCH, "factor": 2.0}), moe(7, 2, 52)),
        layer(latent(4, 20, 28, 10, 41, 44, kv_from=1), moe(9, 4, 20)),
        layer(attention(3, 3, 36, 20, 36, base=40.0, scaling=None, softcap=2.0, diff=0.6), dense(100)),
    ], eps=1e-3, logit_scale=1.7),
    # more query columns per key head than an MFMA tile has, heads and latents beyond one column block, more
    # experts than a wave has lanes
    "wide": config(160, 203, [
        layer(latent(40, 72, 144, 64, 96, 288, base=5000.0), moe(70, 5, 64)),
        layer(latent(18, 136, 136, 64, 64, 288, base=5000.0, kv_from=0), moe(66, 4, 32)),
        layer(attention(34, 2, 72, 144, 32, base=500.0), dense(240)),
    ], eps=1e-6, logit_scale=0.3),
    # the smallest parts, and sizes the matrix-core kernels do not cover: everything runs token by token
    "ends": config(96, 97, [
        layer(latent(1, 8, 16, 2, 16, 520), moe(4, 4, 32)),
        layer(attention(2, 2, 136, 48, 2), None),
        layer(latent(2, 64, 32, 72, 40, 40), dense(8)),
        layer(latent(17, 8, 8, 72, 8, 40, kv_from=2), moe(3, 1, 40)),
        layer(attention(1, 1, 8, 8, 8), dense(33)),
    ], eps=1e-2, logit_scale=2.0),
    # every token uses every expert, so rounding cannot change a choice: bfloat16 is held to every row
    "calm": config(128, 113, [
        layer(attention(8, 2, 32, 64, 24), dense(160)),
        layer(latent(4, 64, 48, 32, 64, 96), moe(3, 3, 32)),
        layer(latent(6, 32, 64, 32, 96, 96, kv_from=1), moe(2, 2, 64)),
        layer(attention(4, 4, 64, 32, 64, scaling=None), None),
    ]),
}


def weights(cfg, seed):
    """bf16 tensors under the names a model folder uses."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s, std=1.0: torch.randn(*s, generator=g) * std
    W = cfg["width"]
    lin = lambda o, i, gain=1.0: r(o, i, std=gain * i ** -0.5)
    t = {"embed": r(cfg["vocab"], W), "head": lin(cfg["vocab"], W, 2.0)}

    def norm(name):
        t[name], t[name + ".b"], t[name + ".alpha"] = 1 + r(W, std=0.3), r(W, std=0.3), 0.6 + 0.2 * torch.rand((), generator=g)
    norm("final.norm")
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        norm(p + "norm1")
        if l["mlp"] is not None:
            norm(p + "norm2")
        H, D, V, q = m["heads"], m["dim"], m["vdim"], p + "mix."
        if l["type"] == "attention":
            G = m["kv_heads"]
            # scores of a few units: single keys carry visible weight, and the cap bends them
            gain = math.sqrt(3.0 / (m["scale"] * math.sqrt(D)))
            t[q + "q"], t[q + "k"], t[q + "v"] = lin(H * 2 * D, W, gain), lin(G * 2 * D, W, gain), lin(G * V, W)
            t[q + "q.b"], t[q + "k.b"], t[q + "v.b"] = r(H * 2 * D, std=0.4), r(G * 2 * D, std=0.4), r(G * V, std=0.4)
            for k in ("lq1", "lk1", "lq2", "lk2"):
                t[q + k] = r(D, std=0.6 * D ** -0.25)
            t[q + "g"], t[q + "o"] = lin(H * V, W, 2.0), lin(W, H * V, 2.0)
        else:
            R, Q, P = m["kv_rank"], m["q_rank"], m["rot_dim"]
            gain = 3.0 / (m["scale"] * math.sqrt(D + P))
            t[q + "dq"], t[q + "dq.norm"], t[q + "uq"] = lin(Q, W), 1 + r(Q, std=0.3), lin(H * (D + P), Q, gain)
            if m.get("kv_from") is None:
                t[q + "dkv"], t[q + "dkv.norm"] = lin(R + P, W), 1 + r(R, std=0.3)
            t[q + "uk"], t[q + "uv"], t[q + "o"] = lin(H * D, R), lin(H * V, R), lin(W, H * V, 2.0)
        if l["mlp"] is not None:
            c, q = l["mlp"], p + "mlp."
            if c["kind"] == "dense":
                t[q + "up"], t[q + "down"] = lin(c["ff"], W), lin(W, c["ff"])
                continue
            E, ff = c["router"]["experts"], c["expert"]["ff"]
            # scores that differ by far more than rounding: neighbours in rank must not change places
            t[q + "router"] = lin(E, W, 2.0)
            for e in range(E):
                t[f"{q}e{e}.gate"], t[f"{q}e{e}.up"], t[f"{q}e{e}.down"] = lin(ff, W, 2.0), lin(ff, W), lin(W, ff)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


_cache: dict = {}


def case(name):
    """(config, weights) of a named configuration."""
    if name not in _cache:
        _cache[name] = (CONFIGS[name], weights(CONFIGS[name], 300 + len(name)))
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
    """float32: every row.  bfloat16: rounding may swap two experts of nearly equal score, which moves that
    token and, through keys, a little of the tokens behind it: there the median row counts, and every row
    where no choice can change."""
    e = row_errors(got, want, whole)
    if dtype == torch.float32:
        assert float(e.max()) < 1e-4, float(e.max())
    elif name == "calm":
        assert float(e.max()) < 0.15, float(e.max())
        assert len(e) < 20 or float(e.quantile(0.9)) < 0.06, float(e.quantile(0.9))
    else:
        assert len(e) < 20 or float(e.median()) < 0.1, float(e.median())
