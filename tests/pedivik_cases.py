"""Small Pedivik configurations with seeded weights that make every mechanism show in the logits."""
import math

import torch

from oracle import pedivik_oracle as O


def layer(heads, dim, vdim, q_rank, kv_rank, window, ff, scale=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": scale if scale is not None else dim ** -0.5, "mask": {"size": window}},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, eps=1e-5, logit_scale=0.5, max_positions=640):
    return {"architecture": "Pedivik", "width": width, "vocab": vocab, "max_positions": max_positions,
            "logit_scale": logit_scale, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # nothing is a multiple of anything; every layer its own sizes and window; one without feed-forward
    "odd": config(76, 131, [layer(5, 24, 40, 52, 44, 7, 100), layer(3, 40, 24, 20, 72, 33, None, 0.21),
                            layer(1, 8, 16, 36, 20, 90, 60)], eps=1e-3, logit_scale=1.75),
    # more heads than two MFMA tiles, value size beyond one column block, one window for all
    "wide": config(160, 203, [layer(37, 32, 136, 64, 160, 50, 224), layer(37, 32, 136, 64, 160, 50, 224)],
                   eps=1e-6, logit_scale=0.125),
    # a token that sees itself alone, and a window longer than any sequence; latent larger than 256
    "ends": config(96, 97, [layer(2, 64, 48, 40, 288, 1, 72), layer(18, 72, 32, 80, 32, 4096, 80)],
                   eps=1e-2, logit_scale=1.0),
}


def weights(cfg, seed):
    """bf16 tensors under the names a model folder uses."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s, std=1.0: torch.randn(*s, generator=g) * std
    W = cfg["width"]
    t = {"embed": r(cfg["vocab"], W), "pos": r(cfg["max_positions"], W, std=0.7),
         "final.norm": r(W, std=0.3)}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        H, D, V, Q, R = m["heads"], m["dim"], m["vdim"], m["q_rank"], m["kv_rank"]
        t[p + "norm1"] = r(W, std=0.3)
        t[p + "mix.dq"], t[p + "mix.dkv"] = r(Q, W, std=W ** -0.5), r(R, W, std=W ** -0.5)
        t[p + "mix.dq.norm"], t[p + "mix.dkv.norm"] = 1 + r(Q, std=0.3), 1 + r(R, std=0.3)
        # scores of a few units: single keys carry visible weight
        gain = math.sqrt(2.0 / (m["scale"] * math.sqrt(D)))
        t[p + "mix.uq"], t[p + "mix.uk"] = r(H * D, Q, std=gain * Q ** -0.5), r(H * D, R, std=gain * R ** -0.5)
        t[p + "mix.uv"] = r(H * V, R, std=R ** -0.5)
        t[p + "mix.o"] = r(W, H * V, std=2 * (H * V) ** -0.5)
        if l["mlp"] is not None:
            F = l["mlp"]["ff"]
            t[p + "norm2"] = r(W, std=0.3)
            t[p + "mlp.up"], t[p + "mlp.down"] = r(F, W, std=W ** -0.5), r(W, F, std=F ** -0.5)
            t[p + "mlp.act"] = torch.tensor([0.4, -0.7]) + r(2, std=0.3)
        t[p + "dwa"] = torch.cat([r(i + 1, std=0.4), torch.tensor([0.9])])
    return {k: v.to(torch.bfloat16) for k, v in t.items()}


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


_cache: dict = {}


def case(name):
    """(config, weights) of a named configuration."""
    if name not in _cache:
        _cache[name] = (CONFIGS[name], weights(CONFIGS[name], 100 + len(name)))
    return _cache[name]


def expected(name, toks):
    """Oracle logits of a whole sequence (float64), kept per sequence."""
    key = (name, tuple(toks))
    if key not in _cache:
        cfg, w = case(name)
        _cache[key] = O.forward(cfg, w, toks)[0]
    return _cache[key]


def error(got, want):
    """Root mean square difference of the logits (their mean taken off), in units of their spread;
    the worst row."""
    d = got.double().cpu() - want
    d = d - d.mean(dim=-1, keepdim=True)
    spread = (want - want.mean(dim=-1, keepdim=True)).square().mean().sqrt()
    return float((d.square().mean(dim=-1).sqrt() / spread).max())


LIMIT = {torch.float32: 3e-5, torch.bfloat16: 4e-2}
