"""Pedivik decoder: latent attention without positions under a sliding window, dense xIELU
feed-forward, learned position vectors, and after every layer a weighted average over the embedding
output and all layer results so far.

The residual stream and every layer result stay in fp32; matrix products run in the model's dtype.
A layer is five products and a handful of HIP launches: the residual add, the depth average and the
norm of whatever comes next are one launch.  Per token and layer the cache holds one latent of
kv_rank elements.
"""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch
import torch.nn.functional as F

from zipage_amd.layers.latent import LatentAttention
from zipage_amd.layers.linear import ResidualLinear, fit
from zipage_amd.layers.residual import embed_norm, residual_norm, xielu


@dataclass(frozen=True)
class PedivikLayer:
    heads: int
    dim: int                # query / key dimensions per head
    vdim: int               # value dimensions per head
    q_rank: int
    kv_rank: int
    scale: float
    window: int             # tokens a position sees, itself included
    ff: int | None          # None: no feed-forward


@dataclass(frozen=True)
class PedivikShape:
    vocab: int
    width: int
    layers: tuple[PedivikLayer, ...]
    max_positions: int
    eps: float
    logit_scale: float

    @classmethod
    def from_config(cls, c: dict) -> "PedivikShape":
        """Reader of config.json.  A key of a layer it does not know is refused: it would change the
        model."""
        def take(d: dict, where: str, *keys):
            extra = set(d) - set(keys)
            missing = set(keys) - set(d)
            if extra or missing:
                raise ValueError(f"Pedivik config, {where}: unknown {sorted(extra)}, missing {sorted(missing)}")
            return [d[k] for k in keys]

        keys = ("layers", "logit_scale", "max_positions", "norm", "vocab", "width")
        entries, logit_scale, max_positions, norm, vocab, width = take(
            {k: v for k, v in c.items() if k in keys}, "model", *keys)
        (eps,) = take(norm, "norm", "eps")
        layers = []
        for i, e in enumerate(entries):
            mixer, mlp, kind = take(e, f"layer {i}", "mixer", "mlp", "type")
            if kind != "latent_attention":
                raise ValueError(f"Pedivik config, layer {i}: unknown mixer {kind!r}")
            dim, heads, kv_rank, mask, q_rank, scale, vdim = take(
                mixer, f"layer {i} mixer", "dim", "heads", "kv_rank", "mask", "q_rank", "scale", "vdim")
            (size,) = take(mask, f"layer {i} mask", "size")
            ff = None
            if mlp is not None:
                ff, mlp_kind = take(mlp, f"layer {i} mlp", "ff", "kind")
                if mlp_kind != "dense":
                    raise ValueError(f"Pedivik config, layer {i}: unknown feed-forward {mlp_kind!r}")
            if size < 1:
                raise ValueError(f"Pedivik config, layer {i}: a window of {size} tokens sees nothing")
            layers.append(PedivikLayer(heads, dim, vdim, q_rank, kv_rank, float(scale), size, ff))
        return cls(vocab, width, tuple(layers), max_positions, float(eps), float(logit_scale))


class Pedivik:
    # what the engine asks a model: no KV compression (every key inside the window counts), and
    # steps that hold portions of prompts beside decoded tokens
    compressible = False
    portions = True
    recurrent = False

    def __init__(self, shape: PedivikShape, device, dtype=torch.bfloat16, seed: int = 0,
                 weights: dict[str, torch.Tensor] | None = None):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Pedivik runs in bfloat16 or float32, not {dtype}")
        self.shape, self.device, self.dtype = shape, torch.device(device), dtype
        self.padded_width = -(-shape.width // 8) * 8
        self.max_positions = shape.max_positions
        self.vocab = shape.vocab
        self.mixers = [LatentAttention(shape.width, l.heads, l.dim, l.vdim, l.q_rank, l.kv_rank, l.scale,
                                       l.window, shape.eps) for l in shape.layers]
        self.sights = sorted({l.window for l in shape.layers})
        # the furthest a token looks back, and the shortest portion attended as a run
        self.lookback = max(self.sights, default=1)
        self.run_min = 16 if dtype == torch.bfloat16 and all(m.can_expand for m in self.mixers) else None
        self.caches: list[torch.Tensor] = []
        if weights is None:
            self._random(seed)
        else:
            self._load(weights)

    # ------------------------------------------------------------------ weights
    def _load(self, tensors: dict[str, torch.Tensor]):
        """Tensor names: embed, pos, final.norm and, per layer i, l<i>.norm1, l<i>.norm2, l<i>.mix.*,
        l<i>.mlp.up / .down / .act, l<i>.dwa."""
        s, W, left = self.shape, self.padded_width, dict(tensors)

        def get(name, *shape):
            if name not in left:
                raise KeyError(f"the model folder has no tensor {name}")
            t = left.pop(name)
            if tuple(t.shape) != shape:
                raise ValueError(f"tensor {name} has shape {tuple(t.shape)}, the configuration says {shape}")
            return t

        dev = lambda t, dt=None: t.to(device=self.device, dtype=dt or self.dtype).contiguous()
        f32 = lambda t: dev(t, torch.float32)
        vec = lambda name: f32(fit(get(name, s.width), W))
        self.embed = dev(fit(get("embed", s.vocab, s.width), s.vocab, W))
        self.pos = dev(fit(get("pos", s.max_positions, s.width), s.max_positions, W))
        self.final_norm = vec("final.norm")
        self.layers = []
        for i, (l, mixer) in enumerate(zip(s.layers, self.mixers)):
            pre = f"l{i}."
            mixer.load({k: get(f"{pre}mix.{k}", *shape) for k, shape in mixer.shapes().items()}, self.dtype, self.device)
            p = dict(norm1=vec(pre + "norm1"), dwa=f32(get(pre + "dwa", i + 2)))
            if l.ff is not None:
                ffp = -(-l.ff // 8) * 8
                p["norm2"] = vec(pre + "norm2")
                p["up"] = dev(fit(get(pre + "mlp.up", l.ff, s.width), ffp, W))
                p["down"] = ResidualLinear(dev(fit(get(pre + "mlp.down", s.width, l.ff), W, ffp)))
                act = get(pre + "mlp.act", 2).double().tolist()
                softplus = lambda a: math.log1p(math.exp(-abs(a))) + max(a, 0.0)
                p["act"] = (softplus(act[0]), 0.5 + softplus(act[1]))
            else:
                left.pop(pre + "norm2", None)     # without a feed-forward nothing reads it
            self.layers.append(p)
        if left:
            raise ValueError(f"tensors the configuration does not name: {sorted(left)[:8]}")

    def _random(self, seed: int, std: float = 0.02):
        """Weights drawn on the device, for benchmarks."""
        s, W = self.shape, self.padded_width
        g = torch.Generator(device=self.device).manual_seed(seed)
        w = lambda *d: torch.empty(*d, device=self.device, dtype=self.dtype).normal_(0.0, std, generator=g)
        zeros = lambda: torch.zeros(W, device=self.device)
        self.embed, self.pos = fit(w(s.vocab, s.width), s.vocab, W), fit(w(s.max_positions, s.width), s.max_positions, W)
        self.final_norm = zeros()
        self.layers = []
        for i, (l, mixer) in enumerate(zip(s.layers, self.mixers)):
            mixer.random(self.dtype, self.device, g, std)
            p = dict(norm1=zeros(), dwa=torch.tensor([0.1 / (i + 1)] * (i + 1) + [0.9], device=self.device))
            if l.ff is not None:
                ffp = -(-l.ff // 8) * 8
                p.update(norm2=zeros(), up=fit(w(l.ff, s.width), ffp, W),
                         down=ResidualLinear(fit(w(s.width, l.ff), W, ffp)), act=(0.8, 1.3))
            self.layers.append(p)

    # ------------------------------------------------------------------ cache
    def allocate_caches(self, num_pages: int, page_size: int, num_slots: int):
        """One page pool per layer; a page holds page_size latents of that layer."""
        self.caches = [m.allocate(num_pages, page_size, self.dtype, self.device) for m in self.mixers]

    # ------------------------------------------------------------------ forward
    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, ctx, trace: list | None = None) -> torch.Tensor:
        """Normed and scaled output rows (N, padded width) for compute_logits.  `trace`, when given,
        receives the stream after every layer."""
        s, W = self.shape, self.padded_width
        N, L = input_ids.shape[0], len(self.layers)
        # plane j holds the embedding output (0) or the result of layer j - 1
        history = torch.empty((L + 1, N, W), dtype=torch.float32, device=self.device)
        x = history[0]
        after = torch.empty((N, W), dtype=torch.float32, device=self.device)     # layer input
        inner = torch.empty((N, W), dtype=torch.float32, device=self.device)     # after the mixer
        norms = [p["norm1"] for p in self.layers] + [self.final_norm]
        scales = [1.0] * L + [s.logit_scale]          # the last norm's rows leave with the logits' scale
        h = embed_norm(input_ids, positions.to(torch.int32), self.embed, self.pos, x, norms[0], s.eps,
                       s.width, weight_offset=1.0)
        for i, (p, mixer) in enumerate(zip(self.layers, self.mixers)):
            y = mixer.forward(h, self.caches[i], ctx)
            if "up" in p:
                h = residual_norm(x, y, p["norm2"], s.eps, s.width, weight_offset=1.0, x_out=inner)
                x, y = inner, p["down"].forward(xielu(F.linear(h, p["up"]), *p["act"]))
            h = residual_norm(x, y, norms[i + 1], s.eps, s.width, weight_offset=1.0, out_scale=scales[i + 1],
                              x_out=after, result=history[i + 1], history=history, mix=p["dwa"])
            x = after
            if trace is not None:
                trace.append(x[:, :s.width].clone())
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.embed)
