"""Rutevik decoder: latent attention with a rotated key part that all heads share, some layers of which read
an earlier layer's cache, between differential attention over grouped heads; dense or mixed feed-forwards;
norms that are a scaled tanh without statistics.

The residual stream stays in fp32; matrix products run in the model's dtype.  The residual add and the norm of
whatever comes next are one launch.  Per token a latent layer holds its latent and the shared key part, a
layer that reads another one's cache holds nothing.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn.functional as F

from zipage_amd.layers.grouped import GroupedAttention
from zipage_amd.layers.latent import LatentAttention
from zipage_amd.layers.linear import ResidualLinear, fit, pad_to_multiple
from zipage_amd.layers.moe import Experts
from zipage_amd.layers.residual import embed_norm, relu_square, residual_norm
from zipage_amd.layers.rotary import Rotary
from zipage_amd.sight import EVERYTHING


@dataclass(frozen=True)
class LatentMixer:
    heads: int
    dim: int                # query / key dimensions per head that are not rotated
    vdim: int
    q_rank: int
    kv_rank: int
    rotary: Rotary          # of the rotated part, all of whose dimensions turn
    scale: float
    source: int             # the layer whose cache it reads: its own index, or an earlier one


@dataclass(frozen=True)
class DifferentialMixer:
    heads: int
    kv_heads: int
    dim: int                # of each map
    vdim: int
    rotary: Rotary
    scale: float
    softcap: float
    diff: float


@dataclass(frozen=True)
class DenseShape:
    ff: int


@dataclass(frozen=True)
class MixtureShape:
    experts: int
    top: int
    ff: int


@dataclass(frozen=True)
class RutevikLayer:
    mixer: LatentMixer | DifferentialMixer
    mlp: DenseShape | MixtureShape | None


@dataclass(frozen=True)
class RutevikShape:
    vocab: int
    width: int
    layers: tuple[RutevikLayer, ...]
    eps: float
    logit_scale: float

    @classmethod
    def from_config(cls, c: dict) -> "RutevikShape":
        """Reader of config.json.  A key it does not know inside a layer is refused: it would change the
        model."""
        def take(d: dict, where: str, *keys, **optional):
            extra = set(d) - set(keys) - set(optional)
            missing = set(keys) - set(d)
            if extra or missing:
                raise ValueError(f"Rutevik config, {where}: unknown {sorted(extra)}, missing {sorted(missing)}")
            return [d[k] for k in keys] + [d.get(k, v) for k, v in optional.items()]

        def rotary(d: dict, where: str) -> Rotary:
            base, dims, scaling = take(d, where, "base", "dims", scaling=None)
            if scaling is not None:
                scaling = tuple(float(v) for v in take(scaling, f"{where} scaling", "factor", "low", "high", "original"))
            return Rotary(float(base), dims, scaling)

        keys = ("layers", "logit_scale", "norm", "vocab", "width")
        entries, logit_scale, norm, vocab, width = take({k: v for k, v in c.items() if k in keys}, "model", *keys)
        (eps,) = take(norm, "norm", "eps")
        layers = []
        for i, e in enumerate(entries):
            mixer, kind, mlp = take(e, f"layer {i}", "mixer", "type", mlp=None)
            if kind == "latent_attention":
                dim, heads, kv_rank, q_rank, rot, rot_dim, scale, vdim, source = take(
                    mixer, f"layer {i} mixer", "dim", "heads", "kv_rank", "q_rank", "rot", "rot_dim", "scale", "vdim",
                    kv_from=None)
                turn = rotary(rot, f"layer {i} rot")
                if turn.dims != rot_dim:
                    raise ValueError(f"Rutevik config, layer {i}: {turn.dims} rotated dimensions of {rot_dim}")
                m = LatentMixer(heads, dim, vdim, q_rank, kv_rank, turn, float(scale), i if source is None else source)
                if source is not None:
                    held = layers[source].mixer if 0 <= source < i else None
                    if not isinstance(held, LatentMixer) or held.source != source or \
                            (held.kv_rank, held.rotary) != (m.kv_rank, m.rotary):
                        raise ValueError(f"Rutevik config, layer {i}: layer {source} holds no latent for it")
            elif kind == "attention":
                diff, dim, heads, kv_heads, rot, scale, cap, vdim = take(
                    mixer, f"layer {i} mixer", "diff", "dim", "heads", "kv_heads", "rot", "scale", "softcap", "vdim")
                m = DifferentialMixer(heads, kv_heads, dim, vdim, rotary(rot, f"layer {i} rot"), float(scale), float(cap),
                                      float(diff))
                if m.softcap <= 0:
                    raise ValueError(f"Rutevik config, layer {i}: a soft cap of {m.softcap}")
            else:
                raise ValueError(f"Rutevik config, layer {i}: unknown mixer {kind!r}")
            f = None
            if mlp is not None and mlp.get("kind") == "dense":
                f = DenseShape(take(mlp, f"layer {i} mlp", "ff", "kind")[0])
            elif mlp is not None and mlp.get("kind") == "moe":
                expert, router, _ = take(mlp, f"layer {i} mlp", "expert", "router", "kind")
                (ff,) = take(expert, f"layer {i} expert", "ff")
                f = MixtureShape(*take(router, f"layer {i} router", "experts", "top"), ff)
            elif mlp is not None:
                raise ValueError(f"Rutevik config, layer {i}: unknown feed-forward {mlp.get('kind')!r}")
            layers.append(RutevikLayer(m, f))
        return cls(vocab, width, tuple(layers), float(eps), float(logit_scale))


class Differential:
    """The mixer of a DifferentialMixer layer with its input and output products."""

    def __init__(self, m: DifferentialMixer, width: int, padded_width: int, eps: float):
        self.padded_width = padded_width
        self.core = GroupedAttention(width, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, None, m.rotary, softcap=m.softcap,
                                     diff=m.diff, eps=eps, bias=True, gated=True)

    @property
    def can_run(self) -> bool:
        return self.core.can_run

    def shapes(self) -> dict:
        return self.core.shapes()

    def load(self, w: dict, dtype, device):
        into, out = self.core.load(w, dtype, device, self.padded_width)
        put = lambda t: t.to(device=device, dtype=dtype).contiguous()
        self.into, self.out = put(into), ResidualLinear(put(out))

    def allocate(self, num_pages: int, page_size: int, dtype, device):
        return self.core.allocate(num_pages, page_size, dtype, device)

    def forward(self, h, cache, ctx, positions, held):
        mixed = torch.empty((h.shape[0], self.core.out_columns), dtype=h.dtype, device=h.device)
        self.core.attend(F.linear(h, self.into), positions, cache, ctx, mixed)
        return self.out.forward(mixed)


class Dense:
    """down(relu(up h)^2)."""

    def __init__(self, width: int, padded_width: int, ff: int):
        self.width, self.padded_width, self.ff, self.ff_p = width, padded_width, ff, pad_to_multiple(ff, 8)

    def shapes(self) -> dict:
        return {"up": (self.ff, self.width), "down": (self.width, self.ff)}

    def load(self, w: dict, dtype, device):
        put = lambda t, *shape: fit(t.to(device=device, dtype=dtype), *shape)
        self.up = put(w["up"], self.ff_p, self.padded_width)
        self.down = ResidualLinear(put(w["down"], self.padded_width, self.ff_p))

    def random(self, dtype, device, generator, std: float):
        self.load({k: torch.empty(*s, dtype=dtype, device=device).normal_(0.0, std, generator=generator)
                   for k, s in self.shapes().items()}, dtype, device)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        return self.down.forward(relu_square(F.linear(h, self.up)))


class Rutevik:
    # what the engine asks a model: no KV compression, steps that hold portions of prompts beside decoded
    # tokens, no state but what the pages hold
    compressible = False
    portions = True
    recurrent = False

    def __init__(self, shape: RutevikShape, device, dtype=torch.bfloat16, seed: int = 0,
                 weights: dict[str, torch.Tensor] | None = None):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Rutevik runs in bfloat16 or float32, not {dtype}")
        self.shape, self.device, self.dtype = shape, torch.device(device), dtype
        self.padded_width = W = pad_to_multiple(shape.width, 32)
        self.vocab = shape.vocab

        def mixer(i: int, m):
            if isinstance(m, DifferentialMixer):
                return Differential(m, shape.width, W, shape.eps)
            return LatentAttention(shape.width, m.heads, m.dim, m.vdim, m.q_rank, m.kv_rank, m.scale, None, shape.eps,
                                   rotary=m.rotary, own_latent=m.source == i, padded_width=W)

        def mlp(f):
            if isinstance(f, MixtureShape):
                return Experts(shape.width, f.experts, f.top, f.ff, 0.0, score="sigmoid", act="silu")
            return None if f is None else Dense(shape.width, W, f.ff)

        self.mixers = [mixer(i, l.mixer) for i, l in enumerate(shape.layers)]
        self.mlps = [mlp(l.mlp) for l in shape.layers]
        # the layer whose pages a layer reads
        self.source = [getattr(l.mixer, "source", i) for i, l in enumerate(shape.layers)]
        self.sights = [None]
        # the furthest a token looks back, and the shortest portion attended as a run
        self.lookback = EVERYTHING
        fits = all(m.can_expand if isinstance(m, LatentAttention) else m.can_run for m in self.mixers)
        self.run_min = 16 if dtype == torch.bfloat16 and fits else None
        self.caches: list[torch.Tensor | None] = []
        if weights is None:
            self._random(seed)
        else:
            self._load(weights)

    # ------------------------------------------------------------------ weights
    def _load(self, tensors: dict[str, torch.Tensor]):
        """Tensor names: embed, head, final.norm and, per layer i, l<i>.norm1 / norm2, l<i>.mix.* and l<i>.mlp.*;
        a norm has .b and .alpha beside its weight."""
        s, W, left = self.shape, self.padded_width, dict(tensors)

        def get(name, *shape):
            if name not in left:
                raise KeyError(f"the model folder has no tensor {name}")
            t = left.pop(name)
            if tuple(t.shape) != shape:
                raise ValueError(f"tensor {name} has shape {tuple(t.shape)}, the configuration says {shape}")
            return t

        put = lambda t: t.to(device=self.device, dtype=self.dtype).contiguous()
        vec = lambda name: fit(get(name, s.width), W).to(device=self.device, dtype=torch.float32).contiguous()
        norm = lambda name: dict(norm_weight=vec(name), norm_bias=vec(name + ".b"), norm_alpha=float(get(name + ".alpha")))
        self.embed = put(fit(get("embed", s.vocab, s.width), s.vocab, W))
        self.head = put(fit(get("head", s.vocab, s.width), s.vocab, W))
        self.final_norm = norm("final.norm")
        self.norms = []
        for i, (mixer, mlp) in enumerate(zip(self.mixers, self.mlps)):
            pre = f"l{i}."
            mixer.load({k: get(f"{pre}mix.{k}", *shape) for k, shape in mixer.shapes().items()}, self.dtype, self.device)
            norms = [norm(pre + "norm1")]
            if mlp is not None:
                norms.append(norm(pre + "norm2"))
                mlp.load({k: get(f"{pre}mlp.{k}", *shape) for k, shape in mlp.shapes().items()}, self.dtype, self.device)
            else:
                for k in ("norm2", "norm2.b", "norm2.alpha"):      # without a feed-forward nothing reads them
                    left.pop(pre + k, None)
            self.norms.append(norms)
        if left:
            raise ValueError(f"tensors the configuration does not name: {sorted(left)[:8]}")

    def _random(self, seed: int, std: float = 0.02):
        """Weights drawn on the device, for benchmarks."""
        s, W = self.shape, self.padded_width
        g = torch.Generator(device=self.device).manual_seed(seed)
        r = lambda *d: torch.empty(*d, device=self.device, dtype=self.dtype).normal_(0.0, std, generator=g)
        full = lambda v: fit(torch.full((s.width,), v, device=self.device), W)
        norm = lambda: dict(norm_weight=full(1.0), norm_bias=full(0.1), norm_alpha=0.6)
        self.embed, self.head = (fit(r(s.vocab, s.width), s.vocab, W) for _ in range(2))
        self.final_norm, self.norms = norm(), []
        for mixer, mlp in zip(self.mixers, self.mlps):
            if isinstance(mixer, LatentAttention):
                mixer.random(self.dtype, self.device, g, std)
            else:
                mixer.load({k: r(*shape) for k, shape in mixer.shapes().items()}, self.dtype, self.device)
            if mlp is not None:
                mlp.random(self.dtype, self.device, g, std)
            self.norms.append([norm(), norm()])

    # ------------------------------------------------------------------ cache
    def allocate_caches(self, num_pages: int, page_size: int, num_slots: int):
        """One page pool per layer that holds keys of its own, None for the others."""
        self.caches = [m.allocate(num_pages, page_size, self.dtype, self.device) for m in self.mixers]

    # ------------------------------------------------------------------ forward
    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, ctx, trace: list | None = None) -> torch.Tensor:
        """Normed and scaled output rows (N, padded width) for compute_logits.  `trace`, when given, receives the
        stream after every layer."""
        s, W, N = self.shape, self.padded_width, input_ids.shape[0]
        positions = positions.to(torch.int32)
        x = torch.empty((N, W), dtype=torch.float32, device=self.device)
        # the last norm's rows leave with the logits' scale
        after = [n[0] for n in self.norms[1:]] + [dict(self.final_norm, out_scale=s.logit_scale)]
        held: list[dict] = [{} for _ in self.mixers]
        h = embed_norm(input_ids, positions, self.embed, None, x, eps=s.eps, norm_width=s.width, **self.norms[0][0])
        for i, (mixer, mlp) in enumerate(zip(self.mixers, self.mlps)):
            j = self.source[i]
            y = mixer.forward(h, self.caches[j], ctx, positions, held[j])
            if mlp is not None:
                h = residual_norm(x, y, eps=s.eps, norm_width=s.width, x_out=x, **self.norms[i][1])
                y = mlp.forward(h)
            h = residual_norm(x, y, eps=s.eps, norm_width=s.width, x_out=x, **after[i])
            if trace is not None:
                trace.append(x[:, :s.width].clone())
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.head)
