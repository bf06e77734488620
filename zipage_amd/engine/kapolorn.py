"""Kapolorn decoder: layers that mix tokens either with chunked sink attention beside a matrix memory or
with a gated delta rule, mixtures of experts, norms before and after every sublayer, and a run of layers
that may be passed several times with the same weights.

The residual stream stays in fp32; matrix products run in the model's dtype.  Mixers that read the same
input share one input and one output product.  Every pass of a layer has its own pages (attention) and its
own states by sequence slot (recurrences).
"""
from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn.functional as F

from zipage_amd.layers.grouped import GroupedAttention
from zipage_amd.layers.linear import ResidualLinear, fit, pad_to_multiple
from zipage_amd.layers.moe import Experts
from zipage_amd.layers.recurrent import ChannelDelta, MatrixMemory
from zipage_amd.layers.residual import embed_norm, residual_norm, softcap
from zipage_amd.layers.rotary import Rotary
from zipage_amd.sight import Chunk


@dataclass(frozen=True)
class ParallelMixer:
    """Chunked attention with sinks (left) beside a matrix memory (right)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int                  # tokens see their own block of this many positions
    rot_base: float
    rot_dims: int
    left_scale: float
    memory_heads: int
    memory_dim: int
    memory_vdim: int
    gate_cap: float
    right_scale: float


@dataclass(frozen=True)
class DeltaMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int


@dataclass(frozen=True)
class ExpertsShape:
    experts: int
    top: int
    groups: int
    keep: int
    ff: int
    limit: float
    shared_ff: int
    shared_limit: float


@dataclass(frozen=True)
class KapolornLayer:
    mixer: ParallelMixer | DeltaMixer
    mlp: ExpertsShape | None


@dataclass(frozen=True)
class KapolornShape:
    vocab: int
    width: int
    layers: tuple[KapolornLayer, ...]
    loop: tuple[int, int, int]          # layers start .. stop - 1 run this many times in a row
    eps: float
    embed_scale: float
    logit_softcap: float

    @property
    def order(self) -> list[int]:
        """Layer indices in the order they run."""
        start, stop, times = self.loop
        return [*range(start), *list(range(start, stop)) * times, *range(stop, len(self.layers))]

    @classmethod
    def from_config(cls, c: dict) -> "KapolornShape":
        """Reader of config.json.  A key it does not know inside a layer is refused: it would change the
        model."""
        def take(d: dict, where: str, *keys):
            extra = set(d) - set(keys)
            missing = set(keys) - set(d)
            if extra or missing:
                raise ValueError(f"Kapolorn config, {where}: unknown {sorted(extra)}, missing {sorted(missing)}")
            return [d[k] for k in keys]

        keys = ("embedding", "layers", "logit_softcap", "loop", "norm", "vocab", "width")
        embedding, entries, cap, loop, norm, vocab, width = take(
            {k: v for k, v in {"loop": None, **c}.items() if k in keys}, "model", *keys)
        (embed_scale,) = take(embedding, "embedding", "scale")
        (eps,) = take(norm, "norm", "eps")
        loop = tuple(take(loop, "loop", "start", "stop", "times")) if loop is not None else (0, 0, 1)
        if not 0 <= loop[0] <= loop[1] <= len(entries) or loop[2] < 1:
            raise ValueError(f"Kapolorn config: loop {loop} over {len(entries)} layers")
        layers = []
        for i, e in enumerate(entries):
            mixer, mlp, kind = take(e, f"layer {i}", "mixer", "mlp", "type")
            if kind == "parallel":
                left, left_scale, right, right_scale = take(mixer, f"layer {i} mixer", "left", "left_scale", "right",
                                                            "right_scale")
                dim, heads, kv_heads, mask, rot, scale, vdim = take(
                    left, f"layer {i} left", "dim", "heads", "kv_heads", "mask", "rot", "scale", "vdim")
                (size,) = take(mask, f"layer {i} mask", "size")
                base, dims = take(rot, f"layer {i} rot", "base", "dims")
                if size < 1:
                    raise ValueError(f"Kapolorn config, layer {i}: a chunk of {size} tokens")
                r_dim, gate_cap, r_heads, r_vdim = take(right, f"layer {i} right", "dim", "gate_cap", "heads", "vdim")
                m = ParallelMixer(heads, kv_heads, dim, vdim, float(scale), size, float(base), dims, float(left_scale),
                                  r_heads, r_dim, r_vdim, float(gate_cap), float(right_scale))
            elif kind == "channel_delta":
                conv, dim, heads, kv_heads, vdim = take(mixer, f"layer {i} mixer", "conv", "dim", "heads", "kv_heads",
                                                        "vdim")
                m = DeltaMixer(heads, kv_heads, dim, vdim, conv)
            else:
                raise ValueError(f"Kapolorn config, layer {i}: unknown mixer {kind!r}")
            f = None
            if mlp is not None:
                expert, mlp_kind, router, shared = take(mlp, f"layer {i} mlp", "expert", "kind", "router", "shared")
                if mlp_kind != "moe":
                    raise ValueError(f"Kapolorn config, layer {i}: unknown feed-forward {mlp_kind!r}")
                ff, limit = take(expert, f"layer {i} expert", "ff", "limit")
                s_ff, s_limit = take(shared, f"layer {i} shared", "ff", "limit")
                experts, groups, top = take(router, f"layer {i} router", "experts", "groups", "top")
                count, keep = take(groups, f"layer {i} groups", "count", "keep")
                f = ExpertsShape(experts, top, count, keep, ff, float(limit), s_ff, float(s_limit))
            layers.append(KapolornLayer(m, f))
        return cls(vocab, width, tuple(layers), loop, float(eps), float(embed_scale), float(cap))


class Parallel:
    """The two mixers of a ParallelMixer layer on one input and one output product; their scales ride on
    the rows that enter the latter."""

    def __init__(self, m: ParallelMixer, width: int, eps: float):
        self.left = GroupedAttention(width, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, Chunk(m.chunk),
                                     Rotary(m.rot_base, m.rot_dims), sinks=True, out_scale=m.left_scale)
        self.right = MatrixMemory(width, m.memory_heads, m.memory_dim, m.memory_vdim, m.gate_cap, eps,
                                  out_scale=m.right_scale)
        self.out_columns = self.left.out_columns + self.right.out_columns
        self.sight = self.left.sight

    def shapes(self, tensors: dict) -> dict:
        return {**{f"left.{k}": s for k, s in self.left.shapes().items()},
                **{f"right.{k}": s for k, s in self.right.shapes().items()}}

    def load(self, w: dict, dtype, device, padded_width: int):
        side = lambda s: {k[len(s) + 1:]: t for k, t in w.items() if k.startswith(s + ".")}
        parts = [m.load(side(s), dtype, device, padded_width) for m, s in ((self.left, "left"), (self.right, "right"))]
        return torch.cat([p[0] for p in parts]), torch.cat([p[1] for p in parts], dim=1)

    def allocate(self, num_pages: int, page_size: int, num_slots: int, dtype, device):
        return self.left.allocate(num_pages, page_size, dtype, device), self.right.allocate(num_slots, dtype, device)

    def mix(self, h, proj, positions, cache, ctx, out):
        cut, edge = self.left.columns, self.left.out_columns
        self.left.attend(proj[:, :cut], positions, cache[0], ctx, out[:, :edge])
        self.right.scan(h, proj[:, cut:], cache[1], ctx, out[:, edge:])


class Delta:
    """The mixer of a DeltaMixer layer."""
    sight = None

    def __init__(self, m: DeltaMixer, width: int, eps: float):
        self.core = ChannelDelta(width, m.heads, m.kv_heads, m.dim, m.vdim, m.taps, eps)
        self.out_columns = self.core.out_columns

    def shapes(self, tensors: dict) -> dict:
        """The ranks of the low-rank products are those of the tensors."""
        rank = lambda k: tensors[k].shape[0] if k in tensors else 1
        return self.core.shapes(rank("a1"), rank("g1"))

    def load(self, w: dict, dtype, device, padded_width: int):
        return self.core.load(w, dtype, device, padded_width)

    def allocate(self, num_pages: int, page_size: int, num_slots: int, dtype, device):
        return self.core.allocate(num_slots, dtype, device)

    def mix(self, h, proj, positions, cache, ctx, out):
        self.core.scan(proj, cache, ctx, out)


class Kapolorn:
    # what the engine asks a model: no KV compression, steps that hold portions of prompts beside decoded
    # tokens, and states that only running a sequence's tokens can build
    compressible = False
    portions = True
    recurrent = True

    def __init__(self, shape: KapolornShape, device, dtype=torch.bfloat16, seed: int = 0,
                 weights: dict[str, torch.Tensor] | None = None):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Kapolorn runs in bfloat16 or float32, not {dtype}")
        self.shape, self.device, self.dtype = shape, torch.device(device), dtype
        self.padded_width = pad_to_multiple(shape.width, 32)
        self.vocab = shape.vocab
        kinds = {ParallelMixer: Parallel, DeltaMixer: Delta}
        self.mixers = [kinds[type(l.mixer)](l.mixer, shape.width, shape.eps) for l in shape.layers]
        self.mlps = [None if l.mlp is None else
                     Experts(shape.width, l.mlp.experts, l.mlp.top, l.mlp.ff, l.mlp.limit, l.mlp.groups, l.mlp.keep,
                             l.mlp.shared_ff, l.mlp.shared_limit) for l in shape.layers]
        attention = [m.left for m in self.mixers if isinstance(m, Parallel)]
        self.sights = sorted({a.sight for a in attention}, key=lambda s: s.size)
        # the furthest a token looks back, and the shortest portion attended as a run
        self.lookback = max((s.size for s in self.sights), default=1)
        self.run_min = 16 if dtype == torch.bfloat16 and all(a.can_run for a in attention) else None
        self.caches: list = []
        if weights is None:
            self._random(seed)
        else:
            self._load(weights)

    # ------------------------------------------------------------------ weights
    def _load(self, tensors: dict[str, torch.Tensor]):
        """Tensor names: embed, final.norm and, per layer i, l<i>.norm1 / norm1b / norm2 / norm2b, l<i>.mix.*
        and l<i>.mlp.*."""
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
        self.embed = put(fit(get("embed", s.vocab, s.width), s.vocab, W))
        self.final_norm = vec("final.norm")
        self.layers = []
        for i, (mixer, mlp) in enumerate(zip(self.mixers, self.mlps)):
            pre = f"l{i}."
            own = {k[len(pre) + 4:]: t for k, t in tensors.items() if k.startswith(pre + "mix.")}
            w = {k: get(f"{pre}mix.{k}", *shape) for k, shape in mixer.shapes(own).items()}
            into, out = mixer.load(w, self.dtype, self.device, W)
            p = dict(norm1=vec(pre + "norm1"), norm1b=vec(pre + "norm1b"), into=put(into), out=ResidualLinear(put(out)))
            if mlp is not None:
                p.update(norm2=vec(pre + "norm2"), norm2b=vec(pre + "norm2b"))
                mlp.load({k: get(f"{pre}mlp.{k}", *shape) for k, shape in mlp.shapes().items()}, self.dtype,
                         self.device)
            else:
                for k in ("norm2", "norm2b"):         # without a feed-forward nothing reads them
                    left.pop(pre + k, None)
            self.layers.append(p)
        if left:
            raise ValueError(f"tensors the configuration does not name: {sorted(left)[:8]}")

    def _random(self, seed: int, std: float = 0.02):
        """Weights drawn on the device, for benchmarks."""
        s, W = self.shape, self.padded_width
        g = torch.Generator(device=self.device).manual_seed(seed)
        r = lambda *d: torch.empty(*d, device=self.device, dtype=self.dtype).normal_(0.0, std, generator=g)
        ones = lambda: torch.ones(W, device=self.device)
        self.embed, self.final_norm = fit(r(s.vocab, s.width), s.vocab, W), ones()
        self.layers = []
        for mixer, mlp in zip(self.mixers, self.mlps):
            ranks = {"a1": torch.empty(128, 0), "g1": torch.empty(128, 0)}
            into, out = mixer.load({k: r(*shape).cpu() for k, shape in mixer.shapes(ranks).items()}, self.dtype,
                                   self.device, W)
            put = lambda t: t.to(self.device).contiguous()
            p = dict(norm1=ones(), norm1b=ones(), into=put(into), out=ResidualLinear(put(out)))
            if mlp is not None:
                p.update(norm2=ones(), norm2b=ones())
                mlp.random(self.dtype, self.device, g, std)
            self.layers.append(p)

    # ------------------------------------------------------------------ cache
    def allocate_caches(self, num_pages: int, page_size: int, num_slots: int):
        """One entry per pass of a layer: a page pool for attention, states by sequence slot for
        recurrences."""
        self.caches = [self.mixers[i].allocate(num_pages, page_size, num_slots, self.dtype, self.device)
                       for i in self.shape.order]

    # ------------------------------------------------------------------ forward
    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, ctx, trace: list | None = None) -> torch.Tensor:
        """Normed output rows (N, padded width) for compute_logits.  `trace`, when given, receives the stream
        after every layer run."""
        s, W, N = self.shape, self.padded_width, input_ids.shape[0]
        positions = positions.to(torch.int32)
        order = s.order
        x = torch.empty((N, W), dtype=torch.float32, device=self.device)
        norms = [self.layers[i]["norm1"] for i in order] + [self.final_norm]
        h = embed_norm(input_ids, positions, self.embed, None, x, norms[0], s.eps, s.width, embed_scale=s.embed_scale)
        for run, i in enumerate(order):
            p, mixer, mlp = self.layers[i], self.mixers[i], self.mlps[i]
            mixed = torch.empty((N, mixer.out_columns), dtype=self.dtype, device=self.device)
            mixer.mix(h, F.linear(h, p["into"]), positions, self.caches[run], ctx, mixed)
            y, w = p["out"].forward(mixed), p["norm1b"]
            if mlp is not None:
                h = residual_norm(x, y, p["norm2"], s.eps, s.width, x_out=x, y_weight=w)
                y, w = mlp.forward(h), p["norm2b"]
            h = residual_norm(x, y, norms[run + 1], s.eps, s.width, x_out=x, y_weight=w)
            if trace is not None:
                trace.append(x[:, :s.width].clone())
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """fp32 logits under the soft cap."""
        return softcap(F.linear(hidden, self.embed), self.shape.logit_softcap)
