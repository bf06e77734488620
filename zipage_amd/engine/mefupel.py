"""Mefupel decoder: windowed attention whose values turn with their position, gated linear attention, and
attention over its own keys beside retention; mixer and feed-forward of a layer read one norm and join the
stream together; a run of layers may be passed several times, each pass starting from the stream, the embedding
and a learned vector.

The residual stream stays in fp32; matrix products run in the model's dtype.  All products of a layer that read
its norm are one, and so are those that write to the stream, except where a mixer's result is normed first.  The
join of all branches, what comes before a pass, and the next norm are one launch.  Every pass of a layer has its
own pages (attention) and its own states by sequence slot (recurrences).
"""
from __future__ import annotations

from dataclasses import dataclass

import torch
import torch.nn.functional as F

from zipage_amd.layers.grouped import GroupedAttention
from zipage_amd.layers.linear import ResidualLinear, fit, pad_to_multiple
from zipage_amd.layers.recurrent import LinearAttention
from zipage_amd.layers.residual import embed_norm, normed_powers, residual_norm
from zipage_amd.layers.rotary import Rotary


@dataclass(frozen=True)
class TurningMixer:
    """Attention whose values turn too."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    window: int
    rotary: Rotary
    scale: float


@dataclass(frozen=True)
class GatedMixer:
    """Linear attention with a decay per key channel."""
    heads: int
    dim: int
    vdim: int
    tau: float


@dataclass(frozen=True)
class PairMixer:
    """Attention over its own keys, with sinks (left), beside retention (right)."""
    heads: int
    kv_heads: int
    dim: int
    window: int
    rotary: Rotary
    scale: float
    memory_heads: int
    memory_dim: int
    memory_vdim: int
    memory_rotary: Rotary
    decay: tuple[float, ...]


@dataclass(frozen=True)
class MefupelLayer:
    mixer: TurningMixer | GatedMixer | PairMixer
    ff: int | None              # None: no feed-forward


@dataclass(frozen=True)
class MefupelShape:
    vocab: int
    width: int
    layers: tuple[MefupelLayer, ...]
    loop: tuple[int, int, int] | None   # layers start .. stop - 1 run this many times in a row
    eps: float

    @property
    def order(self) -> list[tuple[int, int | None]]:
        """The layers in the order they run, each with the number of the pass that it opens, if it does."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        start, stop, times = self.loop
        body = [(i, t if i == start else None) for t in range(times) for i in range(start, stop)]
        return [(i, None) for i in range(start)] + body + [(i, None) for i in range(stop, n)]

    @classmethod
    def from_config(cls, c: dict) -> "MefupelShape":
        """Reader of config.json.  A key it does not know inside a layer is refused: it would change the
        model."""
        def take(d: dict, where: str, *keys, **optional):
            extra = set(d) - set(keys) - set(optional)
            missing = set(keys) - set(d)
            if extra or missing:
                raise ValueError(f"Mefupel config, {where}: unknown {sorted(extra)}, missing {sorted(missing)}")
            return [d[k] for k in keys] + [d.get(k, v) for k, v in optional.items()]

        def rotary(d: dict, where: str, interleaved: bool = False) -> Rotary:
            base, dims = take(d, f"{where} rot", "base", "dims")
            return Rotary(float(base), dims, interleaved=interleaved)

        def attention(d: dict, where: str, interleaved: bool = False):
            dim, heads, kv_heads, mask, rot, scale, vdim = take(
                d, where, "dim", "heads", "kv_heads", "mask", "rot", "scale", "vdim")
            (size,) = take(mask, f"{where} mask", "size")
            if size < 1:
                raise ValueError(f"Mefupel config, {where}: a window of {size} tokens sees nothing")
            return heads, kv_heads, dim, vdim, size, rotary(rot, where, interleaved), float(scale)

        keys = ("layers", "loop", "norm", "vocab", "width")
        entries, loop, norm, vocab, width = take({k: v for k, v in {"loop": None, **c}.items() if k in keys}, "model", *keys)
        (eps,) = take(norm, "norm", "eps")
        if loop is not None:
            loop = tuple(take(loop, "loop", "start", "stop", "times"))
            if not 0 <= loop[0] <= loop[1] <= len(entries) or loop[2] < 1:
                raise ValueError(f"Mefupel config: loop {loop} over {len(entries)} layers")
        layers = []
        for i, e in enumerate(entries):
            mixer, kind, mlp = take(e, f"layer {i}", "mixer", "type", mlp=None)
            if kind == "attention":
                m = TurningMixer(*attention(mixer, f"layer {i} mixer", interleaved=True))
            elif kind == "gla":
                dim, heads, tau, vdim = take(mixer, f"layer {i} mixer", "dim", "heads", "tau", "vdim")
                m = GatedMixer(heads, dim, vdim, float(tau))
            elif kind == "parallel":
                left, right = take(mixer, f"layer {i} mixer", "left", "right")
                heads, kv_heads, dim, vdim, size, rot, scale = attention(left, f"layer {i} left")
                if vdim != dim:
                    raise ValueError(f"Mefupel config, layer {i} left: values of {vdim} that are keys of {dim}")
                decay, r_dim, r_heads, r_rot, r_vdim = take(right, f"layer {i} right", "decay", "dim", "heads", "rot", "vdim")
                m = PairMixer(heads, kv_heads, dim, size, rot, scale, r_heads, r_dim, r_vdim,
                              rotary(r_rot, f"layer {i} right"), tuple(float(v) for v in decay))
            else:
                raise ValueError(f"Mefupel config, layer {i}: unknown mixer {kind!r}")
            ff = None
            if mlp is not None:
                ff, mlp_kind = take(mlp, f"layer {i} mlp", "ff", "kind")
                if mlp_kind != "dense":
                    raise ValueError(f"Mefupel config, layer {i}: unknown feed-forward {mlp_kind!r}")
            layers.append(MefupelLayer(m, ff))
        return cls(vocab, width, tuple(layers), loop, float(eps))


def _rank(tensors: dict) -> int:
    """Of a low-rank product, which is that of the tensors."""
    return tensors["a1"].shape[0] if "a1" in tensors else 1


class Attention:
    """The mixer of a TurningMixer layer."""

    def __init__(self, m: TurningMixer, width: int, eps: float):
        self.attention = GroupedAttention(width, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.window, m.rotary,
                                          turn_values=True)

    def shapes(self, tensors: dict) -> dict:
        return self.attention.shapes()

    def load(self, w: dict, dtype, device, padded_width: int):
        into, out = self.attention.load(w, dtype, device, padded_width)
        return into, [out]

    def allocate(self, num_pages: int, page_size: int, num_slots: int, dtype, device):
        return self.attention.allocate(num_pages, page_size, dtype, device)

    def mix(self, proj, positions, cache, ctx, outs):
        self.attention.attend(proj, positions, cache, ctx, outs[0])


class Gated:
    """The mixer of a GatedMixer layer."""
    attention = None

    def __init__(self, m: GatedMixer, width: int, eps: float):
        self.core = LinearAttention(width, m.heads, m.dim, m.vdim, eps, q_scale=m.dim ** -0.5, tau=m.tau, weighted=True)

    def shapes(self, tensors: dict) -> dict:
        return self.core.shapes(_rank(tensors))

    def load(self, w: dict, dtype, device, padded_width: int):
        into, out = self.core.load(w, dtype, device, padded_width)
        return into, [out]

    def allocate(self, num_pages: int, page_size: int, num_slots: int, dtype, device):
        return self.core.allocate(num_slots, dtype, device)

    def mix(self, proj, positions, cache, ctx, outs):
        self.core.scan(proj, cache, ctx, outs[0])


class Pair:
    """The two mixers of a PairMixer layer.  Each has an output product of its own: the results are normed before
    they join the stream, and the half of each is in the weights of its norm."""

    def __init__(self, m: PairMixer, width: int, eps: float):
        self.attention = GroupedAttention(width, m.heads, m.kv_heads, m.dim, m.dim, m.scale, m.window, m.rotary, sinks=True,
                                          eps=eps, qk_norm=True, tied=True)
        self.memory = LinearAttention(width, m.memory_heads, m.memory_dim, m.memory_vdim, eps, k_scale=m.memory_dim ** -0.5,
                                      decay=m.decay, rotary=m.memory_rotary)
        self.width = width

    def shapes(self, tensors: dict) -> dict:
        return {**{f"left.{k}": s for k, s in self.attention.shapes().items()},
                **{f"right.{k}": s for k, s in self.memory.shapes().items()},
                "left.out": (self.width,), "right.out": (self.width,)}

    def load(self, w: dict, dtype, device, padded_width: int):
        side = lambda s: {k[len(s) + 1:]: t for k, t in w.items() if k.startswith(s + ".")}
        parts = [m.load(side(s), dtype, device, padded_width) for m, s in ((self.attention, "left"), (self.memory, "right"))]
        self.out_norms = [0.5 * fit(w[k], padded_width).to(device=device, dtype=torch.float32) for k in ("left.out", "right.out")]
        return torch.cat([p[0] for p in parts]), [p[1] for p in parts]

    def allocate(self, num_pages: int, page_size: int, num_slots: int, dtype, device):
        return self.attention.allocate(num_pages, page_size, dtype, device), self.memory.allocate(num_slots, dtype, device)

    def mix(self, proj, positions, cache, ctx, outs):
        cut = self.attention.columns
        self.attention.attend(proj[:, :cut], positions, cache[0], ctx, outs[0])
        self.memory.scan(proj[:, cut:], cache[1], ctx, outs[1])


KINDS = {TurningMixer: Attention, GatedMixer: Gated, PairMixer: Pair}


class Layer:
    """A mixer beside a feed-forward of normed powers.  Their input products are one; `outs` are the output
    products, each with the weights of the norm on its result, or None.  Where the mixer's result joins as it is,
    it shares the feed-forward's output product."""

    def __init__(self, l: MefupelLayer, width: int, padded_width: int, eps: float):
        self.mixer, self.ff, self.eps = KINDS[type(l.mixer)](l.mixer, width, eps), l.ff, eps
        self.width, self.padded_width = width, padded_width

    def shapes(self, mix: dict) -> dict:
        W, ff = self.width, self.ff
        return {**{f"mix.{k}": s for k, s in self.mixer.shapes(mix).items()},
                **({} if ff is None else {"mlp.up": (ff, W), "mlp.down": (W, ff), "mlp.act": (4,)})}

    def load(self, w: dict, dtype, device):
        W = self.padded_width
        put = lambda t: t.to(device=device, dtype=dtype).contiguous()
        into, outs = self.mixer.load({k[4:]: t for k, t in w.items() if k.startswith("mix.")}, dtype, device, W)
        self.mixed = into.shape[0]              # columns of the mixer's projections
        self.spans = [o.shape[1] for o in outs]
        self.norms = list(getattr(self.mixer, "out_norms", [None]))
        if self.ff is not None:
            shared = self.norms[0] is None
            self.ff_p = pad_to_multiple(self.ff + shared * self.spans[0], 32) - shared * self.spans[0]
            into = torch.cat([into, fit(w["mlp.up"], self.ff_p, W)])
            down = fit(w["mlp.down"], W, self.ff_p)
            self.act = tuple(w["mlp.act"].double().tolist())
            if shared:
                outs = [torch.cat([outs[0], down], dim=1)]
            else:
                outs.append(down)
                self.norms.append(None)
                self.spans.append(0)
        self.into, self.outs = put(into), [ResidualLinear(put(o)) for o in outs]

    def forward(self, h: torch.Tensor, positions: torch.Tensor, cache, ctx) -> list:
        """The branches that join the stream, with the weights of their norms."""
        proj = F.linear(h, self.into)
        rows = [torch.empty((h.shape[0], o.w.shape[1]), dtype=h.dtype, device=h.device) for o in self.outs]
        self.mixer.mix(proj[:, :self.mixed], positions, cache, ctx, [r[:, :n] for r, n in zip(rows, self.spans)])
        if self.ff is not None:
            normed_powers(proj[:, self.mixed:], self.act, self.eps, self.ff, rows[-1][:, self.spans[-1]:])
        return [(o.forward(r), n) for o, r, n in zip(self.outs, rows, self.norms)]


class Mefupel:
    # what the engine asks a model: no KV compression, steps that hold portions of prompts beside decoded
    # tokens, and states that only running a sequence's tokens can build
    compressible = False
    portions = True
    recurrent = True

    def __init__(self, shape: MefupelShape, device, dtype=torch.bfloat16, seed: int = 0,
                 weights: dict[str, torch.Tensor] | None = None):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"Mefupel runs in bfloat16 or float32, not {dtype}")
        self.shape, self.device, self.dtype = shape, torch.device(device), dtype
        self.padded_width = pad_to_multiple(shape.width, 32)
        self.vocab = shape.vocab
        self.layers = [Layer(l, shape.width, self.padded_width, shape.eps) for l in shape.layers]
        attention = [l.mixer.attention for l in self.layers if l.mixer.attention is not None]
        self.sights = sorted({a.sight for a in attention})
        # the furthest a token looks back, and the shortest portion attended as a run
        self.lookback = max(self.sights, default=1)
        self.run_min = 16 if dtype == torch.bfloat16 and all(a.can_run for a in attention) else None
        self.caches: list = []
        if weights is None:
            self._random(seed)
        else:
            self._load(weights)
        # before a pass but the first the embedding joins the stream
        self.again = torch.ones(2, device=self.device)

    # ------------------------------------------------------------------ weights
    def _load(self, tensors: dict[str, torch.Tensor]):
        """Tensor names: embed, head, final.norm, loop.step and, per layer i, l<i>.norm1, l<i>.mix.* and
        l<i>.mlp.*."""
        s, W, left = self.shape, self.padded_width, dict(tensors)

        def get(name, *shape):
            if name not in left:
                raise KeyError(f"the model folder has no tensor {name}")
            t = left.pop(name)
            if tuple(t.shape) != shape:
                raise ValueError(f"tensor {name} has shape {tuple(t.shape)}, the configuration says {shape}")
            return t

        put = lambda t: t.to(device=self.device, dtype=self.dtype).contiguous()
        rows = lambda t: fit(t, *t.shape[:-1], W).to(device=self.device, dtype=torch.float32).contiguous()
        self.embed = put(fit(get("embed", s.vocab, s.width), s.vocab, W))
        self.head = put(fit(get("head", s.vocab, s.width), s.vocab, W))
        self.final_norm = rows(get("final.norm", s.width))
        self.step = None if s.loop is None else rows(get("loop.step", s.loop[2], s.width))
        self.norms = []
        for i, layer in enumerate(self.layers):
            pre = f"l{i}."
            mix = {k[len(pre) + 4:]: t for k, t in tensors.items() if k.startswith(pre + "mix.")}
            self.norms.append(rows(get(pre + "norm1", s.width)))
            layer.load({k: get(pre + k, *shape) for k, shape in layer.shapes(mix).items()}, self.dtype, self.device)
        if left:
            raise ValueError(f"tensors the configuration does not name: {sorted(left)[:8]}")

    def _random(self, seed: int, std: float = 0.02):
        """Weights drawn on the device, for benchmarks."""
        s, W = self.shape, self.padded_width
        g = torch.Generator(device=self.device).manual_seed(seed)
        r = lambda *d: torch.empty(*d, device=self.device, dtype=self.dtype).normal_(0.0, std, generator=g)
        zeros = lambda *d: torch.zeros(*d, W, device=self.device)
        self.embed, self.head = (fit(r(s.vocab, s.width), s.vocab, W) for _ in range(2))
        self.final_norm, self.norms = zeros(), [zeros() for _ in self.layers]
        self.step = None if s.loop is None else zeros(s.loop[2])
        for layer in self.layers:
            layer.load({k: r(*shape) for k, shape in layer.shapes({"a1": torch.empty(16, 0)}).items()}, self.dtype, self.device)

    # ------------------------------------------------------------------ cache
    def allocate_caches(self, num_pages: int, page_size: int, num_slots: int):
        """One entry per pass of a layer: a page pool for attention, states by sequence slot for
        recurrences."""
        self.caches = [self.layers[i].mixer.allocate(num_pages, page_size, num_slots, self.dtype, self.device)
                       for i, _ in self.shape.order]

    # ------------------------------------------------------------------ forward
    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, ctx, trace: list | None = None) -> torch.Tensor:
        """Normed output rows (N, padded width) for compute_logits.  `trace`, when given, receives the stream
        after every layer run."""
        s, W, N = self.shape, self.padded_width, input_ids.shape[0]
        positions = positions.to(torch.int32)
        order = s.order
        new = lambda *d: torch.empty((*d, N, W), dtype=torch.float32, device=self.device)
        x, embedded = new(), new(1) if s.loop is not None and s.loop[2] > 1 else None
        norms = [self.norms[i] for i, _ in order] + [self.final_norm]

        def before(run: int) -> dict:
            """What joins the stream ahead of a layer run, with the norm that the layer reads."""
            opened = order[run][1] if run < len(order) else None
            return dict(norm_weight=norms[run], weight_offset=1.0, eps=s.eps, norm_width=s.width,
                        **({} if opened is None else dict(shift=self.step[opened])),
                        **({} if not opened else dict(history=embedded, mix=self.again)))

        h = embed_norm(input_ids, positions, self.embed, None, x, result=None if embedded is None else embedded[0], **before(0))
        for run, (i, _) in enumerate(order):
            (y, w), *more = self.layers[i].forward(h, positions, self.caches[run], ctx)
            after = None if trace is None else new()
            h = residual_norm(x, y, y_weight=w, more=tuple(more), x_out=x, result=after, **before(run + 1))
            if trace is not None:
                trace.append(after[:, :s.width])
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.head)
