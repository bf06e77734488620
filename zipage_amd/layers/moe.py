"""Mixture of experts: routing and the expert products without a host decision, so that a step of any
routing replays the same graph."""
from __future__ import annotations

import torch

from zipage_amd import _lib

from .linear import fit, pad_to_multiple


def small_linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x (N, K), w (M, K) -> (N, M) in fp32, for products with few outputs."""
    N, K = x.shape
    assert x.stride(1) == 1 and w.is_contiguous() and w.dtype == x.dtype and w.shape[1] == K
    out = torch.empty((N, w.shape[0]), dtype=torch.float32, device=x.device)
    _lib.call_models("zp_small_linear", _lib.dev_ptr(x), _lib.dev_ptr(w), _lib.dev_ptr(out), N, K, w.shape[0],
                     x.stride(0), _lib.dtype_tag(x), _lib.stream_ptr(x))
    return out


def moe_select(logits: torch.Tensor, experts: int, top: int, groups: int = 1, keep: int = 1,
               score: int = _lib.SCORE_SOFTMAX):
    """Softmax over the first `experts` logits of each row (fp32), or their sigmoids, the `keep` groups with the
    best single score, the `top` best experts of those: (ids, scores, cleared counters for the plan)."""
    N = logits.shape[0]
    assert logits.dtype == torch.float32 and logits.stride(1) == 1
    dev = logits.device
    ids = torch.empty((N, top), dtype=torch.int32, device=dev)
    weights = torch.empty((N, top), dtype=torch.float32, device=dev)
    counts = torch.empty(experts + 1, dtype=torch.int32, device=dev)
    _lib.call_models("zp_moe_select", _lib.dev_ptr(logits), _lib.dev_ptr(ids), _lib.dev_ptr(weights),
                     _lib.dev_ptr(counts), N, experts, top, groups, keep, score, logits.stride(0),
                     _lib.stream_ptr(logits))
    return ids, weights, counts


class Plan:
    """Assignments (token * slots + slot) in the order of their experts, and row tiles over them."""

    def __init__(self, ids: torch.Tensor, counts: torch.Tensor, experts: int, shared: bool, dtype):
        N, top = ids.shape
        lib, dev = _lib.load_models("moe"), ids.device
        self.n, self.experts, self.top, self.shared, self.slots = N, experts, top, int(shared), top + int(shared)
        self.rows = lib.zp_moe_tile_rows(N, experts, top, _lib._DTYPES[dtype])
        self.max_tiles = lib.zp_moe_max_tiles(N, experts, top, self.shared, self.rows)
        self.sorted = torch.empty(N * self.slots, dtype=torch.int32, device=dev)
        self.tiles = torch.empty((self.max_tiles, 4), dtype=torch.int32, device=dev)
        self.ntiles = torch.empty(1, dtype=torch.int32, device=dev)
        size = lib.zp_moe_plan_workspace(N, experts, top)
        ws = torch.empty(size, dtype=torch.uint8, device=dev)
        _lib.call_models("zp_moe_plan", _lib.dev_ptr(ids), _lib.dev_ptr(counts), _lib.dev_ptr(self.sorted),
                         _lib.dev_ptr(self.tiles), _lib.dev_ptr(self.ntiles), N, experts, top, self.shared, self.rows,
                         self.max_tiles, _lib.dev_ptr(ws), size, _lib.stream_ptr(ids))


def tile_order(w: torch.Tensor) -> torch.Tensor:
    """(..., out, in) in the order the expert kernels read: [out / 16][in / step][16-byte piece][row]."""
    piece = 16 // w.element_size()
    *lead, out, inn = w.shape
    t = w.reshape(*lead, out // 16, 16, inn // (4 * piece), 4, piece)
    n = len(lead)
    return t.permute(*range(n), n, n + 2, n + 3, n + 1, n + 4).contiguous()


def gate_up_order(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """16 rows of the gate, then the 16 of `up` that belong to them, and so on."""
    *lead, m, k = gate.shape
    pair = torch.stack([gate.reshape(*lead, m // 16, 16, k), up.reshape(*lead, m // 16, 16, k)], dim=-3)
    return pair.reshape(*lead, 2 * m, k)


class Experts:
    """Gated experts of which every token uses `top`, chosen among its best `keep` of `groups` groups, weighted
    with their scores as they are; and, if `shared_ff` is given, one more for every token.  Scores are a
    softmax or sigmoids.  `act` "clamped": g = min(gate, limit), u = clamp(up, +-limit), w g sigmoid(1.702 g)
    (u + 1) with the weight w on the output; "silu": g sigmoid(g) u with the weight on the expert's input."""

    def __init__(self, width: int, experts: int, top: int, ff: int, limit: float, groups: int = 1, keep: int = 1,
                 shared_ff: int | None = None, shared_limit: float = 0.0, score: str = "softmax",
                 act: str = "clamped"):
        if experts % groups or not 0 < keep <= groups or not 0 < top <= experts // groups * keep:
            raise ValueError(f"{top} of {experts} experts in {keep} of {groups} groups")
        self.width, self.experts, self.top, self.ff, self.limit = width, experts, top, ff, limit
        self.groups, self.keep, self.shared_ff, self.shared_limit = groups, keep, shared_ff, shared_limit
        self.score = {"softmax": _lib.SCORE_SOFTMAX, "sigmoid": _lib.SCORE_SIGMOID}[score]
        self.act = {"clamped": _lib.GATE_CLAMPED, "silu": _lib.GATE_SILU}[act]
        self.ff_p = pad_to_multiple(ff, 32)
        self.shared_p = pad_to_multiple(shared_ff, 32) if shared_ff else 0
        self.width_p = pad_to_multiple(width, 32)

    def shapes(self) -> dict:
        def one(p, ff):
            return {f"{p}.gate": (ff, self.width), f"{p}.up": (ff, self.width), f"{p}.down": (self.width, ff)}
        out = {"router": (self.experts, self.width)}
        for e in range(self.experts):
            out.update(one(f"e{e}", self.ff))
        if self.shared_ff:
            out.update(one("shared", self.shared_ff))
        return out

    def load(self, w: dict, dtype, device):
        E, W = self.experts, self.width_p
        put = lambda t: t.to(device=device, dtype=dtype)
        self.router = fit(put(w["router"]), pad_to_multiple(E, 4), W)

        def pack(names, ff_p):
            gate, up = (torch.stack([fit(put(w[f"{p}.{k}"]), ff_p, W) for p in names]) for k in ("gate", "up"))
            down = torch.stack([fit(put(w[f"{p}.down"]), W, ff_p) for p in names])
            return tile_order(gate_up_order(gate, up)), tile_order(down)
        self.gate_up, self.down = pack([f"e{e}" for e in range(E)], self.ff_p)
        self.shared_gate_up = self.shared_down = None
        if self.shared_ff:
            self.shared_gate_up, self.shared_down = pack(["shared"], self.shared_p)

    def random(self, dtype, device, generator, std: float = 0.02):
        """Random weights straight into their final layout."""
        r = lambda *s: torch.empty(*s, dtype=dtype, device=device).normal_(0.0, std, generator=generator)
        E, W = self.experts, self.width_p
        assert self.width == W and self.ff == self.ff_p and (self.shared_ff or 0) == self.shared_p
        self.router = fit(r(E, W), pad_to_multiple(E, 4), W)
        self.gate_up, self.down = r(E, 2 * self.ff_p * W), r(E, W * self.ff_p)
        self.shared_gate_up = self.shared_down = None
        if self.shared_ff:
            self.shared_gate_up, self.shared_down = r(2 * self.shared_p * W), r(W * self.shared_p)

    # ------------------------------------------------------------------ forward
    def route(self, h: torch.Tensor):
        return moe_select(small_linear(h, self.router), self.experts, self.top, self.groups, self.keep, self.score)

    def gate_up_rows(self, h: torch.Tensor, plan: Plan, weights: torch.Tensor) -> torch.Tensor:
        """Activations by position in plan.sorted, times the assignment's weight."""
        assert h.stride(1) == 1 and h.shape == (plan.n, self.width_p)
        ff = max(self.ff_p, self.shared_p)
        act = torch.empty((plan.n * plan.slots, ff), dtype=h.dtype, device=h.device)
        _lib.call_models("zp_moe_gate_up", _lib.dev_ptr(h), _lib.dev_ptr(self.gate_up), _lib.dev_ptr(self.shared_gate_up),
                         _lib.dev_ptr(act), _lib.dev_ptr(plan.sorted), _lib.dev_ptr(plan.tiles), _lib.dev_ptr(plan.ntiles),
                         _lib.dev_ptr(weights), plan.n, self.experts, self.top, plan.shared, plan.rows, plan.max_tiles,
                         self.width_p, self.ff_p, self.shared_p, h.stride(0), ff, self.act, self.limit, self.shared_limit,
                         _lib.dtype_tag(h), _lib.stream_ptr(h))
        return act

    def down_planes(self, act: torch.Tensor, plan: Plan) -> torch.Tensor:
        """(slots, N, width) parts of the output, to be added up."""
        out = torch.empty((plan.slots, plan.n, self.width_p), dtype=act.dtype, device=act.device)
        _lib.call_models("zp_moe_down", _lib.dev_ptr(act), _lib.dev_ptr(self.down), _lib.dev_ptr(self.shared_down),
                         _lib.dev_ptr(out), _lib.dev_ptr(plan.sorted), _lib.dev_ptr(plan.tiles), _lib.dev_ptr(plan.ntiles),
                         plan.n, self.experts, self.top, plan.shared, plan.rows, plan.max_tiles, self.ff_p, self.shared_p,
                         self.width_p, act.stride(0), self.width_p, _lib.dtype_tag(act), _lib.stream_ptr(act))
        return out

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        """h (N, padded width) -> planes (slots, N, padded width) that `residual_norm` adds up in fp32."""
        ids, weights, counts = self.route(h)
        plan = Plan(ids, counts, self.experts, self.shared_ff is not None, h.dtype)
        return self.down_planes(self.gate_up_rows(h, plan, weights), plan)
