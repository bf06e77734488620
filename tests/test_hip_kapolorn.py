"""Kapolorn on the GPU: every mechanism alone, the model against the oracle in every way a sequence can be
cut and batched, and generation through the engine."""
import io
import json
import types

import pytest
import torch

from oracle import kapolorn_oracle as O
from tests import kapolorn_cases as C

pytestmark = pytest.mark.gpu
BF16, F32 = torch.bfloat16, torch.float32
DTYPES = [BF16, F32]
ids = lambda v: str(v).replace("torch.", "")


def _rand(dev, dtype, *shape, seed=0, std=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * std).to(dtype).to(dev)


def _close(got, want, dtype, factor=1.0):
    """Within a few roundings of `dtype`, relative to each row's largest value."""
    got, want = got.double().cpu(), want.double().cpu()
    eps = {BF16: 2.0 ** -8, F32: 2.0 ** -20}[dtype]
    top = want.abs().amax(dim=-1, keepdim=True).clamp_min(1e-30)
    worst = float(((got - want).abs() / top).max())
    assert worst <= factor * eps, worst


# ------------------------------------------------------------------ row steps
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,width,norm_width", [(1, 96, 76), (3, 512, 512), (17, 1024, 1000), (2, 8192, 8192)])
@pytest.mark.parametrize("planes", [1, 2, 5, 9])
def test_residual_norm_of_a_normed_branch(dev, dtype, n, width, norm_width, planes):
    from zipage_amd.layers import residual_norm
    x, y = _rand(dev, F32, n, width, seed=1), _rand(dev, dtype, planes, n, width, seed=2)
    x[:, norm_width:] = 0
    y[..., norm_width:] = 0
    w, b = _rand(dev, F32, width, seed=3), _rand(dev, F32, width, seed=4)
    c = slice(0, norm_width)
    branch = O.norm(y.double().sum(0)[:, c], b.double()[c], 1e-3)
    want = x.double()[:, c] + branch
    after = torch.empty_like(x)
    h = residual_norm(x, y, w, 1e-3, norm_width, x_out=after, y_weight=b)
    _close(after[:, c], want, F32)
    _close(h[:, c], O.norm(want, w.double()[c], 1e-3), dtype)
    assert not h[:, norm_width:].any() and not after[:, norm_width:].any()
    inplace = x.clone()
    assert residual_norm(inplace, y, None, 1e-3, norm_width, x_out=inplace, y_weight=b) is None
    assert torch.equal(inplace, after)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_embedding_scale_and_softcap(dev, dtype):
    from zipage_amd.layers import embed_norm, softcap
    embed, w = _rand(dev, dtype, 11, 96, seed=1), _rand(dev, F32, 96, seed=3)
    tok, at = torch.tensor([3, 10, 0, 7], device=dev), torch.zeros(4, dtype=torch.int32, device=dev)
    x = torch.empty(4, 96, device=dev)
    h = embed_norm(tok, at, embed, None, x, w, 1e-2, 96, embed_scale=0.3)
    _close(x, embed.double()[tok] * 0.3, F32)
    _close(h, O.norm(embed.double()[tok] * 0.3, w.double(), 1e-2), dtype)
    for n, v in ((1, 7), (3, 131), (5, 4096)):
        z = _rand(dev, dtype, n, v, seed=5, std=12.0)
        got = softcap(z, 7.5)
        assert got.dtype == F32
        _close(got, 7.5 * torch.tanh(z.double() / 7.5), F32)


# ------------------------------------------------------------------ attention
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,G,D,V,rot", [(4, 2, 32, 48, 32), (6, 3, 32, 16, 10), (5, 1, 96, 128, 64), (2, 2, 64, 32, 2),
                                         (3, 3, 32, 32, 0), (8, 2, 256, 256, 256)])
def test_rotary_store(dev, dtype, H, G, D, V, rot):
    from zipage_amd.layers import rotary_store
    n, pages, BS = 9, 3, 16
    cols = H * D + G * (D + V)
    wide = _rand(dev, dtype, n, cols + 24, seed=1)              # the projections of another mixer follow
    pos = torch.tensor([0, 1, 7, 100, 4095, 3, 50000, 12, 13], dtype=torch.int32, device=dev)
    slots = torch.tensor([5, -1, 47, 0, 12, 13, 48, 8, 7], dtype=torch.int32, device=dev)     # 48: past the end
    cache = torch.full((pages, BS, G * (D + V)), 7.0, dtype=dtype, device=dev)
    f = torch.tensor([300.0 ** (-2 * i / max(rot, 1)) for i in range(rot // 2)], device=dev)
    q, kv = rotary_store(wide[:, :cols], pos, f, H, G, D, V, cache, slots, return_kv=True)
    x = wide[:, :cols].double().cpu()
    angle = (pos.cpu().float()[:, None] * f.cpu()).double()[:, None]           # positions and angles are fp32

    def turn(t):
        u, v = t[..., :rot // 2], t[..., rot // 2:rot]
        return torch.cat([u * angle.cos() - v * angle.sin(), v * angle.cos() + u * angle.sin(), t[..., rot:]], -1)
    if rot:
        small = torch.arange(9)
        keep, angle = angle, (small[:, None] * f.cpu().double())[:, None]
        assert torch.allclose(turn(x[:, :H * D].view(n, H, D)), O.rotate(x[:, :H * D].view(n, H, D), small, 300.0, rot), atol=1e-5)
        angle = keep
    factor = 1.0
    _close(q, turn(x[:, :H * D].view(n, H, D)).flatten(1), dtype, factor)
    _close(kv[:, :G * D], turn(x[:, H * D:(H + G) * D].reshape(n, G, D)).flatten(1), dtype, factor)
    assert torch.equal(kv[:, G * D:], wide[:, (H + G) * D:cols])
    flat = cache.view(-1, G * (D + V))
    kept = [i for i, s in enumerate(slots.tolist()) if 0 <= s < 48]
    assert torch.equal(flat[slots[kept].long()], kv[kept])
    assert (flat[sorted(set(range(48)) - set(slots[kept].tolist()))] == 7).all()
    assert torch.equal(rotary_store(wide[:, :cols], pos, f, H, G, D, V, cache, slots), q)


def _seen(c, window, chunk):
    """First key of the last of c tokens."""
    return max(0, c - window) if window else ((c - 1) // chunk * chunk if chunk else 0)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,G,D,V,BS,window,chunk", [
    (1, 1, 32, 16, 16, None, None), (6, 3, 64, 48, 64, None, 95), (34, 2, 160, 144, 16, None, 33), (16, 1, 128, 128, 48, None, 1),
    (8, 8, 32, 256, 32, None, 70), (40, 2, 256, 96, 64, None, 257), (12, 4, 96, 32, 256, 31, None), (4, 2, 64, 64, 16, None, 5000)])
def test_grouped_rows_attention(dev, dtype, H, G, D, V, BS, window, chunk):
    """Ragged contexts over scattered pages; most queries point at one key: the oldest they see, the one
    just before that, or one at a page's border.  With a sink per head, some of them dominant."""
    from zipage_amd.layers import grouped_rows_attention
    ctx = [1, 2, 31, 32, 33, BS, BS + 1, 95, 96, 97, 98, 300, 0, 511, 512, 513, 640]
    n, B, NB = len(ctx), len(ctx) + 2, -(-640 // BS)
    pages = B * NB + 3
    g = torch.Generator().manual_seed(H * D)
    tables = torch.randperm(pages, generator=g)[:B * NB].view(B, NB).int()
    trows = torch.randperm(B, generator=g)[:n].int()
    cache = _rand("cpu", dtype, pages, BS, G * (D + V), seed=1)
    q = _rand("cpu", dtype, n, H, D, seed=2, std=0.5)
    sinks = _rand("cpu", F32, H, seed=3, std=3.0)
    flat = cache.view(-1, G * (D + V))
    scale = D ** -0.5
    at = lambda i, t: int(tables[trows[i], t // BS]) * BS + t % BS
    want = torch.zeros(n, H, V, dtype=torch.float64)
    for i, c in enumerate(ctx):
        if c == 0:
            continue
        low = _seen(c, window, chunk)
        key = (low, low - 1, (c - 1) // BS * BS)[i % 3]
        keys = flat[[at(i, t) for t in range(c)]].double()
        k, v = keys[:, :G * D].view(c, G, D), keys[:, G * D:].view(c, G, V)
        for h in range(H):
            b = h // (H // G)
            if key >= 0 and h % 4:
                q[i, h] = (k[key, b] * (8.0 / (scale * float(k[key, b] @ k[key, b])))).to(dtype)
            s = k[low:, b] @ q[i, h].double() * scale
            want[i, h] = O.sink_softmax(s[None], sinks[h].double())[0] @ v[low:, b]
    for i, c in enumerate(ctx):                  # entries in front of what is seen are never read
        if c:
            tables[trows[i], :_seen(c, window, chunk) // BS] = -1
    t = lambda a: torch.as_tensor(a, dtype=torch.int32).to(dev)
    tol = 2.0 if dtype == BF16 else 4.0

    def run(rows):
        wide = torch.full((len(rows), H * V + 8), 3.0, dtype=dtype, device=dev)      # part of wider rows
        grouped_rows_attention(q[rows].flatten(1).to(dev), cache.to(dev), H, G, D, V, t(tables), t([ctx[i] for i in rows]),
                               scale, wide[:, :H * V], window=window, chunk=chunk, sinks=sinks.to(dev),
                               table_rows=t([int(trows[i]) for i in rows]), out_scale=1.5)
        assert (wide[:, H * V:] == 3).all()
        return wide[:, :H * V].view(len(rows), H, V)
    got = run(list(range(n)))
    assert not got[ctx.index(0)].any()
    live = [i for i, c in enumerate(ctx) if c]
    _close(got[live], want[live] * 1.5, dtype, tol)
    for i in (4, 11, 16):                        # one token at a time: other splits of the keys
        _close(run([i]), want[i:i + 1] * 1.5, dtype, tol)
    plain = torch.empty(1, H * V, dtype=dtype, device=dev)                           # without a sink
    grouped_rows_attention(q[16:17].flatten(1).to(dev), cache.to(dev), H, G, D, V, t(tables), t([640]), scale, plain,
                           window=window, chunk=chunk, table_rows=trows[16:17].to(dev))
    low = _seen(640, window, chunk)
    keys = flat[[at(16, j) for j in range(low, 640)]].double()
    for h in range(H):
        b = h // (H // G)
        s = torch.softmax(keys[:, b * D:(b + 1) * D] @ q[16, h].double() * scale, 0)
        _close(plain.view(H, V)[h], s @ keys[:, G * D + b * V:G * D + (b + 1) * V], dtype, tol)


@pytest.mark.parametrize("H,G,D,V,window,chunk", [(1, 1, 32, 32, None, 100), (6, 3, 64, 88, None, 33), (8, 2, 128, 128, None, 1),
                                                  (3, 1, 160, 136, None, 128), (4, 4, 256, 256, None, 200), (9, 3, 96, 48, 64, None),
                                                  (10, 2, 64, 48, None, 4096)])
def test_run_attention(dev, H, G, D, V, window, chunk):
    """Runs at the start, behind cached context and of all lengths about a tile's; queries that point at the
    first key inside and outside what they see; sinks."""
    import numpy as np
    from zipage_amd.engine.inputs import plan_runs
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import run_attention
    from zipage_amd.sight import Chunk
    BS, sight = 16, window or Chunk(chunk)
    parts, page = [], 0
    for start, count in ((0, 127), (0, 128), (0, 129), (45, 16), (300, 257), (7, 300), (1, 2)):
        s = Sequence([0] * (start + count), block_size=BS)
        need = -(-(start + count) // BS)
        s.block_table = list(range(page, page + need))
        page += need
        parts.append(Portion(s, start, count))
    runs = plan_runs(parts, BS, sight)
    total = sum(p.count for p in parts)
    k, v = _rand("cpu", BF16, page * BS, G, D, seed=1), _rand("cpu", BF16, page * BS, G, V, seed=2)
    q, sinks = _rand("cpu", BF16, total, H, D, seed=3, std=0.5), _rand("cpu", F32, H, seed=4, std=3.0)
    scale, rep = D ** -0.5, torch.arange(H) // (H // G)
    want, r = torch.empty(total, H, V, dtype=torch.float64), 0
    for p in parts:
        base, m = p.seq.block_table[0] * BS, p.start + p.count
        low = [_seen(t + 1, window, chunk) for t in range(p.start, m)]
        for i, t in enumerate(range(p.start, m)):
            key = (low[i], low[i] - 1, t)[t % 3]
            if key >= 0:
                row = k[base + key][rep].float()
                q[r + i, 1:] = (row * (8.0 / (scale * (row * row).sum(-1, keepdim=True)))).to(BF16)[1:]
        kk, vv, j = k[base:base + m].double(), v[base:base + m].double(), torch.arange(m)[None]
        pos = torch.arange(p.start, m)[:, None]
        seen = (j <= pos) & (j >= torch.tensor(low)[:, None])
        for h in range(H):
            sc = (q[r:r + p.count, h].double() @ kk[:, rep[h]].T * scale).masked_fill(~seen, float("-inf"))
            want[r:r + p.count, h] = O.sink_softmax(sc, sinks[h].double()) @ vv[:, rep[h]]
        r += p.count
    if runs.key_slots is None:
        runs.key_slots = np.concatenate([np.arange(p.start, p.start + p.count) + p.seq.block_table[0] * BS for p in parts])
    slots = torch.as_tensor(runs.key_slots).long()
    kv = torch.cat([k[slots].flatten(1), v[slots].flatten(1)], dim=1).to(dev)
    out = torch.full((total, H * V + 16), float("nan"), dtype=BF16, device=dev)
    run_attention(q.flatten(1).to(dev), kv, H, G, D, V, torch.as_tensor(runs.tiles).to(dev), scale, out[:, :H * V],
                  window=window, chunk=chunk, sinks=sinks.to(dev), out_scale=0.75)
    _close(out[:, :H * V].view(total, H, V), want * 0.75, BF16, 2.0)


# ------------------------------------------------------------------ recurrences
def _segments(dev, parts, run_min=None):
    """parts: (row, count, slot, start), those of run_min tokens and more behind the others."""
    from zipage_amd.engine.qwen3 import Segments
    made = []
    for some in ([p for p in parts if run_min is None or p[1] < run_min], [p for p in parts if run_min and p[1] >= run_min]):
        t = torch.tensor(some, dtype=torch.int32).view(-1, 4).T.contiguous().to(dev)
        # steps of single tokens only take the kernels of decoding
        made.append(Segments(*t, first_row=some[0][0], longest=max(p[1] for p in some),
                             max_count=int(all(p[1] == 1 for p in parts))) if some else None)
    return types.SimpleNamespace(segments=made[0], run_segments=made[1])


CUTS = [[70], [1], [2, 3, 16, 17, 1, 1], [15, 25, 30], [16, 16, 8], [33, 7]]


def _scan_in_cuts(dev, step, n, cuts, slots, run_min):
    """Sequences of n tokens run together, each cut its own way, states in the given slots; step(rows of the
    sequences, segments) -> output rows.  Returns the outputs in sequence order."""
    seqs = len(cuts)
    at, out = [0] * seqs, [[] for _ in range(seqs)]
    turn = 0
    while any(a < n for a in at):
        parts, rows, row = [], [], 0
        count = lambda s: min(cuts[s][len(out[s]) % len(cuts[s])], n - at[s])
        for s in sorted(range(seqs), key=lambda s: run_min is not None and count(s) >= run_min):
            if at[s] == n or (turn + s) % 4 == 3:            # it pauses
                continue
            c = count(s)
            parts.append((row, c, slots[s], at[s]))
            rows += [(s, t) for t in range(at[s], at[s] + c)]
            row += c
        turn += 1
        if not parts:
            continue
        got = step(rows, _segments(dev, parts, run_min))
        for (r, c, slot, _), s in zip(parts, [slots.index(p[2]) for p in parts]):
            out[s].append(got[r:r + c])
            at[s] += c
    return [torch.cat(o) for o in out]


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("run_min", [None, 16, 2])
@pytest.mark.parametrize("H,D,V", [(3, 20, 24), (2, 64, 64), (1, 128, 128), (300, 32, 40), (2, 40, 136), (1, 130, 250)])
def test_matrix_memory(dev, dtype, run_min, H, D, V):
    """Prompts against token by token against portions, in blocks and token by token, states in slots that
    others used before."""
    from zipage_amd.layers import MatrixMemory
    W, n, cap, eps = 64, 70, 3.0, 1e-3
    r = lambda *s, seed, std=1.0: _rand("cpu", dtype, *s, seed=seed, std=std)
    w = {"q": r(H * D, W, seed=1, std=.2), "k": r(H * D, W, seed=2, std=.2), "v": r(H * V, W, seed=3, std=.2),
         "g": r(H * V, W, seed=4, std=.2), "o": r(W, H * V, seed=5), "norm": 1 + r(H * V, seed=6, std=.3),
         "i": r(H, W, seed=7, std=.3), "i.b": r(H, seed=8), "f": r(H, W, seed=9, std=.2), "f.b": 3 + r(H, seed=10)}
    m = MatrixMemory(W, H, D, V, cap, eps, out_scale=1.5)
    into, _ = m.load(w, dtype, dev, W)
    into = into.to(dev)
    h = r(len(CUTS), n, W, seed=11).to(dev)
    h[:, 20] *= 3                                            # a token whose gate raises the maximum
    proj = (h.flatten(0, 1).float() @ into.float().T).to(dtype).view(len(CUTS), n, -1)
    state = m.allocate(len(CUTS) + 2, dtype, dev).fill_(float("nan"))
    Dp, Vp = m.dim_p, m.vdim_p

    def step(rows, seg):
        s, t = [a for a, _ in rows], [b for _, b in rows]
        out = torch.full((len(rows), H * Vp + 8), 7.0, dtype=dtype, device=dev)
        m.scan(h[s, t].contiguous(), proj[s, t].contiguous(), state, seg, out[:, :H * Vp])
        assert (out[:, H * Vp:] == 7).all()
        return out[:, :H * Vp].view(len(rows), H, Vp)[..., :V].clone()
    for round_, slots in enumerate(([3, 0, 6, 1, 5, 2], [0, 1, 2, 3, 4, 5])):
        got = _scan_in_cuts(dev, step, n, CUTS, slots, run_min)
        for s in range(len(CUTS)):
            P = proj[s].double().cpu()
            part = lambda at, d, dp: P[:, at:at + H * dp].view(n, H, dp)[..., :d]
            hh = h[s].double().cpu()
            i = cap * torch.tanh((hh @ w["i"].double().T + w["i.b"].double()) / cap)
            f = torch.nn.functional.logsigmoid(cap * torch.tanh((hh @ w["f"].double().T + w["f.b"].double()) / cap))
            o = O.mlstm_recurrence(part(0, D, Dp) * D ** -0.5, part(H * Dp, D, Dp), part(2 * H * Dp, V, Vp), i, f)
            o = O.rms(o, eps) * w["norm"].double().view(H, V) * torch.sigmoid(part(2 * H * Dp + H * Vp, V, Vp)) * 1.5
            # a small denominator amplifies rounding
            _close(got[s].flatten(1), o.flatten(1), dtype, 1.0 if dtype == BF16 else 512.0)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("run_min", [None, 16, 7])
@pytest.mark.parametrize("H,G,D,V,taps", [(6, 2, 24, 40, 3), (2, 2, 64, 64, 4), (2, 1, 128, 128, 8), (200, 50, 32, 32, 2), (1, 1, 40, 136, 1),
                                          (2, 2, 200, 250, 8)])
def test_channel_delta(dev, dtype, run_min, H, G, D, V, taps):
    """As above; some channels keep everything, others forget within a token."""
    from zipage_amd.layers import ChannelDelta
    W, n, eps = 64, 70, 1e-3
    r = lambda *s, seed, std=1.0: _rand("cpu", dtype, *s, seed=seed, std=std)
    ra, rg = 5, 11
    w = {"q": r(G * D, W, seed=1, std=.2), "k": r(G * D, W, seed=2, std=.2), "v": r(H * V, W, seed=3, std=.2),
         "q.conv": r(G * D, taps, seed=4), "k.conv": r(G * D, taps, seed=5), "v.conv": r(H * V, taps, seed=6),
         "b": r(H, W, seed=7, std=.2), "A_log": r(H, seed=8, std=.5), "norm": 1 + r(V, seed=9, std=.3),
         "a1": r(ra, W, seed=10, std=.1), "a2": r(H * D, ra, seed=11, std=.4), "dt_bias": -3 + 6 * r(H * D, seed=12),
         "g1": r(rg, W, seed=13, std=.1), "g2": r(H * V, rg, seed=14, std=.4), "o": r(W, H * V, seed=15)}
    assert {k: tuple(t.shape) for k, t in w.items()} == ChannelDelta(W, H, G, D, V, taps, eps).shapes(ra, rg)
    m = ChannelDelta(W, H, G, D, V, taps, eps, out_scale=1.5)
    into, _ = m.load(w, dtype, dev, W)
    h = r(len(CUTS), n, W, seed=16).to(dev)
    proj = (h.flatten(0, 1).float() @ into.to(dev).float().T).to(dtype).view(len(CUTS), n, -1)
    S, tail = m.allocate(len(CUTS) + 2, dtype, dev)
    state = (S.fill_(float("nan")), tail.fill_(float("nan")))
    Dp, Vp = m.dim_p, m.vdim_p

    def step(rows, seg):
        s, t = [a for a, _ in rows], [b for _, b in rows]
        out = torch.full((len(rows), H * Vp), 7.0, dtype=dtype, device=dev)
        m.scan(proj[s, t].contiguous(), state, seg, out)
        return out.view(len(rows), H, Vp)[..., :V].clone()
    head = torch.arange(H) // (H // G)
    for round_, slots in enumerate(([3, 0, 6, 1, 5, 2], [0, 1, 2, 3, 4, 5])):
        got = _scan_in_cuts(dev, step, n, CUTS, slots, run_min)
        for s in range(len(CUTS)):
            P = proj[s].double().cpu()
            part = lambda at, k, d, dp: P[:, at:at + k * dp].reshape(n, k, dp)[..., :d].reshape(n, k * d)
            conv = lambda x, k: O.short_conv(x, w[k + ".conv"].double())
            q = O.unit(conv(part(0, G, D, Dp), "q").view(n, G, D)) * D ** -0.5
            k = O.unit(conv(part(G * Dp, G, D, Dp), "k").view(n, G, D))
            v = conv(part(2 * G * Dp, H, V, Vp), "v").view(n, H, V)
            beta = torch.sigmoid(P[:, m.b_at:m.b_at + H])
            # the low-rank products' rounding is the library's: take its rows
            low = torch.nn.functional.linear(proj[s][:, m.low_at:m.low_at + m.low_rank], m.low).double().cpu()
            a = low[:, :H * Dp].view(n, H, Dp)[..., :D] + w["dt_bias"].double().view(H, D)
            gate = low[:, H * Dp:].view(n, H, Vp)[..., :V]
            g = torch.exp(-torch.exp(w["A_log"].double())[None, :, None] * torch.nn.functional.softplus(a))
            o = O.norm(O.delta_recurrence(q[:, head], k[:, head], v, g, beta), w["norm"].double(), eps)
            _close(got[s].flatten(1), (o * torch.sigmoid(gate) * 1.5).flatten(1), dtype, 1.0 if dtype == BF16 else 64.0)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_inert_segments_leave_states_alone(dev, dtype):
    """The padding of a decode batch: rows without a token write zeros and touch no state."""
    from zipage_amd.engine.qwen3 import Segments
    from zipage_amd.layers import MatrixMemory
    m = MatrixMemory(32, 2, 32, 32, 5.0, 1e-3)
    r = lambda *s: _rand("cpu", dtype, *s, seed=len(s), std=.2)
    into, _ = m.load({k: r(*s) for k, s in m.shapes().items()}, dtype, dev, 32)
    h = _rand(dev, dtype, 4, 32, seed=2)
    proj, state = (h.float() @ into.to(dev).float().T).to(dtype), m.allocate(5, dtype, dev)
    t = lambda *a: torch.tensor(a, dtype=torch.int32, device=dev)
    out = torch.full((4, 64), 9.0, dtype=dtype, device=dev)
    m.scan(h, proj, state, types.SimpleNamespace(
        segments=Segments(None, t(1, 0, 900, 0), t(1, 4, 2, 4), t(0, 0, 0, 0), max_count=1), run_segments=None), out)
    assert not out[1].any() and not out[3].any() and out[0].any() and out[2].any()
    assert not state[[0, 3, 4]].any() and state[1].any() and state[2].any()


# ------------------------------------------------------------------ experts
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,K,M", [(1, 32, 4), (5, 96, 12), (64, 512, 64), (4100, 64, 72)])
def test_small_linear(dev, dtype, n, K, M):
    from zipage_amd.layers import small_linear
    x, w = _rand(dev, dtype, n, K + 8, seed=1)[:, :K], _rand(dev, dtype, M, K, seed=2)
    got = small_linear(x, w)
    assert got.dtype == F32
    _close(got, x.double().cpu() @ w.double().cpu().T, F32, 4.0)


@pytest.mark.parametrize("E,top,groups,keep", [(1, 1, 1, 1), (12, 2, 2, 1), (10, 3, 5, 2), (64, 6, 1, 1), (66, 4, 3, 2), (256, 8, 8, 4),
                                               (300, 5, 300, 7), (1000, 3, 4, 4)])
def test_selection(dev, E, top, groups, keep):
    from zipage_amd.layers.moe import moe_select
    z = _rand(dev, F32, 37, E + 3, seed=E, std=2.0)
    ids_, s, counts = moe_select(z, E, top, groups, keep)
    want = O.route(z[:, :E].double().cpu(), top, groups, keep)
    got = torch.zeros(37, E, dtype=torch.float64).scatter_(1, ids_.long().cpu(), s.double().cpu())
    assert torch.equal(got > 0, want > 0) and not counts.any()
    _close(got, want, F32, 4.0)


@pytest.mark.parametrize("n", [1, 2, 63, 500, 3000])
@pytest.mark.parametrize("E,top,shared", [(12, 3, True), (70, 5, False), (4, 4, True)])
def test_plan_covers_every_assignment_once(dev, n, E, top, shared):
    from zipage_amd.layers.moe import Plan, moe_select
    z = _rand(dev, F32, n, E, seed=n, std=2.0)
    z[:, 0] += 4                                             # one expert is much fuller than the others
    ids_, s, counts = moe_select(z, E, top)
    p = Plan(ids_, counts, E, shared, BF16)
    order, tiles = p.sorted.cpu().tolist(), p.tiles[:int(p.ntiles)].cpu().tolist()
    assert sorted(order) == list(range(n * p.slots))
    expert = torch.cat([ids_.cpu(), torch.full((n, 1), E, dtype=torch.int32)], 1)[:, :p.slots].flatten().tolist()
    at = 0
    for e, first, rows, _ in tiles:
        assert first == at and 1 <= rows <= p.rows
        assert all(expert[a] == e for a in order[first:first + rows])
        at += rows
    assert at == n * p.slots and [t[0] for t in tiles] == sorted(t[0] for t in tiles)


def _expert_weights(E, W, ff, sff, dtype):
    r = lambda o, i, seed: _rand("cpu", dtype, o, i, seed=seed, std=i ** -0.5)
    w = {"router": r(E, W, 1) * 3}
    for e in range(E):
        w.update({f"e{e}.gate": r(ff, W, 3 * e + 2), f"e{e}.up": r(ff, W, 3 * e + 3), f"e{e}.down": r(W, ff, 3 * e + 4)})
    if sff:
        w.update({"shared.gate": r(sff, W, 9001), "shared.up": r(sff, W, 9002), "shared.down": r(W, sff, 9003)})
    return w


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n", [1, 3, 40, 129, 700, 2500])
@pytest.mark.parametrize("E,top,groups,keep,W,ff,sff", [(12, 2, 2, 1, 96, 44, 72), (5, 3, 1, 1, 160, 96, 32), (66, 4, 3, 2, 64, 32, None),
                                                        (3, 2, 1, 1, 256, 160, 320)])
def test_experts(dev, dtype, n, E, top, groups, keep, W, ff, sff):
    from zipage_amd.layers import Experts
    m = Experts(W, E, top, ff, 0.8, groups, keep, sff, 1.3)
    w = _expert_weights(E, W, ff, sff, dtype)
    m.load(w, dtype, dev)
    h = _rand(dev, dtype, n, m.width_p, seed=5, std=1.5)
    h[:, W:] = 0
    planes = m.forward(h)
    assert planes.shape == (top + (1 if sff else 0), n, m.width_p) and not planes[..., W:].any()
    ids_, s, _ = m.route(h)
    d = {k: v.double() for k, v in w.items()}
    x = h[:, :W].double().cpu()
    part = lambda e: {k[len(e) + 1:]: v for k, v in d.items() if k.startswith(e + ".")}
    want = torch.zeros(top + (1 if sff else 0), n, W, dtype=torch.float64)
    for e in range(E):
        y = O.expert(x, part(f"e{e}"), 0.8)
        for j in range(top):
            hit = (ids_[:, j] == e).cpu()
            want[j, hit] = s[:, j].double().cpu()[hit, None] * y[hit]
    if sff:
        want[top] = O.expert(x, part("shared"), 1.3)
    _close(planes[..., :W], want, dtype, 2.0 if dtype == BF16 else 16.0)
    if dtype == F32:
        z = x @ d["router"].T
        got = torch.zeros(n, E, dtype=torch.float64).scatter_(1, ids_.long().cpu(), s.double().cpu())
        _close(got, O.route(z, top, groups, keep), F32, 16.0)


# ------------------------------------------------------------------ the model
def _engine(name, dtype, tmp, **kw):
    from zipage_amd.engine import EngineConfig, ZipageEngine, read_shape
    from zipage_amd.engine.weights import write_safetensors
    folder = tmp / name
    if not folder.exists():
        folder.mkdir()
        cfg, w = C.case(name)
        (folder / "config.json").write_text(json.dumps(cfg))
        write_safetensors(str(folder / "model.safetensors"), w)
    base = dict(shape=read_shape(str(folder)), model_folder=str(folder), dtype=dtype, num_kvcache_blocks=64,
                kvcache_block_size=16, max_concurrency=6)
    base.update(kw)
    return ZipageEngine(EngineConfig(**base))


@pytest.fixture(scope="module")
def engines(tmp_path_factory):
    """Engines by (case, dtype), kept for the module: pages and slots are used again and again."""
    tmp, made = tmp_path_factory.mktemp("kapolorn"), {}

    def get(name, dtype, **kw):
        if kw:
            return _engine(name, dtype, tmp, **kw)
        if (name, dtype) not in made:
            made[(name, dtype)] = _engine(name, dtype, tmp)
        return made[(name, dtype)]
    yield get
    for e in made.values():
        assert e.scheduler.pool.num_free == 64 and len(e.scheduler.free_rows) == 6


def _feed_all(eng, toks, cuts):
    """Logits of every position, the sequence cut as `cuts` says (the last size repeats)."""
    s, at, out, k = eng.open_request(), 0, [], 0
    while at < len(toks):
        n = min(cuts[min(k, len(cuts) - 1)], len(toks) - at)
        out.append(eng.feed([(s, toks[at:at + n], list(range(n)))]).clone())
        at, k = at + n, k + 1
    eng.close_request(s)
    torch.cuda.synchronize()
    return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
@pytest.mark.parametrize("cuts", [[400], [1], [2], [3, 17, 1, 16, 15, 64], [100, 1], [37], [16]], ids=lambda c: "-".join(map(str, c)))
def test_any_cut_of_a_sequence_gives_the_oracle(dev, engines, name, dtype, cuts):
    toks = C.tokens(C.CONFIGS[name], 150, 3)
    C.close(name, _feed_all(engines(name, dtype), toks, cuts), C.expected(name, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_layer_streams(dev, engines, dtype):
    """The stream after every pass of every layer, a whole prompt in one step."""
    from zipage_amd.engine import Portion
    cfg, w = C.case("calm")
    toks = C.tokens(cfg, 120, 9)
    eng = engines("calm", dtype)
    s = eng.open_request()
    s.token_ids, s.num_tokens, s.num_prompt_tokens = list(toks), 120, 120
    eng.scheduler.pool.grow(s, 120)
    i, p, ctx, _ = eng.runner.prepare_portions([Portion(s, 0, 120)])
    streams = []
    eng.runner.model.forward(i, p, ctx, trace=streams)
    eng.close_request(s)
    want = O.forward(cfg, w, toks)[1]
    assert len(streams) == len(want) == 5
    for got, ref in zip(streams, want):
        if dtype == F32:
            _close(got, ref, F32, 32.0)
        else:
            e = (got.double().cpu() - ref).square().mean(-1).sqrt() / ref.square().mean(-1).sqrt()
            assert float(e.median()) < 0.03 and float(e.quantile(0.9)) < 0.08


@pytest.mark.parametrize("name,dtype", [("odd", F32), ("calm", F32), ("calm", BF16), ("wide", BF16)], ids=ids)
def test_first_tokens_and_page_borders(dev, engines, name, dtype):
    for n in (1, 2, 15, 16, 17, 33, 38):
        toks = C.tokens(C.CONFIGS[name], n, 20 + n)
        C.close(name, _feed_all(engines(name, dtype), toks, [n]), C.expected(name, toks), dtype)
        C.close(name, _feed_all(engines(name, dtype), toks, [n - 1 or 1, 1]), C.expected(name, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_long_decoding(dev, engines, dtype):
    """Many chunks of decoded tokens; the pages behind them are given back on the way."""
    cfg = C.CONFIGS["calm"]
    toks = C.tokens(cfg, 400, 5)
    eng = engines("calm", dtype)
    s = eng.open_request()
    got = [eng.feed([(s, toks[:20], [19])]).clone()]
    for t in range(20, 400):
        got.append(eng.feed([(s, toks[t:t + 1], [0])]).clone())
        assert 64 - eng.scheduler.pool.num_free <= 6           # a chunk of 64 tokens, 16 a page
    eng.close_request(s)
    C.close("calm", torch.cat(got), C.expected("calm", toks)[19:], dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_mixed_batches_equal_each_alone(dev, engines, name, dtype):
    """Portions beside single tokens, requests that pause, end and are followed by others in their pages
    and slots: every logit is the oracle's."""
    cfg = C.CONFIGS[name]
    eng = engines(name, dtype)
    g = torch.Generator().manual_seed(4)
    rnd = lambda lo, hi: int(torch.randint(lo, hi + 1, (1,), generator=g))
    todo = [C.tokens(cfg, n, 40 + i) for i, n in enumerate((60, 1, 110, 33, 150, 2, 77, 128, 19))]
    everything = torch.cat([C.expected(name, t) for t in todo])
    live, rows, wants = [], [], []
    while todo or live:
        while todo and len(live) < 5:
            live.append([eng.open_request(), todo.pop(0), 0])
        batch, meta = [], []
        for item in live:
            s, toks, at = item
            if len(live) > 1 and rnd(0, 5) == 0:
                continue
            n = min((1, 1, 2, 3, 16, 40, 70)[rnd(0, 6)], len(toks) - at)
            batch.append((s, toks[at:at + n], list(range(n))))
            meta.append((item, n))
        if not batch:
            continue
        rows.append(eng.feed(batch).clone())
        for item, n in meta:
            wants.append(C.expected(name, item[1])[item[2]:item[2] + n])
            item[2] += n
            if item[2] == len(item[1]):
                eng.close_request(item[0])
        live = [i for i in live if i[2] < len(i[1])]
    C.close(name, torch.cat(rows), torch.cat(wants), dtype, whole=everything)


def test_graph_replays_equal_eager_steps(dev, engines):
    """The same decode steps through replayed graphs and eagerly, with other work in between."""
    eng, eager = engines("wide", BF16), engines("wide", BF16, use_graph=False)
    toks = [C.tokens(C.CONFIGS["wide"], 90, 60 + i) for i in range(3)]
    a, b = [eng.open_request() for _ in toks], [eager.open_request() for _ in toks]
    for step in range(40):
        n = 30 if step == 0 else 1
        at = 0 if step == 0 else 29 + step
        got = eng.feed([(s, t[at:at + n], [n - 1]) for s, t in zip(a, toks)]).clone()
        junk = torch.randn(256, 256, device=dev) @ torch.randn(256, 256, device=dev)
        want = eager.feed([(s, t[at:at + n], [n - 1]) for s, t in zip(b, toks)]).clone()
        torch.cuda.synchronize()
        assert junk.isfinite().all() and torch.equal(got, want), step
    for s in a:
        eng.close_request(s)


def test_bad_input_is_an_error(dev, engines):
    eng = engines("odd", BF16)
    s = eng.open_request()
    for bad in ([131], [-1], []):
        with pytest.raises(ValueError):
            eng.feed([(s, bad, [])])
    with pytest.raises(ValueError, match="place"):
        eng.feed([(s, [1, 2], [2])])
    assert eng.feed([(s, [1, 2], [])]) is None
    eng.close_request(s)
    from zipage_amd.layers.recurrent import _key_size
    with pytest.raises(ValueError, match="256"):
        _key_size(257)
    from zipage_amd.layers import Experts
    with pytest.raises(ValueError, match="groups"):
        Experts(32, 8, 5, 32, 1.0, 4, 2)


# ------------------------------------------------------------------ generation
def _greedy_ok(name, prompt, got, slack=1e-4):
    """`got` is the oracle's greedy continuation, up to a near tie of two logits."""
    cfg, w = C.case(name)
    lg = O.forward(cfg, w, prompt + got)[0]
    for i, tok in enumerate(got):
        row = lg[len(prompt) - 1 + i]
        assert float(row.max() - row[tok]) < slack * float(row.std()), i


@pytest.mark.parametrize("kw", [{}, dict(max_num_batched_tokens=24), dict(num_kvcache_blocks=14, max_concurrency=2),
                                dict(enable_prefix_cache=True), dict(use_graph=False, enable_async_compress=True)],
                         ids=lambda k: "-".join(k) or "default")
def test_greedy_generation(dev, engines, kw):
    """Through the scheduler: prompts longer than a step, more requests than slots, prompts of one token,
    prompts that share their beginning."""
    from zipage_amd.engine import SamplingParams
    cfg = C.CONFIGS["odd"]
    eng = engines("odd", F32, **(kw or dict(seed=1)))
    first = C.tokens(cfg, 70, 1)
    prompts = [first, C.tokens(cfg, 1, 2), first[:50] + C.tokens(cfg, 9, 3), C.tokens(cfg, 33, 4), first[:64], [5, 6]]
    counts = [30, 40, 7, 1, 20, 60]
    for round_ in range(2):                    # the second round meets used pages and slots
        outs = eng.generate(prompts, [SamplingParams(max_tokens=c, ignore_eos=True) for c in counts])
        for p, c, o in zip(prompts, counts, outs):
            assert len(o["token_ids"]) == c
            _greedy_ok("odd", p, o["token_ids"], 1e-3)
    pool = eng.scheduler.pool
    assert pool.num_free == pool.num_pages and pool.reserved == 0
    assert eng.stats["decode_tokens"] + eng.stats["mixed_decode_tokens"] == 2 * sum(c - 1 for c in counts)


def test_generation_stops_at_eos_and_samples(dev, engines):
    from zipage_amd.engine import SamplingParams
    cfg, w = C.case("calm")
    prompt = C.tokens(cfg, 21, 8)
    want = O.greedy(cfg, w, prompt, 12)
    eos = want[7]
    eng = engines("calm", F32, eos=eos)
    out = eng.generate([prompt], SamplingParams(max_tokens=12))[0]["token_ids"]
    assert out == want[:want.index(eos) + 1]
    cold = eng.generate([prompt] * 3, SamplingParams(temperature=1e-4, max_tokens=6, ignore_eos=True))
    assert all(o["token_ids"] == want[:6] for o in cold)
    hot = eng.generate([prompt] * 4, SamplingParams(temperature=50.0, max_tokens=8, ignore_eos=True))
    assert len({tuple(o["token_ids"]) for o in hot}) > 1


def test_bf16_generation_follows_its_own_logits(dev, engines):
    """Greedy tokens of the bf16 engine are within bf16 error of the oracle's best."""
    from zipage_amd.engine import SamplingParams
    prompts = [C.tokens(C.CONFIGS["calm"], n, 70 + n) for n in (5, 64, 131)]
    eng = engines("calm", BF16, max_num_batched_tokens=50)
    for p, o in zip(prompts, eng.generate(prompts, SamplingParams(max_tokens=60, ignore_eos=True))):
        _greedy_ok("calm", p, o["token_ids"], 0.3)


def test_command_line(dev, engines, tmp_path, capsys, monkeypatch):
    import numpy as np
    from zipage_amd import cli
    folder = engines("ends", F32).cfg.model_folder
    cfg, w = C.case("ends")
    prompt = C.tokens(cfg, 40, 2)
    assert cli.main(["generate", "--model", folder, "--dtype", "float32", "--tokens", ",".join(map(str, prompt)),
                     "--tokens", "3", "--max-tokens", "9", "--batch-tokens", "16"]) == 0
    lines = [json.loads(l) for l in capsys.readouterr().out.splitlines() if l.startswith("{")]
    _greedy_ok("ends", prompt, lines[0]["token_ids"], 1e-3)
    _greedy_ok("ends", [3], lines[1]["token_ids"], 1e-3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": prompt[:33], "want": [0, 32]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": [3, 4], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": [5], "want": [0]}, {"id": "a", "tokens": prompt[33:], "want": [6]}],
              "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "c", "tokens": prompt[:1], "want": [0]}], "end": ["c"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    assert cli.main(["trace", "--model", folder, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "128"]) == 0
    done = [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")]
    assert done == [f"done {i}" for i in range(4)] and not (tmp_path / "1.f32").exists()
    read = lambda i: torch.from_numpy(np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"]))
    full, other = C.expected("ends", prompt), C.expected("ends", [3, 4, 5])
    C.close("ends", read(0), full[[0, 32]], F32, whole=full)
    C.close("ends", read(2), torch.stack([other[2], full[39]]), F32, whole=full)
    C.close("ends", read(3), full[:1], F32, whole=full)
