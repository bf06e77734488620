"""Mefupel on the GPU: every mechanism alone, the model against the oracle in every way a sequence can be cut
and batched, and generation through the engine."""
import io
import json
import types

import pytest
import torch

from oracle import mefupel_oracle as O
from tests import mefupel_cases as C
from tests.test_hip_kapolorn import CUTS, _scan_in_cuts

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


def _angles(positions, freqs):
    """fp32 angles (n, 1, pairs)."""
    return (positions.cpu().float()[:, None] * freqs.cpu()).double()[:, None]


def _turn(x, positions, freqs, back=False, adjacent=False):
    """x (n, heads, dim): pairs half apart, or neighbours."""
    half = freqs.numel()
    a = _angles(positions, freqs) * (-1 if back else 1)
    one = 2 * torch.arange(half) if adjacent else torch.arange(half)
    two = one + (1 if adjacent else half)
    out, u, v = x.clone(), x[..., one], x[..., two]
    out[..., one], out[..., two] = u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin()
    return out


def _freqs(dev, n, base=300.0):
    return torch.tensor([base ** (-i / max(n, 1)) for i in range(n)], device=dev)


# ------------------------------------------------------------------ row steps
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,width,norm_width", [(1, 96, 76), (3, 512, 512), (17, 1024, 1000), (2, 8192, 8192)])
@pytest.mark.parametrize("normed,plain", [((1,), (2,)), ((1, 3), ()), ((2, 1), (4,)), ((), (1, 2, 1)), ((1, 1), (1,))], ids=str)
def test_branches_join_the_stream(dev, dtype, n, width, norm_width, normed, plain):
    """Some normed, some as they are, in any order; with what comes before a pass of a loop."""
    from zipage_amd.layers import residual_norm
    x = _rand(dev, F32, n, width, seed=1)
    made = [(_rand(dev, dtype, p, n, width, seed=10 + i), _rand(dev, F32, width, seed=20 + i) if i < len(normed) else None)
            for i, p in enumerate(normed + plain)]
    embedded, shift, w = (_rand(dev, F32, *s, seed=30 + i) for i, s in enumerate(((1, n, width), (width,), (width,))))
    for t in (x, embedded, shift, w, *(t for pair in made for t in pair if t is not None)):
        t[..., norm_width:] = 0
    want = x.double()
    for y, b in made:
        y = y.double().sum(0)
        want = want + (y if b is None else y / torch.sqrt(y.square().sum(-1, keepdim=True) / norm_width + 1e-3) * b.double())
    unit = lambda t: t / torch.sqrt(t.square().sum(-1, keepdim=True) / norm_width + 1e-3) * (1 + w.double())
    one = torch.ones(2, device=dev)
    for order in (made, made[::-1]):
        (y, b), *more = order
        kept, after = torch.empty_like(x), torch.empty_like(x)
        h = residual_norm(x, y, w, 1e-3, norm_width, weight_offset=1.0, y_weight=b, more=tuple(more), result=kept, x_out=after,
                          history=embedded, mix=one, shift=shift)
        _close(kept, want, F32, 2.0)
        _close(after, want + embedded[0].double() + shift.double(), F32, 2.0)
        _close(h, unit(want + embedded[0].double() + shift.double()), dtype)
        h = residual_norm(x, y, w, 1e-3, norm_width, weight_offset=1.0, y_weight=b, more=tuple(more), x_out=after)
        _close(after, want, F32, 2.0)
        _close(h, unit(want), dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_embedding_with_a_vector_on_top(dev, dtype):
    from zipage_amd.layers import embed_norm
    embed, w, shift = _rand(dev, dtype, 11, 96, seed=1), _rand(dev, F32, 96, seed=2), _rand(dev, F32, 96, seed=3)
    tok, at = torch.tensor([3, 10, 0, 7], device=dev), torch.zeros(4, dtype=torch.int32, device=dev)
    x, kept = torch.empty(4, 96, device=dev), torch.empty(4, 96, device=dev)
    h = embed_norm(tok, at, embed, None, x, w, 1e-2, 96, weight_offset=1.0, shift=shift, result=kept)
    assert torch.equal(kept, embed[tok].float())
    _close(x, embed[tok].double() + shift.double(), F32)
    _close(h, O.norm(embed[tok].double() + shift.double(), w.double(), 1e-2), dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,width,norm_width", [(5, 8, 5), (3, 96, 96), (7, 512, 500), (4, 2048, 2048), (3, 4104, 4100), (2, 8200, 8193),
                                                (2, 16384, 16384), (2, 18432, 18432), (1, 32768, 32700)])
def test_normed_powers(dev, dtype, n, width, norm_width):
    """Rows inside wider ones; one element that towers over the others."""
    from zipage_amd.layers import normed_powers
    wide = _rand(dev, dtype, n, width + 24, seed=1)
    z = wide[:, 16:16 + width]
    z[:, norm_width:] = 0
    z[0, 0] = 40.0
    act, out = (0.7, -1.5, 0.4, 0.3), torch.full((n, width + 8), 9.0, dtype=dtype, device=dev)
    normed_powers(z, act, 1e-3, norm_width, out[:, :width])
    want = O.poly_norm(z[:, :norm_width].double().cpu(), act, 1e-3)
    _close(out[:, :norm_width], want, dtype, 1.0 if dtype == BF16 else 4.0)
    assert (out[:, width:] == 9).all()


# ------------------------------------------------------------------ rotary positions and stores
POSITIONS = [0, 1, 7, 100, 4095, 3, 50000, 12, 13]
SLOTS = [5, -1, 47, 0, 12, 13, 48, 8, 7]                       # 48: past the end


def _check_slots(cache, kv):
    flat = cache.view(-1, kv.shape[1])
    kept = [i for i, s in enumerate(SLOTS) if 0 <= s < 48]
    put = [SLOTS[i] for i in kept]
    assert torch.equal(flat[put], kv[kept])
    assert (flat[sorted(set(range(48)) - set(put))] == 7).all()


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,G,D,V,vdim,rot", [(4, 2, 32, 48, 48, 32), (6, 3, 24, 16, 14, 10), (5, 1, 96, 128, 128, 64), (2, 2, 64, 32, 18, 2),
                                              (3, 3, 32, 32, 2, 0), (2, 1, 256, 256, 256, 256)])
def test_turning_values_are_stored(dev, dtype, H, G, D, V, vdim, rot):
    from zipage_amd.layers import rotary_store, store_form
    n, cols = 9, H * D + G * (D + V)
    wide = _rand(dev, dtype, n, cols + 24, seed=1)
    pos, slots = (torch.tensor(a, dtype=torch.int32, device=dev) for a in (POSITIONS, SLOTS))
    cache = torch.full((3, 16, G * (D + V)), 7.0, dtype=dtype, device=dev)
    f, vf = _freqs(dev, rot // 2), torch.zeros(V // 2, device=dev)
    vf[:vdim // 2] = _freqs(dev, vdim // 2, 40.0)
    turns = torch.full((n, V // 2, 2), float("nan"), device=dev)
    q, kv = rotary_store(wide[:, :cols], pos, f, H, G, D, V, cache, slots, return_kv=True, form=store_form(value_freqs=vf, turns=turns))
    x = wide[:, :cols].double().cpu()
    _close(q, _turn(x[:, :H * D].view(n, H, D), pos, f).flatten(1), dtype)
    _close(kv[:, :G * D], _turn(x[:, H * D:(H + G) * D].reshape(n, G, D), pos, f).flatten(1), dtype)
    _close(kv[:, G * D:], _turn(x[:, (H + G) * D:].reshape(n, G, V), pos, vf, adjacent=True).flatten(1), dtype)
    a = _angles(pos, vf)[:, 0]
    _close(turns, torch.stack([a.cos(), a.sin()], -1), F32)
    _check_slots(cache, kv)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,G,D,dim,rot", [(4, 2, 32, 32, 32), (6, 3, 32, 20, 10), (8, 8, 16, 9, 0), (20, 1, 80, 72, 48), (2, 2, 256, 250, 250)])
def test_keys_that_are_values_and_norms_over_all_heads(dev, dtype, H, G, D, dim, rot):
    from zipage_amd.layers import rotary_store, store_form
    n, cols = 9, (H + G) * D
    x = _rand(dev, dtype, n, cols // D, D, seed=1)
    x[..., dim:] = 0
    x[2] *= 30
    x[3] *= 1e-3
    wide = torch.cat([x.flatten(1), torch.full((n, 8), 5.0, dtype=dtype, device=dev)], 1)
    pos, slots = (torch.tensor(a, dtype=torch.int32, device=dev) for a in (POSITIONS, SLOTS))
    cache = torch.full((3, 16, 2 * G * D), 7.0, dtype=dtype, device=dev)
    f, w = _freqs(dev, rot // 2), _rand(dev, F32, cols, seed=2)
    form = store_form(w, H * dim, G * dim, 1e-3, tied=True)
    q, kv = rotary_store(wide[:, :cols], pos, f, H, G, D, D, cache, slots, return_kv=True, form=form)
    x = x.double().cpu()
    unit = lambda t: t / torch.sqrt(t.square().sum((1, 2), keepdim=True) / (t.shape[1] * dim) + 1e-3)
    wq, wk = w.double().cpu()[:H * D].view(H, D), w.double().cpu()[H * D:].view(G, D)
    _close(q, _turn(unit(x[:, :H]) * wq, pos, f).flatten(1), dtype)
    _close(kv[:, :G * D], _turn(unit(x[:, H:]) * wk, pos, f).flatten(1), dtype)
    assert torch.equal(kv[:, G * D:], wide[:, H * D:cols])                 # as projected
    _check_slots(cache, kv)


# ------------------------------------------------------------------ attention that turns back
def _window_softmax(q, k, v, low, scale, sink=None):
    """q (D), k and v of the keys low .. end."""
    s = torch.cat([k[low:] @ q * scale] + ([] if sink is None else [sink[None]]))
    return torch.softmax(s, 0)[:len(k) - low] @ v[low:]


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,G,D,V,BS,window", [(1, 1, 32, 16, 16, 1), (6, 3, 64, 48, 64, 95), (34, 2, 160, 144, 16, 33), (16, 1, 128, 128, 48, 96),
                                               (8, 8, 32, 256, 32, 300), (40, 2, 256, 96, 64, 512), (4, 2, 64, 64, 16, 5000), (2, 1, 264, 264, 16, 31)])
def test_single_tokens_turn_back(dev, dtype, H, G, D, V, BS, window):
    """Ragged contexts over scattered pages; queries point at the oldest key they see, the one just before that, or
    one at a page's border; with and without sinks."""
    from zipage_amd.layers import attention_form, grouped_rows_attention
    ctx = [1, 2, 31, 32, 33, BS, BS + 1, 95, 96, 97, 98, 300, 0, 511, 512, 513, 640]
    n, B, NB = len(ctx), len(ctx) + 2, -(-640 // BS)
    pages = B * NB + 3
    g = torch.Generator().manual_seed(H * D)
    tables = torch.randperm(pages, generator=g)[:B * NB].view(B, NB).int()
    trows = torch.randperm(B, generator=g)[:n].int()
    cache, q = _rand("cpu", dtype, pages, BS, G * (D + V), seed=1), _rand("cpu", dtype, n, H, D, seed=2, std=0.5)
    sinks, f, scale = _rand("cpu", F32, H, seed=3, std=3.0), _freqs("cpu", V // 2, 40.0), D ** -0.5
    flat = cache.view(-1, G * (D + V))
    low = [max(0, c - window) for c in ctx]
    for i, c in enumerate(ctx):
        rows = flat[[int(tables[trows[i], t // BS]) * BS + t % BS for t in range(c)]].double()
        key = (low[i], low[i] - 1, (c - 1) // BS * BS)[i % 3]
        for h in range(H if key >= 0 and c else 0):
            if h % 4:
                k = rows[key, h // (H // G) * D:][:D]
                q[i, h] = (k * (8.0 / (scale * float(k @ k)))).to(dtype)
    want = {}
    for sink in (None, sinks.double()):
        o = torch.zeros(n, H, V, dtype=torch.float64)
        for i, c in enumerate(ctx):
            rows = flat[[int(tables[trows[i], t // BS]) * BS + t % BS for t in range(c)]].double()
            for h in range(H if c else 0):
                b = h // (H // G)
                o[i, h] = _window_softmax(q[i, h].double(), rows[:, b * D:(b + 1) * D], rows[:, G * D + b * V:][:, :V], low[i], scale,
                                          None if sink is None else sink[h])
        want[sink is None] = _turn(o, torch.tensor([c - 1 for c in ctx]), f, back=True, adjacent=True) * 1.5
    for i, c in enumerate(ctx):                  # entries in front of what is seen are never read
        if c:
            tables[trows[i], :low[i] // BS] = -1
    t = lambda a: torch.as_tensor(a, dtype=torch.int32).to(dev)
    a = _angles(torch.tensor([c - 1 for c in ctx]), f)[:, 0]
    turns = torch.stack([a.cos(), a.sin()], -1).float().to(dev)

    def run(rows, sink):
        wide = torch.full((len(rows), H * V + 8), 3.0, dtype=dtype, device=dev)
        grouped_rows_attention(q[rows].flatten(1).to(dev), cache.to(dev), H, G, D, V, t(tables), t([ctx[i] for i in rows]), scale,
                               wide[:, :H * V], window=window, sinks=sink, table_rows=t([int(trows[i]) for i in rows]), out_scale=1.5,
                               form=attention_form(turns=turns[rows].contiguous()))
        torch.cuda.synchronize()
        assert (wide[:, H * V:] == 3).all()
        return wide[:, :H * V].view(len(rows), H, V)
    live, tol = [i for i, c in enumerate(ctx) if c], 2.0 if dtype == BF16 else 4.0
    for sink in (None, sinks.to(dev)):
        got = run(list(range(n)), sink)
        assert not got[ctx.index(0)].any()
        _close(got[live], want[sink is None][live], dtype, tol)
        for i in (4, 11, 16):                    # one token at a time: other splits of the keys
            _close(run([i], sink), want[sink is None][i:i + 1], dtype, tol)


@pytest.mark.parametrize("H,G,D,V,window", [(1, 1, 32, 32, 100), (6, 3, 64, 88, 33), (8, 2, 128, 128, 1), (3, 1, 160, 136, 128), (4, 4, 256, 256, 200),
                                            (9, 3, 96, 48, 64), (10, 2, 64, 16, 4096), (2, 2, 192, 128, 65)])
def test_runs_turn_back(dev, H, G, D, V, window):
    """Runs at the start, behind cached context and of all lengths about a tile's; queries that point at the first key
    inside and outside the window."""
    import numpy as np
    from zipage_amd.engine.inputs import plan_runs
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import attention_form, run_attention
    BS, parts, page = 16, [], 0
    for start, count in ((0, 127), (0, 128), (0, 129), (45, 16), (300, 257), (7, 300), (1, 2)):
        s = Sequence([0] * (start + count), block_size=BS)
        need = -(-(start + count) // BS)
        s.block_table = list(range(page, page + need))
        page += need
        parts.append(Portion(s, start, count))
    runs = plan_runs(parts, BS, window)
    total, scale, rep = sum(p.count for p in parts), D ** -0.5, torch.arange(H) // (H // G)
    k, v = _rand("cpu", BF16, page * BS, G, D, seed=1), _rand("cpu", BF16, page * BS, G, V, seed=2)
    q, f = _rand("cpu", BF16, total, H, D, seed=3, std=0.5), _freqs("cpu", V // 2, 40.0)
    want, pos, r = torch.empty(total, H, V, dtype=torch.float64), [], 0
    for p in parts:
        base, m = p.seq.block_table[0] * BS, p.start + p.count
        for i, t in enumerate(range(p.start, m)):
            low = max(0, t - window + 1)
            key = (low, low - 1, t)[t % 3]
            if key >= 0:
                row = k[base + key][rep].float()
                q[r + i, 1:] = (row * (8.0 / (scale * (row * row).sum(-1, keepdim=True)))).to(BF16)[1:]
        kk, vv, at = k[base:base + m].double(), v[base:base + m].double(), torch.arange(p.start, m)
        far = at[:, None] - torch.arange(m)[None]
        for h in range(H):
            sc = (q[r:r + p.count, h].double() @ kk[:, rep[h]].T * scale).masked_fill((far < 0) | (far >= window), float("-inf"))
            want[r:r + p.count, h] = torch.softmax(sc, -1) @ vv[:, rep[h]]
        pos.append(at)
        r += p.count
    want = _turn(want, torch.cat(pos), f, back=True, adjacent=True)
    if runs.key_slots is None:
        runs.key_slots = np.concatenate([np.arange(p.start, p.start + p.count) + p.seq.block_table[0] * BS for p in parts])
    slots = torch.as_tensor(runs.key_slots).long()
    kv = torch.cat([k[slots].flatten(1), v[slots].flatten(1)], dim=1).to(dev)
    a = _angles(torch.cat(pos), f)[:, 0]
    turns = torch.stack([a.cos(), a.sin()], -1).float().to(dev)
    out = torch.full((total, H * V + 16), float("nan"), dtype=BF16, device=dev)
    run_attention(q.flatten(1).to(dev), kv, H, G, D, V, torch.as_tensor(runs.tiles).to(dev), scale, out[:, :H * V], window=window,
                  form=attention_form(turns=turns))
    _close(out[:, :H * V].view(total, H, V), want, BF16, 2.0)


# ------------------------------------------------------------------ linear attention
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("run_min", [None, 16, 2])
@pytest.mark.parametrize("gated", [True, False], ids=["gated", "retention"])
@pytest.mark.parametrize("H,D,V,rot", [(3, 20, 24, 10), (2, 64, 64, 64), (1, 128, 128, 0), (300, 32, 40, 18), (2, 40, 136, 40), (1, 130, 250, 130),
                                       (5, 8, 96, 2), (2, 100, 8, 36)])
def test_linear_attention(dev, dtype, run_min, gated, H, D, V, rot):
    """Prompts against token by token against portions, in blocks and token by token, states in slots that others used
    before; channels that keep everything beside some that forget within a token."""
    from zipage_amd.layers import LinearAttention, Rotary
    W, n, eps, tau = 64, 70, 1e-3, 3.0
    r = lambda *s, seed, std=1.0: _rand("cpu", dtype, *s, seed=seed, std=std)
    decay = tuple([0.0, 1.0, 0.5, 0.97, 0.999][i % 5] for i in range(H))
    turning = not gated and rot > 0
    m = LinearAttention(W, H, D, V, eps, q_scale=0.7, k_scale=1.3, tau=tau if gated else None, decay=None if gated else decay,
                        rotary=Rotary(200.0, rot) if turning else None, weighted=gated)
    w = {k: r(*s, seed=i, std=.2) for i, (k, s) in enumerate(m.shapes(5).items())}
    if gated:
        w["norm"], w["a1"], w["a2.b"] = 1 + r(V, seed=20, std=.3), r(5, W, seed=21, std=.1), 6 * r(H * D, seed=22)
    into, _ = m.load(w, dtype, dev, W)
    h = r(len(CUTS), n, W, seed=23).to(dev)
    proj = (h.flatten(0, 1).float() @ into.to(dev).float().T).to(dtype).view(len(CUTS), n, -1)
    state = m.allocate(len(CUTS) + 2, dtype, dev).fill_(float("nan"))
    Dp, Vp = m.dim_p, m.vdim_p

    def step(rows, seg):
        s, t = [a for a, _ in rows], [b for _, b in rows]
        wide = torch.full((len(rows), H * Vp + 8), 7.0, dtype=dtype, device=dev)
        m.scan(proj[s, t].contiguous(), state, seg, wide[:, :H * Vp])
        torch.cuda.synchronize()
        assert (wide[:, H * Vp:] == 7).all()
        return wide[:, :H * Vp].view(len(rows), H, Vp)[..., :V].clone()
    for slots in ([3, 0, 6, 1, 5, 2], [0, 1, 2, 3, 4, 5]):
        got = _scan_in_cuts(dev, step, n, CUTS, slots, run_min)
        for s in range(len(CUTS)):
            P = proj[s].double().cpu()
            part = lambda at, d, dp: P[:, at:at + H * dp].reshape(n, H, dp)[..., :d]
            q, k = part(0, D, Dp) * 0.7, part(H * Dp, D, Dp) * 1.3
            if turning:
                q, k = (_turn(x, torch.arange(n), m.freqs) for x in (q, k))
            if gated:                            # the low-rank product's rounding is the library's: take its rows
                low = torch.nn.functional.linear(proj[s][:, m.low_at:m.low_at + m.low_rank], m.low).double().cpu()
                z = low.view(n, H, Dp)[..., :D] + w["a2.b"].double().view(H, D)
                alpha = torch.sigmoid(z) ** (1 / tau)
            else:
                alpha = torch.tensor(decay, dtype=torch.float64)[None, :, None].expand(n, H, D)
            o = O.rms(O.linear_recurrence(q, k, part(2 * H * Dp, V, Vp), alpha), eps)
            o = o * (w["norm"].double() if gated else 1) * O.silu(part(2 * H * Dp + H * Vp, V, Vp))
            # a read-out near zero, normed, amplifies rounding
            _close(got[s].flatten(1), o.flatten(1), dtype, 1.0 if dtype == BF16 else 512.0)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_far_tokens_of_a_recurrence(dev, dtype):
    """A token far back that alone has the direction asked for: what is left of it is exactly its decay."""
    from zipage_amd.layers import LinearAttention, Rotary
    n, H, D = 600, 2, 32
    m = LinearAttention(D, H, D, D, 0.0, decay=(0.999, 0.98), rotary=Rotary(50.0, 16))
    proj = torch.zeros(n, 4 * H * D)
    proj[:, 2 * H * D:3 * H * D] = _rand("cpu", F32, n, H * D, seed=1)          # values
    proj[:, 3 * H * D:] = 1.0
    for h in range(H):
        proj[:, H * D + h * D + 20] = 1.0                                        # keys: channel 20, which does not turn
        proj[3, H * D + h * D + 20] = 0.0
        proj[3, H * D + h * D + 21] = 1.0                                        # but token 3: channel 21
        proj[n - 40:, h * D + 21] = 1.0                                          # late queries ask for it alone
    m.load({k: torch.zeros(*s) for k, s in m.shapes().items()}, dtype, dev, D)
    proj = proj.to(dtype).to(dev)
    seg = lambda *a: types.SimpleNamespace(**_segments_of(dev, *a))
    v = proj[3, 2 * H * D:3 * H * D].double().cpu().view(H, D)
    want = (v / v.square().mean(-1, keepdim=True).sqrt() * torch.sigmoid(torch.ones(1).double())).flatten()
    for cuts in ([n], [n - 1, 1], [n - 30, 7, 23], [37] * 16 + [8]):
        state, at, rows = m.allocate(2, dtype, dev).fill_(float("nan")), 0, []
        for c in cuts:
            out = torch.empty(c, H * D, dtype=dtype, device=dev)
            m.scan(proj[at:at + c], state, seg(c, 1, at, dtype), out)
            rows.append(out)
            at += c
        got = torch.cat(rows)
        assert at == n
        _close(got[n - 40:], want.expand(40, -1), dtype, 1.0 if dtype == BF16 else 8.0)


def _segments_of(dev, count, slot, start, dtype):
    from zipage_amd.engine.qwen3 import Segments
    t = [torch.tensor([a], dtype=torch.int32, device=dev) for a in (0, count, slot, start)]
    s = Segments(*t, first_row=0, longest=count, max_count=int(count == 1))
    run = dtype == BF16 and count >= 16
    return dict(segments=None if run else s, run_segments=s if run else None)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_inert_segments_leave_states_alone(dev, dtype):
    """The padding of a decode batch: rows without a token write zeros and touch no state."""
    from zipage_amd.engine.qwen3 import Segments
    from zipage_amd.layers import LinearAttention
    m = LinearAttention(32, 2, 32, 32, 1e-3, tau=2.0, weighted=True)
    r = lambda *s: _rand("cpu", dtype, *s, seed=len(s), std=.2)
    into, _ = m.load({k: r(*s) for k, s in m.shapes(4).items()}, dtype, dev, 32)
    h = _rand(dev, dtype, 4, 32, seed=2)
    proj, state = (h.float() @ into.to(dev).float().T).to(dtype), m.allocate(5, dtype, dev)
    t = lambda *a: torch.tensor(a, dtype=torch.int32, device=dev)
    out = torch.full((4, 64), 9.0, dtype=dtype, device=dev)
    m.scan(proj, state, types.SimpleNamespace(
        segments=Segments(None, t(1, 0, 900, 0), t(1, 4, 2, 4), t(0, 0, 0, 0), max_count=1), run_segments=None), out)
    assert not out[1].any() and not out[3].any() and out[0].any() and out[2].any()
    assert not state[[0, 3, 4]].any() and state[1].any() and state[2].any()


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
    tmp, made = tmp_path_factory.mktemp("mefupel"), {}

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
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_layer_streams(dev, engines, name, dtype):
    """The stream after every pass of every layer, a whole prompt in one step."""
    from zipage_amd.engine import Portion
    cfg, w = C.case(name)
    toks = C.tokens(cfg, 120, 9)
    eng = engines(name, dtype)
    s = eng.open_request()
    s.token_ids, s.num_tokens, s.num_prompt_tokens = list(toks), 120, 120
    eng.scheduler.pool.grow(s, 120)
    i, p, ctx, _ = eng.runner.prepare_portions([Portion(s, 0, 120)])
    streams = []
    eng.runner.model.forward(i, p, ctx, trace=streams)
    eng.close_request(s)
    want = O.forward(cfg, w, toks)[1]
    assert len(streams) == len(want) == len(O.layer_runs(cfg))
    for got, ref in zip(streams, want):
        if dtype == F32:
            _close(got, ref, F32, 32.0)
        else:
            e = (got.double().cpu() - ref).square().mean(-1).sqrt() / ref.square().mean(-1).sqrt()
            assert float(e.median()) < 0.03 and float(e.quantile(0.9)) < 0.06


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("window", [40, 200])
@pytest.mark.parametrize("kind", ["turning", "keys"])
def test_far_keys_of_a_layer(dev, kind, window, dtype):
    """A mixer on pages: sharp scores, so that nearly each token's weight lies on one key anywhere in its window, in a
    prompt's portion and decoded alone; another page table must not matter."""
    from zipage_amd.engine.inputs import Runs, plan_portions
    from zipage_amd.engine.model_runner import StepContext
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import GroupedAttention, Rotary
    W, n, BS = 64, 200, 16
    if kind == "turning":
        m = C.attention(4, 2, 32, 48, window, 16, 2000.0)
        mix = GroupedAttention(W, 4, 2, 32, 48, m["scale"], window, Rotary(2000.0, 16, interleaved=True), turn_values=True)
    else:
        m = C.attention(4, 2, 40, 40, window, 16, 2000.0)
        mix = GroupedAttention(W, 4, 2, 40, 40, m["scale"], window, Rotary(2000.0, 16), sinks=True, eps=1e-5, qk_norm=True, tied=True)
    w = {k: _rand("cpu", BF16, *s, seed=i, std=s[-1] ** -0.5 if len(s) == 2 else 1.0) for i, (k, s) in enumerate(mix.shapes().items())}
    w["q" if kind == "turning" else "q.norm"] *= 14.0
    h = _rand("cpu", BF16, n, W, seed=50)
    into, out = mix.load(w, dtype, dev, W)
    into, out = into.to(dev, dtype), out.to(dev, dtype)
    w64 = {k: v.double() for k, v in w.items()}
    want = O.rotated_value_attention(h.double(), w64, m) if kind == "turning" else O.key_value_attention(h.double(), w64, m, 1e-5)
    for seed, cuts in ((0, [n]), (1, [150, 50]), (2, [180, 2, 17, 1]), (3, [199, 1]), (4, [39, 1, 1, 38, 41, 2, 78])):
        cache = mix.allocate(20, BS, dtype, dev)
        cache.fill_(float("nan"))                                       # what nobody wrote must not be read
        table = torch.randperm(20, generator=torch.Generator().manual_seed(seed))[:-(-n // BS)].tolist()
        at, got = 0, []
        for c in cuts:
            s = Sequence([0] * (at + c), block_size=BS)
            s.block_table = table
            plan = plan_portions([Portion(s, at, c)], BS, [window], 16 if dtype == BF16 else None)
            t = lambda a: None if a is None else torch.as_tensor(a).to(dev)
            ctx = StepContext(False, t(plan.slots), None, t(plan.context_lens), t(plan.tables), table_rows=t(plan.table_rows),
                              runs={k: Runs(t(r.tiles), t(r.key_slots)) for k, r in plan.runs.items()})
            mixed = torch.empty(c, mix.out_columns, dtype=dtype, device=dev)
            mix.attend(torch.nn.functional.linear(h[at:at + c].to(dev, dtype), into), t(plan.positions), cache, ctx, mixed)
            got.append(torch.nn.functional.linear(mixed, out).float())
            at += c
        got = torch.cat(got).double().cpu()
        e = (got - want).square().mean(-1).sqrt() / want.square().mean(-1).sqrt()
        assert float(e.max()) < (5e-5 if dtype == F32 else 0.3), (cuts, float(e.max()))
        assert float(e.median()) < (2e-6 if dtype == F32 else 0.05), (cuts, float(e.median()))


@pytest.mark.parametrize("name,dtype", [("odd", F32), ("ends", F32), ("calm", F32), ("calm", BF16), ("wide", BF16)], ids=ids)
def test_first_tokens_and_page_borders(dev, engines, name, dtype):
    for n in (1, 2, 15, 16, 17, 33, 38):
        toks = C.tokens(C.CONFIGS[name], n, 20 + n)
        C.close(name, _feed_all(engines(name, dtype), toks, [n]), C.expected(name, toks), dtype)
        C.close(name, _feed_all(engines(name, dtype), toks, [n - 1 or 1, 1]), C.expected(name, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_long_decoding(dev, engines, dtype):
    """Many windows of decoded tokens; the pages behind them are given back on the way."""
    cfg = C.CONFIGS["calm"]
    toks = C.tokens(cfg, 400, 5)
    eng = engines("calm", dtype)
    s = eng.open_request()
    got = [eng.feed([(s, toks[:20], [19])]).clone()]
    for t in range(20, 400):
        got.append(eng.feed([(s, toks[t:t + 1], [0])]).clone())
        assert 64 - eng.scheduler.pool.num_free <= 6           # a window of 70 tokens, 16 a page
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


@pytest.mark.parametrize("name", ["calm", "odd"])
def test_graph_replays_equal_eager_steps(dev, engines, name):
    """The same decode steps through replayed graphs and eagerly, with other work in between."""
    eng, eager = engines(name, BF16), engines(name, BF16, use_graph=False)
    toks = [C.tokens(C.CONFIGS[name], 90, 60 + i) for i in range(3)]
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
    from zipage_amd.layers import attention_form, normed_powers, residual_norm, run_attention
    t = lambda *s: torch.zeros(*s, dtype=BF16, device=dev)
    x, w = torch.zeros(2, 64, device=dev), torch.ones(64, device=dev)
    with pytest.raises(RuntimeError, match="normed"):            # at most two branches are
        residual_norm(x, t(2, 64), w, 1e-3, 64, y_weight=w, more=((t(2, 64), w), (t(2, 64), w)))
    with pytest.raises(RuntimeError, match="32768"):
        normed_powers(t(1, 32776), (1, 1, 1, 1), 1e-3, 32776, t(1, 32776))
    with pytest.raises(RuntimeError, match="soft cap"):          # turns go with plain scores
        run_attention(t(4, 32), t(4, 48), 1, 1, 32, 16, torch.tensor([[0, 4, 0, 0]], dtype=torch.int32, device=dev), 1.0, t(4, 16),
                      form=attention_form(5.0, turns=torch.zeros(4, 8, 2, device=dev)))


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
    for again in range(2):                     # the second time meets used pages and slots
        outs = eng.generate(prompts, [SamplingParams(max_tokens=c, ignore_eos=True) for c in counts])
        for p, c, o in zip(prompts, counts, outs):
            assert len(o["token_ids"]) == c
            _greedy_ok("odd", p, o["token_ids"], 1e-3)
    pool = eng.scheduler.pool
    assert pool.num_free == pool.num_pages and pool.reserved == 0
    assert eng.stats["decode_tokens"] + eng.stats["mixed_decode_tokens"] == 2 * sum(c - 1 for c in counts)
    assert eng.stats["prefill_tokens"] == 2 * sum(map(len, prompts))


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
