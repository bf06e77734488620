"""Rutevik on the GPU: every mechanism alone, the model against the oracle in every way a sequence can be cut
and batched, and generation through the engine."""
import io
import json

import pytest
import torch

from oracle import rutevik_oracle as O
from tests import rutevik_cases as C

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


def _turn(x, positions, freqs):
    """x (n, heads, dim), fp32 angles."""
    half = freqs.numel()
    a = (positions.cpu().float()[:, None] * freqs.cpu()).double()[:, None]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), x[..., 2 * half:]], -1)


def _freqs(dev, n, base=300.0):
    return torch.tensor([base ** (-i / max(n, 1)) for i in range(n)], device=dev)


# ------------------------------------------------------------------ row steps
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,width,norm_width", [(1, 96, 76), (3, 512, 512), (17, 1024, 1000), (2, 8192, 8192)])
def test_tanh_norm(dev, dtype, n, width, norm_width):
    """Behind the embedding and behind the residual add of several planes; arguments from 1e-4 to far out."""
    from zipage_amd.layers import embed_norm, residual_norm
    embed = _rand(dev, dtype, 11, width, seed=1)
    embed *= torch.logspace(-4, 1.5, 11, device=dev)[:, None].to(dtype)
    w, b = _rand(dev, F32, width, seed=3), _rand(dev, F32, width, seed=4, std=0.1)
    for t in (embed.T, w, b):
        t[norm_width:] = 0
    tok, at = torch.arange(n, device=dev) % 11, torch.zeros(n, dtype=torch.int32, device=dev)
    x = torch.empty(n, width, device=dev)
    want = embed.double()[tok]
    h = embed_norm(tok, at, embed, None, x, w, 1e-3, norm_width, norm_bias=b, norm_alpha=0.8)
    _close(h, O.dyt(want, w.double(), b.double(), 0.8), dtype)
    assert torch.equal(x, embed[tok].float())
    for planes in (1, 3):
        y = _rand(dev, dtype, planes, n, width, seed=5)
        y[..., norm_width:] = 0
        want = x.double() + y.double().sum(0)
        after = torch.empty_like(x)
        h = residual_norm(x, y, w, 1e-3, norm_width, out_scale=0.4, x_out=after, norm_bias=b, norm_alpha=0.3)
        _close(after, want, F32)
        _close(h, O.dyt(want, w.double(), b.double(), 0.3) * 0.4, dtype)
        assert not h[:, norm_width:].any()


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_tanh_norm_keeps_small_arguments(dev, dtype):
    """Every element on its own, relative: a difference of near-equal terms would lose the small ones."""
    from zipage_amd.layers import residual_norm
    x = torch.logspace(-6, 2, 4096, device=dev).view(1, -1) * torch.tensor([1.0, -1.0], device=dev).repeat(2048)
    one, none = torch.ones(4096, device=dev), torch.zeros(4096, device=dev)
    h = residual_norm(x, torch.zeros(1, 4096, device=dev, dtype=dtype), one, 0.0, 4096, norm_bias=none, norm_alpha=0.5)
    want = torch.tanh(0.5 * x.double())
    assert float(((h.double() - want) / want).abs().max()) < {BF16: 2.0 ** -8, F32: 1e-6}[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_relu_square(dev, dtype):
    from zipage_amd.layers import relu_square
    z = _rand(dev, dtype, 37, 88, seed=1, std=3.0)
    _close(relu_square(z), torch.relu(z.double()) ** 2, dtype)


# ------------------------------------------------------------------ rotary positions and stores
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,G,D,V,rot", [(4, 2, 24, 48, 16), (6, 3, 8, 16, 6), (5, 1, 48, 96, 48), (3, 3, 32, 32, 0)])
def test_rotary_store_with_bias_of_two_maps(dev, dtype, H, G, D, V, rot):
    from zipage_amd.layers import rotary_store
    n, BS = 7, 16
    cols = 2 * (H + G) * D + G * V
    wide = _rand(dev, dtype, n, cols + H * V, seed=1)              # a gate's columns follow
    bias = _rand(dev, F32, cols, seed=2)
    pos = torch.tensor([0, 1, 7, 100, 4095, 3, 50000], dtype=torch.int32, device=dev)
    slots = torch.tensor([5, -1, 47, 0, 12, 13, 48], dtype=torch.int32, device=dev)     # 48: past the end
    cache = torch.full((3, BS, G * (2 * D + V)), 7.0, dtype=dtype, device=dev)
    f = _freqs(dev, rot // 2)
    q, kv = rotary_store(wide[:, :cols], pos, f, H, G, D, V, cache, slots, return_kv=True, maps=2, bias=bias)
    x = (wide[:, :cols].double() + bias.double()).cpu()
    want = _turn(x[:, :2 * (H + G) * D].reshape(n, 2 * (H + G), D), pos, f).flatten(1)
    _close(q, want[:, :2 * H * D], dtype)
    _close(kv[:, :2 * G * D], want[:, 2 * H * D:], dtype)
    _close(kv[:, 2 * G * D:], x[:, 2 * (H + G) * D:], dtype)
    flat = cache.view(-1, G * (2 * D + V))
    kept = [i for i, s in enumerate(slots.tolist()) if 0 <= s < 48]
    assert torch.equal(flat[slots[kept].long()], kv[kept])
    assert (flat[sorted(set(range(48)) - set(slots[kept].tolist()))] == 7).all()


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("Q,R,P,rot,qn,cn", [(64, 96, 32, 32, 50, 90), (32, 32, 8, 2, 32, 32), (512, 544, 72, 70, 500, 530),
                                             (1536, 512, 0, 0, 1536, 512), (96, 0, 0, 0, 90, 0)])
def test_latent_norm_store(dev, dtype, Q, R, P, rot, qn, cn):
    from zipage_amd.layers.latent import latent_norm_store
    n = 7
    x = _rand(dev, dtype, n, Q + R + P, seed=1)
    x[:, qn:Q] = 0
    x[:, Q + cn:Q + R] = 0
    wq, wc = _rand(dev, F32, Q, seed=2), _rand(dev, F32, R, seed=3) if R else None
    pos = torch.tensor([0, 1, 7, 100, 4095, 3, 50000], dtype=torch.int32, device=dev)
    slots = torch.tensor([5, -1, 47, 0, 12, 13, 48], dtype=torch.int32, device=dev)
    cache = torch.full((3, 16, R + P), 7.0, dtype=dtype, device=dev) if R else None
    f = _freqs(dev, rot // 2) if rot else None
    out = latent_norm_store(x, wq, wc, qn, cn, 1e-2, cache, slots if R else None, return_c=R > 0, positions=pos, freqs=f)
    q, c = out if R else (out, None)
    part = lambda a, b, size, w: x[:, a:b].double() / torch.sqrt(x[:, a:b].double().square().sum(-1, keepdim=True) / size + 1e-2) * w.double()
    _close(q, part(0, Q, qn, wq), dtype)
    if not R:
        return
    _close(c[:, :R], part(Q, Q + R, cn, wc), dtype)
    if P:
        _close(c[:, R:], _turn(x[:, Q + R:].double().cpu()[:, None], pos, f)[:, 0], dtype)
    flat = cache.view(-1, R + P)
    kept = [i for i, s in enumerate(slots.tolist()) if 0 <= s < 48]
    assert torch.equal(flat[slots[kept].long()], c[kept])
    assert (flat[sorted(set(range(48)) - set(slots[kept].tolist()))] == 7).all()


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,H,K,M,tail,rot", [(1, 3, 32, 64, 8, 2), (37, 5, 64, 96, 32, 32), (130, 2, 128, 32, 72, 70), (9, 40, 32, 16, 16, 0)])
def test_headwise_product_and_turned_tail(dev, dtype, n, H, K, M, tail, rot):
    from zipage_amd.layers.latent import headwise_linear, rotate_heads
    x, w = _rand(dev, dtype, n, H, K + tail, seed=1), _rand(dev, dtype, H, M, K, seed=2)
    pos = (torch.arange(n, device=dev, dtype=torch.int32) * 37) % 5000
    f = _freqs(dev, rot // 2) if rot else None
    got = headwise_linear(x, w, positions=pos, freqs=f)
    want = torch.einsum("nhk,hmk->nhm", x[..., :K].double().cpu(), w.double().cpu())
    _close(got[..., :M], want, dtype, 2.0 if dtype == BF16 else 4.0)
    turned = _turn(x[..., K:].double().cpu(), pos, f) if rot else x[..., K:]
    _close(got[..., M:], turned, dtype)
    if rot:                                  # the same in place, as part of wider rows
        wide = torch.cat([x.flatten(1), torch.full((n, 8), 3.0, dtype=dtype, device=dev)], dim=1)
        rotate_heads(wide[:, :-8], pos, f, H, K)
        assert (wide[:, -8:] == 3).all()
        y = wide[:, :-8].view(n, H, K + tail)
        assert torch.equal(y[..., :K], x[..., :K])
        _close(y[..., K:], turned, dtype)


# ------------------------------------------------------------------ single tokens over pages
CTX = [1, 2, 31, 32, 33, 16, 17, 95, 96, 97, 300, 0, 511, 512, 513, 640]


def _paged(dtype, BS, row, seed):
    n, B, NB = len(CTX), len(CTX) + 2, -(-640 // BS)
    pages = B * NB + 3
    g = torch.Generator().manual_seed(seed)
    tables = torch.randperm(pages, generator=g)[:B * NB].view(B, NB).int()
    trows = torch.randperm(B, generator=g)[:n].int()
    cache = _rand("cpu", dtype, pages, BS, row, seed=1)
    flat = cache.view(-1, row)
    of = lambda i: flat[[int(tables[trows[i], t // BS]) * BS + t % BS for t in range(CTX[i])]].double()
    return tables, trows, cache, of


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,R,P,BS", [(1, 32, 8, 16), (5, 64, 32, 64), (40, 288, 64, 16), (17, 512, 64, 64), (20, 96, 24, 32),
                                      (3, 544, 16, 16), (4, 96, 72, 64), (16, 256, 48, 256), (33, 384, 64, 128)])
def test_latent_rows_with_a_rotated_part(dev, dtype, H, R, P, BS):
    """Ragged contexts over scattered pages; most queries point at one key, the oldest, the newest or one at a
    page's border, some through the rotated part alone."""
    from zipage_amd.layers import latent_rows_attention
    tables, trows, cache, of = _paged(dtype, BS, R + P, H * R)
    n, scale = len(CTX), (R + P) ** -0.5
    q = _rand("cpu", dtype, n, H, R + P, seed=2, std=0.5)
    want = torch.zeros(n, H, R, dtype=torch.float64)
    for i, c in enumerate(CTX):
        if c == 0:
            continue
        rows = of(i)
        key = (0, c - 1, (c - 1) // BS * BS)[i % 3]
        for h in range(H):
            if h % 3 == 1:
                q[i, h] = (rows[key] * (8.0 / (scale * float(rows[key] @ rows[key])))).to(dtype)
            elif h % 3 == 2:
                q[i, h, :R] = 0
                q[i, h, R:] = (rows[key, R:] * (8.0 / (scale * float(rows[key, R:] @ rows[key, R:])))).to(dtype)
        want[i] = torch.softmax(q[i].double() @ rows.T * scale, -1) @ rows[:, :R]
    t = lambda a: torch.as_tensor(a, dtype=torch.int32).to(dev)

    def run(which):
        return latent_rows_attention(q[which].to(dev), cache.to(dev), t(tables), t([CTX[i] for i in which]), scale,
                                     table_rows=t([int(trows[i]) for i in which]), rank=R)
    got = run(list(range(n)))
    assert not got[CTX.index(0)].any()
    live = [i for i, c in enumerate(CTX) if c]
    tol = 2.0 if dtype == BF16 else 4.0
    _close(got[live], want[live], dtype, tol)
    for i in (4, 10, 15):                        # one token at a time: other splits of the keys
        _close(run([i]), want[i:i + 1], dtype, tol)


def _pair(q1, q2, k1, k2, v, seen, scale, cap, balance, eps, vdim, diff_scale, gate):
    """One head over whole contexts: (queries, keys) masks, fp64."""
    o = []
    for q, k in ((q1, k1), (q2, k2)):
        s = O.capped(q @ k.T * scale, cap) if cap else q @ k.T * scale
        o.append(torch.softmax(s.masked_fill(~seen, float("-inf")), -1) @ v)
    o = o[0] - balance * o[1]
    o = o / torch.sqrt(o.square().sum(-1, keepdim=True) / vdim + eps) * diff_scale
    return o if gate is None else o * torch.sigmoid(gate)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,G,D,V,vdim,BS,cap,gated", [
    (1, 1, 8, 16, 16, 16, 3.0, True), (6, 3, 24, 48, 40, 64, 0.0, True), (34, 2, 72, 144, 144, 16, 20.0, True),
    (16, 1, 64, 128, 128, 48, 6.0, True), (8, 8, 40, 64, 57, 32, 2.0, False), (20, 2, 128, 96, 96, 64, 50.0, True),
    (4, 4, 136, 48, 48, 256, 9.0, True), (6, 2, 128, 256, 256, 16, 4.0, True), (12, 4, 32, 32, 32, 64, 90.0, True)])
def test_differential_rows(dev, dtype, H, G, D, V, vdim, BS, cap, gated):
    """Two maps over the same values; each map points at a key of its own; the soft cap bends large scores."""
    from zipage_amd.layers import attention_form, grouped_rows_attention
    tables, trows, cache, of = _paged(dtype, BS, G * (2 * D + V), H * D)
    cache[..., 2 * G * D:].view(*cache.shape[:2], G, V)[..., vdim:] = 0
    n, scale, balance, eps = len(CTX), D ** -0.5, 0.4, 1e-3
    q = _rand("cpu", dtype, n, H, 2, D, seed=2, std=0.5)
    gate = _rand("cpu", dtype, n, H * V + 8, seed=3)
    want = torch.zeros(n, H, V, dtype=torch.float64)
    for i, c in enumerate(CTX):
        if c == 0:
            continue
        rows = of(i)
        k, v = rows[:, :2 * G * D].view(c, G, 2, D), rows[:, 2 * G * D:].view(c, G, V)
        key = (0, c - 1, (c - 1) // BS * BS)[i % 3]
        for h in range(H):
            b = h // (H // G)
            for j in range(2):
                if h % 4 > j:                    # the second map elsewhere
                    x = k[(key + j * (c // 2)) % c, b, j]
                    q[i, h, j] = (x * (8.0 / (scale * float(x @ x)))).to(dtype)
            want[i, h] = _pair(*q[i, h].double().unsqueeze(1), k[:, b, 0], k[:, b, 1], v[:, b], torch.ones(1, c, dtype=torch.bool),
                               scale, cap, balance, eps, vdim, 1.5, gate[i, h * V:(h + 1) * V].double() if gated else None)[0]
    t = lambda a: torch.as_tensor(a, dtype=torch.int32).to(dev)
    gate = gate.to(dev)

    def run(which):
        wide = torch.full((len(which), H * V + 8), 3.0, dtype=dtype, device=dev)
        own = gate[which].contiguous()
        form = attention_form(cap, 2, balance, eps, vdim, own[:, :H * V] if gated else None)
        grouped_rows_attention(q[which].flatten(1).to(dev), cache.to(dev), H, G, D, V, t(tables), t([CTX[i] for i in which]), scale,
                               wide[:, :H * V], table_rows=t([int(trows[i]) for i in which]), out_scale=1.5, form=form)
        torch.cuda.synchronize()
        assert (wide[:, H * V:] == 3).all()
        return wide[:, :H * V].view(len(which), H, V)
    got = run(list(range(n)))
    assert not got[CTX.index(0)].any()
    live = [i for i, c in enumerate(CTX) if c]
    tol = 3.0 if dtype == BF16 else 16.0
    _close(got[live], want[live], dtype, tol)
    for i in (4, 10, 15):
        _close(run([i]), want[i:i + 1], dtype, tol)


# ------------------------------------------------------------------ runs of prompt tokens
def _run_parts(BS):
    from zipage_amd.engine.inputs import plan_runs
    from zipage_amd.engine.sequence import Portion, Sequence
    parts, page = [], 0
    for start, count in ((0, 127), (0, 128), (0, 129), (45, 16), (300, 257), (7, 300), (1, 2)):
        s = Sequence([0] * (start + count), block_size=BS)
        need = -(-(start + count) // BS)
        s.block_table = list(range(page, page + need))
        page += need
        parts.append(Portion(s, start, count))
    return parts, page * BS, plan_runs(parts, BS, None)


@pytest.mark.parametrize("H,D,P,V", [(1, 32, 8, 16), (6, 24, 40, 88), (8, 128, 64, 128), (3, 64, 32, 144), (4, 192, 64, 256), (5, 40, 24, 64)])
def test_run_attention_with_a_shared_key_part(dev, H, D, P, V):
    from zipage_amd.layers.latent import latent_tiles_attention
    parts, rows, runs = _run_parts(16)
    total = sum(p.count for p in parts)
    k, v, ks = (_rand("cpu", BF16, rows, H, D, seed=1), _rand("cpu", BF16, rows, H, V, seed=2), _rand("cpu", BF16, rows, P, seed=5))
    q = _rand("cpu", BF16, total, H, D + P, seed=3, std=0.5)
    scale, want, r = (D + P) ** -0.5, torch.empty(total, H, V, dtype=torch.float64), 0
    for p in parts:
        base, m = p.seq.block_table[0] * 16, p.start + p.count
        kk = torch.cat([k[base:base + m], ks[base:base + m, None].expand(m, H, P)], -1)
        for i, t in enumerate(range(p.start, m)):
            key = kk[(0, t, t // 2)[t % 3]].float()
            if i % 2:                            # through the shared part alone
                q[r + i, :, :D] = 0
                q[r + i, :, D:] = (key[:, D:] * (8.0 / (scale * key[:, D:].square().sum(-1, keepdim=True)))).to(BF16)
            else:
                q[r + i] = (key * (8.0 / (scale * key.square().sum(-1, keepdim=True)))).to(BF16)
        seen = torch.arange(m)[None] <= torch.arange(p.start, m)[:, None]
        for h in range(H):
            sc = (q[r:r + p.count, h].double() @ kk[:, h].double().T * scale).masked_fill(~seen, float("-inf"))
            want[r:r + p.count, h] = torch.softmax(sc, -1) @ v[base:base + m, h].double()
        r += p.count
    slots = torch.as_tensor(runs.key_slots).long()
    held = torch.cat([torch.zeros(len(slots), 8, dtype=BF16), ks[slots]], dim=1).to(dev)      # part of wider rows
    out = torch.full((total, H * V), float("nan"), dtype=BF16, device=dev)
    latent_tiles_attention(q.flatten(1).to(dev), torch.cat([k[slots].flatten(1), v[slots].flatten(1)], 1).to(dev), H, D, V,
                           torch.as_tensor(runs.tiles).to(dev), scale, None, out, held[:, 8:])
    _close(out.view(total, H, V), want, BF16, 2.0)


@pytest.mark.parametrize("H,G,D,V,vdim,cap,gated", [(1, 1, 8, 16, 16, 3.0, True), (6, 3, 24, 48, 40, 0.0, True), (8, 2, 64, 128, 128, 30.0, True),
                                                    (3, 1, 128, 144, 130, 5.0, False), (4, 4, 96, 256, 256, 80.0, True), (10, 5, 128, 64, 64, 2.0, True)])
def test_differential_runs(dev, H, G, D, V, vdim, cap, gated):
    from zipage_amd.layers import attention_form, run_attention
    parts, rows, runs = _run_parts(16)
    total, scale, balance, eps = sum(p.count for p in parts), D ** -0.5, 0.4, 1e-3
    k, v = _rand("cpu", BF16, rows, G, 2, D, seed=1), _rand("cpu", BF16, rows, G, V, seed=2)
    v[..., vdim:] = 0
    q, gate = _rand("cpu", BF16, total, H, 2, D, seed=3, std=0.5), _rand("cpu", BF16, total, H * V + 16, seed=4)
    want, r, rep = torch.empty(total, H, V, dtype=torch.float64), 0, torch.arange(H) // (H // G)
    for p in parts:
        base, m = p.seq.block_table[0] * 16, p.start + p.count
        for i, t in enumerate(range(p.start, m)):
            for j, key in enumerate(((0, t, t // 2)[t % 3], (t // 3, 0, t)[t % 3])):
                if (t + j) % 4:
                    x = k[base + key][rep, j].float()
                    q[r + i, :, j] = (x * (8.0 / (scale * x.square().sum(-1, keepdim=True)))).to(BF16)
        kk, vv = k[base:base + m].double(), v[base:base + m].double()
        seen = torch.arange(m)[None] <= torch.arange(p.start, m)[:, None]
        for h in range(H):
            b, mine = rep[h], slice(r, r + p.count)
            want[mine, h] = _pair(q[mine, h, 0].double(), q[mine, h, 1].double(), kk[:, b, 0], kk[:, b, 1], vv[:, b], seen, scale, cap,
                                  balance, eps, vdim, 0.75, gate[mine, h * V:(h + 1) * V].double() if gated else None)
        r += p.count
    slots = torch.as_tensor(runs.key_slots).long()
    out = torch.full((total, H * V + 16), float("nan"), dtype=BF16, device=dev)
    gate = gate.to(dev)
    run_attention(q.flatten(1).to(dev), torch.cat([k[slots].flatten(1), v[slots].flatten(1)], 1).to(dev), H, G, D, V,
                  torch.as_tensor(runs.tiles).to(dev), scale, out[:, :H * V], out_scale=0.75,
                  form=attention_form(cap, 2, balance, eps, vdim, gate[:, :H * V] if gated else None))
    _close(out[:, :H * V].view(total, H, V), want, BF16, 3.0)


@pytest.mark.parametrize("cap", [4.0, 50.0, 90.0])
@pytest.mark.parametrize("low", [False, True], ids=["spread", "low"])
def test_soft_cap_of_one_map(dev, cap, low):
    """Scores all over the cap's range, and all of them deep below zero, where a softmax without a running maximum
    has only tiny weights; with a sink that is as low."""
    from zipage_amd.layers import attention_form, grouped_rows_attention, run_attention
    parts, rows, runs = _run_parts(16)
    H, G, D, V, scale = 6, 2, 64, 64, 0.125
    total = sum(p.count for p in parts)
    k, v, q = _rand("cpu", BF16, rows, G, D, seed=1), _rand("cpu", BF16, rows, G, V, seed=2), _rand("cpu", BF16, total, H, D, seed=3)
    sinks = torch.linspace(-2.0, 2.0, H)
    if low:                                      # every key near one direction, every query against it
        k, q = 1 + 0.1 * k, -1.1 * cap / (scale * D) + 0.2 * q
        sinks -= 0.8 * cap
    want, r = torch.empty(total, H, V, dtype=torch.float64), 0
    for p in parts:
        base, m = p.seq.block_table[0] * 16, p.start + p.count
        seen = torch.arange(m)[None] <= torch.arange(p.start, m)[:, None]
        for h in range(H):
            sc = O.capped(q[r:r + p.count, h].double() @ k[base:base + m, h // 3].double().T * scale, cap)
            sc = torch.cat([sc.masked_fill(~seen, float("-inf")), sinks[h].double().expand(p.count, 1)], -1)
            want[r:r + p.count, h] = torch.softmax(sc, -1)[:, :-1] @ v[base:base + m, h // 3].double()
        r += p.count
    kv = torch.cat([k.flatten(1), v.flatten(1)], 1)
    t = lambda a: torch.as_tensor(a, dtype=torch.int32).to(dev)
    out = torch.full((total, H * V), float("nan"), dtype=BF16, device=dev)
    run_attention(q.flatten(1).to(dev), kv[torch.as_tensor(runs.key_slots).long()].to(dev), H, G, D, V, t(runs.tiles), scale, out,
                  sinks=sinks.to(dev), form=attention_form(cap))
    _close(out.view(total, H, V), want, BF16, 3.0)
    # the last token of every part, singly
    ends = torch.tensor([p.count for p in parts]).cumsum(0) - 1
    width = max(len(p.seq.block_table) for p in parts)
    tables = t([p.seq.block_table + [-1] * (width - len(p.seq.block_table)) for p in parts])
    for dtype in DTYPES:
        out = torch.full((len(parts), H * V), float("nan"), dtype=dtype, device=dev)
        grouped_rows_attention(q[ends].flatten(1).to(dev, dtype), kv.view(-1, 16, kv.shape[1]).to(dev, dtype), H, G, D, V, tables,
                               t([p.start + p.count for p in parts]), scale, out, sinks=sinks.to(dev), form=attention_form(cap))
        _close(out.view(-1, H, V), want[ends], dtype, 3.0 if dtype == BF16 else 64.0)


# ------------------------------------------------------------------ experts
@pytest.mark.parametrize("E,top", [(3, 3), (16, 1), (70, 5), (300, 8)])
def test_sigmoid_choice(dev, E, top):
    from zipage_amd import _lib
    from zipage_amd.layers.moe import moe_select
    z = _rand(dev, F32, 37, E + 4, seed=E, std=2.0)
    ids_, wts, counts = moe_select(z, E, top, score=_lib.SCORE_SIGMOID)
    want = O.route(z[:, :E].double().cpu(), top)
    got = torch.zeros(37, E, dtype=torch.float64).scatter_(1, ids_.long().cpu(), wts.double().cpu())
    assert float((got - want).abs().max()) < 1e-6 and not counts.any()


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,width,E,top,ff", [(1, 96, 4, 1, 40), (7, 76, 10, 3, 44), (40, 160, 66, 4, 32), (300, 128, 3, 3, 72),
                                              (700, 256, 8, 2, 160)])
def test_experts_weighted_at_their_input(dev, dtype, n, width, E, top, ff):
    """From a row per expert to tiles of 128."""
    from zipage_amd.layers import Experts
    m = Experts(width, E, top, ff, 0.0, score="sigmoid", act="silu")
    w = {k: _rand("cpu", BF16, *s, seed=i, std=2.0 * s[-1] ** -0.5) for i, (k, s) in enumerate(m.shapes().items())}
    m.load(w, dtype, dev)
    h = torch.zeros(n, m.width_p, dtype=dtype, device=dev)
    h[:, :width] = _rand(dev, dtype, n, width, seed=99)
    x, w64 = h[:, :width].double().cpu(), {k: v.double() for k, v in w.items()}
    z = x @ w64["router"].T
    gap = z.sort(-1, descending=True).values
    sure = torch.ones(n, dtype=torch.bool) if top == E else gap[:, top - 1] - gap[:, top] > 1e-3
    got = m.forward(h).double().sum(0)[:, :width].cpu()
    want = O.experts(x, w64, C.moe(E, top, ff))
    assert int(sure.sum()) >= 0.8 * n
    _close(got[sure], want[sure], dtype, 3.0 if dtype == BF16 else 16.0)


# ------------------------------------------------------------------ the model
def _engine(name, dtype, tmp, **kw):
    from zipage_amd.engine import EngineConfig, ZipageEngine, read_shape
    from zipage_amd.engine.weights import write_safetensors
    cfg, w = C.case(name)
    folder = tmp / name
    if not folder.exists():
        folder.mkdir()
        (folder / "config.json").write_text(json.dumps(cfg))
        write_safetensors(str(folder / "model.safetensors"), w)
    base = dict(shape=read_shape(str(folder)), model_folder=str(folder), dtype=dtype, num_kvcache_blocks=64,
                kvcache_block_size=16, max_concurrency=6, max_model_len=1024)
    base.update(kw)
    return ZipageEngine(EngineConfig(**base))


@pytest.fixture(scope="module")
def engines(tmp_path_factory):
    """Engines by (case, dtype), kept for the module: pages and slots are used again and again."""
    tmp, made = tmp_path_factory.mktemp("rutevik"), {}

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
@pytest.mark.parametrize("name", ["odd", "calm"])
def test_layer_streams(dev, engines, name, dtype):
    """The stream after every layer, a whole prompt in one step."""
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
    assert len(streams) == len(want) == len(cfg["layers"])
    for got, ref in zip(streams, want):
        if dtype == F32:
            _close(got, ref, F32, 32.0)
        else:
            e = (got.double().cpu() - ref).square().mean(-1).sqrt() / ref.square().mean(-1).sqrt()
            assert float(e.median()) < 0.03 and (name == "odd" or float(e.quantile(0.9)) < 0.06)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("layer", ["latent", "reader", "differential"])
def test_far_keys_of_a_layer(dev, layer, dtype):
    """A mixer on pages: the last tokens of a long sequence point at one far key, the first token, a page's
    first or last one, in a prompt's portion and decoded alone; another page table must not matter."""
    from zipage_amd.engine.inputs import plan_portions
    from zipage_amd.engine.model_runner import StepContext
    from zipage_amd.engine.inputs import Runs
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import GroupedAttention, LatentAttention, Rotary
    W, n, BS = 64, 200, 16
    rot = {"base": 2000.0, "dims": 16}
    if layer == "differential":
        m = C.attention(4, 2, 32, 48, 16, base=2000.0, scaling=None, softcap=12.0)
        mix = GroupedAttention(W, 4, 2, 32, 48, m["scale"], None, Rotary(2000.0, 16), softcap=12.0, diff=m["diff"], eps=1e-5,
                               bias=True, gated=True)
    else:
        m = C.latent(3, 24, 40, 16, 48, 40, base=2000.0)
        mix = LatentAttention(W, 3, 24, 40, 48, 40, m["scale"], None, 1e-5, Rotary(2000.0, 16), padded_width=W)
        reader = LatentAttention(W, 3, 24, 40, 48, 40, m["scale"], None, 1e-5, Rotary(2000.0, 16), own_latent=False, padded_width=W)
    assert m["rot"] == rot
    w = {k: _rand("cpu", BF16, *s, seed=i, std=s[-1] ** -0.5 if len(s) == 2 else 0.3) for i, (k, s) in enumerate(mix.shapes().items())}
    sharp = 14.0 if layer == "differential" else 5.0
    w["q" if layer == "differential" else "uq"] *= sharp               # one key takes nearly all of a row
    h = _rand("cpu", BF16, n, W, seed=50)
    if layer == "differential":
        into, out = mix.load(w, dtype, dev, W)
        into, out = into.to(dev, dtype), out.to(dev, dtype)
        want = O.differential_attention(h.double(), {k: v.double() for k, v in w.items()}, m, 1e-5)
    else:
        mix.load(w, dtype, dev)
        own = {k: v for k, v in w.items() if not k.startswith("dkv")}
        reader.load(own, dtype, dev)
        w64 = {k: v.double() for k, v in w.items()}
        want = O.latent_attention(h.double(), w64, m, 1e-5, O.shared_keys(h.double(), w64, m, 1e-5))
    for seed, cuts in ((0, [n]), (1, [150, 50]), (2, [180, 2, 17, 1]), (3, [199, 1])):
        cache = mix.allocate(20, BS, dtype, dev)
        cache.fill_(float("nan"))                                       # what nobody wrote must not be read
        table = torch.randperm(20, generator=torch.Generator().manual_seed(seed))[:-(-n // BS)].tolist()
        at, got = 0, []
        for c in cuts:
            s = Sequence([0] * (at + c), block_size=BS)
            s.block_table = table
            plan = plan_portions([Portion(s, at, c)], BS, [None], 16 if dtype == BF16 else None)
            t = lambda a: None if a is None else torch.as_tensor(a).to(dev)
            ctx = StepContext(False, t(plan.slots), None, t(plan.context_lens), t(plan.tables), table_rows=t(plan.table_rows),
                              runs={k: Runs(t(r.tiles), t(r.key_slots)) for k, r in plan.runs.items()})
            x, pos = h[at:at + c].to(dev, dtype), t(plan.positions)
            if layer == "differential":
                mixed = torch.empty(c, mix.out_columns, dtype=dtype, device=dev)
                mix.attend(torch.nn.functional.linear(x, into), pos, cache, ctx, mixed)
                got.append(torch.nn.functional.linear(mixed, out).float())
            else:
                held = {}
                y = mix.forward(x, cache, ctx, pos, held)
                if layer == "reader":
                    y = reader.forward(x, cache, ctx, pos, held)
                got.append(y.float().sum(0))
            at += c
        got = torch.cat(got).double().cpu()
        e = (got - want).square().mean(-1).sqrt() / want.square().mean(-1).sqrt()
        assert float(e.max()) < (2e-5 if dtype == F32 else 0.3), (cuts, float(e.max()))
        assert float(e.median()) < (2e-6 if dtype == F32 else 0.05), (cuts, float(e.median()))


@pytest.mark.parametrize("name,dtype", [("odd", F32), ("calm", F32), ("calm", BF16), ("wide", BF16)], ids=ids)
def test_first_tokens_and_page_borders(dev, engines, name, dtype):
    for n in (1, 2, 15, 16, 17, 33, 38):
        toks = C.tokens(C.CONFIGS[name], n, 20 + n)
        C.close(name, _feed_all(engines(name, dtype), toks, [n]), C.expected(name, toks), dtype)
        C.close(name, _feed_all(engines(name, dtype), toks, [n - 1 or 1, 1]), C.expected(name, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_long_decoding(dev, engines, dtype):
    cfg = C.CONFIGS["calm"]
    toks = C.tokens(cfg, 400, 5)
    eng = engines("calm", dtype)
    s = eng.open_request()
    got = [eng.feed([(s, toks[:20], [19])]).clone()]
    for t in range(20, 400):
        got.append(eng.feed([(s, toks[t:t + 1], [0])]).clone())
        assert 64 - eng.scheduler.pool.num_free == t // 16 + 1
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


@pytest.mark.parametrize("name", ["wide", "odd"])
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
    from zipage_amd.layers import GroupedAttention, Rotary, attention_form, run_attention
    with pytest.raises(ValueError, match="rotated"):
        GroupedAttention(32, 2, 1, 16, 16, 1.0, None, Rotary(10.0, 18))
    t = lambda *s: torch.zeros(*s, dtype=BF16, device=dev)
    with pytest.raises(RuntimeError, match="two maps"):          # sinks go with one map
        run_attention(t(4, 64), t(4, 80), 1, 1, 32, 16, torch.tensor([[0, 4, 0, 0]], dtype=torch.int32, device=dev), 1.0, t(4, 16),
                      sinks=torch.zeros(1, device=dev), form=attention_form(0.0, 2, 0.5, 1e-5, 16))


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
    prompt_tokens = 2 * sum(map(len, prompts))
    assert eng.stats["prefill_tokens"] < prompt_tokens if "enable_prefix_cache" in kw else eng.stats["prefill_tokens"] == prompt_tokens


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
