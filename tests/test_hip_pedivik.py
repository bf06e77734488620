"""Pedivik on the GPU: every mechanism alone, the model against the oracle in every way a sequence can
be cut and batched, and generation through the engine."""
import io
import json

import pytest
import torch

from oracle import pedivik_oracle as O
from tests import pedivik_cases as C

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
@pytest.mark.parametrize("width,norm_width", [(8, 8), (80, 76), (520, 520), (4096, 4090), (8192, 8192)])
def test_embed_norm(dev, dtype, width, norm_width):
    from zipage_amd.layers import embed_norm
    embed, pos = _rand(dev, dtype, 11, width, seed=1), _rand(dev, dtype, 9, width, seed=2)
    embed[:, norm_width:] = 0
    pos[:, norm_width:] = 0
    tok = torch.tensor([3, 10, 0, 3, 7], device=dev)
    at = torch.tensor([0, 8, 1, 1, 5], device=dev, dtype=torch.int32)
    w = _rand(dev, F32, width, seed=3, std=0.3)
    for table in (pos, None):
        x = torch.empty(5, width, device=dev)
        h = embed_norm(tok, at, embed, table, x, w, 1e-2, norm_width, weight_offset=1.0)
        want = embed[tok].double()
        if table is not None:
            want = O.embedding(tok, at.long(), embed.double(), table.double())
        _close(x, want, F32)
        n = O.norm_around_one(want[:, :norm_width], w.double()[:norm_width], 1e-2)
        _close(h[:, :norm_width], n, dtype)
        assert not h[:, norm_width:].any()


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,width,norm_width", [(1, 80, 76), (3, 512, 512), (17, 1024, 1000), (2, 8192, 8192)])
@pytest.mark.parametrize("planes", [None, 1, 3, 4, 9])
def test_residual_norm(dev, dtype, n, width, norm_width, planes):
    from zipage_amd.layers import residual_norm
    x, y = _rand(dev, F32, n, width, seed=1), _rand(dev, dtype, n, width, seed=2)
    x[:, norm_width:] = 0
    y[:, norm_width:] = 0
    w = _rand(dev, F32, width, seed=3)
    s = x.double() + y.double()
    hist = mix = None
    want = s
    if planes is not None:
        hist = _rand(dev, F32, planes + 2, n, width, seed=4)
        hist[..., norm_width:] = 0
        mix = _rand(dev, F32, planes + 1, seed=5)
        want = O.depth_average([*hist[:planes].double(), s], mix.double().tolist())
    for offset, scale in ((1.0, 0.25), (0.0, 1.0)):
        after, result = torch.empty_like(x), torch.empty_like(x)
        h = residual_norm(x, y, w, 1e-3, norm_width, weight_offset=offset, out_scale=scale, x_out=after,
                          result=result, history=hist, mix=mix)
        _close(result, s, F32)
        _close(after, want, F32)
        normed = O.rms(want[:, :norm_width], 1e-3) * (offset + w.double()[:norm_width]) * scale
        _close(h[:, :norm_width], normed, dtype)
    parts = torch.stack([y * 0.25, y * 0.5, y * 0.25])       # planes of partial sums: exact halves
    residual_norm(x, parts, None, 1e-3, norm_width, x_out=after, history=hist, mix=mix)
    _close(after, want, F32)
    inplace = x.clone()
    assert residual_norm(inplace, y, None, 1e-3, norm_width, x_out=inplace, history=hist, mix=mix) is None
    _close(inplace, want, F32)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_xielu(dev, dtype):
    from zipage_amd.layers import xielu
    z = torch.cat([torch.linspace(-30, 8, 4096), torch.linspace(-0.3, 0.3, 4096), torch.logspace(-12, -1, 1024),
                   -torch.logspace(-12, -1, 1024)]).to(dtype).to(dev)
    p, q = 0.6, -1.1
    sp = lambda t: float(torch.nn.functional.softplus(torch.tensor(t, dtype=torch.float64)))
    got = xielu(z.view(-1, 8), sp(p), 0.5 + sp(q)).view(-1).double().cpu()
    want = O.xielu(z.double().cpu(), p, q)
    eps = {BF16: 2.0 ** -8, F32: 2.0 ** -20}[dtype]
    z = z.double().cpu()          # for z < 0 the two terms cancel near one point: measure against z there
    assert ((got - want).abs() <= eps * torch.where(z < -0.125, z.abs(), want.abs()) + 1e-30).all()


@pytest.mark.parametrize("n", [1, 7, 64, 1024, 1030])
@torch.inference_mode()                       # as the engine captures: one process, one kind of graph state
def test_residual_linear_in_parts(dev, n):
    """A long contraction in parts and whole, against fp64; captured into a graph and replayed."""
    from zipage_amd.layers.linear import ResidualLinear
    w, x = _rand(dev, BF16, 96, 8192, seed=1, std=0.02), _rand(dev, BF16, n, 8192, seed=2)
    lin = ResidualLinear(w)
    planes = lin.forward(x)
    assert planes.shape == (4 if n <= 1024 else 1, n, 96)
    want = x.double().cpu() @ w.double().cpu().T
    _close(planes.double().sum(0), want, BF16)
    assert ResidualLinear(w[:, :4000].contiguous()).parts is None and ResidualLinear(w.float()).parts is None
    s = torch.cuda.Stream()
    s.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(s):
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g, stream=s):
            held = lin.forward(x)
        for i in range(4):
            x.copy_(_rand(dev, BF16, n, 8192, seed=10 + i))
            eager = lin.forward(x)
            g.replay()
            s.synchronize()
            assert torch.equal(held, eager), i


# ------------------------------------------------------------------ latent pieces
@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("q,qp,r,rp", [(52, 64, 44, 64), (96, 96, 512, 512), (1536, 1536, 20, 32)])
def test_latent_norm_store_and_gather(dev, dtype, q, qp, r, rp):
    from zipage_amd.layers.latent import latent_norm_store
    from zipage_amd.layers.runs import gather_rows
    n, pages, BS = 9, 4, 8
    down = _rand(dev, dtype, n, qp + rp, seed=1)
    down[:, q:qp] = 0
    down[:, qp + r:] = 0
    wq, wc = _rand(dev, F32, qp, seed=2), _rand(dev, F32, rp, seed=3)
    cache = torch.full((pages, BS, rp), 7.0, dtype=dtype, device=dev)
    slots = torch.tensor([5, -1, 31, 0, 12, 13, 32, 8, 7], dtype=torch.int32, device=dev)  # 32: past the end
    cq, c = latent_norm_store(down, wq, wc, q, r, 1e-2, cache, slots, return_c=True)
    _close(cq[:, :q], O.norm_plain(down[:, :q].double(), wq.double()[:q], 1e-2), dtype)
    _close(c[:, :r], O.norm_plain(down[:, qp:qp + r].double(), wc.double()[:r], 1e-2), dtype)
    assert not cq[:, q:].any() and not c[:, r:].any()
    flat = cache.view(-1, rp)
    kept = [i for i, s in enumerate(slots.tolist()) if 0 <= s < 32]
    assert torch.equal(flat[slots[kept].long()], c[kept])
    untouched = sorted(set(range(32)) - set(slots[kept].tolist()))
    assert (flat[untouched] == 7).all()
    rows = torch.tensor([31, 0, 5, 5, 13], dtype=torch.int32, device=dev)
    assert torch.equal(gather_rows(cache, rows), flat[rows.long()])


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("n,H,K,M", [(1, 1, 32, 16), (5, 3, 64, 80), (64, 2, 160, 32), (133, 5, 96, 288), (300, 37, 64, 160)])
def test_headwise_linear(dev, dtype, n, H, K, M):
    from zipage_amd.layers.latent import headwise_linear
    x, w = _rand(dev, dtype, n, H, K, seed=1), _rand(dev, dtype, H, M, K, seed=2)
    want = torch.stack([x[:, h].double().cpu() @ w[h].double().cpu().T for h in range(H)], dim=1)
    _close(headwise_linear(x, w), want, dtype)


def _rows_reference(q, flat, tables, ctx, trows, BS, scale, window):
    out = torch.zeros(q.shape, dtype=torch.float64)
    for i in range(q.shape[0]):
        n = int(ctx[i])
        keys = list(range(max(0, n - window) if window else 0, n))
        if not keys:
            continue
        c = flat[[int(tables[trows[i], t // BS]) * BS + t % BS for t in keys]]
        s = torch.softmax(q[i] @ c.T * scale, dim=-1)
        out[i] = s @ c
    return out


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("H,R,BS,window", [
    (1, 32, 16, None), (5, 96, 64, 95), (16, 128, 48, 33), (17, 160, 16, 1), (37, 288, 32, 70), (64, 512, 64, 257),
    (128, 256, 256, 31), (3, 384, 16, 500), (2, 544, 16, 40)])
def test_latent_rows_attention(dev, dtype, H, R, BS, window):
    """Ragged contexts over scattered pages; every third token's query points at one key: the oldest
    it sees, the one just before that, or one at a page's border."""
    from zipage_amd.layers import latent_rows_attention
    ctx = [1, 2, 31, 32, 33, BS, BS + 1, 95, 96, 97, 98, 300, 0, 511, 512, 513, 640]
    n, B, NB = len(ctx), len(ctx) + 2, -(-640 // BS)
    pages = B * NB + 3
    g = torch.Generator().manual_seed(H * R)
    tables = torch.randperm(pages, generator=g)[:B * NB].view(B, NB).int()
    trows = torch.randperm(B, generator=g)[:n].int()
    cache = _rand("cpu", dtype, pages, BS, R, seed=1)
    q = _rand("cpu", dtype, n, H, R, seed=2, std=0.5)
    flat = cache.view(-1, R)
    scale = R ** -0.5
    for i, c in enumerate(ctx):
        if c == 0:
            continue
        low = max(0, c - window) if window else 0
        key = (low, low - 1, (c - 1) // BS * BS)[i % 3]
        if low - 1 < key and key >= 0 or key == low - 1 >= 0:
            row = flat[int(tables[trows[i], key // BS]) * BS + key % BS].float()
            q[i] = (row * (12.0 / (scale * float(row @ row)))).to(dtype)
    # entries in front of the window are never read
    for i, c in enumerate(ctx):
        if window:
            tables[trows[i], :max(0, c - window) // BS] = -1
    want = _rows_reference(q.double(), flat.double(), tables, ctx, trows, BS, scale, window)
    t = lambda a: torch.as_tensor(a, dtype=torch.int32).to(dev)
    got = latent_rows_attention(q.to(dev), cache.to(dev), t(tables), t(ctx), scale, window, t(trows))
    assert not got[ctx.index(0)].any()
    live = [i for i, c in enumerate(ctx) if c]
    _close(got[live], want[live], dtype, 2.0 if dtype == BF16 else 4.0)
    # one token at a time: other launch shapes, other splits of the keys
    for i in (4, 11, 16):
        alone = latent_rows_attention(q[i:i + 1].to(dev), cache.to(dev), t(tables), t(ctx[i:i + 1]), scale, window,
                                      t(trows[i:i + 1]))
        _close(alone, want[i:i + 1], dtype, 2.0 if dtype == BF16 else 4.0)


@pytest.mark.parametrize("H,D,V,window", [(1, 32, 16, None), (5, 64, 88, 100), (8, 128, 128, 33), (3, 160, 136, 1),
                                          (2, 256, 256, 200), (9, 96, 48, 64)])
def test_latent_tiles_attention(dev, H, D, V, window):
    """Runs at the start, behind cached context and of all lengths about a tile's; queries that point at
    the first key inside and outside their window."""
    import numpy as np
    from zipage_amd.engine.inputs import plan_runs
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import latent_tiles_attention
    BS = 16
    parts, page = [], 0
    for start, count in ((0, 127), (0, 128), (0, 129), (45, 16), (300, 257), (7, 300), (1, 2)):
        s = Sequence([0] * (start + count), block_size=BS)
        need = -(-(start + count) // BS)
        s.block_table = list(range(page, page + need))
        page += need
        parts.append(Portion(s, start, count))
    runs = plan_runs(parts, BS, window)
    total = sum(p.count for p in parts)
    k = _rand("cpu", BF16, page * BS, H, D, seed=1)
    v = _rand("cpu", BF16, page * BS, H, V, seed=2)
    q = _rand("cpu", BF16, total, H, D, seed=3, std=0.5)
    scale = D ** -0.5
    want = torch.empty(total, H, V, dtype=torch.float64)
    r = 0
    for p in parts:
        base = p.seq.block_table[0] * BS
        for t in range(p.start, p.start + p.count):
            low = 0 if window is None else max(0, t - window + 1)
            key = (low, low - 1, t)[t % 3]
            if key >= 0:
                row = k[base + key].float()
                q[r] = (row * (12.0 / (scale * (row * row).sum(-1, keepdim=True)))).to(BF16)
            r += 1
        n, m = p.count, p.start + p.count
        qi, kk, vv = q[r - n:r].double(), k[base:base + m].double(), v[base:base + m].double()
        pos = torch.arange(p.start, m)
        seen = pos[:, None] >= torch.arange(m)[None]
        if window is not None:
            seen &= pos[:, None] - torch.arange(m)[None] < window
        for h in range(H):
            sc = (qi[:, h] @ kk[:, h].T * scale).masked_fill(~seen, float("-inf"))
            want[r - n:r, h] = torch.softmax(sc, -1) @ vv[:, h]
    if runs.key_slots is None:
        runs.key_slots = np.concatenate([np.arange(p.start, p.start + p.count) + p.seq.block_table[0] * BS
                                         for p in parts])
    slots = torch.as_tensor(runs.key_slots).long()
    kv = torch.cat([k[slots].flatten(1), v[slots].flatten(1)], dim=1).to(dev)
    out = torch.full((total, H * V), float("nan"), dtype=BF16, device=dev)
    latent_tiles_attention(q.flatten(1).to(dev), kv, H, D, V, torch.as_tensor(runs.tiles).to(dev), scale, window, out)
    _close(out.view(total, H, V), want, BF16, 2.0)


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
    tmp, made = tmp_path_factory.mktemp("pedivik"), {}

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
@pytest.mark.parametrize("cuts", [[400], [1], [2], [3, 17, 1, 16, 15, 64], [100, 1], [128], [16]],
                         ids=lambda c: "-".join(map(str, c)))
def test_any_cut_of_a_sequence_gives_the_oracle(dev, engines, name, dtype, cuts):
    toks = C.tokens(C.CONFIGS[name], 150, 3)
    assert C.error(_feed_all(engines(name, dtype), toks, cuts), C.expected(name, toks)) < C.LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_layer_streams(dev, engines, dtype):
    """The stream after every layer, a whole prompt in one step."""
    from zipage_amd.engine import Portion
    cfg, w = C.case("odd")
    toks = C.tokens(cfg, 120, 9)
    eng = engines("odd", dtype)
    s = eng.open_request()
    s.token_ids, s.num_tokens, s.num_prompt_tokens = list(toks), 120, 120
    eng.scheduler.pool.grow(s, 120)
    i, p, ctx, _ = eng.runner.prepare_portions([Portion(s, 0, 120)])
    streams = []
    eng.runner.model.forward(i, p, ctx, trace=streams)
    eng.close_request(s)
    want = O.forward(cfg, w, toks)[1]
    assert len(streams) == len(want) == 3
    for got, ref in zip(streams, want):
        _close(got, ref, dtype, 8.0 if dtype == BF16 else 16.0)


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_first_tokens_and_page_borders(dev, engines, name, dtype):
    for n in (1, 2, 15, 16, 17, 33):
        toks = C.tokens(C.CONFIGS[name], n, 20 + n)
        assert C.error(_feed_all(engines(name, dtype), toks, [n]), C.expected(name, toks)) < C.LIMIT[dtype], n
        assert C.error(_feed_all(engines(name, dtype), toks, [n - 1 or 1, 1]), C.expected(name, toks)) < C.LIMIT[dtype], n


@pytest.mark.parametrize("dtype", DTYPES, ids=ids)
def test_long_decoding(dev, engines, dtype):
    """Several windows of decoded tokens; the pages behind the windows are given back on the way."""
    cfg = C.CONFIGS["odd"]
    toks = C.tokens(cfg, 420, 5)
    eng = engines("odd", dtype)
    s = eng.open_request()
    got = [eng.feed([(s, toks[:20], [19])]).clone()]
    for t in range(20, 420):
        got.append(eng.feed([(s, toks[t:t + 1], [0])]).clone())
        assert 64 - eng.scheduler.pool.num_free <= 7           # 90 tokens of window, 16 a page
    eng.close_request(s)
    assert C.error(torch.cat(got), C.expected("odd", toks)[19:]) < C.LIMIT[dtype]


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
    live, worst = [], 0.0
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
        logits, at = eng.feed(batch).clone(), 0
        for item, n in meta:
            want = C.expected(name, item[1])[item[2]:item[2] + n]
            scale_rows = C.expected(name, item[1])
            d = logits[at:at + n].double().cpu() - want
            d -= d.mean(-1, keepdim=True)
            spread = (scale_rows - scale_rows.mean(-1, keepdim=True)).square().mean().sqrt()
            worst = max(worst, float((d.square().mean(-1).sqrt() / spread).max()))
            at += n
            item[2] += n
            if item[2] == len(item[1]):
                eng.close_request(item[0])
        live = [i for i in live if i[2] < len(i[1])]
    assert worst < C.LIMIT[dtype]


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
    with pytest.raises(ValueError, match="once"):
        eng.feed([(s, [1], []), (s, [2], [])])
    assert eng.feed([(s, [1, 2], [])]) is None
    eng.close_request(s)
    from zipage_amd.engine import SamplingParams
    with pytest.raises(ValueError, match="positions"):
        eng.add_request([1] * 600, SamplingParams(max_tokens=50, ignore_eos=True))
    small = engines("ends", F32, num_kvcache_blocks=2)
    with pytest.raises(ValueError, match="pages"):
        small.add_request([1] * 60, SamplingParams(max_tokens=5))


# ------------------------------------------------------------------ generation
def _greedy_ok(name, prompt, got):
    """`got` is the oracle's greedy continuation, up to a near tie of two logits."""
    cfg, w = C.case(name)
    lg = O.forward(cfg, w, prompt + got)[0]
    for i, tok in enumerate(got):
        row = lg[len(prompt) - 1 + i]
        assert float(row.max() - row[tok]) < 1e-4 * float(row.std()), i


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
    counts = [30, 40, 7, 1, 20, 100]
    for round_ in range(2):                    # the second round meets used pages and, if kept, its prefixes
        outs = eng.generate(prompts, [SamplingParams(max_tokens=c, ignore_eos=True) for c in counts])
        for p, c, o in zip(prompts, counts, outs):
            assert len(o["token_ids"]) == c
            _greedy_ok("odd", p, o["token_ids"])
    pool = eng.scheduler.pool
    assert pool.num_free == pool.num_pages and pool.reserved == 0
    assert eng.stats["decode_tokens"] + eng.stats["mixed_decode_tokens"] == 2 * sum(c - 1 for c in counts)


def test_generation_stops_at_eos_and_samples(dev, engines):
    from zipage_amd.engine import SamplingParams
    cfg, w = C.case("odd")
    prompt = C.tokens(cfg, 21, 8)
    want, _ = O.greedy(cfg, w, prompt, 12)
    eos = want[7]
    eng = engines("odd", F32, eos=eos)
    out = eng.generate([prompt], SamplingParams(max_tokens=12))[0]["token_ids"]
    assert out == want[:want.index(eos) + 1]
    # drawn tokens: a cold distribution is greedy, a hot one is not
    cold = eng.generate([prompt] * 3, SamplingParams(temperature=1e-4, max_tokens=6, ignore_eos=True))
    assert all(o["token_ids"] == want[:6] for o in cold)
    hot = eng.generate([prompt] * 4, SamplingParams(temperature=50.0, max_tokens=8, ignore_eos=True))
    assert len({tuple(o["token_ids"]) for o in hot}) > 1


def test_bf16_generation_follows_its_own_logits(dev, engines):
    """Greedy tokens of the bf16 engine are within bf16 error of the oracle's best."""
    from zipage_amd.engine import SamplingParams
    cfg, w = C.case("wide")
    prompts = [C.tokens(cfg, n, 70 + n) for n in (5, 64, 131)]
    eng = engines("wide", BF16, max_num_batched_tokens=50)
    for p, o in zip(prompts, eng.generate(prompts, SamplingParams(max_tokens=60, ignore_eos=True))):
        lg = O.forward(cfg, w, p + o["token_ids"])[0]
        for i, tok in enumerate(o["token_ids"]):
            row = lg[len(p) - 1 + i]
            assert float(row.max() - row[tok]) < 6 * C.LIMIT[BF16] * float(row.std())


def test_command_line(dev, engines, tmp_path, capsys, monkeypatch):
    import numpy as np
    from zipage_amd import cli
    eng = engines("ends", F32)
    folder = eng.cfg.model_folder
    cfg, w = C.case("ends")
    prompt = C.tokens(cfg, 40, 2)
    assert cli.main(["generate", "--model", folder, "--dtype", "float32", "--tokens", ",".join(map(str, prompt)),
                     "--tokens", "3", "--max-tokens", "9", "--batch-tokens", "16"]) == 0
    lines = [json.loads(l) for l in capsys.readouterr().out.splitlines() if l.startswith("{")]
    _greedy_ok("ends", prompt, lines[0]["token_ids"])
    _greedy_ok("ends", [3], lines[1]["token_ids"])
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
    assert C.error(read(0), full[[0, 32]]) < C.LIMIT[F32]
    assert C.error(read(2), torch.stack([other[2], full[39]])) < C.LIMIT[F32]
    assert C.error(read(3), full[:1]) < C.LIMIT[F32]
