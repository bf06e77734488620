"""Pedivik or Kapolorn beside Qwen3, Rutevik or Mefupel beside Pedivik and Kapolorn, at equal size: prefill and decode
throughput through the engine (random weights), and every kernel between the matrix products against its
roofline, beside the kernel of the other model that does the like work.

Equal size: same width, heads, head dimensions and vocabulary; Pedivik's ungated feed-forward is 1.5
times as wide as Qwen3's gated one, so both hold the same parameters; a Kapolorn token passes three of 32
experts and the shared one, each a quarter as wide as Qwen3's feed-forward, a Rutevik token four of 32 such
experts; its differential layers have half the heads, with values of twice the size.  Mefupel's feed-forwards are
as wide as Pedivik's.  Kernels are timed as
replays of a graph of many launches over buffers that together exceed the caches.
"""
from __future__ import annotations

import time
from dataclasses import replace
from types import SimpleNamespace

import torch

HBM = 8.0e12          # bytes/s
MFMA = 2.5e15         # dense bf16 FLOP/s
FP32 = 157e12         # fp32 FLOP/s, vector or matrix
BF16 = torch.bfloat16

SIZES = {
    # width, heads, kv_heads (Qwen3), head dim, gated ff, layers, vocab, q_rank, kv_rank, window
    "1k": (1024, 16, 8, 128, 3072, 8, 32768, 512, 256, 1024),
    "4k": (4096, 32, 8, 128, 12288, 8, 32768, 1536, 512, 1024),
}


def shapes(size: str):
    from zipage_amd.engine import PedivikLayer, PedivikShape, Qwen3Shape
    W, H, HK, D, FF, L, V, QR, KR, win = SIZES[size]
    layer = PedivikLayer(H, D, D, QR, KR, D ** -0.5, win, FF * 3 // 2)
    return (PedivikShape(V, W, (layer,) * L, 8192, 1e-6, 1.0),
            Qwen3Shape(L, W, H, HK, D, FF, V, max_position=8192))


def kapolorn_shapes(size: str):
    from zipage_amd.engine import KapolornShape, Qwen3Shape
    from zipage_amd.engine.kapolorn import DeltaMixer, ExpertsShape, KapolornLayer, ParallelMixer
    W, H, HK, D, FF, L, V, _, _, chunk = SIZES[size]
    moe = ExpertsShape(32, 3, 4, 2, FF // 4, 7.0, FF // 4, 7.0)
    par = KapolornLayer(ParallelMixer(H, HK, D, D, D ** -0.5, chunk, 1e6, D, 0.8, H // 2, D, D, 15.0, 1.1), moe)
    delta = KapolornLayer(DeltaMixer(H, H // 2, D, D, 4), moe)
    return (KapolornShape(V, W, (par, delta) * (L // 2), (0, 0, 1), 1e-6, 1.0, 15.0),
            Qwen3Shape(L, W, H, HK, D, FF, V, max_position=8192))


def rutevik_shapes(size: str):
    """One differential layer (the first with a dense feed-forward) to three latent ones, of which one reads the
    cache of the one before it.  Pedivik's window holds everything here, Kapolorn keeps its chunks."""
    from zipage_amd.engine import KapolornShape, PedivikShape, RutevikShape
    from zipage_amd.engine.rutevik import DenseShape, DifferentialMixer, LatentMixer, MixtureShape, RutevikLayer
    from zipage_amd.layers import Rotary
    W, H, HK, D, FF, L, V, QR, KR, _ = SIZES[size]
    moe, rot = MixtureShape(32, 4, FF // 4), Rotary(5e5, D // 2)
    diff = DifferentialMixer(H // 2, HK // 2, D, 2 * D, Rotary(5e5, D, (8.0, 1.0, 4.0, 2048.0)), D ** -0.5, 30.0, 0.4)
    layers = []
    for i in range(L):
        source = i - 1 if i % 4 == 2 else i
        m = LatentMixer(H, D, D, QR, KR, rot, (D * 3 // 2) ** -0.5, source) if i % 4 else diff
        layers.append(RutevikLayer(m, moe if i else DenseShape(FF * 3 // 2)))
    pedivik, kapolorn = shapes(size)[0], kapolorn_shapes(size)[0]
    everything = lambda layer: replace(layer, window=8192)
    return {"rutevik": RutevikShape(V, W, tuple(layers), 1e-6, 1.0),
            "pedivik": replace(pedivik, layers=tuple(map(everything, pedivik.layers))), "kapolorn": kapolorn}


def throughput(shape, batch: int, prompt: int, out_tokens: int) -> dict:
    """One generate() call per figure: prefill in steps of up to 32768 tokens, then decode steps."""
    from zipage_amd.engine import EngineConfig, SamplingParams, ZipageEngine
    total = prompt + out_tokens
    per = -(-total // 256) + 1
    cfg = EngineConfig(shape=shape, max_concurrency=batch, max_num_seqs=batch, num_kvcache_blocks=batch * per + 8,
                       max_cache_blocks_per_seq=per, max_model_len=total + 1, kvcache_block_size=256,
                       max_num_batched_tokens=32768)
    eng = ZipageEngine(cfg)
    g = torch.Generator().manual_seed(0)
    prompts = torch.randint(0, shape.vocab, (batch, prompt), generator=g).tolist()
    run = lambda n: eng.generate(prompts, SamplingParams(max_tokens=n, ignore_eos=True))
    run(out_tokens)                           # products, graphs and allocator warm up
    for k in ("prefill_s", "decode_s", "decode_tokens", "decode_steps", "prefill_tokens"):
        eng.stats[k] = 0
    run(out_tokens)
    st = eng.stats
    # the step alone: replays of the decode graph at the last step's inputs
    r = eng.runner
    g_ = r._graphs[max(r._graphs)][0]
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    with torch.cuda.stream(r.run_stream):
        for _ in range(20):
            g_.replay()
    torch.cuda.synchronize()
    step = (time.perf_counter() - t0) / 20
    del eng, r
    torch.cuda.empty_cache()
    return {"prefill_tok_per_s": round(st["prefill_tokens"] / st["prefill_s"]),
            "decode_tok_per_s": round(st["decode_tokens"] / st["decode_s"]),
            "ms_per_decode_step": round(st["decode_s"] / st["decode_steps"] * 1e3, 3),
            "ms_layers_of_a_decode_step": round(step * 1e3, 3)}


@torch.inference_mode()
def timed(fn, variants: int, launches: int = 24) -> float:
    """Seconds per call of fn(i): a graph of `launches` calls over `variants` buffer sets."""
    torch.cuda.synchronize()                  # the inputs were made on another stream
    s = torch.cuda.Stream()
    with torch.cuda.stream(s):
        for i in range(min(variants, 3)):
            fn(i)
        s.synchronize()
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g, stream=s):
            for i in range(launches):
                fn(i % variants)
        g.replay()
        best = float("inf")
        for _ in range(5):
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record(s)
            g.replay()
            b.record(s)
            b.synchronize()
            best = min(best, a.elapsed_time(b))
    del g
    torch.cuda.empty_cache()
    return best / launches / 1e3


def _sets(nbytes: int) -> int:
    """Buffer sets that together exceed the 256 MB last-level cache."""
    return max(2, min(24, -(-(1 << 30) // max(nbytes, 1))))


def kernels(size: str, decode_batch: int, prompts: int, prompt: int) -> list[dict]:
    """Rows of (kernel, like kernel): time, roofline time and the fraction of each."""
    import torch.nn.functional as F
    from zipage_amd.engine.inputs import plan_runs
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import (latent_rows_attention, latent_tiles_attention, paged_decode_attention,
                                   qk_norm_rope_store, residual_norm, rms_norm, silu_and_mul, xielu)
    from zipage_amd.layers.latent import headwise_linear, latent_norm_store
    W, H, HK, D, FF, L, V, QR, KR, win = SIZES[size]
    dev, BS = torch.device("cuda:0"), 256
    rnd = lambda *s, dt=BF16: torch.randn(*s, device=dev, dtype=torch.float32).to(dt)
    rows = []

    def put(name, where, secs, byts, flops=0.0):
        roof = max(byts / HBM, flops / MFMA)
        rows.append({"kernel": name, "at": where, "us": round(secs * 1e6, 1),
                     "bound": "hbm" if byts / HBM >= flops / MFMA else "mfma",
                     "roofline_us": round(roof * 1e6, 1), "frac": round(roof / secs, 3)})

    for phase, N in (("decode", decode_batch), ("prefill", prompts * prompt)):
        at = f"{phase}, {N} tokens"
        big = N * W
        # norms of the stream
        k = _sets(big * 14)
        xs, ys = [rnd(N, W, dt=torch.float32) for _ in range(k)], [rnd(N, W) for _ in range(k)]
        w32, w16 = torch.zeros(W, device=dev), torch.ones(W, device=dev, dtype=BF16)
        put("residual_norm (fp32 stream)", at,
            timed(lambda i: residual_norm(xs[i], ys[i], w32, 1e-6, W, 1.0, x_out=xs[i]), k), big * (4 + 2 + 4 + 2))
        planes = L // 2 + 1
        kh = max(1, min(k, (8 << 30) // (planes * big * 4)))
        hist = [rnd(planes + 1, N, W, dt=torch.float32) for _ in range(kh)]
        mix = torch.full((planes + 1,), 0.3, device=dev)
        put(f"residual_norm with depth average over {planes} planes", at,
            timed(lambda i: residual_norm(xs[i], ys[i], w32, 1e-6, W, 1.0, x_out=xs[i], result=hist[i][planes],
                                          history=hist[i], mix=mix), kh), big * (4 + 2 + 4 + 4 + 2 + 4 * planes))
        del hist
        rs = [rnd(N, W) for _ in range(k)]
        put("like: add_rms_norm (16-bit stream)", at, timed(lambda i: rms_norm(ys[i], w16, 1e-6, rs[i]), k),
            big * (2 + 2 + 2 + 2))
        del xs, ys, rs
        # activations
        k = _sets(N * FF * 3 // 2 * 4)
        zs = [rnd(N, FF * 3 // 2) for _ in range(k)]
        put("xielu", at, timed(lambda i: xielu(zs[i], 0.8, 1.3), k), N * FF * 3 // 2 * 4)
        del zs
        gs = [rnd(N, 2 * FF) for _ in range(k)]
        put("like: silu_and_mul", at, timed(lambda i: silu_and_mul(gs[i]), k), N * FF * 6)
        del gs
        # norms and stores of the attention inputs
        slots = torch.randperm(N, device=dev).int()
        k = _sets(N * (QR + KR) * 6)
        downs = [rnd(N, QR + KR) for _ in range(k)]
        caches = [rnd(-(-N // BS), BS, KR) for _ in range(k)]
        wq, wc = torch.ones(QR, device=dev), torch.ones(KR, device=dev)
        put("latent_norm_store", at, timed(lambda i: latent_norm_store(downs[i], wq, wc, QR, KR, 1e-6, caches[i],
                                                                        slots), k), N * (QR + KR) * 4)
        del downs, caches
        qkv_w = (H + 2 * HK) * D
        k = _sets(N * qkv_w * 4)
        qkvs = [rnd(N, qkv_w) for _ in range(k)]
        kcs = [rnd(-(-N // BS), BS, HK, D) for _ in range(2 * k)]
        pos = torch.arange(N, device=dev, dtype=torch.int32) % 4096
        cos, sin = rnd(8192, D // 2, dt=torch.float32), rnd(8192, D // 2, dt=torch.float32)
        nw = torch.ones(D, device=dev, dtype=BF16)
        put("like: qk_norm_rope_store", at,
            timed(lambda i: qk_norm_rope_store(qkvs[i], pos, cos, sin, nw, nw, H, HK, D, 1e-6, kcs[2 * i], kcs[2 * i + 1],
                                               slots), k), N * qkv_w * 4)
        del qkvs, kcs
    # ---- decode attention
    ctx_len = prompt
    per = -(-ctx_len // BS)
    for B in (64, decode_batch):
        at = f"decode, {B} sequences, context {ctx_len}"
        k = _sets(B * win * KR * 2)
        caches = [rnd(B * per, BS, KR) for _ in range(k)]
        tables = torch.randperm(B * per, device=dev).int().view(B, per)
        ctx = torch.full((B,), ctx_len, device=dev, dtype=torch.int32)
        q = rnd(B, H, KR)
        seen = min(win, ctx_len)
        put(f"latent_rows_attention, window {win}", at,
            timed(lambda i: latent_rows_attention(q, caches[i], tables, ctx, D ** -0.5, win), k),
            B * seen * KR * 2 + 2 * B * H * KR * 2, 4.0 * B * H * seen * KR)
        del caches
        k = max(2, _sets(2 * B * ctx_len * HK * D * 2))
        kcs = [rnd(B * per, BS, HK, D) for _ in range(2 * k)]
        qd = rnd(B, H, D)
        put("like: paged_decode_attention", at,
            timed(lambda i: paged_decode_attention(qd, kcs[2 * i], kcs[2 * i + 1], ctx, tables, D ** -0.5), k),
            2 * B * ctx_len * HK * D * 2 + 2 * B * H * D * 2, 4.0 * B * H * ctx_len * D)
        del kcs
    k = _sets(H * KR * D * 2)
    ws, wv = [rnd(H, KR, D) for _ in range(k)], [rnd(H, D, KR) for _ in range(k)]
    x1, x2 = rnd(B, H, D), rnd(B, H, KR)
    byts, fl = H * KR * D * 2 + B * H * (KR + D) * 2, 2.0 * B * H * KR * D
    put("headwise_linear, q into the latent space", at, timed(lambda i: headwise_linear(x1, ws[i]), k), byts, fl)
    put("headwise_linear, values out of it", at, timed(lambda i: headwise_linear(x2, wv[i]), k), byts, fl)
    lin = [rnd(W, H * D) for _ in range(_sets(W * H * D * 2))]
    xl = rnd(B, H * D)
    put("like: output projection (library product)", at, timed(lambda i: F.linear(xl, lin[i]), len(lin)),
        W * H * D * 2 + B * (W + H * D) * 2, 2.0 * B * W * H * D)
    del ws, wv, lin
    # ---- prefill attention
    N = prompts * prompt
    at = f"prefill, {prompts} x {prompt} tokens"
    seqs = [Sequence([0] * prompt) for _ in range(prompts)]
    for s in seqs:
        s.block_table = list(range(per))
    tiles = torch.as_tensor(plan_runs([Portion(s, 0, prompt) for s in seqs], BS, win).tiles).to(dev)
    k = 2
    qs, kvs = [rnd(N, H * D) for _ in range(k)], [rnd(N, H * 2 * D) for _ in range(k)]
    out = torch.empty(N, H * D, device=dev, dtype=BF16)
    pairs = sum(min(i + 1, win) for i in range(prompt)) * prompts
    put(f"latent_tiles_attention, window {win}", at,
        timed(lambda i: latent_tiles_attention(qs[i], kvs[i], H, D, D, tiles, D ** -0.5, win, out), k, 6),
        N * H * D * 2 * 4, 4.0 * pairs * H * D)
    full = torch.as_tensor(plan_runs([Portion(s, 0, prompt) for s in seqs], BS, None).tiles).to(dev)
    pairs = prompt * (prompt + 1) / 2 * prompts
    put("latent_tiles_attention, no window", at,
        timed(lambda i: latent_tiles_attention(qs[i], kvs[i], H, D, D, full, D ** -0.5, None, out), k, 6),
        N * H * D * 2 * 4, 4.0 * pairs * H * D)
    del kvs
    ks = [rnd(prompts, prompt, HK, D) for _ in range(2 * k)]
    put("like: scaled_dot_product_attention (library, causal)", at,
        timed(lambda i: F.scaled_dot_product_attention(
            qs[i].view(prompts, prompt, H, D).transpose(1, 2), ks[2 * i].transpose(1, 2), ks[2 * i + 1].transpose(1, 2),
            is_causal=True, enable_gqa=True), k, 6), N * (2 * H + 2 * HK) * D * 2, 4.0 * pairs * H * D)
    return rows


def kapolorn_kernels(size: str, decode_batch: int, prompts: int, prompt: int) -> list[dict]:
    """The same for Kapolorn's kernels.  Recurrences run in fp32: their roofline is that of fp32 arithmetic
    (7 or 5 operations per state element and token) or of the state's bytes, whichever is longer."""
    import torch.nn.functional as F
    from zipage_amd.engine.inputs import plan_runs
    from zipage_amd.engine.qwen3 import Segments
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import (ChannelDelta, Experts, MatrixMemory, grouped_rows_attention, paged_decode_attention,
                                   qk_norm_rope_store, residual_norm, rms_norm, rotary_store, run_attention,
                                   silu_and_mul, small_linear, softcap)
    from zipage_amd.layers.moe import Plan, moe_select
    from zipage_amd.sight import Chunk
    W, H, HK, D, FF, L, V, _, _, chunk = SIZES[size]
    dev, BS = torch.device("cuda:0"), 256
    rnd = lambda *s, dt=BF16: torch.randn(*s, device=dev, dtype=torch.float32).to(dt)
    i32 = lambda a: torch.as_tensor(a, dtype=torch.int32, device=dev)
    rows = []

    def put(name, where, secs, byts, flops=0.0, peak=MFMA):
        roof = max(byts / HBM, flops / peak)
        bound = "hbm" if byts / HBM >= flops / peak else ("mfma" if peak == MFMA else "fp32")
        rows.append({"kernel": name, "at": where, "us": round(secs * 1e6, 1), "bound": bound,
                     "roofline_us": round(roof * 1e6, 1), "frac": round(roof / secs, 3)})

    gen = torch.Generator(device=dev).manual_seed(0)
    moe = Experts(W, 32, 3, FF // 4, 7.0, 4, 2, FF // 4, 7.0)
    moe.random(BF16, dev, gen)
    E, S = moe.experts, moe.top + 1
    plan_of = lambda r: Plan(r[0], r[2], E, True, BF16)
    gu, dn = [rnd(2 * FF, W) for _ in range(2)], [rnd(W, FF) for _ in range(2)]
    for phase, N in (("decode", 64), ("decode", decode_batch), ("prefill", prompts * prompt)):
        at, big = f"{phase}, {N} tokens", N * W
        seqs = N if phase == "decode" else prompts
        # norms of the stream
        for planes in (1, S):
            k = _sets(big * (10 + 2 * planes))
            xs, ys = [rnd(N, W, dt=torch.float32) for _ in range(k)], [rnd(planes, N, W) for _ in range(k)]
            w32, w16 = torch.ones(W, device=dev), torch.ones(W, device=dev, dtype=BF16)
            put(f"residual_norm of a normed branch, {planes} planes", at,
                timed(lambda i: residual_norm(xs[i], ys[i], w32, 1e-6, W, x_out=xs[i], y_weight=w32), k), big * (10 + 2 * planes))
            if planes == 1:
                rs = [rnd(N, W) for _ in range(k)]
                put("like: add_rms_norm (16-bit stream)", at, timed(lambda i: rms_norm(ys[i][0], w16, 1e-6, rs[i]), k), big * 8)
                del rs
            del xs, ys
        # rotary positions and the store
        width = (H + 2 * HK) * D
        slots, pos = torch.randperm(N, device=dev).int(), torch.arange(N, device=dev, dtype=torch.int32) % 4096
        k = _sets(N * width * 4)
        qkvs, caches = [rnd(N, width) for _ in range(k)], [rnd(-(-N // BS), BS, 2 * HK * D) for _ in range(k)]
        freqs = rnd(D // 2, dt=torch.float32).abs()
        put("rotary_store", at, timed(lambda i: rotary_store(qkvs[i], pos, freqs, H, HK, D, D, caches[i], slots), k), N * width * 4)
        cos, sin, nw = rnd(8192, D // 2, dt=torch.float32), rnd(8192, D // 2, dt=torch.float32), torch.ones(D, device=dev, dtype=BF16)
        kcs = [rnd(-(-N // BS), BS, HK, D) for _ in range(2 * k)]
        put("like: qk_norm_rope_store", at,
            timed(lambda i: qk_norm_rope_store(qkvs[i], pos, cos, sin, nw, nw, H, HK, D, 1e-6, kcs[2 * i], kcs[2 * i + 1], slots), k),
            N * width * 4)
        del qkvs, caches, kcs
        # recurrences
        n = N // seqs
        seg = Segments(i32(range(0, N, n)), i32([n] * seqs), i32(torch.randperm(seqs)), i32([5] * seqs), longest=n,
                       max_count=int(n == 1))
        seg = SimpleNamespace(segments=seg if n < 16 else None, run_segments=None if n < 16 else seg)
        for name, mixer, ops in ((f"mlstm_scan, {H // 2} heads", MatrixMemory(W, H // 2, D, D, 15.0, 1e-6), 5),
                                 (f"delta_scan, {H} heads", ChannelDelta(W, H, H // 2, D, D, 4, 1e-6), 7)):
            small = {q: torch.randn(*s) * 0.02 for q, s in (mixer.shapes() if ops == 5 else mixer.shapes(128, 128)).items()}
            mixer.load({q: t.to(BF16) for q, t in small.items()}, BF16, dev, W)
            h = rnd(N, W)
            k = 2
            projs = [rnd(N, mixer.columns) for _ in range(k)]
            states = [mixer.allocate(seqs + 1, BF16, dev) for _ in range(k)]
            out = torch.empty(N, mixer.out_columns, device=dev, dtype=BF16)
            state = 2 * seqs * mixer.heads * D * D * 4
            inner = (lambda i: mixer.scan(h, projs[i], states[i], seg, out)) if ops == 5 else \
                (lambda i: mixer.scan(projs[i], states[i], seg, out))
            extra = timed((lambda i: small_linear(h, mixer.gates)) if ops == 5 else
                          (lambda i: F.linear(projs[i][:, mixer.low_at:mixer.low_at + mixer.low_rank], mixer.low)), k, 6)
            low = 0 if ops == 5 else N * H * 2 * D * 2
            put(name, at, max(timed(inner, k, 6) - extra, 1e-9), state + N * (mixer.columns + mixer.out_columns) * 2 + low,
                float(ops) * N * mixer.heads * D * D, FP32)
            del projs, states, out
        # experts
        h = [rnd(N, W) for _ in range(2)]
        put("small_linear (router)", at, timed(lambda i: small_linear(h[i], moe.router), 2), N * W * 2 + E * W * 2)
        z = rnd(N, E, dt=torch.float32)
        ids, wts, counts = moe_select(z, E, 3, 4, 2)
        put("moe_select", at, timed(lambda i: moe_select(z, E, 3, 4, 2), 2), N * E * 4 + N * 24)
        put("moe_plan (after moe_select)", at,
            timed(lambda i: plan_of(moe_select(z, E, 3, 4, 2)), 2) - timed(lambda i: moe_select(z, E, 3, 4, 2), 2),
            N * 3 * 12)
        plan = plan_of((ids, wts, counts))
        act = moe.gate_up_rows(h[0], plan, wts)
        used = min(E, N * 3) + 1
        fl = 2.0 * N * S * W * (FF // 4)
        put("moe_gate_up", at, timed(lambda i: moe.gate_up_rows(h[i], plan, wts), 2, 6),
            used * 2 * (FF // 4) * W * 2 + N * W * 2 + N * FF * 2, 2 * fl)
        put("like: gate and up (library product), silu_and_mul", at, timed(lambda i: silu_and_mul(F.linear(h[i], gu[i])), 2, 6),
            2 * FF * W * 2 + N * W * 2 + N * FF * 2, 2 * fl)
        put("moe_down", at, timed(lambda i: moe.down_planes(act, plan), 2, 6),
            used * (FF // 4) * W * 2 + N * FF * 2 + S * N * W * 2, fl)
        full = rnd(N, FF)
        put("like: down (library product)", at, timed(lambda i: F.linear(full, dn[i]), 2, 6), FF * W * 2 + N * FF * 2 + N * W * 2, fl)
        del h, act, full
        m = N if phase == "decode" else prompts
        z = rnd(m, V)
        put("softcap", f"{m} rows of logits", timed(lambda i: softcap(z, 15.0), 1), m * V * 6)
    # ---- decode attention
    per = -(-prompt // BS)
    for B in (64, decode_batch):
        for ctx_len in (chunk, prompt):
            at = f"decode, {B} sequences, context {ctx_len}"
            k = _sets(B * ctx_len * HK * D * 4)
            caches = [rnd(B * per, BS, 2 * HK * D) for _ in range(k)]
            tables, ctx = torch.randperm(B * per, device=dev).int().view(B, per), i32([ctx_len] * B)
            q, sinks, out = rnd(B, H * D), rnd(H, dt=torch.float32), torch.empty(B, H * D, device=dev, dtype=BF16)
            for name, size_ in ((f"grouped_rows_attention, chunk {chunk}", chunk), ("grouped_rows_attention, no limit", None)):
                seen = ctx_len if size_ is None else (ctx_len - 1) % size_ + 1
                put(name, at, timed(lambda i: grouped_rows_attention(q, caches[i], H, HK, D, D, tables, ctx, D ** -0.5, out,
                                                                     chunk=size_, sinks=sinks), k),
                    2 * B * seen * HK * D * 2 + 2 * B * H * D * 2, 4.0 * B * H * seen * D)
            del caches
            kcs = [rnd(B * per, BS, HK, D) for _ in range(2 * k)]
            qd = rnd(B, H, D)
            put("like: paged_decode_attention", at,
                timed(lambda i: paged_decode_attention(qd, kcs[2 * i], kcs[2 * i + 1], ctx, tables, D ** -0.5), k),
                2 * B * ctx_len * HK * D * 2 + 2 * B * H * D * 2, 4.0 * B * H * ctx_len * D)
            del kcs
    # ---- prefill attention
    N, at, k = prompts * prompt, f"prefill, {prompts} x {prompt} tokens", 2
    parts = []
    for _ in range(prompts):
        s = Sequence([0] * prompt)
        s.block_table = list(range(per))
        parts.append(Portion(s, 0, prompt))
    qs, kvs = [rnd(N, H * D) for _ in range(k)], [rnd(N, 2 * HK * D) for _ in range(k)]
    out = torch.empty(N, H * D, device=dev, dtype=BF16)
    for name, size_ in ((f"run_attention, chunk {chunk}", chunk), ("run_attention, no limit", None)):
        tiles = i32(plan_runs(parts, BS, None if size_ is None else Chunk(size_)).tiles)
        pairs = sum((i % size_ if size_ else i) + 1 for i in range(prompt)) * prompts
        put(name, at, timed(lambda i: run_attention(qs[i], kvs[i], H, HK, D, D, tiles, D ** -0.5, out, chunk=size_, sinks=sinks), k, 6),
            N * (2 * H + 2 * HK) * D * 2, 4.0 * pairs * H * D)
    ks = [rnd(prompts, prompt, HK, D) for _ in range(2 * k)]
    put("like: scaled_dot_product_attention (library, causal)", at,
        timed(lambda i: F.scaled_dot_product_attention(
            qs[i].view(prompts, prompt, H, D).transpose(1, 2), ks[2 * i].transpose(1, 2), ks[2 * i + 1].transpose(1, 2),
            is_causal=True, enable_gqa=True), k, 6), N * (2 * H + 2 * HK) * D * 2, 4.0 * prompt * (prompt + 1) / 2 * prompts * H * D)
    return rows


def rutevik_kernels(size: str, decode_batch: int, prompts: int, prompt: int) -> list[dict]:
    """The same for Rutevik's kernels; each has the like kernel of Pedivik or Kapolorn behind it."""
    from zipage_amd.engine.inputs import plan_runs
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import (Experts, Rotary, attention_form, grouped_rows_attention, latent_rows_attention,
                                   latent_tiles_attention, relu_square, residual_norm, rotary_store, rotate_heads,
                                   run_attention, xielu)
    from zipage_amd.layers.latent import headwise_linear, latent_norm_store
    from zipage_amd.layers.moe import Plan, moe_select
    W, H, HK, D, FF, L, V, QR, KR, _ = SIZES[size]
    P, H2, HK2, V2 = D // 2, H // 2, HK // 2, 2 * D             # rotated part; heads of the differential layers
    dev, BS = torch.device("cuda:0"), 256
    rnd = lambda *s, dt=BF16: torch.randn(*s, device=dev, dtype=torch.float32).to(dt)
    i32 = lambda a: torch.as_tensor(a, dtype=torch.int32, device=dev)
    rows = []

    def put(name, where, secs, byts, flops=0.0):
        roof = max(byts / HBM, flops / MFMA)
        rows.append({"kernel": name, "at": where, "us": round(secs * 1e6, 1),
                     "bound": "hbm" if byts / HBM >= flops / MFMA else "mfma",
                     "roofline_us": round(roof * 1e6, 1), "frac": round(roof / secs, 3)})

    gen = torch.Generator(device=dev).manual_seed(0)
    silu = Experts(W, 32, 4, FF // 4, 0.0, score="sigmoid", act="silu")
    clamped = Experts(W, 32, 4, FF // 4, 7.0)
    silu.random(BF16, dev, gen)
    clamped.router, clamped.gate_up, clamped.down = silu.router, silu.gate_up, silu.down
    clamped.shared_gate_up = clamped.shared_down = None
    freqs, turn = rnd(D // 2, dt=torch.float32).abs(), Rotary(5e5, P).frequencies(dev)
    w32, b32 = torch.ones(W, device=dev), torch.zeros(W, device=dev)
    per, E = -(-prompt // BS), 32
    form = lambda gate: attention_form(30.0, 2, 0.5, 1e-6, V2, gate)
    for phase, N in (("decode", 64), ("decode", decode_batch), ("prefill", prompts * prompt)):
        at, big = f"{phase}, {N} tokens", N * W
        pos, slots = torch.arange(N, device=dev, dtype=torch.int32) % prompt, torch.randperm(N, device=dev).int()
        for planes in (1, 4):
            k = _sets(big * (10 + 2 * planes))
            xs, ys = [rnd(N, W, dt=torch.float32) for _ in range(k)], [rnd(planes, N, W) for _ in range(k)]
            for name, more in (("residual_norm, tanh norm", dict(norm_bias=b32, norm_alpha=0.6)), ("like: residual_norm, RMS norm", {})):
                put(f"{name}, {planes} planes", at,
                    timed(lambda i: residual_norm(xs[i], ys[i], w32, 1e-6, W, x_out=xs[i], **more), k), big * (10 + 2 * planes))
            del xs, ys
        n = N * FF * 3 // 2
        zs = [rnd(N, FF * 3 // 2) for _ in range(_sets(n * 4))]
        put("relu_square", at, timed(lambda i: relu_square(zs[i]), len(zs)), n * 4)
        put("like: xielu", at, timed(lambda i: xielu(zs[i], 0.8, 1.3), len(zs)), n * 4)
        del zs
        # latent rows
        wq, wc = torch.ones(QR, device=dev), torch.ones(KR, device=dev)
        for name, p, more in (("latent_norm_store, rotated part", P, dict(positions=pos, freqs=turn)), ("like: latent_norm_store", 0, {})):
            k = _sets(N * (QR + KR + p) * 4)
            downs, caches = [rnd(N, QR + KR + p) for _ in range(k)], [rnd(-(-N // BS), BS, KR + p) for _ in range(k)]
            put(name, at, timed(lambda i: latent_norm_store(downs[i], wq, wc, QR, KR, 1e-6, caches[i], slots, **more), k),
                N * (QR + KR + p) * 4)
            del downs, caches
        k = _sets(N * QR * 4)
        downs = [rnd(N, QR) for _ in range(k)]
        put("latent_norm_store, queries alone", at, timed(lambda i: latent_norm_store(downs[i], wq, None, QR, 0, 1e-6, None, None), k), N * QR * 4)
        del downs
        # queries, keys and values of the grouped heads
        width, kvw = (2 * H2 + 2 * HK2) * D + HK2 * V2, 2 * HK2 * D + HK2 * V2
        bias = rnd(width, dt=torch.float32)
        k = _sets(N * width * 4)
        qkvs, caches = [rnd(N, width) for _ in range(k)], [rnd(-(-N // BS), BS, kvw) for _ in range(k)]
        put("rotary_store, two maps, bias", at, timed(lambda i: rotary_store(
            qkvs[i], pos, freqs, H2, HK2, D, V2, caches[i], slots, maps=2, bias=bias), k), N * width * 4)
        put("like: rotary_store", at, timed(lambda i: rotary_store(qkvs[i], pos, freqs, H, HK, D, D, caches[i], slots), k), N * width * 4)
        del qkvs, caches
        if phase == "prefill":
            k = _sets(N * H * (D + P) * 2)
            qs = [rnd(N, H * (D + P)) for _ in range(k)]
            put("rotate_heads (the rotated part's bytes)", at, timed(lambda i: rotate_heads(qs[i], pos, turn, H, D), k), N * H * P * 4)
            del qs
        else:
            for name, w_, tail in (("q into the latent space", rnd(H, KR, D), P), ("values out of it", rnd(H, D, KR), 0)):
                M, K = w_.shape[1:]
                ws = [w_] + [rnd(H, M, K) for _ in range(_sets(H * M * K * 2) - 1)]
                for label, t in (((f"headwise_linear, {name}, turned tail", tail),) if tail else ()) + ((f"like: headwise_linear, {name}", 0),):
                    x = rnd(N, H, K + t)
                    more = dict(positions=pos, freqs=turn) if t else {}
                    put(label, at, timed(lambda i: headwise_linear(x, ws[i], **more), len(ws)),
                        H * M * K * 2 + N * H * (K + M + 2 * t) * 2, 2.0 * N * H * K * M)
                del ws
        # experts
        h, z = [rnd(N, W) for _ in range(2)], rnd(N, E, dt=torch.float32)
        for name, moe in (("sigmoids, silu, weight on the input", silu), ("softmax, clamped", clamped)):
            label = "like: " if moe is clamped else ""
            put(f"{label}moe_select, {name}", at, timed(lambda i: moe_select(z, E, 4, score=moe.score), 2), N * (E * 4 + 32))
            ids, wts, counts = moe_select(z, E, 4, score=moe.score)
            plan = Plan(ids, counts, E, False, BF16)
            act, used, fl = moe.gate_up_rows(h[0], plan, wts), min(E, N * 4), 2.0 * N * W * FF
            put(f"{label}moe_gate_up, {name}", at, timed(lambda i: moe.gate_up_rows(h[i], plan, wts), 2, 6),
                used * (FF // 2) * W * 2 + N * W * 2 + N * FF * 2, 2 * fl)
        put("moe_down (the same for both)", at, timed(lambda i: silu.down_planes(act, plan), 2, 6),
            used * (FF // 4) * W * 2 + N * FF * 2 + 4 * N * W * 2, fl)
        del h, act
    # ---- decode attention
    for B, ctx_len in ((1, prompt), (64, prompt), (decode_batch, prompt), (8, 4 * prompt)):
        at, pages = f"decode, {B} sequences, context {ctx_len}", -(-ctx_len // BS)
        tables, ctx = torch.randperm(B * pages, device=dev).int().view(B, pages), i32([ctx_len] * B)
        for name, p in (("latent_rows_attention, rotated part", P), ("like: latent_rows_attention", 0)):
            k = _sets(B * ctx_len * (KR + p) * 2)
            caches, q = [rnd(B * pages, BS, KR + p) for _ in range(k)], rnd(B, H, KR + p)
            put(name, at, timed(lambda i: latent_rows_attention(q, caches[i], tables, ctx, D ** -0.5, rank=KR), k),
                B * ctx_len * (KR + p) * 2 + B * H * (2 * KR + p) * 2, 2.0 * B * H * ctx_len * (2 * KR + p))
            del caches
        k = _sets(B * ctx_len * HK * D * 4)
        caches, q = [rnd(B * pages, BS, 2 * HK * D) for _ in range(k)], rnd(B, H * D)
        out, gate = torch.empty(B, H * D, device=dev, dtype=BF16), rnd(B, H * D)
        byts = 2 * B * ctx_len * HK * D * 2 + 2 * B * H * D * 2
        put("grouped_rows_attention, differential, soft cap, gate", at,
            timed(lambda i: grouped_rows_attention(q, caches[i], H2, HK2, D, V2, tables, ctx, D ** -0.5, out, form=form(gate)), k),
            byts + B * H * D * 2, 6.0 * B * H * ctx_len * D)
        put("like: grouped_rows_attention", at,
            timed(lambda i: grouped_rows_attention(q, caches[i], H, HK, D, D, tables, ctx, D ** -0.5, out), k), byts,
            4.0 * B * H * ctx_len * D)
        del caches
    # ---- prefill attention
    N, at, k = prompts * prompt, f"prefill, {prompts} x {prompt} tokens", 2
    parts = []
    for _ in range(prompts):
        s = Sequence([0] * prompt)
        s.block_table = list(range(per))
        parts.append(Portion(s, 0, prompt))
    tiles, pairs = i32(plan_runs(parts, BS, None).tiles), prompt * (prompt + 1) / 2 * prompts
    out, gate = torch.empty(N, H * D, device=dev, dtype=BF16), rnd(N, H * D)
    qs, kvs = [rnd(N, H * (D + P)) for _ in range(k)], [rnd(N, 2 * H * D) for _ in range(k)]
    shared = [rnd(N, KR + P)[:, KR:] for _ in range(k)]
    put("latent_tiles_attention, shared rotated part", at,
        timed(lambda i: latent_tiles_attention(qs[i], kvs[i], H, D, D, tiles, D ** -0.5, None, out, shared[i]), k, 6),
        N * (H * (4 * D + P) + P) * 2, 2.0 * pairs * H * (2 * D + P))
    qs = [rnd(N, H * D) for _ in range(k)]
    put("like: latent_tiles_attention", at,
        timed(lambda i: latent_tiles_attention(qs[i], kvs[i], H, D, D, tiles, D ** -0.5, None, out), k, 6),
        N * H * D * 4 * 2, 4.0 * pairs * H * D)
    kvs = [rnd(N, 2 * HK * D) for _ in range(k)]
    put("run_attention, differential, soft cap, gate", at,
        timed(lambda i: run_attention(qs[i], kvs[i], H2, HK2, D, V2, tiles, D ** -0.5, out, form=form(gate)), k, 6),
        N * (3 * H + 2 * HK) * D * 2, 6.0 * pairs * H * D)
    put("like: run_attention", at,
        timed(lambda i: run_attention(qs[i], kvs[i], H, HK, D, D, tiles, D ** -0.5, out), k, 6),
        N * (2 * H + 2 * HK) * D * 2, 4.0 * pairs * H * D)
    return rows


def mefupel_shapes(size: str):
    """Two attention layers with turning values, one of gated linear attention and one of attention over its keys
    beside retention, in turn, without a loop.  Pedivik and Kapolorn keep their windows and chunks of the same length."""
    from zipage_amd.engine import MefupelShape
    from zipage_amd.engine.mefupel import GatedMixer, MefupelLayer, PairMixer, TurningMixer
    from zipage_amd.layers import Rotary
    W, H, HK, D, FF, L, V, _, _, win = SIZES[size]
    turning = TurningMixer(H, HK, D, D, win, Rotary(5e5, D, interleaved=True), D ** -0.5)
    pair = PairMixer(H, HK, D, win, Rotary(2e4, D // 2), D ** -0.5, H // 2, D, D, Rotary(1e6, D),
                     tuple(1 - 2.0 ** (-5 - 6 * i / (H // 2)) for i in range(H // 2)))
    layers = tuple(MefupelLayer((turning, turning, GatedMixer(H, D, D, 16.0), pair)[i % 4], FF * 3 // 2) for i in range(L))
    return {"mefupel": MefupelShape(V, W, layers, None, 1e-6), "pedivik": shapes(size)[0], "kapolorn": kapolorn_shapes(size)[0]}


def mefupel_kernels(size: str, decode_batch: int, prompts: int, prompt: int) -> list[dict]:
    """The same for Mefupel's kernels; each has the like kernel of Kapolorn, Rutevik or Pedivik behind it."""
    import torch.nn.functional as F
    from zipage_amd.engine.inputs import plan_runs
    from zipage_amd.engine.qwen3 import Segments
    from zipage_amd.engine.sequence import Portion, Sequence
    from zipage_amd.layers import (ChannelDelta, LinearAttention, MatrixMemory, Rotary, attention_form, grouped_rows_attention,
                                   normed_powers, residual_norm, rotary_store, run_attention, small_linear, store_form, xielu)
    from zipage_amd.sight import Chunk
    W, H, HK, D, FF, L, V, _, _, win = SIZES[size]
    dev, BS = torch.device("cuda:0"), 256
    rnd = lambda *s, dt=BF16: torch.randn(*s, device=dev, dtype=torch.float32).to(dt)
    i32 = lambda a: torch.as_tensor(a, dtype=torch.int32, device=dev)
    rows = []

    def put(name, where, secs, byts, flops=0.0, peak=MFMA):
        roof = max(byts / HBM, flops / peak)
        bound = "hbm" if byts / HBM >= flops / peak else ("mfma" if peak == MFMA else "fp32")
        rows.append({"kernel": name, "at": where, "us": round(secs * 1e6, 1), "bound": bound,
                     "roofline_us": round(roof * 1e6, 1), "frac": round(roof / secs, 3)})

    w32, one, per = torch.ones(W, device=dev), torch.ones(2, device=dev), -(-prompt // BS)
    for phase, N in (("decode", 64), ("decode", decode_batch), ("prefill", prompts * prompt)):
        at, big = f"{phase}, {N} tokens", N * W
        seqs = N if phase == "decode" else prompts
        # branches joining the stream
        k = _sets(big * 16)
        xs, ys = [rnd(N, W, dt=torch.float32) for _ in range(k)], [rnd(3, N, W) for _ in range(k)]
        held = [rnd(1, N, W, dt=torch.float32) for _ in range(k)]
        put("residual_norm, two normed branches and a plain one", at,
            timed(lambda i: residual_norm(xs[i], ys[i][0], w32, 1e-6, W, 1.0, x_out=xs[i], y_weight=w32,
                                          more=((ys[i][1], w32), (ys[i][2], None))), k), big * 16)
        put("residual_norm, embedding and vector before a pass", at,
            timed(lambda i: residual_norm(xs[i], ys[i][0], w32, 1e-6, W, 1.0, x_out=xs[i], history=held[i], mix=one, shift=w32), k),
            big * 16)
        put("residual_norm, one plain branch", at,
            timed(lambda i: residual_norm(xs[i], ys[i][0], w32, 1e-6, W, 1.0, x_out=xs[i]), k), big * 12)
        put("like: residual_norm of a normed branch", at,
            timed(lambda i: residual_norm(xs[i], ys[i][0], w32, 1e-6, W, x_out=xs[i], y_weight=w32), k), big * 12)
        del xs, ys, held
        n = N * FF * 3 // 2
        zs, out = [rnd(N, FF * 3 // 2) for _ in range(_sets(n * 4))], rnd(N, FF * 3 // 2)
        put("normed_powers", at, timed(lambda i: normed_powers(zs[i], (0.7, -0.5, 0.4, 0.3), 1e-6, FF * 3 // 2, out), len(zs)), n * 4)
        put("like: xielu", at, timed(lambda i: xielu(zs[i], 0.8, 1.3), len(zs)), n * 4)
        del zs, out
        # queries, keys and values of the grouped heads
        pos, slots = torch.arange(N, device=dev, dtype=torch.int32) % prompt, torch.randperm(N, device=dev).int()
        width, freqs, half = (H + 2 * HK) * D, Rotary(5e5, D).frequencies(dev), Rotary(2e4, D // 2).frequencies(dev)
        k = _sets(N * width * 4)
        qkvs, caches = [rnd(N, width) for _ in range(k)], [rnd(-(-N // BS), BS, 2 * HK * D) for _ in range(k)]
        turns, qk = torch.empty(N, D // 2, 2, device=dev), torch.ones((H + HK) * D, device=dev)
        turning, keys = store_form(value_freqs=freqs, turns=turns), store_form(qk, H * D, HK * D, 1e-6, tied=True)
        put("rotary_store, turning values", at,
            timed(lambda i: rotary_store(qkvs[i], pos, freqs, H, HK, D, D, caches[i], slots, form=turning), k), N * (width + 2 * D) * 4)
        put("rotary_store, norms, keys as values", at,
            timed(lambda i: rotary_store(qkvs[i], pos, half, H, HK, D, D, caches[i], slots, form=keys), k),
            N * (2 * width - HK * D) * 2)
        put("like: rotary_store", at, timed(lambda i: rotary_store(qkvs[i], pos, freqs, H, HK, D, D, caches[i], slots), k), N * width * 4)
        del qkvs, caches
        # recurrences
        n = N // seqs
        seg = Segments(i32(range(0, N, n)), i32([n] * seqs), i32(torch.randperm(seqs)), i32([5] * seqs), longest=n,
                       max_count=int(n == 1))
        seg = SimpleNamespace(segments=seg if n < 16 else None, run_segments=None if n < 16 else seg)
        retention = LinearAttention(W, H // 2, D, D, 1e-6, decay=(0.99,) * (H // 2), rotary=Rotary(1e6, D))
        for name, mixer, ops in ((f"linear attention, a decay per channel, {H} heads", LinearAttention(W, H, D, D, 1e-6, tau=16.0, weighted=True), 5),
                                 (f"like: delta_scan, {H} heads", ChannelDelta(W, H, H // 2, D, D, 4, 1e-6), 7),
                                 (f"linear attention, retention, {H // 2} heads", retention, 4),
                                 (f"like: mlstm_scan, {H // 2} heads", MatrixMemory(W, H // 2, D, D, 15.0, 1e-6), 5)):
            ranks = (128, 128) if isinstance(mixer, ChannelDelta) else () if isinstance(mixer, MatrixMemory) else (16,)
            small = {q: torch.randn(*s) * 0.02 for q, s in mixer.shapes(*ranks).items()}
            mixer.load({q: t.to(BF16) for q, t in small.items()}, BF16, dev, W)
            h, k = rnd(N, W), 2
            projs = [rnd(N, mixer.columns) for _ in range(k)]
            states = [mixer.allocate(seqs + 1, BF16, dev) for _ in range(k)]
            out = torch.empty(N, mixer.out_columns, device=dev, dtype=BF16)
            byts = 2 * seqs * mixer.heads * D * D * 4 + N * (mixer.columns + mixer.out_columns) * 2
            gates = isinstance(mixer, MatrixMemory)
            secs = timed((lambda i: mixer.scan(h, projs[i], states[i], seg, out)) if gates else
                         (lambda i: mixer.scan(projs[i], states[i], seg, out)), k, 6)
            if gates:
                secs -= timed(lambda i: small_linear(h, mixer.gates), k, 6)
            elif mixer.low is not None:
                secs -= timed(lambda i: F.linear(projs[i][:, mixer.low_at:mixer.low_at + mixer.low_rank], mixer.low), k, 6)
                byts += N * mixer.low.shape[0] * 2
            put(name, at, max(secs, 1e-9), byts, float(ops) * N * mixer.heads * D * D, FP32)
            del projs, states, out
    # ---- decode attention
    sinks = rnd(H, dt=torch.float32)
    for B, ctx_len in ((1, prompt), (64, prompt), (decode_batch, prompt)):
        at, pages = f"decode, {B} sequences, context {ctx_len}", -(-ctx_len // BS)
        tables, ctx = torch.randperm(B * pages, device=dev).int().view(B, pages), i32([ctx_len] * B)
        k = _sets(B * win * HK * D * 4)
        caches, q = [rnd(B * pages, BS, 2 * HK * D) for _ in range(k)], rnd(B, H * D)
        out, form = torch.empty(B, H * D, device=dev, dtype=BF16), attention_form(turns=rnd(B, D // 2, 2, dt=torch.float32))
        for name, seen, more in ((f"grouped_rows_attention, window {win}, turning back", min(win, ctx_len), dict(window=win, form=form)),
                                 (f"grouped_rows_attention, window {win}, sinks", min(win, ctx_len), dict(window=win, sinks=sinks)),
                                 (f"like: grouped_rows_attention, chunk {win}, sinks", (ctx_len - 1) % win + 1, dict(chunk=win, sinks=sinks))):
            put(name, at, timed(lambda i: grouped_rows_attention(q, caches[i], H, HK, D, D, tables, ctx, D ** -0.5, out, **more), k),
                2 * B * seen * HK * D * 2 + 2 * B * H * D * 2, 4.0 * B * H * seen * D)
        del caches
    # ---- prefill attention
    N, at, k = prompts * prompt, f"prefill, {prompts} x {prompt} tokens", 2
    parts = []
    for _ in range(prompts):
        s = Sequence([0] * prompt)
        s.block_table = list(range(per))
        parts.append(Portion(s, 0, prompt))
    qs, kvs, out = [rnd(N, H * D) for _ in range(k)], [rnd(N, 2 * HK * D) for _ in range(k)], torch.empty(N, H * D, device=dev, dtype=BF16)
    form, chunk = attention_form(turns=rnd(N, D // 2, 2, dt=torch.float32)), Chunk(win)
    window, blocks = i32(plan_runs(parts, BS, win).tiles), i32(plan_runs(parts, BS, chunk).tiles)
    pairs = sum(min(i + 1, win) for i in range(prompt)) * prompts
    for name, tiles, seen, more in ((f"run_attention, window {win}, turning back", window, pairs, dict(window=win, form=form)),
                                    (f"run_attention, window {win}, sinks", window, pairs, dict(window=win, sinks=sinks)),
                                    (f"like: run_attention, chunk {win}, sinks", blocks, sum(i % win + 1 for i in range(prompt)) * prompts,
                                     dict(chunk=win, sinks=sinks))):
        put(name, at, timed(lambda i: run_attention(qs[i], kvs[i], H, HK, D, D, tiles, D ** -0.5, out, **more), k, 6),
            N * (2 * H + 2 * HK) * D * 2, 4.0 * seen * H * D)
    return rows


def beside_qwen3(model: str, make):
    return lambda size: dict(zip((model, "qwen3"), make(size)))


MODELS = {"pedivik": (beside_qwen3("pedivik", shapes), kernels),
          "kapolorn": (beside_qwen3("kapolorn", kapolorn_shapes), kapolorn_kernels),
          "rutevik": (rutevik_shapes, rutevik_kernels),
          "mefupel": (mefupel_shapes, mefupel_kernels)}


def compare(model: str = "pedivik", sizes=("1k", "4k"), out_tokens: int = 64) -> dict:
    """The whole report.  The headline figure is the model's decode rate at the largest size and batch."""
    import sys
    report = {"sizes": {}}
    make, table = MODELS[model]
    for size in sizes:
        entry = {name: {} for name in make(size)}
        for batch, prompt in ((1, 2048), (64, 2048), (256, 2048)):
            for name, shape in make(size).items():
                entry[name][f"{batch} x {prompt}"] = throughput(shape, batch, prompt, out_tokens)
                print(f"{size}: {name}, {batch} x {prompt} tokens", file=sys.stderr, flush=True)
        entry["kernels"] = table(size, 256, 8, 2048)
        report["sizes"][size] = entry
    return report
