"""Kapolorn on the host, no GPU: the oracle's mechanisms against other forms of the same equations, that the
test cases would show the faults they are there for, readers, step plans, pages and scheduling."""
import copy
import json

import numpy as np
import pytest
import torch

from oracle import kapolorn_oracle as O
from tests import kapolorn_cases as C
from zipage_amd.engine import EngineConfig, KapolornShape, PagePool, SamplingParams, Scheduler, Sequence
from zipage_amd.engine.inputs import plan_portions, plan_runs
from zipage_amd.engine.registry import arch_for_shape, read_shape
from zipage_amd.engine.sequence import Portion
from zipage_amd.sight import Chunk, first_seen


def _r(g, *s):
    return torch.randn(*s, generator=g, dtype=torch.float64)


# ------------------------------------------------------------------ the oracle itself
def test_oracle_attention_against_loops():
    g = torch.Generator().manual_seed(0)
    m = {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 3, "scale": 0.7, "mask": {"size": 4}, "rot": {"base": 50.0, "dims": 4}}
    h = _r(g, 11, 5)
    w = {"q": _r(g, 24, 5), "k": _r(g, 12, 5), "v": _r(g, 6, 5), "sink": _r(g, 4), "o": _r(g, 5, 12)}
    got = O.sink_attention(h, w, m)

    def turned(x, p):                    # complex numbers for the pairs (i, i + 2)
        z = [complex(x[i], x[i + 2]) * np.exp(1j * p * 50.0 ** (-2 * i / 4)) for i in range(2)]
        return np.array([z[0].real, z[1].real, z[0].imag, z[1].imag, x[4], x[5]])
    for i in range(11):
        out = []
        for a in range(4):
            b = a // 2
            q = turned((w["q"] @ h[i])[a * 6:a * 6 + 6].tolist(), i)
            e, vs = [], []
            for j in range(i // 4 * 4, i + 1):
                k = turned((w["k"] @ h[j])[b * 6:b * 6 + 6].tolist(), j)
                e.append(np.exp(0.7 * q @ k))
                vs.append((w["v"] @ h[j])[b * 3:b * 3 + 3].numpy())
            out.append(sum(x * v for x, v in zip(e, vs)) / (sum(e) + np.exp(float(w["sink"][a]))))
        assert np.allclose(got[i].numpy(), w["o"].numpy() @ np.concatenate(out), atol=1e-12)


def test_oracle_recurrences_against_closed_forms():
    g = torch.Generator().manual_seed(1)
    n, H, D, V = 9, 2, 3, 4
    q, k, v = _r(g, n, H, D), _r(g, n, H, D), _r(g, n, H, V)
    i, f = 2 * _r(g, n, H), -torch.rand(n, H, generator=g, dtype=torch.float64)
    got = O.mlstm_recurrence(q, k, v, i, f)
    for h in range(H):
        for t in range(n):
            F = [float(f[s + 1:t + 1, h].sum()) for s in range(t + 1)]
            m = max([float(f[:t + 1, h].sum())] + [F[s] + float(i[s, h]) for s in range(t + 1)])
            a = torch.tensor([np.exp(F[s] + float(i[s, h]) - m) for s in range(t + 1)]) * (k[:t + 1, h] @ q[t, h])
            den = max(abs(float(a.sum())), np.exp(-m)) + 1e-6
            assert torch.allclose(got[t, h], a @ v[:t + 1, h] / den, atol=1e-12)
    # the delta rule as a product of matrices: S_t = (I - beta k k^T) diag(g) S_{t-1} + beta k v^T
    gd, beta = torch.rand(n, H, D, generator=g, dtype=torch.float64), torch.rand(n, H, generator=g, dtype=torch.float64)
    got = O.delta_recurrence(q, k, v, gd, beta)
    for h in range(H):
        S = torch.zeros(D, V, dtype=torch.float64)
        for t in range(n):
            kk = k[t, h][:, None]
            S = (torch.eye(D) - beta[t, h] * kk @ kk.T) @ torch.diag(gd[t, h]) @ S + beta[t, h] * kk @ v[t, h][None]
            assert torch.allclose(got[t, h], S.T @ q[t, h], atol=1e-12)
    x, w = _r(g, 7, 5), _r(g, 5, 3)
    y = torch.nn.functional.conv1d(torch.cat([torch.zeros(2, 5), x]).T[None], w[:, None], groups=5)[0].T
    assert torch.allclose(O.short_conv(x, w), torch.nn.functional.silu(y), atol=1e-12)


def test_oracle_routing():
    z = torch.tensor([[3.0, 0.0, 2.0, 1.9, -1.0, 2.5]], dtype=torch.float64)
    s = torch.softmax(z, -1)[0]
    for count, keep, top, want in ((3, 1, 2, [0, 1]), (3, 2, 3, [0, 5, 1]), (1, 1, 3, [0, 5, 2]), (2, 1, 2, [0, 2])):
        a = O.route(z, top, count, keep)[0]
        assert sorted(a.nonzero().flatten().tolist()) == sorted(want)
        assert torch.equal(a[want], s[want])
    w = {"gate": torch.tensor([[2.0], [-3.0]]).double(), "up": torch.tensor([[-4.0], [0.5]]).double(), "down": torch.eye(2).double()}
    y = O.expert(torch.ones(1, 1).double(), w, 1.0)[0]
    want = [1 / (1 + np.exp(-1.702)) * 0.0, -3 / (1 + np.exp(3 * 1.702)) * 1.5]      # min, no lower clamp; clamp
    assert np.allclose(y.numpy(), want, atol=1e-12)


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_cases_show_planted_faults(name, monkeypatch):
    """Each fault, planted in the oracle, moves the logits far beyond what the float32 GPU tests allow."""
    cfg, w = C.case(name)
    toks = C.tokens(cfg, 80, 3)
    right = C.expected(name, toks)
    limit = 1e-2

    def fault(change_cfg=None, change_w=None):
        c, t = copy.deepcopy(cfg), dict(w)
        if change_cfg:
            change_cfg(c)
        if change_w:
            change_w(t)
        return float(C.row_errors(O.forward(c, t, toks)[0], right).max())

    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        change = lambda f: fault(lambda c: f(c["layers"][i]))
        scaled = lambda k, by: fault(change_w=lambda t: t.update({p + k: t[p + k] * by}))
        if l["type"] == "parallel":
            size = m["left"]["mask"]["size"]
            if size < 80:
                assert change(lambda l: l["mixer"]["left"]["mask"].update(size=size + 1)) > limit, i
                assert size == 1 or change(lambda l: l["mixer"]["left"]["mask"].update(size=size - 1)) > limit, i
            for k in ("left_scale", "right_scale"):
                assert change(lambda l: l["mixer"].update({k: m[k] * 1.5})) > limit, (i, k)
            if size > 1:
                assert change(lambda l: l["mixer"]["left"].update(scale=m["left"]["scale"] * 1.5)) > limit, i
                assert change(lambda l: l["mixer"]["left"]["rot"].update(base=3.0)) > limit or m["left"]["rot"]["dims"] <= 2, i
            assert change(lambda l: l["mixer"]["right"].update(gate_cap=1.0)) > limit, i
            assert fault(change_w=lambda t: t.update({p + "mix.left.sink": t[p + "mix.left.sink"] - 40})) > limit, i
            for k in ("i.b", "f.b"):
                assert fault(change_w=lambda t: t.update({p + "mix.right." + k: t[p + "mix.right." + k] + 1})) > limit, (i, k)
            for k in ("norm", "g"):
                assert scaled("mix.right." + k, -1) > limit, (i, k)
        else:
            for k in ("norm", "g1", "b", "a1", "A_log", "dt_bias", "v.conv") + (("q.conv", "k.conv") if m["conv"] > 1 else ()):
                flip = (lambda t: t.update({p + "mix." + k: t[p + "mix." + k].flip(-1)})) if k.endswith("conv") and m["conv"] > 1 \
                    else (lambda t: t.update({p + "mix." + k: t[p + "mix." + k] * -2}))
                assert fault(change_w=flip) > limit, (i, k)
        for k in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] else ()):
            assert scaled(k, -2) > limit, (i, k)
        if l["mlp"]:
            c = l["mlp"]
            assert change(lambda l: l["mlp"]["expert"].update(limit=0.2)) > limit, i
            assert change(lambda l: l["mlp"]["shared"].update(limit=0.2)) > limit, i
            if c["router"]["top"] > 1:
                assert change(lambda l: l["mlp"]["router"].update(top=c["router"]["top"] - 1)) > limit, i
            if c["router"]["groups"]["keep"] < c["router"]["groups"]["count"]:
                assert change(lambda l: l["mlp"]["router"]["groups"].update(keep=c["router"]["groups"]["count"])) > limit, i
    assert fault(lambda c: c["loop"].update(times=cfg["loop"]["times"] + 1)) > limit
    assert fault(lambda c: c.update(logit_softcap=cfg["logit_softcap"] * 1.3)) > limit
    assert fault(lambda c: c["embedding"].update(scale=cfg["embedding"]["scale"] * 3)) > limit
    # a state that is lost between two tokens, in one place
    for mech in ("mlstm_recurrence", "delta_recurrence"):
        if mech == "delta_recurrence" or any(l["type"] == "parallel" for l in cfg["layers"]):
            whole = getattr(O, mech)
            monkeypatch.setattr(O, mech, lambda *a: torch.cat([whole(*(x[:40] for x in a)), whole(*(x[40:] for x in a))]))
            assert fault() > limit, mech
            monkeypatch.setattr(O, mech, whole)


# ------------------------------------------------------------------ readers
def test_config_reader_and_registry(tmp_path):
    cfg = C.CONFIGS["odd"]
    s = KapolornShape.from_config(cfg)
    assert (s.width, s.vocab, s.eps, s.embed_scale, s.logit_softcap) == (76, 131, 1e-3, 0.7, 9.0)
    assert s.order == [0, 1, 2, 1, 2, 1, 2]
    a = s.layers[0].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.chunk, a.rot_dims, a.memory_heads, a.memory_dim, a.memory_vdim) == \
        (6, 3, 24, 40, 7, 10, 3, 20, 24)
    assert (s.layers[2].mixer.scale, s.layers[2].mixer.gate_cap, s.layers[2].mixer.left_scale) == (0.21, 2.5, 1.3)
    assert (s.layers[1].mixer.taps, s.layers[1].mlp) == (3, None)
    f = s.layers[0].mlp
    assert (f.experts, f.top, f.groups, f.keep, f.ff, f.limit, f.shared_ff, f.shared_limit) == (10, 3, 5, 2, 44, 0.8, 72, 2.0)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert read_shape(str(tmp_path)) == s and arch_for_shape(s).name == "Kapolorn"
    for path, value in ((("mixer", "left", "softcap"), 1), (("mixer", "left", "mask", "kind"), "window"), (("mlp", "kind"), "dense"),
                        (("mixer", "left", "mask", "size"), 0), (("type",), "conv"), (("mlp", "router", "bias"), True),
                        (("mixer", "right", "conv"), 4), (("mlp", "shared", "top"), 1)):
        bad = copy.deepcopy(cfg)
        d = bad["layers"][0]
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            KapolornShape.from_config(bad)
    for loop in ({"start": 2, "stop": 1, "times": 2}, {"start": 0, "stop": 4, "times": 1}, {"start": 0, "stop": 1, "times": 0}):
        with pytest.raises(ValueError, match="loop"):
            KapolornShape.from_config({**cfg, "loop": loop})


def test_load_refuses_wrong_shapes_and_leftovers():
    from zipage_amd.engine import Kapolorn
    cfg, w = C.case("odd")
    shape = KapolornShape.from_config(cfg)
    m = Kapolorn(shape, "cpu", weights=dict(w))
    assert m.lookback == 33 and m.sights == [Chunk(7), Chunk(33)] and m.padded_width == 96
    m.allocate_caches(3, 16, 5)
    assert len(m.caches) == 7 and m.caches[1][0].dtype == torch.float32 and m.caches[1][0].shape[:2] == (5, 6)
    for name in ("l1.mix.a1", "l0.mlp.e9.up", "l2.mix.left.sink"):
        with pytest.raises(KeyError, match=name):
            Kapolorn(shape, "cpu", weights={k: v for k, v in w.items() if k != name})
    with pytest.raises(ValueError, match="final.norm"):
        Kapolorn(shape, "cpu", weights={**w, "final.norm": w["final.norm"][:-1]})
    with pytest.raises(ValueError, match="extra"):
        Kapolorn(shape, "cpu", weights={**w, "extra": w["embed"]})
    with pytest.raises(ValueError, match="float16"):
        Kapolorn(shape, "cpu", dtype=torch.float16, weights=dict(w))


def test_expert_weights_in_tile_order():
    """Element (row, column) of an expert matrix is where the kernels look for it."""
    from zipage_amd.layers.moe import gate_up_order, tile_order
    for dtype, piece in ((torch.bfloat16, 8), (torch.float32, 4)):
        w = torch.arange(48 * 64).view(48, 64).to(torch.float32)
        t = tile_order(w.to(dtype)).flatten()
        w = w.to(dtype)
        for row, col in ((0, 0), (5, 63), (17, 8), (47, 33), (31, 31)):
            step, inside = divmod(col, 4 * piece)
            g, e = divmod(inside, piece)
            at = ((row // 16) * (64 // (4 * piece)) + step) * 64 * piece + (g * 16 + row % 16) * piece + e
            assert t[at] == w[row, col]
    gate, up = torch.arange(32.0).view(32, 1), 100 + torch.arange(32.0).view(32, 1)
    both = gate_up_order(gate, up).flatten().tolist()
    assert both == [*range(16), *range(100, 116), *range(16, 32), *range(116, 132)]


# ------------------------------------------------------------------ plans and pages
def _seq(n, bs=16, max_tokens=8, base=0):
    return Sequence([base + i for i in range(n)], SamplingParams(max_tokens=max_tokens, ignore_eos=True), bs)


def test_chunked_run_plan_covers_every_visible_key():
    rng = np.random.default_rng(0)
    for size in (1, 5, 64, 300, 4096):
        seqs = []
        for start, count in ((0, 130), (37, 16), (200, 257), (64, 2)):
            s = _seq(start + count)
            s.block_table = list(rng.permutation(100)[: -(-len(s) // 16)])
            seqs.append(Portion(s, start, count))
        runs = plan_runs(seqs, 16, Chunk(size))
        if runs.key_slots is None:
            runs.key_slots = np.concatenate([[p.seq.block_table[t // 16] * 16 + t % 16 for t in
                                              range(p.start, p.start + p.count)] for p in seqs])
        rows = [(p, t) for p in seqs for t in range(p.start, p.start + p.count)]
        met = 0
        for q0, n, k0, rel in runs.tiles.tolist():
            for i in range(n):
                p, t = rows[q0 + i]
                low = (rel + i) // size * size               # the run's first key starts a chunk
                got = runs.key_slots[k0 + low:k0 + rel + i + 1].tolist()
                assert got == [p.seq.block_table[j // 16] * 16 + j % 16 for j in range(t // size * size, t + 1)]
                met += 1
        assert met == len(rows)
    assert [first_seen(p, Chunk(5)) for p in (0, 4, 5, 9, 10)] == [0, 0, 5, 5, 10]
    assert [first_seen(p, 5) for p in (0, 4, 5, 9)] == [0, 0, 1, 5] and first_seen(7, None) == 0


def test_portion_plan_names_the_segments():
    a, b, c = _seq(20), _seq(50, base=100), _seq(9, base=200)
    a.query_id, b.query_id, c.query_id = 3, 1, 2
    a.block_table, b.block_table, c.block_table = [5, 6], [-1, 1, 2, 3], [9]
    plan = plan_portions([Portion(b, 20, 30), Portion(a, 19, 1), Portion(c, 5, 3)], 16, [Chunk(33)], 16)
    assert plan.first_row == [4, 0, 1]
    assert plan.short == 2
    assert plan.segments.tolist() == [[0, 1, 4], [1, 3, 30], [3, 2, 1], [19, 5, 20]]


def test_pages_behind_the_chunk_come_back():
    pool, lookback = PagePool(8, 16, 100), 20
    s = _seq(200)
    for upto in range(1, 201):
        pool.grow(s, upto)
        pool.computed(s, upto, lookback)
        for t in range(upto // 20 * 20, upto):               # what the next token sees
            assert s.block_table[t // 16] >= 0
        assert len([p for p in s.block_table if p >= 0]) <= 3
    pool.release(s)
    assert pool.num_free == 8 and not pool.refcount.any()


def test_recurrent_models_share_no_prefix():
    """A state exists only behind tokens that ran: prompts with a common beginning run in full."""
    shape = KapolornShape.from_config(C.CONFIGS["odd"])
    cfg = EngineConfig(shape=shape, kvcache_block_size=16, num_kvcache_blocks=24, max_concurrency=2,
                       max_num_batched_tokens=40, enable_prefix_cache=True)
    sched = Scheduler(cfg)
    for _ in range(3):
        sched.add(_seq(70, max_tokens=3))
    ran = 0
    while not sched.is_finished():
        batch = sched.schedule_portions(33)
        assert batch
        done = []
        for p in batch:
            ran += p.count
            sched.pool.computed(p.seq, p.start + p.count, 33)
            if p.ends:
                done.append(p.seq)
        sched.postprocess(done, None, advance=True)
    assert ran == 3 * 72 and sched.pool.num_free == 24 and sched.pool.reserved == 0
