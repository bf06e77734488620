"""Mefupel on the host, no GPU: the oracle's mechanisms against other forms of the same equations, that the test
cases would show the faults they are there for, readers, orders of dimensions, plans, pages and scheduling."""
import copy
import json
import math

import numpy as np
import pytest
import torch

from oracle import mefupel_oracle as O
from tests import mefupel_cases as C
from zipage_amd.engine import EngineConfig, Mefupel, MefupelShape, PagePool, SamplingParams, Scheduler, Sequence
from zipage_amd.engine.mefupel import GatedMixer, PairMixer, TurningMixer
from zipage_amd.engine.registry import arch_for_shape, read_shape
from zipage_amd.layers import GroupedAttention, LinearAttention
from zipage_amd.layers.rotary import Rotary


def _r(g, *s):
    return torch.randn(*s, generator=g, dtype=torch.float64)


# ------------------------------------------------------------------ the oracle itself
def _turned(x, angle_of, pairs):
    """Complex numbers for the pairs; what belongs to none stays."""
    out = np.array(x, dtype=float)
    for i, (a, b) in enumerate(pairs):
        z = complex(x[a], x[b]) * np.exp(1j * angle_of(i))
        out[a], out[b] = z.real, z.imag
    return out


def test_oracle_turning_values_against_loops():
    g = torch.Generator().manual_seed(0)
    m = C.attention(4, 2, 6, 8, 5, 4, base=50.0, scale=0.7)
    h = _r(g, 12, 5)
    w = {"q": _r(g, 24, 5), "k": _r(g, 12, 5), "v": _r(g, 16, 5), "o": _r(g, 5, 32)}
    n = {k: v.numpy() for k, v in w.items()}
    got = O.rotated_value_attention(h, w, m)
    key = lambda x, p: _turned(x, lambda i: p * 50.0 ** (-2 * i / 4), [(0, 1), (2, 3)])
    val = lambda x, p: _turned(x, lambda i: p * 50.0 ** (-2 * i / 8), [(2 * i, 2 * i + 1) for i in range(4)])
    for i in range(12):
        out = []
        for a in range(4):
            b, lo = a // 2, max(0, i - 4)
            q = key((n["q"] @ h[i].numpy())[a * 6:a * 6 + 6], i)
            e = np.exp([0.7 * q @ key((n["k"] @ h[t].numpy())[b * 6:b * 6 + 6], t) for t in range(lo, i + 1)])
            # each value turned by the distance
            out.append(sum(x * val((n["v"] @ h[t].numpy())[b * 8:b * 8 + 8], t - i) for x, t in zip(e, range(lo, i + 1))) / e.sum())
        assert np.allclose(got[i].numpy(), n["o"] @ np.concatenate(out), atol=1e-11)


def test_oracle_attention_over_its_keys_against_loops():
    g = torch.Generator().manual_seed(1)
    m = C.attention(4, 2, 6, 6, 3, 4, base=20.0, scale=0.4)
    h = _r(g, 9, 5)
    w = {"q": _r(g, 24, 5), "k": _r(g, 12, 5), "o": _r(g, 5, 24), "q.norm": _r(g, 24), "k.norm": _r(g, 12), "sink": _r(g, 4)}
    n = {k: v.numpy() for k, v in w.items()}
    got = O.key_value_attention(h, w, m, 1e-2)
    unit = lambda x: x / np.sqrt((x * x).mean() + 1e-2)
    turn = lambda x, p: _turned(x, lambda i: p * 20.0 ** (-2 * i / 4), [(0, 2), (1, 3)])
    for i in range(9):
        out = []
        for a in range(4):
            b, seen = a // 2, range(max(0, i - 2), i + 1)
            q = turn((unit(n["q"] @ h[i].numpy()) * n["q.norm"])[a * 6:a * 6 + 6], i)
            raw = {t: n["k"] @ h[t].numpy() for t in seen}
            e = {t: math.exp(0.4 * q @ turn((unit(raw[t]) * n["k.norm"])[b * 6:b * 6 + 6], t)) for t in seen}
            out.append(sum(e[t] * raw[t][b * 6:b * 6 + 6] for t in seen) / (sum(e.values()) + math.exp(n["sink"][a])))
        assert np.allclose(got[i].numpy(), n["o"] @ np.concatenate(out), atol=1e-11)


def test_oracle_recurrences_against_attention_forms():
    """Retention and gated linear attention as sums over all earlier tokens with products of decays."""
    g = torch.Generator().manual_seed(2)
    q, k, v = _r(g, 10, 2, 4), _r(g, 10, 2, 4), _r(g, 10, 2, 3)
    decay = torch.rand(10, 2, 4, generator=g, dtype=torch.float64)
    got = O.linear_recurrence(q, k, v, decay)
    for t in range(10):
        want = sum((q[t] * k[s] * decay[s + 1:t + 1].prod(0)).sum(-1)[:, None] * v[s] for s in range(t + 1))
        assert torch.allclose(got[t], want)
    m = C.pair((1, 1, 4, 9, 2), (2, 4, 3), 4, (0.3, 0.8))["right"]
    h = _r(g, 7, 5)
    w = {"q": _r(g, 8, 5), "k": _r(g, 8, 5), "v": _r(g, 6, 5), "g": _r(g, 6, 5), "o": torch.eye(6, dtype=torch.float64)}
    got = O.retention(h, w, m, 1e-3)
    f = [1.0, 300.0 ** -0.5]
    z = lambda x, p: np.array([complex(x[i], x[i + 2]) * np.exp(1j * p * f[i]) for i in range(2)])
    for a, d in ((0, 0.3), (1, 0.8)):
        heads = lambda n_, size: (h @ w[n_].T).view(7, 2, size)[:, a].numpy()
        qs, ks, vs, gs = heads("q", 4), heads("k", 4), heads("v", 3), heads("g", 3)
        for t in range(7):
            o = sum(d ** (t - s) * (z(qs[t], t) * z(ks[s], s).conj()).real.sum() / 2 * vs[s] for s in range(t + 1))
            o = o / np.sqrt((o * o).mean() + 1e-3)
            assert np.allclose(got[t, a * 3:a * 3 + 3].numpy(), o * gs[t] / (1 + np.exp(-gs[t])))


def test_oracle_feed_forward_and_order_of_passes():
    z = torch.tensor([[3.0, -4.0]], dtype=torch.float64)
    want = 2 * z / math.sqrt(12.5) + 3 * z ** 2 / math.sqrt((81 + 256) / 2) - z ** 3 / math.sqrt((27 ** 2 + 64 ** 2) / 2) + 0.5
    assert torch.allclose(O.poly_norm(z, torch.tensor([2.0, 3.0, -1.0, 0.5]).double(), 0.0), want)
    cfg = {"layers": [None] * 5, "loop": {"start": 1, "stop": 3, "times": 2}}
    runs = O.layer_runs(cfg)
    assert runs == [(0, None), (1, 0), (2, 0), (1, 1), (2, 1), (3, None), (4, None)]
    for name, c in C.CONFIGS.items():
        s = MefupelShape.from_config(c)
        assert [i for i, _ in s.order] == [i for i, _ in O.layer_runs(c)], name
        opened = [t if t is not None and i == c["loop"]["start"] else None for i, t in O.layer_runs(c)]
        assert [t for _, t in s.order] == opened, name


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_cases_show_planted_faults(name, monkeypatch):
    """Each fault, planted in the oracle, moves the logits far beyond what the float32 GPU tests allow."""
    cfg, w = C.case(name)
    toks = C.tokens(cfg, 80, 3)
    right = C.expected(name, toks)
    limit = 4e-3

    def fault(change_cfg=None, change_w=None):
        c, t = copy.deepcopy(cfg), dict(w)
        if change_cfg:
            change_cfg(c)
        if change_w:
            change_w(t)
        return float(C.row_errors(O.forward(c, t, toks)[0], right).max())

    def planted(mech, other):
        with monkeypatch.context() as m:
            m.setattr(O, mech, other)
            return fault()

    kinds = set()
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        kinds.add(l["type"])
        scaled = lambda k, by: fault(change_w=lambda t: t.update({p + k: t[p + k] * by}))
        sides = [()] if l["type"] != "parallel" else [("left",), ("right",)]

        def change(side, **kw):
            def put(c):
                m = c["layers"][i]["mixer"]
                (m[side[0]] if side else m).update(kw)
            return fault(put)
        for side in sides:
            m = l["mixer"][side[0]] if side else l["mixer"]
            if "mask" in m:
                size = m["mask"]["size"]
                if size < 60:
                    assert change(side, mask={"size": size + 1}) > limit, (i, side)
                    assert size == 1 or change(side, mask={"size": size - 1}) > limit, (i, side)
                if size > 1:
                    assert change(side, scale=m["scale"] * 1.5) > limit, (i, side)
            if "rot" in m and m.get("mask", {"size": 2})["size"] > 1:
                other = {"base": m["rot"]["base"] * 0.2, "dims": m["rot"]["dims"]}
                if m["rot"]["dims"] > 2 or m["vdim"] > 2 and not side:
                    assert change(side, rot=other) > limit, (i, side)
                assert m["rot"]["dims"] == 2 or change(side, rot={**m["rot"], "dims": m["rot"]["dims"] - 2}) > limit, (i, side)
            if "decay" in m:
                for j, d in enumerate(m["decay"]):
                    assert change(side, decay=[*m["decay"][:j], d * 0.9 + 0.04, *m["decay"][j + 1:]]) > limit, (i, j)
            if "tau" in m:
                assert change(side, tau=m["tau"] * 1.5) > limit, i
        if l["type"] == "gla":
            names = ["mix.a2", "mix.a2.b"]
        elif l["type"] == "parallel":
            names = ["mix.left.sink", "mix.left.out", "mix.right.out"] + ["mix.left.q.norm"] * (l["mixer"]["left"]["mask"]["size"] > 1)
        else:
            names = []
        for k in names + ["norm1"]:
            assert scaled(k, -1) > limit, (i, k)
        if l["type"] == "gla":
            assert fault(change_w=lambda t: t.update({p + "mix.norm": t[p + "mix.norm"].flip(0)})) > limit, i
        if l["mlp"] is not None:
            for j in range(4):
                assert fault(change_w=lambda t: t.update({p + "mlp.act": t[p + "mlp.act"] * (1 - 0.3 * (torch.arange(4) == j)).to(torch.bfloat16)})) \
                    > limit, (i, j)
    assert fault(lambda c: c["norm"].update(eps=cfg["norm"]["eps"] * 100 + 1e-2)) > limit
    if "loop" in cfg:
        assert fault(change_w=lambda t: t.update({"loop.step": t["loop.step"] * 0})) > limit
    if cfg.get("loop", {"times": 1})["times"] > 1:
        assert fault(change_w=lambda t: t.update({"loop.step": t["loop.step"].flip(0)})) > limit
        assert fault(change_w=lambda t: t.update({"loop.step": t["loop.step"][:1].expand_as(t["loop.step"])})) > limit
        once = {**cfg, "loop": None}              # the passes written out, without what joins before each
        order = [i for i, _ in O.layer_runs(cfg)]
        flat = {**once, "layers": [cfg["layers"][i] for i in order]}
        t = {k: v for k, v in w.items() if not k.startswith("l") or k.startswith("loop")}
        for run, i in enumerate(order):
            t.update({f"l{run}." + k[len(f"l{i}."):]: v for k, v in w.items() if k.startswith(f"l{i}.")})
        assert float(C.row_errors(O.forward(flat, t, toks)[0], right).max()) > limit
    turn, weights_of, recurrence, over_keys = O.turn, O.weights_of, O.linear_recurrence, O.key_value_attention
    if "attention" in kinds:
        assert planted("turn", lambda x, p, b, d, layout, back=False: x if back else turn(x, p, b, d, layout)) > limit
        other = {"halves": "interleaved", "interleaved": "halves"}
        assert planted("turn", lambda x, p, b, d, layout, back=False: turn(x, p, b, d, other[layout], back)) > limit
        assert planted("turn", lambda x, p, b, d, layout, back=False: turn(x, p + 1 if back else p, b, d, layout, back)) > limit

    def lost_first(score, seen, sink=None):
        seen = seen.clone()
        seen[1:, 0] = False
        return weights_of(score, seen, sink)
    assert planted("weights_of", lost_first) > limit                                  # forgets the first token
    if "parallel" in kinds:
        scaled_sink = lambda score, seen, sink=None: weights_of(score, seen, None if sink is None else sink * 0.5)
        assert planted("weights_of", scaled_sink) > limit
        assert planted("key_value_attention", lambda h, w_, m, eps: over_keys(h, w_, m, eps * 100 + 1e-1)) > limit

    def decay_after(q, k, v, decay):
        """The decay acts on the token's own write too."""
        return recurrence(q, k * decay, v, decay)
    assert planted("linear_recurrence", decay_after) > limit

    def lost_state(q, k, v, decay):
        """A state that starts again at a block's edge."""
        return torch.cat([recurrence(q[a:a + 32], k[a:a + 32], v[a:a + 32], decay[a:a + 32]) for a in range(0, len(q), 32)])
    assert planted("linear_recurrence", lost_state) > limit


# ------------------------------------------------------------------ readers
def test_config_reader_and_registry(tmp_path):
    cfg = C.CONFIGS["odd"]
    s = MefupelShape.from_config(cfg)
    assert (s.width, s.vocab, s.eps, s.loop, len(s.layers)) == (76, 131, 1e-3, (1, 4, 3), 5)
    assert s.layers[0].mixer == GatedMixer(2, 12, 20, 5.0) and [l.ff for l in s.layers] == [36, 44, None, 52, 100]
    assert s.layers[1].mixer == TurningMixer(6, 3, 20, 14, 7, Rotary(1000.0, 10, interleaved=True), 20 ** -0.5)
    assert s.layers[3].mixer == PairMixer(4, 2, 24, 33, Rotary(50.0, 10), 24 ** -0.5, 3, 20, 12, Rotary(300.0, 6), (0.5, 0.93, 0.999))
    assert MefupelShape.from_config(C.CONFIGS["wide"]).loop is None
    assert MefupelShape.from_config({**C.CONFIGS["wide"], "loop": None}).loop is None
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert read_shape(str(tmp_path)) == s and arch_for_shape(s).name == "Mefupel"
    for i, path, value in ((0, ("mixer", "rot"), {}), (0, ("mlp", "act"), "x"), (0, ("mlp", "kind"), "moe"), (0, ("type",), "delta"),
                           (1, ("mixer", "mask", "kind"), 1), (1, ("mixer", "mask", "size"), 0), (1, ("mixer", "rot", "scaling"), {}),
                           (1, ("mixer", "sink"), True), (3, ("mixer", "left", "vdim"), 20), (3, ("mixer", "right", "tau"), 2.0),
                           (3, ("mixer", "left_scale"), 1.0), (3, ("norm",), 1)):
        bad = copy.deepcopy(cfg)
        d = bad["layers"][i]
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            MefupelShape.from_config(bad)
    for loop in ({"start": 3, "stop": 2, "times": 1}, {"start": 0, "stop": 6, "times": 1}, {"start": 0, "stop": 1, "times": 0},
                 {"start": 0, "stop": 1}):
        with pytest.raises(ValueError):
            MefupelShape.from_config({**cfg, "loop": loop})
    with pytest.raises(ValueError, match="missing"):
        MefupelShape.from_config({k: v for k, v in cfg.items() if k != "norm"})
    bad = copy.deepcopy(cfg)
    bad["layers"][3]["mixer"]["right"]["decay"].pop()
    with pytest.raises(ValueError, match="one per head"):
        Mefupel(MefupelShape.from_config(bad), "cpu", weights=dict(C.case("odd")[1]))


def test_load_refuses_wrong_shapes_and_leftovers():
    cfg, w = C.case("odd")
    shape = MefupelShape.from_config(cfg)
    m = Mefupel(shape, "cpu", weights=dict(w))
    assert m.sights == [7, 18, 33] and m.lookback == 33 and m.padded_width == 96 and m.run_min == 16 and m.recurrent
    m.allocate_caches(3, 16, 5)
    assert tuple(m.caches[0].shape) == (5, 2, 32, 32) and len(m.caches) == 11
    assert [tuple(m.caches[i].shape) for i in (1, 4, 7)] == [(3, 16, 3 * (24 + 16))] * 3
    assert len({m.caches[i].data_ptr() for i in (1, 4, 7)}) == 3                      # a pass has its own pages ..
    assert len({m.caches[i][1].data_ptr() for i in (3, 6, 9)}) == 3                   # .. and states
    assert tuple(m.caches[3][0].shape) == (3, 16, 2 * (32 + 32)) and tuple(m.caches[3][1].shape) == (5, 3, 32, 32)
    # output products: with the mixer's where its result joins as it is, three where results are normed
    assert [len(l.outs) for l in m.layers] == [1, 1, 1, 3, 1] and [n is None for n in m.layers[3].norms] == [False, False, True]
    assert torch.equal(m.layers[3].norms[1][:76], 0.5 * w["l3.mix.right.out"].float())
    assert Mefupel(MefupelShape.from_config(C.CONFIGS["ends"]), "cpu", weights=dict(C.case("ends")[1])).run_min is None
    for name in ("l1.mix.v", "l0.mix.a2.b", "l3.mix.left.k.norm", "l3.mix.right.out", "l4.mlp.act", "loop.step", "head", "l2.norm1"):
        with pytest.raises(KeyError, match=name):
            Mefupel(shape, "cpu", weights={k: v for k, v in w.items() if k != name})
    with pytest.raises(ValueError, match="loop.step"):
        Mefupel(shape, "cpu", weights={**w, "loop.step": w["loop.step"][:2]})
    with pytest.raises(ValueError, match="l0.mix.a2"):
        Mefupel(shape, "cpu", weights={**w, "l0.mix.a2": w["l0.mix.a2"][:, 1:]})
    for extra in ("l3.mix.left.v", "l2.mlp.up", "l1.mix.sink", "l5.norm1"):
        with pytest.raises(ValueError, match=extra):
            Mefupel(shape, "cpu", weights={**w, extra: w["l1.mix.v"]})
    with pytest.raises(ValueError, match="float16"):
        Mefupel(shape, "cpu", dtype=torch.float16, weights=dict(w))


def test_options_that_do_not_go_together():
    rot = Rotary(100.0, 4)
    for kw in (dict(tied=True, turn_values=True), dict(tied=True, bias=True), dict(qk_norm=True, diff=0.5)):
        with pytest.raises(ValueError):
            GroupedAttention(32, 2, 1, 8, 8, 1.0, 4, rot, **kw)
    for vdim, kw in ((6, dict(tied=True)), (7, dict(turn_values=True))):
        with pytest.raises(ValueError):
            GroupedAttention(32, 2, 1, 8, vdim, 1.0, 4, rot, **kw)
    for kw in (dict(), dict(tau=2.0, decay=(0.5, 0.5)), dict(decay=(0.5,)), dict(decay=(0.5, 0.5), rotary=Rotary(10.0, 10))):
        with pytest.raises(ValueError):
            LinearAttention(32, 2, 8, 8, 1e-3, **kw)


def test_orders_of_dimensions():
    """Rows in the kernels' order: keys' pairs half apart, values' pairs neighbours; scores and results as before."""
    x = torch.arange(10.0).double()[None, None] ** 2 + 1
    for inter in (False, True):
        layout = "interleaved" if inter else "halves"
        r = Rotary(20.0, 6, interleaved=inter)
        order = r.order(10)
        assert sorted(order) == list(range(10))
        want = O.turn(x, torch.tensor([3]), 20.0, 6, layout)
        assert torch.allclose(O.turn(x[..., order], torch.tensor([3]), 20.0, 6, "halves"), want[..., order])
        order = Rotary(20.0, 10, interleaved=inter).adjacent_order(10)
        want = O.turn(x, torch.tensor([3]), 20.0, 10, layout)
        assert torch.allclose(O.turn(x[..., order], torch.tensor([3]), 20.0, 10, "interleaved"), want[..., order])
    m = GroupedAttention(32, 4, 2, 6, 10, 1.0, 4, Rotary(20.0, 4, interleaved=True), turn_values=True)
    w = {k: torch.randn(*s) for k, s in m.shapes().items()}
    into, out = m.load(w, torch.float32, "cpu", 32)
    assert into.shape == (m.columns, 32) and m.columns == 6 * 8 + 2 * 16 and out.shape == (32, 4 * 16)
    assert torch.equal(into[8 + 1], w["q"][6 + 2]) and torch.equal(into[32 + 2], w["k"][1]) and torch.equal(into[48 + 3], w["v"][3])
    assert not into[6:8].any() and not into[48 + 10:48 + 16].any() and m.value_freqs.numel() == 8 and not m.value_freqs[5:].any()
    m = GroupedAttention(32, 4, 2, 6, 6, 1.0, 4, Rotary(20.0, 4, interleaved=True), tied=True, qk_norm=True, eps=1e-3)
    w = {k: torch.randn(*s) for k, s in m.shapes().items()}
    assert "v" not in w
    into, out = m.load(w, torch.float32, "cpu", 32)
    assert m.columns == 6 * 16 and torch.equal(into[64 + 1], w["k"][2])
    assert torch.equal(m.norm[64:70], w["k.norm"][[0, 2, 1, 3, 4, 5]])
    assert torch.equal(out[:, 16 + 1], w["o"][:, 6 + 2]) and not out[:, 6:16].any()      # values are keys in that order


# ------------------------------------------------------------------ pages and scheduling
def _seq(n, max_tokens=8, bs=16):
    return Sequence(list(range(n)), SamplingParams(max_tokens=max_tokens, ignore_eos=True), bs)


def test_pages_behind_the_widest_window_are_given_back():
    pool = PagePool(8, 16, 100)
    s = _seq(128)
    for upto in range(1, 129):
        pool.grow(s, upto)
        pool.computed(s, upto, 33)
        first = max(0, upto - 32) // 16                    # the next token sees 32 behind it
        assert [p >= 0 for p in s.block_table] == [j >= first for j in range(-(-upto // 16))]
    pool.release(s)
    assert pool.num_free == 8 and not pool.refcount.any()


def test_scheduler_runs_every_token_of_recurrent_models():
    """No prefix is shared: a state cannot start behind tokens that did not run."""
    shape = MefupelShape.from_config(C.CONFIGS["odd"])
    cfg = EngineConfig(shape=shape, kvcache_block_size=16, num_kvcache_blocks=12, max_concurrency=3,
                       max_num_batched_tokens=40, enable_prefix_cache=True)
    sched = Scheduler(cfg)
    for _ in range(3):
        sched.add(_seq(70, max_tokens=3))
    ran = 0
    while not sched.is_finished():
        batch = sched.schedule_portions(33)
        assert batch and sum(p.count for p in batch) <= 40
        done = []
        for p in batch:
            ran += p.count
            sched.pool.computed(p.seq, p.start + p.count, 33)
            if p.ends:
                done.append(p.seq)
        sched.postprocess(done, None, advance=True)
    assert ran == 3 * 72 and sched.pool.num_free == 12 and sched.pool.reserved == 0
