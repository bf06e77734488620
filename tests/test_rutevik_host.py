"""Rutevik on the host, no GPU: the oracle's mechanisms against other forms of the same equations, that the test
cases would show the faults they are there for, readers, plans, pages and scheduling."""
import copy
import json
import math

import numpy as np
import pytest
import torch

from oracle import rutevik_oracle as O
from tests import rutevik_cases as C
from zipage_amd.engine import EngineConfig, PagePool, RutevikShape, SamplingParams, Scheduler, Sequence
from zipage_amd.engine.inputs import plan_portions
from zipage_amd.engine.registry import arch_for_shape, read_shape
from zipage_amd.engine.sequence import Portion
from zipage_amd.layers.rotary import Rotary
from zipage_amd.sight import EVERYTHING


def _r(g, *s):
    return torch.randn(*s, generator=g, dtype=torch.float64)


# ------------------------------------------------------------------ the oracle itself
def _turned(x, p, freqs):
    """Complex numbers for the pairs (i, i + half)."""
    half = len(freqs)
    z = [complex(x[i], x[i + half]) * np.exp(1j * p * f) for i, f in enumerate(freqs)]
    return np.array([v.real for v in z] + [v.imag for v in z] + list(x[2 * half:]))


def test_oracle_differential_attention_against_loops():
    g = torch.Generator().manual_seed(0)
    m = C.attention(4, 2, 6, 3, 4, base=50.0, scale=0.7, softcap=1.5, diff=0.3, scaling=None)
    h = _r(g, 9, 5)
    w = {"q": _r(g, 48, 5), "k": _r(g, 24, 5), "v": _r(g, 6, 5), "q.b": _r(g, 48), "k.b": _r(g, 24), "v.b": _r(g, 6),
         "g": _r(g, 12, 5), "o": _r(g, 5, 12), **{k: _r(g, 6) * 0.4 for k in ("lq1", "lk1", "lq2", "lk2")}}
    n = {k: v.numpy() for k, v in w.items()}
    freqs = [50.0 ** (-2 * i / 4) for i in range(2)]
    lam = math.exp(n["lq1"] @ n["lk1"]) - math.exp(n["lq2"] @ n["lk2"]) + 0.3
    got = O.differential_attention(h, w, m, 1e-4)
    row = lambda k, i: n[k] @ h[i].numpy() + n[k + ".b"]
    for i in range(9):
        out = []
        for a in range(4):
            b, parts = a // 2, []
            for j in range(2):
                q = _turned(row("q", i)[(a * 2 + j) * 6:][:6], i, freqs)
                e = [math.exp(1.5 * math.tanh(0.7 * q @ _turned(row("k", t)[(b * 2 + j) * 6:][:6], t, freqs) / 1.5))
                     for t in range(i + 1)]
                parts.append(sum(x * row("v", t)[b * 3:b * 3 + 3] for t, x in enumerate(e)) / sum(e))
            o = parts[0] - lam * parts[1]
            out.append(o / np.sqrt((o * o).mean() + 1e-4) * 0.7)
        out = np.concatenate(out) / (1 + np.exp(-n["g"] @ h[i].numpy()))
        assert np.allclose(got[i].numpy(), n["o"] @ out, atol=1e-11)


def test_oracle_latent_attention_against_absorbed_products():
    """Scores and values from the latent itself, head by head."""
    g = torch.Generator().manual_seed(1)
    m = C.latent(3, 4, 5, 6, 7, 8, base=20.0, scale=0.6)
    h, other = _r(g, 8, 6), _r(g, 8, 6)
    w = {"dq": _r(g, 7, 6), "dq.norm": _r(g, 7), "uq": _r(g, 30, 7), "uk": _r(g, 12, 8), "uv": _r(g, 15, 8), "o": _r(g, 6, 15),
         "dkv": _r(g, 14, 6), "dkv.norm": _r(g, 8)}
    held = O.shared_keys(other, w, m, 1e-4)             # another layer's input
    got = O.latent_attention(h, w, m, 1e-4, held)
    n = {k: v.numpy() for k, v in w.items()}
    freqs = [20.0 ** (-2 * i / 6) for i in range(3)]
    unit = lambda x: x / np.sqrt((x * x).mean() + 1e-4)
    down = [n["dkv"] @ x.numpy() for x in other]
    c = np.stack([unit(d[:8]) * n["dkv.norm"] for d in down])
    kr = np.stack([_turned(d[8:], t, freqs) for t, d in enumerate(down)])
    assert np.allclose(held[0].numpy(), c) and np.allclose(held[1].numpy(), kr)
    for i in range(8):
        q = n["uq"] @ (unit(n["dq"] @ h[i].numpy()) * n["dq.norm"])
        out = []
        for a in range(3):
            qa = q[a * 10:a * 10 + 10]
            inner = n["uk"][a * 4:a * 4 + 4].T @ qa[:4]
            e = np.exp(0.6 * (c[:i + 1] @ inner + kr[:i + 1] @ _turned(qa[4:], i, freqs)))
            out.append(n["uv"][a * 5:a * 5 + 5] @ (e @ c[:i + 1] / e.sum()))
        assert np.allclose(got[i].numpy(), n["o"] @ np.concatenate(out), atol=1e-11)


def test_oracle_routing_and_feed_forwards():
    z = torch.tensor([[3.0, 0.0, 2.0, 1.9, -1.0, 2.5]], dtype=torch.float64)
    for top, want in ((1, [0]), (3, [0, 2, 5]), (6, range(6))):
        a = O.route(z, top)[0]
        assert sorted(a.nonzero().flatten().tolist()) == list(want)
        assert torch.allclose(a[list(want)], 1 / (1 + torch.exp(-z[0, list(want)])))
    w = {"gate": torch.tensor([[2.0]]).double(), "up": torch.tensor([[3.0]]).double(), "down": torch.tensor([[1.0]]).double()}
    full = {"router": torch.tensor([[0.0]]).double(), **{f"e0.{k}": v for k, v in w.items()}}
    y = O.experts(torch.ones(1, 1).double(), full, C.moe(1, 1, 1))      # score 0.5 on the input: g = 1, u = 1.5
    assert abs(float(y) - 1.5 / (1 + math.exp(-1))) < 1e-12
    assert O.dense(torch.tensor([[1.0, -2.0]]).double(), {"up": torch.eye(2).double() * 3, "down": torch.ones(1, 2).double()}) == 9.0
    assert torch.allclose(O.dyt(torch.tensor([0.5]).double(), 2.0, 0.1, 0.8), torch.tensor([2 * math.tanh(0.4) + 0.1]).double())


def test_rotary_frequencies():
    """Kept, mixed and divided by the factor, on both sides of both edges; product against oracle."""
    rot = {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 512}}
    f = O.frequencies(rot)
    plain = [10000.0 ** (-2 * i / 64) for i in range(32)]
    kinds = set()
    for a, b in zip(f, plain):
        length = 2 * math.pi / b
        if length < 128:
            kinds.add("kept")
            assert a == b
        elif length > 512:
            kinds.add("divided")
            assert a == b / 8
        else:
            kinds.add("mixed")
            s = (512 / length - 1) / 3
            assert abs(a - ((1 - s) * b / 8 + s * b)) < 1e-15 and b / 8 < a < b
    assert len(kinds) == 3
    got = Rotary(10000.0, 64, (8.0, 1.0, 4.0, 512.0)).frequencies("cpu")
    assert torch.allclose(got, torch.tensor(f, dtype=torch.float64).float(), rtol=2e-7)
    assert torch.equal(Rotary(10000.0, 64).frequencies("cpu"), torch.tensor(plain, dtype=torch.float64).float())
    assert Rotary(5.0, 0).frequencies("cpu").numel() == 0


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_cases_show_planted_faults(name, monkeypatch):
    """Each fault, planted in the oracle, moves the logits far beyond what the float32 GPU tests allow."""
    cfg, w = C.case(name)
    toks = C.tokens(cfg, 80, 3)
    right = C.expected(name, toks)
    limit = 5e-3

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

    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        change = lambda **kw: fault(lambda c: c["layers"][i]["mixer"].update(kw))
        scaled = lambda k, by=-1: fault(change_w=lambda t: t.update({p + k: t[p + k] * by}))
        turn = lambda **kw: change(rot={**m["rot"], **kw})
        assert change(scale=m["scale"] * 1.5) > limit, i
        if m["rot"]["dims"] > 2:
            # a layer that reads another's keys turns its own queries only
            assert turn(base=3.0) > limit, i
        if l["type"] == "attention":
            assert change(softcap=m["softcap"] * 1.5) > limit and change(diff=m["diff"] + 0.1) > limit, i
            if "scaling" in m["rot"] and m["rot"]["dims"] > 2:
                assert turn(scaling=None) > limit, i
            for k in ("q.b", "k.b", "v.b", "lq1", "lq2", "g"):
                assert scaled("mix." + k) > limit, (i, k)
        else:
            for k in ("dq.norm", "uq") + (("dkv.norm", "dkv") if m.get("kv_from") is None else ()):
                half = lambda t: t.update({p + "mix." + k: t[p + "mix." + k].flip(-1)})
                assert fault(change_w=half) > limit, (i, k)
        for k in ("norm1", "norm1.b", "norm1.alpha") + (("norm2", "norm2.b", "norm2.alpha") if l["mlp"] else ()):
            assert scaled(k, 0.5) > limit, (i, k)
        if l["mlp"] and l["mlp"]["kind"] == "moe" and l["mlp"]["router"]["top"] > 1:
            assert fault(lambda c: c["layers"][i]["mlp"]["router"].update(top=l["mlp"]["router"]["top"] - 1)) > limit, i
    assert fault(lambda c: c.update(logit_scale=cfg["logit_scale"] * 1.1)) > limit
    if name != "wide":                                   # there no layer's norm meets a small root mean square
        assert fault(lambda c: c["norm"].update(eps=cfg["norm"]["eps"] * 100 + 1e-2)) > limit
    whole = O.causal_softmax
    late = lambda s: torch.nn.functional.pad(whole(s)[:-1], (0, 0, 1, 0)) + torch.diag((torch.arange(len(s)) == 0).to(s))
    assert planted("causal_softmax", late) > limit                                     # does not see itself

    def lost_first(s):
        s = s.clone()
        s[1:, 0] = -math.inf
        return whole(s)
    assert planted("causal_softmax", lost_first) > limit                              # forgets the oldest token
    if any(l["mlp"] and l["mlp"]["kind"] == "moe" for l in cfg["layers"]):
        def weight_behind(h, w, c):
            a = O.route(h @ w["router"].T, c["router"]["top"])
            return sum(a[:, e:e + 1] * O.expert(h, {k: w[f"e{e}.{k}"] for k in ("gate", "up", "down")})
                       for e in range(c["router"]["experts"]))
        assert planted("experts", weight_behind) > limit
    keys = O.shared_keys
    shift = lambda h, w, m, eps: (keys(h, w, m, eps)[0], keys(h, w, m, eps)[1].roll(1, 0))
    assert planted("shared_keys", shift) > limit                                       # a rotated part of the wrong token


def test_cases_show_a_wrong_source():
    """Reading the nearest latent instead of the named one shows."""
    cfg, w = C.case("odd")
    toks = C.tokens(cfg, 60, 3)
    bad = copy.deepcopy(cfg)
    bad["layers"][3]["mixer"].update(kv_rank=44, rot_dim=10, rot=cfg["layers"][4]["mixer"]["rot"])
    t = dict(w)
    for k, n in (("uk", 7 * 12), ("uv", 7 * 20)):
        t[f"l3.mix.{k}"] = w[f"l3.mix.{k}"][:, :44]
    t["l3.mix.dkv"], t["l3.mix.dkv.norm"] = w["l3.mix.dkv"][:54], w["l3.mix.dkv.norm"][:44]
    t["l3.mix.uq"] = w["l3.mix.uq"][:7 * 22]
    right = O.forward(bad, t, toks)[0]
    bad["layers"][4]["mixer"]["kv_from"] = 3
    assert float(C.row_errors(O.forward(bad, t, toks)[0], right).max()) > 0.1


# ------------------------------------------------------------------ readers
def test_config_reader_and_registry(tmp_path):
    cfg = C.CONFIGS["odd"]
    s = RutevikShape.from_config(cfg)
    assert (s.width, s.vocab, s.eps, s.logit_scale, len(s.layers)) == (76, 131, 1e-3, 1.7, 6)
    a = s.layers[0].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.softcap, a.diff) == (6, 3, 20, 40, 5.0, 0.25)
    assert a.rotary == Rotary(1000.0, 10, (3.0, 1.5, 6.0, 96.0)) and s.layers[5].mixer.rotary.stretch is None
    b = s.layers[2].mixer
    assert (b.heads, b.dim, b.vdim, b.q_rank, b.kv_rank, b.rotary.dims, b.scale) == (3, 40, 24, 37, 44, 10, 0.2)
    assert [getattr(l.mixer, "source", None) for l in s.layers] == [None, 1, 1, 3, 1, None]
    assert (s.layers[1].mlp.ff, s.layers[2].mlp, s.layers[3].mlp.experts, s.layers[3].mlp.top, s.layers[3].mlp.ff) == (52, None, 7, 2, 52)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert read_shape(str(tmp_path)) == s and arch_for_shape(s).name == "Rutevik"
    for i, path, value in ((0, ("mixer", "mask"), 1), (0, ("mixer", "softcap"), 0), (0, ("mixer", "rot", "kind"), "x"),
                           (0, ("mixer", "rot", "scaling", "extra"), 1), (0, ("mlp", "shared"), {}), (0, ("mlp", "router", "groups"), 2),
                           (1, ("mlp", "act"), "relu"), (1, ("mlp", "kind"), "gated"), (1, ("type",), "conv"), (1, ("mixer", "kv_from"), 0),
                           (2, ("mixer", "kv_from"), 3), (2, ("mixer", "kv_from"), 2), (4, ("mixer", "kv_from"), 2),
                           (4, ("mixer", "kv_from"), 3), (2, ("mixer", "kv_rank"), 40), (2, ("mixer", "rot", "base"), 301.0),
                           (1, ("mixer", "rot_dim"), 12), (0, ("scale",), 1), (2, ("mixer", "kv_from"), -1)):
        bad = copy.deepcopy(cfg)
        d = bad["layers"][i]
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            RutevikShape.from_config(bad)
    with pytest.raises(ValueError, match="missing"):
        RutevikShape.from_config({k: v for k, v in cfg.items() if k != "logit_scale"})


def test_load_refuses_wrong_shapes_and_leftovers():
    from zipage_amd.engine import Rutevik
    cfg, w = C.case("odd")
    shape = RutevikShape.from_config(cfg)
    m = Rutevik(shape, "cpu", weights=dict(w))
    assert m.sights == [None] and m.padded_width == 96 and m.source == [0, 1, 1, 3, 1, 5] and m.run_min == 16
    m.allocate_caches(3, 16, 5)
    # [keys of both maps | values] of three heads; latent and rotated part; nothing for those that read another's
    assert [None if c is None else tuple(c.shape) for c in m.caches] == \
        [(3, 16, 3 * (2 * 24 + 48)), (3, 16, 64 + 16), None, (3, 16, 96 + 32), None, (3, 16, 3 * (2 * 40 + 32))]
    core = m.mixers[0].core
    dot = lambda i: math.exp(float(w[f"l0.mix.lq{i}"].double() @ w[f"l0.mix.lk{i}"].double()))
    assert abs(core.balance - (dot(1) - dot(2) + 0.25)) < 1e-9 and abs(core.out_scale - 0.75) < 1e-9
    assert Rutevik(RutevikShape.from_config(C.CONFIGS["ends"]), "cpu", weights=dict(C.case("ends")[1])).run_min is None
    for name in ("l1.mix.dkv", "l0.mlp.e9.up", "l0.mix.lk2", "l3.norm2.alpha", "head"):
        with pytest.raises(KeyError, match=name):
            Rutevik(shape, "cpu", weights={k: v for k, v in w.items() if k != name})
    with pytest.raises(ValueError, match="final.norm.b"):
        Rutevik(shape, "cpu", weights={**w, "final.norm.b": w["final.norm.b"][:-1]})
    with pytest.raises(ValueError, match="l2.mix.dkv"):      # a layer that reads another's cache has none
        Rutevik(shape, "cpu", weights={**w, "l2.mix.dkv": w["l1.mix.dkv"]})
    with pytest.raises(ValueError, match="float16"):
        Rutevik(shape, "cpu", dtype=torch.float16, weights=dict(w))
    # norms of a feed-forward that is not there are not asked for
    Rutevik(shape, "cpu", weights={**w, "l2.norm2": w["l1.norm2"], "l2.norm2.b": w["l1.norm2.b"], "l2.norm2.alpha": w["l1.norm2.alpha"]})


# ------------------------------------------------------------------ plans and pages
def _seq(n, bs=16, max_tokens=8, base=0):
    return Sequence([base + i for i in range(n)], SamplingParams(max_tokens=max_tokens, ignore_eos=True), bs)


def test_run_plan_names_the_whole_context():
    a, b = _seq(40), _seq(100, base=50)
    a.block_table, b.block_table = [7, 2, 5], [9, 8, 1, 0, 4, 6, 3]
    plan = plan_portions([Portion(a, 0, 40), Portion(b, 70, 30)], 16, [None], 16)
    slots = plan.runs[None].key_slots.tolist()
    assert slots == [p.seq.block_table[t // 16] * 16 + t % 16 for p in (Portion(a, 0, 40), Portion(b, 70, 30))
                     for t in range(p.start + p.count)]
    assert plan.runs[None].tiles.tolist() == [[0, 40, 0, 0], [40, 30, 40, 70]]
    own = plan_portions([Portion(a, 0, 40)], 16, [None], 16)
    assert own.runs[None].key_slots is None


def test_every_page_stays_while_its_sequence_lives():
    pool = PagePool(8, 16, 100)
    s = _seq(128)
    for upto in range(1, 129):
        pool.grow(s, upto)
        pool.computed(s, upto, EVERYTHING)
        assert len([p for p in s.block_table if p >= 0]) == -(-upto // 16)
    pool.release(s)
    assert pool.num_free == 8 and not pool.refcount.any()


def test_scheduler_shares_prefixes_and_reserves_whole_sequences():
    """Prompts with a common beginning run its tokens once; no request is admitted that could run out of pages."""
    shape = RutevikShape.from_config(C.CONFIGS["odd"])
    cfg = EngineConfig(shape=shape, kvcache_block_size=16, num_kvcache_blocks=12, max_concurrency=3,
                       max_num_batched_tokens=40, enable_prefix_cache=True)
    sched = Scheduler(cfg)
    assert sched.peak_pages(_seq(70, max_tokens=10), EVERYTHING) == 5
    for _ in range(3):
        sched.add(_seq(70, max_tokens=3))
    ran, most = 0, 0
    while not sched.is_finished():
        batch = sched.schedule_portions(EVERYTHING)
        assert batch
        most = max(most, len(sched.running))
        done = []
        for p in batch:
            ran += p.count
            sched.pool.computed(p.seq, p.start + p.count, EVERYTHING)
            if p.ends:
                done.append(p.seq)
        sched.postprocess(done, None, advance=True)
    assert most == 2 and 72 + 2 * 8 <= ran < 3 * 72
    assert sched.pool.num_free == 12 and sched.pool.reserved == 0
