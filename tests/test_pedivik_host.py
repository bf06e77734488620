"""Pedivik on the host, no GPU: configuration and weight readers, the plan of a step of portions, the
pages of windowed sequences, and that the test cases would show the faults they are there for."""
import copy
import json

import numpy as np
import pytest
import torch

from oracle import pedivik_oracle as O
from tests import pedivik_cases as C
from zipage_amd.engine import EngineConfig, PagePool, PedivikShape, SamplingParams, Scheduler, Sequence
from zipage_amd.engine.inputs import plan_portions, plan_runs
from zipage_amd.engine.registry import architecture_of, read_shape
from zipage_amd.engine.sequence import Portion
from zipage_amd.engine.weights import read_folder, write_safetensors


# ------------------------------------------------------------------ the oracle itself
def test_oracle_mechanisms_against_loops():
    g = torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    h, H, D, V, size, scale = r(9, 6), 2, 3, 4, 3, 0.7
    w = {"dq": r(5, 6), "dq.norm": r(5), "uq": r(H * D, 5), "dkv": r(7, 6), "dkv.norm": r(7),
         "uk": r(H * D, 7), "uv": r(H * V, 7), "o": r(6, H * V)}
    got = O.latent_attention(h, w, H, D, V, scale, size, 1e-3)
    norm = lambda x: x / torch.sqrt((x * x).mean() + 1e-3)
    for i in range(9):
        q = w["uq"] @ (norm(w["dq"] @ h[i]) * w["dq.norm"])
        seen = [j for j in range(9) if j <= i and i - j <= size - 1]
        out = []
        for a in range(H):
            s, vs = [], []
            for j in seen:
                c = norm(w["dkv"] @ h[j]) * w["dkv.norm"]
                s.append(float(q[a * D:(a + 1) * D] @ (w["uk"] @ c)[a * D:(a + 1) * D]) * scale)
                vs.append((w["uv"] @ c)[a * V:(a + 1) * V])
            e = np.exp(np.array(s) - max(s))
            out.append(sum(x * v for x, v in zip(e / e.sum(), vs)))
        assert torch.allclose(got[i], w["o"] @ torch.cat(out), atol=1e-12)
    z = torch.tensor([-3.0, -1e-3, 0.0, 1e-3, 2.0], dtype=torch.float64)
    sp = lambda t: np.log1p(np.exp(t))
    want = [(0.5 + sp(0.2)) * (np.exp(a) - 1 - a) + a / 2 if a <= 0 else sp(-0.3) * a * a + a / 2
            for a in z.tolist()]
    assert np.allclose(O.xielu(z, -0.3, 0.2), want, atol=1e-12)
    xs = [r(2, 3) for _ in range(3)]
    assert torch.allclose(O.depth_average(xs, [0.5, -1.0, 2.0]), 0.5 * xs[0] - xs[1] + 2 * xs[2])


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_cases_show_planted_faults(name):
    """Each fault, planted in the oracle, moves the logits far beyond what the float32 GPU tests allow
    (the bfloat16 attention kernels have tests of their own with keys that stand out)."""
    cfg, w = C.case(name)
    toks = C.tokens(cfg, 130, 3)
    right = C.expected(name, toks)
    limit = 300 * C.LIMIT[torch.float32]

    def fault(change_cfg=None, change_w=None):
        c, t = copy.deepcopy(cfg), dict(w)
        if change_cfg:
            change_cfg(c)
        if change_w:
            change_w(t)
        return C.error(O.forward(c, t, toks)[0], right)

    for i, l in enumerate(cfg["layers"]):
        size = l["mixer"]["mask"]["size"]
        if size < 130:
            assert fault(lambda c: c["layers"][i]["mixer"]["mask"].update(size=size + 1)) > limit, i
            if size > 1:
                assert fault(lambda c: c["layers"][i]["mixer"]["mask"].update(size=size - 1)) > limit, i
        if size > 1:
            assert fault(lambda c: c["layers"][i]["mixer"].update(scale=l["mixer"]["scale"] * 1.5)) > limit, i
        for name_ in (f"l{i}.norm1", f"l{i}.mix.dkv.norm") + ((f"l{i}.norm2", f"l{i}.mlp.act") if l["mlp"] else ()):
            assert fault(change_w=lambda t: t.update({name_: t[name_] * -2})) > limit, name_
        assert fault(change_w=lambda t: t.update({f"l{i}.dwa": t[f"l{i}.dwa"].flip(0)})) > limit, i
    assert fault(change_w=lambda t: t.update(pos=t["pos"].roll(1, 0))) > limit
    assert fault(lambda c: c.update(logit_scale=cfg["logit_scale"] * 1.5)) > limit
    assert fault(change_w=lambda t: t.update({"final.norm": t["final.norm"] * 0})) > limit


# ------------------------------------------------------------------ readers
def test_config_reader_and_registry(tmp_path):
    cfg = C.CONFIGS["odd"]
    s = PedivikShape.from_config(cfg)
    assert (s.width, s.vocab, s.eps, s.logit_scale, s.max_positions) == (76, 131, 1e-3, 1.75, 640)
    assert [l.window for l in s.layers] == [7, 33, 90] and s.layers[1].ff is None
    assert (s.layers[0].heads, s.layers[0].dim, s.layers[0].vdim, s.layers[0].q_rank, s.layers[0].kv_rank,
            s.layers[0].ff) == (5, 24, 40, 52, 44, 100)
    assert s.layers[1].scale == 0.21
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert read_shape(str(tmp_path)) == s
    assert architecture_of({"architectures": ["Qwen3ForCausalLM"]}).name == "Qwen3ForCausalLM"
    with pytest.raises(ValueError, match="no model"):
        architecture_of({"architecture": "Other"})
    for path, value in ((("mixer", "sinks"), 1), (("mixer", "mask", "kind"), "chunk"), (("mlp", "kind"), "gated"),
                        (("mixer", "mask", "size"), 0), (("type",), "conv")):
        bad = copy.deepcopy(cfg)
        d = bad["layers"][0]
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            PedivikShape.from_config(bad)


def test_safetensors_round_trip(tmp_path):
    t = {"a": torch.randn(3, 5).bfloat16(), "odd": torch.arange(7, dtype=torch.uint8), "i": torch.arange(6).int().view(2, 3),
         "f": torch.randn(2, 2), "s": torch.tensor(2.5)}
    write_safetensors(str(tmp_path / "m.safetensors"), t)
    back = read_folder(str(tmp_path))
    assert set(back) == set(t)
    for k in t:
        assert back[k].dtype == t[k].dtype and torch.equal(back[k], t[k])
    from safetensors.torch import load_file
    other = load_file(str(tmp_path / "m.safetensors"))
    assert all(torch.equal(other[k], t[k]) for k in t)
    with pytest.raises(FileNotFoundError):
        read_folder(str(tmp_path / ".."))


def test_load_refuses_wrong_shapes_and_leftovers():
    from zipage_amd.engine import Pedivik
    cfg, w = C.case("odd")
    shape = PedivikShape.from_config(cfg)
    Pedivik(shape, "cpu", weights=dict(w))
    with pytest.raises(KeyError, match="l1.mix.uk"):
        Pedivik(shape, "cpu", weights={k: v for k, v in w.items() if k != "l1.mix.uk"})
    with pytest.raises(ValueError, match="final.norm"):
        Pedivik(shape, "cpu", weights={**w, "final.norm": w["final.norm"][:-1]})
    with pytest.raises(ValueError, match="extra"):
        Pedivik(shape, "cpu", weights={**w, "extra": w["embed"]})
    with pytest.raises(ValueError, match="float16"):
        Pedivik(shape, "cpu", dtype=torch.float16, weights=dict(w))


# ------------------------------------------------------------------ plans and pages
def _seq(n, bs=16, max_tokens=8, base=0):
    return Sequence([base + i for i in range(n)], SamplingParams(max_tokens=max_tokens, ignore_eos=True), bs)


def test_run_plan_covers_every_visible_key():
    """Tiles and key rows of portions, against the definition: query at position p sees
    max(0, p - window + 1) .. p."""
    rng = np.random.default_rng(0)
    for window in (None, 1, 5, 64, 300):
        seqs = []
        for start, count in ((0, 130), (37, 16), (200, 257), (15, 2)):
            s = _seq(start + count)
            s.block_table = list(rng.permutation(100)[: -(-len(s) // 16)])
            seqs.append(Portion(s, start, count))
        runs = plan_runs(seqs, 16, window)
        if runs.key_slots is None:
            assert window == 1
            runs.key_slots = np.concatenate([[p.seq.block_table[t // 16] * 16 + t % 16 for t in
                                              range(p.start, p.start + p.count)] for p in seqs])
        rows = [(p, t) for p in seqs for t in range(p.start, p.start + p.count)]
        met = 0
        for q0, n, k0, rel in runs.tiles.tolist():
            assert 1 <= n <= 128
            for i in range(n):
                p, t = rows[q0 + i]
                low = 0 if window is None else max(0, rel + i - window + 1)
                got = runs.key_slots[k0 + low:k0 + rel + i + 1].tolist()
                first = 0 if window is None else max(0, t - window + 1)
                assert got == [p.seq.block_table[j // 16] * 16 + j % 16 for j in range(first, t + 1)]
                met += 1
        assert met == len(rows)
    s = _seq(40)
    s.block_table = [2, 0, 1]
    only = plan_runs([Portion(s, 0, 40)], 16, 5)
    assert only.key_slots is None           # a prompt from its start needs no gather


def test_portion_plan_orders_singles_first():
    a, b, c = _seq(20), _seq(50, base=100), _seq(9, base=200)
    a.num_tokens += 1                       # a token that is on the device only
    a.query_id, b.query_id, c.query_id = 3, 1, 2
    a.block_table, b.block_table, c.block_table = [5, 6], [-1, 1, 2, 3], [9]
    plan = plan_portions([Portion(b, 20, 30), Portion(a, 20, 1), Portion(c, 5, 3)], 16, [33], 16)
    assert plan.first_row == [4, 0, 1]
    assert plan.ids[:4].tolist() == [0, 205, 206, 207] and plan.rows[:4].tolist() == [3, -1, -1, -1]
    assert plan.positions[:4].tolist() == [20, 5, 6, 7] and plan.context_lens.tolist() == [21, 6, 7, 8]
    assert plan.table_rows.tolist() == [1, 2, 2, 2] and plan.tables[1].tolist() == [5, 6, -1, -1]
    assert plan.slots[:5].tolist() == [6 * 16 + 4, 9 * 16 + 5, 9 * 16 + 6, 9 * 16 + 7, 1 * 16 + 4]
    assert plan.runs[33].key_slots is not None and list(plan.runs) == [33]
    none = plan_portions([Portion(b, 20, 30)], 16, [33], None)
    assert not none.runs and len(none.context_lens) == 30


def test_pages_leave_with_the_window_and_come_back():
    pool = PagePool(8, 16, 100)
    s, lookback = _seq(200), 20
    for upto in range(1, 201):
        pool.grow(s, upto)
        pool.computed(s, upto, lookback)
        for t in range(max(0, upto - lookback + 1), upto):     # what the next token sees
            assert s.block_table[t // 16] >= 0
        held = [p for p in s.block_table if p >= 0]
        assert len(held) <= 3 and len(set(held)) == len(held)
        assert pool.num_free == 8 - len(held)
    pool.release(s)
    assert pool.num_free == 8 and not pool.refcount.any()
    with pytest.raises(RuntimeError, match="empty"):
        pool.grow(_seq(200), 200)


def test_prefix_pages_are_shared_only_when_computed():
    pool = PagePool(16, 16, 100, enable_prefix_cache=True)
    a, b, c = _seq(50), _seq(50), _seq(33)
    pool.grow(a, 40)
    pool.computed(a, 40, 1000)
    pool.share_prefix(b, 1000)
    assert b.num_computed_tokens == 32 and b.block_table == a.block_table[:2]
    pool.grow(a, 50)
    pool.computed(a, 50, 1000)
    pool.release(a)
    pool.share_prefix(c, 10)                 # the last token runs; pages behind the window are not held
    assert c.num_computed_tokens == 32 and c.block_table[0] == -1 and c.block_table[1] == b.block_table[1]
    pool.release(b)
    pool.release(c)
    assert pool.num_free == 16 and not pool.refcount.any()


def test_scheduler_mixes_decodes_and_portions():
    """Random requests through the scheduler: no step exceeds its tokens, every token of every
    sequence runs exactly once and in order, nobody waits for a page, everything returns."""
    shape = PedivikShape.from_config(C.CONFIGS["odd"])
    rng = np.random.default_rng(1)
    for prefix in (False, True):
        cfg = EngineConfig(shape=shape, kvcache_block_size=16, num_kvcache_blocks=24, max_concurrency=4,
                           max_num_batched_tokens=40, max_num_seqs=8, enable_prefix_cache=prefix)
        sched, lookback = Scheduler(cfg), 90
        seqs = [_seq(int(rng.integers(1, 200)), max_tokens=int(rng.integers(1, 60))) for _ in range(14)]
        for s in seqs:
            sched.add(s)
        ran = {id(s): 0 for s in seqs}
        mixed = steps = 0
        while not sched.is_finished():
            batch = sched.schedule_portions(lookback)
            assert batch and sum(p.count for p in batch) <= 40
            steps += 1
            mixed += len({p.count > 1 for p in batch}) == 2
            done = []
            for p in batch:
                if ran[id(p.seq)] == 0:
                    ran[id(p.seq)] = p.start
                assert p.start == ran[id(p.seq)] and p.count >= 1
                for t in range(max(0, p.start - lookback + 1), p.start + p.count):
                    assert p.seq.block_table[t // 16] >= 0
                ran[id(p.seq)] += p.count
                sched.pool.computed(p.seq, p.start + p.count, lookback)
                if p.ends:
                    done.append(p.seq)
            sched.postprocess(done, None, advance=True)
        assert mixed > 5
        for s in seqs:
            assert ran[id(s)] == s.num_prompt_tokens + s.params.max_tokens - 1
        assert sched.pool.num_free == 24 and sched.pool.reserved == 0 and len(sched.free_rows) == 4
