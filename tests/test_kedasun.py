"""Kedasun on the CPU: config and weights, caches and convolution state, portions
of prompts, value mixing across stages, and greedy generation, against the plain
model of kedasun_oracle.py."""
from __future__ import annotations

import random

import pytest
import torch

import llm_sharding_demo_amd.runtime.trace as trace
from llm_sharding_demo_amd.config import AttentionSpec, DenseSpec, EngineConfig, RopeSpec, SamplingParams, get_model_config
from llm_sharding_demo_amd.ops import reference as ref
from llm_sharding_demo_amd.parallel.partition import layer_cuts, make_unit_plan, unit_costs
from llm_sharding_demo_amd.runtime.engine import Engine
from llm_sharding_demo_amd.runtime.kv_cache import PAGE, PagedCache, layer_cache, pad_up

from . import kedasun_oracle as orc


def model(tmp_path, layers, seed=0, **kw):
    cfg = orc.config(layers, **kw)
    w = orc.random_weights(cfg, seed)
    orc.save(str(tmp_path), cfg, w)
    return cfg, w


def all_kinds():
    """Both mixers twice with other sizes, a layer without a feed-forward, one that
    keeps its own values, all dimensions rotated and none."""
    mixed = dict(kv_heads=2, vdim=24)
    return [orc.full(v_mix=False, heads=3, kv_heads=1, dim=16, vdim=20, rot=16), orc.windowed(**mixed),
            orc.full(**mixed), orc.windowed(heads=4, dim=16, conv=1, size=9, keep=0, ff=0, **mixed),
            orc.full(heads=2, dim=8, rot=0, ff=24, limit=7.0, **mixed),
            orc.windowed(v_mix=False, heads=3, kv_heads=3, dim=8, vdim=12, conv=5, size=33, keep=70)]


def engine(path, **kw):
    kw = {"device": "cpu", "max_batch": 4, "max_seq_len": 320, "kv_tokens": 640, **kw}
    return Engine(EngineConfig(model_id=str(path), weights=str(path), **kw))


def ids_of(n, vocab=200, seed=0):
    r = random.Random(seed)
    return [r.randrange(vocab) for _ in range(n)]


def close(got, want, tol=1e-4):
    return float((got.double() - want).abs().max()) < tol * float(want.double().pow(2).mean().sqrt())


# -- configuration and weights ------------------------------------------------

def test_config_reader(tmp_path):
    cfg, w = model(tmp_path, all_kinds(), eps=3e-6, groups=8)
    mc = get_model_config(str(tmp_path))
    assert (mc.arch, mc.vocab_size, mc.hidden, mc.n_layers) == ("kedasun", 200, 88, 6)
    assert (mc.norm_eps, mc.norm_groups, mc.embed_scale, mc.eos_token_id) == (3e-6, 8, 0.7, -1)
    assert mc.layers[0].mixer == AttentionSpec(3, 1, 16, 20, 0.2, rope=RopeSpec(16, 1000.0, interleaved=True), talking=False)
    assert mc.layers[1].mixer == AttentionSpec(6, 2, 40, 24, 0.3, 70, talk_weights=True, keep_first=5, distance_bias=True,
                                               conv=3, qk_norm=True, bias=True, head_gate=True, mix_values=1)
    assert [l.mixer.mix_values for l in mc.layers] == [None, 1, 1, 1, 1, None]
    assert mc.layers[4].mixer.rope is None and mc.layers[3].mlp is None and mc.layers[4].mlp == DenseSpec(24, 7.0)
    assert mc.mixed_values == mc.layers[1].mixer and mc.boundary == 88 + 2 * 24
    assert mc.stage_params(range(6)) + 2 * mc.embed_params() + 88 == sum(torch.Size(s).numel()
                                                                          for s in orc.shapes(cfg).values())
    assert mc.layers[1].mixer.slopes() == pytest.approx(orc.slopes(6), rel=1e-14)


@pytest.mark.parametrize("bad,kw", [
    (orc.full(heads=5), {}), (orc.full(rot=7), {}), (orc.windowed(size=0), {}), (orc.windowed(keep=-1), {}),
    (orc.windowed(vdim=32), {}), (orc.windowed(kv_heads=3), {}), (orc.full(), {"groups": 3}), (orc.full(), {"groups": 0}),
    ({**orc.full(), "type": "x"}, {}), ({**orc.full(), "mlp": {"kind": "moe", "ff": 8, "limit": 1.0}}, {})])
def test_config_rejects(tmp_path, bad, kw):
    """Also values of other sizes than those that are mixed in."""
    orc.save(str(tmp_path), orc.config([orc.full(), bad], **kw), {"x": torch.zeros(1)})
    with pytest.raises(ValueError):
        get_model_config(str(tmp_path))


def test_presets_run():
    eng = Engine(EngineConfig(model_id="kedasun-test", device="cpu", max_batch=2, max_seq_len=64))
    out = eng.generate_ids([[3, 4, 5]], SamplingParams(greedy=True, max_new_tokens=4))
    assert len(out[0]) == 4


def test_layer_caches():
    c = layer_cache(AttentionSpec(6, 2, 40, 24, 1.0, conv=3), pad_up)
    assert c.pages == ((2, PAGE, 64), (2, PAGE, 32)) and c.ring == ((3, 8 * 64 + 2 * 32),)
    assert layer_cache(AttentionSpec(6, 2, 40, 24, 1.0)).ring == ()


# -- mechanisms ----------------------------------------------------------------

def test_grouped_norm_and_clamped_gate():
    g = torch.Generator().manual_seed(0)
    x, w = torch.randn(5, 24, generator=g) * torch.linspace(0.1, 8, 24), torch.randn(24, generator=g)
    for groups in (1, 2, 3, 24):
        assert close(ref.group_rmsnorm(x, w, 1e-3, groups), orc.group_norm(x.double(), w.double(), groups, 1e-3), 1e-6)
    gate, up = 3 * torch.randn(5, 24, generator=g), 3 * torch.randn(5, 24, generator=g)
    eye = torch.eye(24, dtype=torch.float64)
    w = {"gate": torch.cat([eye, 0 * eye], 1), "up": torch.cat([0 * eye, eye], 1), "down": eye}
    want = orc.feed_forward(torch.cat([gate, up], 1).double(), lambda n: w[n], 1.5)
    assert close(ref.clamped_glu(gate, up, 1.5, 1.702), want, 1e-6)


def test_interleaved_rotation():
    x, pos = torch.randn(5, 3, 20, generator=torch.Generator().manual_seed(0)), torch.tensor([0, 1, 63, 64, 1000])
    got = ref.partial_rope(x, pos, RopeSpec(12, 100.0, interleaved=True))
    assert close(got, orc.rotate(x.double(), pos.tolist(), 12, 100.0), 1e-6)
    assert torch.equal(got[..., 12:], x[..., 12:])


def test_window_kept_tokens_and_mixed_weights():
    """A key whose score stands out is seen at the last place of the window and not
    one further, among the kept first tokens and not one behind them, also at page
    borders; and it reaches the heads that the mixing matrix sends it to."""
    H, G, D, V, n, slot = 4, 2, 6, 5, 3 * PAGE, 1
    kv = PagedCache([layer_cache(AttentionSpec(H, G, D, V, 1.0))], 2, 8, n, torch.float32, "cpu")
    kv.assign([(slot, (5, 0, 3))])
    g = torch.Generator().manual_seed(2)
    pos, slots = torch.arange(n, dtype=torch.int32), torch.full((n,), slot)
    k, v = torch.randn(n, G, D, generator=g) * 0.1, torch.randn(n, G, V, generator=g)
    talk = torch.tensor([[1.0, 0, 0, 0], [0, 0, 0, 1.0], [0.5, -1.0, 0.5, 0], [0, 0, 0, 1.0]])
    slope = torch.tensor([1e-3] * H)
    q = torch.ones(1, H, D)
    i32 = dict(dtype=torch.int32)
    for W, keep in ((1, 0), (7, 3), (PAGE, 1), (PAGE + 1, PAGE), (2 * PAGE, 70), (None, 0), (5, n)):
        for p in (3, PAGE - 1, PAGE, 2 * PAGE, n - 1):
            edge = p if W is None else max(0, p - W)
            for key in {edge, min(p, edge + 1), 0, min(p, max(0, keep - 1)), min(p, keep), p}:
                kk, vv = k.clone(), v.clone()
                kk[key, 0] = 8.0  # the heads of the first group
                vv[key] = 100.0
                for pool, x in zip(kv.entries[0], (kk, vv)):
                    ref.paged_append(pool, kv.table, x, slots, pos)
                o = ref.talking_attention(q, *kv.entries[0], kv.table, torch.tensor([slot], **i32), torch.tensor([p], **i32),
                                          torch.tensor([0, 1], **i32), talk, 1.0, None, W, True, slope, keep)
                want = orc.attend(q.double(), kk[: p + 1].double(), vv[: p + 1].double(), 1.0, W, keep, slope.tolist(),
                                  talk.double(), first=p)
                assert close(o, want)
                assert (float(o[0, 0].mean()) > 50) == orc.visible(p, key, W, keep)


# -- cache, portions, batches ---------------------------------------------------

def run_portions(ses, rid, ids, sizes, end=True):
    out, at, sizes = [], 0, list(sizes)
    while at < len(ids):
        n = min(sizes.pop(0) if sizes else 1, len(ids) - at)
        out.append(ses.step([{"id": rid, "tokens": ids[at:at + n], "want": list(range(n))}],
                            [rid] if end and at + n == len(ids) else []))
        at += n
    return torch.cat(out)


@pytest.mark.parametrize("groups", [1, 4, 11])
def test_whole_prompts(tmp_path, groups):
    cfg, w = model(tmp_path, all_kinds(), seed=3, groups=groups)
    ids = ids_of(120)
    got = run_portions(trace.TraceSession(engine(tmp_path)), "a", ids, [120])
    assert close(got, orc.forward(cfg, w, ids))


def test_every_mechanism_counts(tmp_path):
    """Each of the design's mechanisms changes the logits by far more than the
    comparisons here let pass."""
    cfg, w = model(tmp_path, all_kinds(), seed=3)
    ids = ids_of(120)
    want = orc.forward(cfg, w, ids)

    def off(cfg2=cfg, **tensors):
        d = orc.forward(cfg2, {**w, **tensors}, ids) - want
        return float(d.abs().max() / want.pow(2).mean().sqrt())

    def other(i, **mixer):
        layers = [dict(l, mixer={**l["mixer"], **mixer}) if j == i else l for j, l in enumerate(cfg["layers"])]
        return {**cfg, "layers": layers}

    assert off(other(1, mask={"size": 70, "keep_first": 4})) > 1e-2 and off(other(1, mask={"size": 71, "keep_first": 5})) > 1e-2
    assert off(other(2, rot={"dims": 22, "base": 1000.0})) > 1e-2
    for name in ("l1.mix.vmix", "l2.mix.vmix", "l1.mix.talk", "l1.mix.g", "l1.mix.k.conv", "l1.mix.v.b", "l3.mix.o.b"):
        changed = off(**{name: w[name] * 0})
        assert (changed == 0) if name == "l1.mix.vmix" else changed > 1e-2, name


@pytest.mark.parametrize("sizes", [[2] * 75, [63, 1, 2, 60, 24], [1] * 150, [64, 64, 22], [7, 130, 13]])
def test_portions(tmp_path, sizes):
    cfg, w = model(tmp_path, all_kinds()[1:4])
    ids = ids_of(150)
    assert close(run_portions(trace.TraceSession(engine(tmp_path)), "a", ids, sizes), orc.forward(cfg, w, ids))


def test_mixed_batches_and_reused_slots(tmp_path):
    """Unequal requests in one batch, finished ones' pages and slots used again."""
    cfg, w = model(tmp_path, all_kinds()[1:])
    eng = engine(tmp_path, kv_tokens=6 * PAGE)
    ses = trace.TraceSession(eng)
    seqs = {k: ids_of(n, seed=n) for k, n in (("a", 100), ("b", 5), ("c", 131), ("d", 66))}
    want = {k: orc.forward(cfg, w, v) for k, v in seqs.items()}
    steps = [[("a", 70), ("b", 1)], [("a", 1), ("b", 3), ("c", 2)], [("b", 1), ("c", 61), ("a", 1)],
             [("c", 1), ("a", 28), ("d", 60)], [("d", 1), ("c", 2)], [("c", 65), ("d", 5)]]
    at = dict.fromkeys(seqs, 0)
    for _ in range(2):
        for st in steps:
            ent = [{"id": k, "tokens": seqs[k][at[k]:at[k] + n], "want": list(range(n))} for k, n in st]
            rows = [want[k][at[k] + j] for k, n in st for j in range(n)]
            for k, n in st:
                at[k] += n
            got = ses.step(ent, [k for k, _ in st if at[k] == len(seqs[k])])
            assert close(got, torch.stack(rows))
        assert not ses.live and eng.page_pools[0].available == 6 and eng.slots.available == 4
        at = dict.fromkeys(seqs, 0)


# -- scheduler and engine ---------------------------------------------------------

@pytest.mark.parametrize("kw", [{}, {"num_microbatches": 2}, {"prefill_chunk": 7}, {"kv_tokens": 4 * PAGE}])
def test_greedy_generation(tmp_path, kw):
    cfg, w = model(tmp_path, all_kinds()[1:4])
    eng = engine(tmp_path, **kw)
    prompts = [ids_of(n, seed=n) for n in (1, 70, 13, 40)]
    sp = [SamplingParams(greedy=True, max_new_tokens=n) for n in (8, 5, 10, 3)]
    for _ in range(2):  # the second session finds the first one's rows in its slots
        out = eng.generate_ids(prompts, sp)
        assert [len(o) for o in out] == [s.max_new_tokens for s in sp]
        assert all(orc.is_greedy(cfg, w, p, o) for p, o in zip(prompts, out))
        assert eng.page_pools[0].available == eng.kv_pages and eng.slots.available == eng.kv_slots


@pytest.mark.parametrize("split", [1, 2, 3])
def test_two_stages_and_compat_forwards(tmp_path, split):
    """The cut may fall in front of the first layer whose values are mixed in, or
    behind it: they cross the boundary beside the residual."""
    layers = all_kinds()
    cfg, w = model(tmp_path, [layers[0], layers[1], layers[2], layers[3]])
    eng = engine(tmp_path, num_stages=2, split_points=[split], transport="strict")
    prompts = [ids_of(n, seed=n) for n in (30, 5, 66)]
    out = eng.generate_ids(prompts, SamplingParams(greedy=True, max_new_tokens=4))
    assert all(len(o) == 4 and orc.is_greedy(cfg, w, p, o) for p, o in zip(prompts, out))
    hid = eng.forward_a(prompts[0])
    assert hid.shape == (30, 88 + 2 * 24)
    assert close(eng.forward_b(hid), orc.forward(cfg, w, prompts[0]))
    eng.shutdown()


def test_partition_and_memory_budget(tmp_path):
    mc = get_model_config("kedasun-2b")
    assert layer_cuts(mc) == list(range(1, mc.n_layers))
    costs, head, _ = unit_costs(mc)
    assert len(costs) == 2 * mc.n_layers and min(costs[::2]) > 0 and max(costs[1::2]) == 0 and head > 0
    plan = make_unit_plan(mc, 3)
    assert [u % 2 for p in plan for u in p] == [0] * 6
    model(tmp_path, all_kinds())
    eng = engine(tmp_path)
    slot = sum(layer_cache(l.mixer).slot_bytes(4) for l in eng.mcfg.layers)
    page = sum(layer_cache(l.mixer).page_bytes(4) for l in eng.mcfg.layers)
    kv = eng.stages[0].kv
    assert kv.nbytes == (eng.kv_slots + 2) * slot + (eng.kv_pages + 1) * page + 4 * kv.table.numel()
    assert eng._weight_bytes(0) == 2 * (eng.mcfg.stage_params(range(6)) + 2 * eng.mcfg.embed_params())


def test_routing_of_the_attention_kernels():
    """Splits fill the chip with few sequences and vanish with many; never more than there are tiles."""
    from llm_sharding_demo_amd.ops.routing import Routing

    r = Routing()
    assert r.paged_splits(4, 1028) == 17 and r.paged_splits(4096, 1028) == 1 and r.paged_splits(1, 3) == 1
    assert r.mix_splits(1, 1028, 16, 4) == 19 and r.mix_splits(256, 1028, 16, 4) == 1
    assert r.mix_splits(128, 1028, 32, 8) == 2 and r.mix_splits(1, 1, 4, 4) <= 2
