"""Timisun on an MI355X: every kernel against the plain functions of
timisun_oracle.py, then whole models -- prompts, portions, mixed batches,
decoding, reused pages -- in bf16 and in fp32, and greedy generation through
the scheduler with captured graphs."""
from __future__ import annotations

import random

import pytest
import torch

from . import timisun_oracle as orc

pytestmark = pytest.mark.gpu
DEV = "cuda"
F64 = torch.float64
PAGE = 64


@pytest.fixture(scope="module")
def C():
    from llm_sharding_demo_amd.ops.hip import _load

    return _load()


def rand(*shape, seed=0, scale=1.0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def err(got, want):
    """RMS of the difference over the RMS of the wanted values."""
    got, want = got.detach().cpu().to(F64), want.to(F64)
    return float((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())


def tol(dtype, bf16):
    return 2e-6 if dtype == torch.float32 else bf16


def pad(t, *shape):
    out = torch.zeros(shape, dtype=t.dtype)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


DTYPES = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])


# -- norms, embedding ------------------------------------------------------------

@DTYPES
@pytest.mark.parametrize("rows,width,padded,splits", [(3, 100, 128, 0), (5, 192, 192, 3), (300, 320, 320, 12),
                                                      (1, 2048, 2048, 6)])
def test_norm_around_zero_with_padding(C, dtype, rows, width, padded, splits):
    x = pad(rand(rows, width), rows, padded)
    w = rand(width, seed=1, scale=0.3).to(dtype)
    slab = pad(rand(max(splits, 1), rows, width, seed=2).to(dtype), max(splits, 1), rows, padded)
    total = x.to(F64) + (slab.to(F64).sum(0) if splits else 0)
    xd = x.to(DEV)
    wd, sd = pad(w, padded).to(DEV), slab.to(DEV) if splits else None
    if dtype == torch.float32:
        out = C.norm_fp32(xd, sd, wd, 1e-3, None, True, width, 1.0)
    else:
        out = C.norm(xd, sd, None, wd, None, 1e-3, True, None, True, width, 1.0)
    want = orc.norm(total[:, :width], w.to(F64), 1e-3)
    assert err(out[:, :width], want) < tol(dtype, 3e-3)
    assert float(out[:, width:].abs().max()) == 0 if padded > width else True
    assert err(xd, total) < 1e-6


@DTYPES
def test_scaled_embedding(C, dtype):
    table, ids = rand(50, 64).to(dtype), torch.tensor([3, 49, 0, 3], dtype=torch.int32)
    if dtype == torch.float32:
        out = C.embed_fp32(ids.to(DEV), table.to(DEV), 3.7)
    else:
        out = C.embed(ids.to(DEV), ids.to(DEV), table.to(DEV), None, 3.7)
    assert err(out, orc.embed(ids.tolist(), table.to(F64), 3.7)) < 1e-6


# -- latent append, router -----------------------------------------------------------

@DTYPES
@pytest.mark.parametrize("rank,E,top", [(40, 6, 2), (64, 1, 1), (200, 70, 5), (512, 300, 8), (24, 100, 90)])
def test_latent_post(C, dtype, rank, E, top):
    T, nq, rp = 9, 128, -(-rank // 64) * 64
    f32 = dtype == torch.float32
    y = rand(T, (nq + rank + E + 7) // 4 * 4, seed=3).to(DEV)
    gain, corr = rand(rank, seed=4), rand(E, seed=5)
    cache = torch.zeros(6, PAGE, rp, dtype=dtype, device=DEV)
    table = torch.tensor([[5, 5, 5], [2, 4, 0]], dtype=torch.int32, device=DEV)
    pos = torch.tensor([0, 63, 64, 65, 127, 128, 190, 191, 1], dtype=torch.int32)
    slots = torch.ones(T, dtype=torch.int32)
    q, ids, wts = C.latent_post(y, nq, True, f32, cache, rank, gain.to(DEV), 1e-4, table, slots.to(DEV), pos.to(DEV),
                                corr.to(DEV), top)
    yc = y.cpu().to(F64)
    assert err(q, yc[:, :nq]) < tol(dtype, 3e-3)
    c = orc.rms(yc[:, nq:nq + rank], 1e-4) * gain.to(F64)
    for t in range(T):
        p = int(pos[t])
        row = cache[int(table[1, p // PAGE]), p % PAGE]
        assert err(row[:rank], c[t]) < tol(dtype, 4e-3) and (rp == rank or float(row[rank:].abs().max()) == 0)
        order, ws = orc.route(torch.ones(1, dtype=F64), yc[t, nq + rank:nq + rank + E, None], corr.to(F64), top)
        assert ids[t].tolist() == order
        assert err(wts[t], ws) < 1e-5


# -- attention in the latent space --------------------------------------------------

def paged(c, dtype, rp, seed=0):
    """The latents c [n, rank] in shuffled pages of a pool full of other values."""
    n = c.shape[0]
    k = -(-n // PAGE)
    order = list(range(k + 3))
    random.Random(seed).shuffle(order)
    pool = rand(k + 3, PAGE, rp, seed=9, scale=4.0)
    for i in range(n):
        pool[order[i // PAGE], i % PAGE] = 0
        pool[order[i // PAGE], i % PAGE, : c.shape[1]] = c[i]
    table = torch.zeros(2, k, dtype=torch.int32)
    table[1] = torch.tensor(order[:k])
    return pool.to(dtype).to(DEV), table.to(DEV)


def latent_tokens(C, q, pool, table, pos, H, window, scale, splits=1):
    slots = torch.ones(len(pos), dtype=torch.int32, device=DEV)
    return C.latent_decode(q, pool, table, slots, torch.tensor(pos, dtype=torch.int32, device=DEV), H, window, scale,
                           splits)


@DTYPES
@pytest.mark.parametrize("rank", [64, 128, 192, 256, 320, 384, 448, 512, 576, 640])
def test_latent_attention_ranks(C, dtype, rank):
    """Prefill and decode kernels on every instantiated rank (640: the kernel
    without MFMA), heads over one 16-head group."""
    from llm_sharding_demo_amd.ops.hip import latent_tiles

    H, n, W, scale = 17, 150, 61, rank ** -0.5
    c = rand(n, rank, seed=1).to(dtype)
    q = rand(n, H, rank, seed=2).to(dtype)
    pool, table = paged(c, dtype, rank)
    want = orc.attend(q.to(F64), c.to(F64), scale, W)
    qd = q.reshape(n, -1).contiguous().to(DEV)
    got = latent_tokens(C, qd, pool, table, list(range(n)), H, W, scale, splits=2)
    assert err(got.reshape(n, H, rank), want) < tol(dtype, 4e-3)
    rows = C.latent_tile_rows(rank)
    if dtype == torch.float32 or rows == 0:
        return

    class Meta:
        host_qlens = [n - 37]
    i32 = dict(dtype=torch.int32, device=DEV)
    got = C.latent_prefill(qd[37:].contiguous(), pool, table, latent_tiles(Meta, H, rows).to(DEV),
                           torch.tensor([1], **i32), torch.tensor([37], **i32), torch.tensor([0, n - 37], **i32), H, W,
                           scale)
    assert err(got.reshape(n - 37, H, rank), want[37:]) < 4e-3


@DTYPES
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 63, 64, 65, 100, 1 << 30])
def test_window_edges_show(C, dtype, window):
    """One key stands out: its latent is the answer exactly where it is the
    window's last, and absent one token further; also at page borders."""
    from llm_sharding_demo_amd.ops.hip import latent_tiles

    R, H, n = 64, 3, 260
    base = rand(n, R, seed=1, scale=0.05)
    for key in (0, 1, 62, 63, 64, 65, 127, 128, 150):
        c = base.clone()
        c[key] = 2.0
        c = c.to(dtype)
        pool, table = paged(c, dtype, R, seed=key)
        q = torch.full((n, H, R), 1.0, dtype=dtype)
        want = orc.attend(q[:, :1].to(F64), c.to(F64), 1.0, window).expand(n, H, R)
        qd = q.reshape(n, -1).to(DEV)
        outs = [latent_tokens(C, qd, pool, table, list(range(n)), H, window, 1.0, s) for s in (1, 3)]
        if dtype == torch.bfloat16:
            class Meta:
                host_qlens = [n]
            i32 = dict(dtype=torch.int32, device=DEV)
            outs.append(C.latent_prefill(qd, pool, table, latent_tiles(Meta, H, 128).to(DEV), torch.tensor([1], **i32),
                                         torch.tensor([0], **i32), torch.tensor([0, n], **i32), H, window, 1.0))
        for o in outs:
            o = o.reshape(n, H, R).cpu().to(F64)
            assert err(o, want) < tol(dtype, 5e-3)
            for p in range(n):
                assert (float(o[p].mean()) > 1.5) == orc.visible(p, key, window), (p, key)


def test_far_key_among_many(C):
    """A key 3000 tokens back decides; the pages lie in random order."""
    R, H, n = 128, 16, 3100
    c = rand(n, R, seed=3, scale=0.05)
    c[57] = 2.0
    c = c.to(torch.bfloat16)
    pool, table = paged(c, torch.bfloat16, R)
    q = torch.full((1, H * R), 1.0, dtype=torch.bfloat16, device=DEV)
    for splits in (1, 4, 24):
        o = latent_tokens(C, q, pool, table, [n - 1], H, 1 << 30, 0.5, splits)
        assert abs(float(o.float().mean()) - 2.0) < 0.02
        o = latent_tokens(C, q, pool, table, [n - 1], H, n - 58, 0.5, splits)
        assert float(o.float().abs().mean()) < 0.1


@pytest.mark.parametrize("dim,vdim", [(64, 64), (64, 80), (128, 16), (128, 128)])
@pytest.mark.parametrize("window", [1, 33, 64, 90, 1 << 30])
def test_expanded_attention(C, dim, vdim, window):
    """Ragged portions over gathered latents: keys and values made per row."""
    from llm_sharding_demo_amd.ops.hip import latent_tiles

    R, H, n = 192, 3, 330
    c = rand(n, R, seed=1).to(torch.bfloat16)
    c[100] *= 3  # one key stands out
    pool, table = paged(c, torch.bfloat16, R)
    wk, wv = rand(H * dim, R, seed=2, scale=R ** -0.5), rand(H * vdim, R, seed=3, scale=R ** -0.5)
    k, v = (c.to(F64) @ wk.to(F64).T).reshape(n, H, dim), (c.to(F64) @ wv.to(F64).T).reshape(n, H, vdim)
    starts, lens = [0, 70, 129], [141, 3, 201]
    lo = [max(0, s - window + 1) if i < 2 else s - window + 1 for i, s in enumerate(starts)]  # below 0: zero rows
    if window > n:
        lo = [0, 0, -5]
    cu_k = [0]
    for s, m, a in zip(starts, lens, lo):
        cu_k.append(cu_k[-1] + s + m - a)
    i32 = dict(dtype=torch.int32, device=DEV)
    T = sum(lens)
    q = rand(T, H, dim, seed=4).to(torch.bfloat16)
    slots, klo, cuk = torch.tensor([1, 1, 1], **i32), torch.tensor(lo, **i32), torch.tensor(cu_k, **i32)
    rows = C.latent_gather(pool, table, slots, klo, cuk, cu_k[-1])
    for i in range(3):
        part = rows[cu_k[i]:cu_k[i + 1]].cpu()
        cut = max(0, -lo[i])
        assert torch.equal(part[cut:], c[max(0, lo[i]):starts[i] + lens[i]]) and not part[:cut].any()
    kk = (rows.float() @ wk.T.to(DEV)).to(torch.bfloat16)
    vv = (rows.float() @ wv.T.to(DEV)).to(torch.bfloat16)

    class Meta:
        host_qlens = lens
    cu_q = [0, lens[0], lens[0] + lens[1], T]
    got = C.latent_expanded(q.reshape(T, -1).to(DEV), kk, vv, latent_tiles(Meta, 1, 128).to(DEV),
                            torch.tensor(cu_q, **i32), torch.tensor(starts, **i32), klo, cuk, H, window, dim ** -0.5)
    got = got.reshape(T, H, vdim).cpu()
    for i in range(3):
        for j in range(0, lens[i], 7):
            p = starts[i] + j
            keys = [x for x in range(p + 1) if orc.visible(p, x, window)]
            for h in range(H):
                s = k[keys, h] @ q[cu_q[i] + j, h].to(F64) * dim ** -0.5
                assert err(got[cu_q[i] + j, h], torch.softmax(s, 0) @ v[keys, h]) < 0.02


# -- grouped GEMMs ---------------------------------------------------------------------

@DTYPES
@pytest.mark.parametrize("M,G,N,K", [(1, 3, 16, 64), (33, 4, 80, 128), (130, 2, 272, 192), (70, 16, 128, 512)])
def test_batch_linear(C, dtype, M, G, N, K):
    a, w = rand(M, G * K, seed=1).to(dtype), rand(G, N, K, seed=2).to(dtype)
    want = torch.einsum("mgk,gnk->mgn", a.to(F64).reshape(M, G, K), w.to(F64)).reshape(M, -1)
    for tm in ((64,) if dtype == torch.float32 else (32, 64, 128)):
        assert err(C.batch_linear(a.to(DEV), w.to(DEV), tm), want) < tol(dtype, 4e-3)


def test_linear_fp32(C):
    a, w, x = rand(70, 192, seed=1), rand(100, 192, seed=2), rand(70, 100, seed=3)
    want = a.to(F64) @ w.to(F64).T
    assert err(C.linear_fp32(a.to(DEV), w.to(DEV)), want) < 2e-6
    xd = x.to(DEV)
    C.linear_fp32(a.to(DEV), w.to(DEV), xd)
    assert err(xd, want + x.to(F64)) < 2e-6


@pytest.mark.parametrize("n,E,tm", [(1, 1, 32), (7, 5, 32), (3000, 64, 64), (5000, 1000, 128)])
def test_moe_group(C, n, E, tm):
    ids = torch.randint(0, E, (n, 1), generator=torch.Generator().manual_seed(n), dtype=torch.int32)
    perm, tiles = (t.cpu() for t in C.moe_group(ids.to(DEV), E, tm))
    assert sorted(perm.tolist()) == list(range(n))
    seen = torch.zeros(n, dtype=torch.int32)
    for e, s0, k, _ in tiles.tolist():
        assert k <= tm
        for r in range(s0, s0 + k):
            assert int(ids[perm[r]]) == e
            seen[r] += 1
    assert int(seen.min()) == int(seen.max()) == 1


def moe_case(T, H, E, top, F, Fs, dtype, seed=0):
    d = dict(gate=rand(E, F, H, seed=seed, scale=H ** -0.5 * 2), up=rand(E, F, H, seed=seed + 1, scale=H ** -0.5 * 2),
             down=rand(E, H, F, seed=seed + 2, scale=F ** -0.5), h=rand(T, H, seed=seed + 3))
    if Fs:
        d.update(sgate=rand(Fs, H, seed=seed + 4, scale=H ** -0.5 * 2),
                 sup=rand(Fs, H, seed=seed + 5, scale=H ** -0.5 * 2), sdown=rand(H, Fs, seed=seed + 6, scale=Fs ** -0.5))
    d = {k: v.to(dtype) for k, v in d.items()}
    g = torch.Generator().manual_seed(seed)
    ids = torch.rand(T, E, generator=g).topk(top, 1).indices.int()
    wts = torch.rand(T, top, generator=g) + 0.1
    lim, slim = 0.8, 1.6
    x = {k: v.to(F64) for k, v in d.items()}
    parts = torch.zeros(top + bool(Fs), T, H, dtype=F64)
    for t in range(T):
        for k in range(top):
            e = int(ids[t, k])
            parts[k, t] = float(wts[t, k]) * orc.expert(x["h"][t:t + 1], x["gate"][e], x["up"][e], x["down"][e], lim)[0]
    if Fs:
        parts[top] = orc.expert(x["h"], x["sgate"], x["sup"], x["sdown"], slim)
    return d, ids, wts, lim, slim, parts


def moe_weights(d, H, F, Fs):
    from llm_sharding_demo_amd.ops.hip import interleave_experts, pad_to

    fp, fsp = -(-F // 64) * 64, -(-Fs // 64) * 64
    w = interleave_experts(torch.cat([d["gate"], d["up"]], 1), fp, H).to(DEV)
    dn = pad_to(d["down"], d["down"].shape[0], H, fp).to(DEV)
    ws = dns = None
    if Fs:
        ws = interleave_experts(torch.cat([d["sgate"], d["sup"]], 0), fsp, H).to(DEV)
        dns = pad_to(d["sdown"], H, fsp).to(DEV)
    return w, dn, ws, dns


MOE_SIZES = pytest.mark.parametrize("T,H,E,top,F,Fs", [(1, 64, 1, 1, 16, 0), (3, 128, 6, 2, 40, 56), (5, 192, 9, 9, 64, 32),
                                                      (4, 576, 8, 3, 600, 1100), (40, 128, 4, 2, 64, 128),
                                                      (300, 192, 5, 3, 96, 200)])


@DTYPES
@MOE_SIZES
def test_experts_grouped(C, dtype, T, H, E, top, F, Fs):
    d, ids, wts, lim, slim, parts = moe_case(T, H, E, top, F, Fs, dtype)
    w, dn, ws, dns = moe_weights(d, H, F, Fs)
    f32 = dtype == torch.float32
    for tm in ((64,) if f32 else (32, 64, 128)):
        perm, tiles = C.moe_group(ids.to(DEV), E, tm)
        mid, mids = C.moe_up(d["h"].to(DEV), perm, tiles, top, w, lim, 1.702, ws, slim, tm)
        slab = torch.full((parts.shape[0], T, H), 7.0, dtype=dtype, device=DEV)
        C.moe_down(mid, mids if Fs else None, perm, tiles, wts.to(DEV), dn, dns, slab, tm)
        assert err(slab, parts) < tol(dtype, 6e-3)
        if not f32:
            slab = torch.full((parts.shape[0], T, H), 7.0, device=DEV)
            C.moe_down(mid, mids if Fs else None, perm, tiles, wts.to(DEV), dn, dns, slab, tm)
            assert err(slab, parts) < 6e-3


@MOE_SIZES
def test_experts_streamed(C, T, H, E, top, F, Fs):
    if T > 64:
        pytest.skip("grouped kernels only")
    d, ids, wts, lim, slim, parts = moe_case(T, H, E, top, F, Fs, torch.bfloat16)
    w, dn, ws, dns = moe_weights(d, H, F, Fs)
    x = rand(T, H, seed=8).to(DEV)
    want = x.cpu().to(F64) + parts.sum(0)
    C.moe_few(d["h"].to(DEV), ids.to(DEV), wts.to(DEV), w, dn, lim, 1.702, ws, dns, slim, x)
    assert err(x, want) < 5e-3


# -- whole models -------------------------------------------------------------------------

def layers_a():
    return [orc.layer(), orc.layer(kv_from=0, heads=2, dim=16, vdim=20, window=9, experts=3, top=1, ff=24),
            orc.layer(rank=24, heads=5, window=33, mlp=False), orc.layer(kv_from=0, window=140, experts=4, top=4)]


def layers_b():
    """Ranks above the MFMA kernels and above one tile, many heads, one expert,
    no shared expert, a window of one token and no window at all."""
    a = orc.layer(rank=130, heads=18, dim=72, vdim=8, window=1, experts=1, top=1, ff=130)
    b = orc.layer(rank=600, heads=2, dim=8, vdim=100, window=77, experts=20, top=7, ff=8, shared_ff=8)
    b["mlp"]["shared"] = None
    c = orc.layer(rank=130, kv_from=0, heads=1, dim=1, vdim=1, experts=2, top=2, ff=1, shared_ff=3)
    c["mixer"]["mask"] = None
    return [a, b, c]


def layers_c():
    """Ranks wide against the heads, so prompts expand keys and values."""
    return [orc.layer(rank=256, dim=20, vdim=24, window=60), orc.layer(rank=256, dim=64, vdim=10, window=None, kv_from=0),
            orc.layer(rank=500, dim=16, vdim=16, heads=2, window=130)]


MODELS = {"a": (layers_a, dict(vocab=200, width=96)), "b": (layers_b, dict(vocab=131, width=70, eps=1e-3)),
          "c": (layers_c, dict(vocab=97, width=128))}
# per position: RMS of the logit difference over the standard deviation of the
# logits
LIMIT = {"fp32": 2e-5, "bf16": 0.025}


@pytest.fixture(scope="module", params=[f"{m}-{d}" for m in sorted(MODELS) for d in ("fp32", "bf16")])
def case(request, tmp_path_factory):
    """(dtype, model directory, config, weights, requests, their logits).  In
    bf16, rounding may settle a router's close call the other way, so there the
    corrections decide (3 apart, the scores within 1); the kernel tests above
    route every token its own way in both types."""
    name, dtype = request.param.split("-")
    make, kw = MODELS[name]
    cfg = orc.config(make(), **kw)
    w = orc.random_weights(cfg, 3)
    if dtype == "bf16":
        for k in w:
            if k.endswith("correction"):
                g = torch.Generator().manual_seed(len(k) + int(k[1]))
                w[k] = (3.0 * torch.randperm(len(w[k]), generator=g)).to(w[k].dtype)
    path = str(tmp_path_factory.mktemp("model"))
    orc.save(path, cfg, w)
    seqs = {k: ids_of(n, cfg["vocab"], n) for k, n in (("a", 170), ("b", 5), ("c", 131), ("d", 66))}
    return dtype, path, cfg, w, seqs, {k: orc.forward(cfg, w, v) for k, v in seqs.items()}


@pytest.fixture(autouse=True)
def expand_any_prompt(monkeypatch):
    """Test prompts are short: let the expanded form take them from two tokens."""
    from llm_sharding_demo_amd.ops.hip import HipBackend

    monkeypatch.setattr(HipBackend, "R", HipBackend.R.replace(latent_expand_t=2))


def ids_of(n, vocab, seed=0):
    r = random.Random(seed)
    return [r.randrange(vocab) for _ in range(n)]


def make_engine(path, dtype, **kw):
    from llm_sharding_demo_amd.config import EngineConfig
    from llm_sharding_demo_amd.runtime.engine import Engine

    return Engine(EngineConfig(model_id=path, weights=path, dtype=dtype, device=DEV,
                               **{"max_batch": 4, "max_seq_len": 320, "kv_tokens": 640, **kw}))


def check(got, want, dtype):
    e = (got.to(F64) - want).pow(2).mean(1).sqrt() / want.std(1)
    assert float(e.max()) < LIMIT[dtype], float(e.max())


def test_model_portions(case):
    """Whole prompts, portions down to two tokens, and token by token."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    dtype, path, _, _, seqs, want = case
    ses = TraceSession(make_engine(path, dtype))
    ids = seqs["a"]
    for sizes in ([170], [64, 64, 42], [2] * 85, [63, 1, 2, 70, 34], [130] + [1] * 40, [7, 1, 1, 150, 11]):
        out, at = [], 0
        for n in sizes:
            last = at + n == len(ids)
            out.append(ses.step([{"id": "r", "tokens": ids[at:at + n], "want": list(range(n))}], ["r"] if last else []))
            at += n
        check(torch.cat(out), want["a"], dtype)


def test_model_mixed_batches(case):
    """Requests of unequal length in one batch; pages and slots used again."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    dtype, path, _, _, seqs, want = case
    eng = make_engine(path, dtype, kv_tokens=8 * PAGE)
    ses = TraceSession(eng)
    steps = [[("a", 70), ("b", 1)], [("a", 1), ("b", 3), ("c", 2)], [("b", 1), ("c", 61), ("a", 1)],
             [("c", 1), ("a", 98), ("d", 60)], [("d", 1), ("c", 2)], [("c", 65), ("d", 5)]]
    for _ in range(3):
        at = dict.fromkeys(seqs, 0)
        for st in steps:
            ent = [{"id": k, "tokens": seqs[k][at[k]:at[k] + n], "want": list(range(n))} for k, n in st]
            rows = torch.stack([want[k][at[k] + j] for k, n in st for j in range(n)])
            for k, n in st:
                at[k] += n
            check(ses.step(ent, [k for k, _ in st if at[k] == len(seqs[k])]), rows, dtype)
        assert not ses.live and eng.page_pools[0].available == 8


def test_residual_after_every_layer(case):
    from llm_sharding_demo_amd.runtime.batch import BatchMeta

    dtype, path, cfg, w, seqs, _ = case
    st = make_engine(path, dtype, kv_tokens=0, max_batch=1).stages[0]
    st.kv.assign([(0, tuple(range(5)))])
    want, got = [], []
    orc.forward(cfg, w, seqs["d"], want)
    ids = torch.tensor(seqs["d"], dtype=torch.int32, device=DEV)
    st.forward(BatchMeta.build([0], [0], [len(ids)], DEV), ids, residuals=got)
    assert len(got) == len(want) == len(cfg["layers"])
    for g, x in zip(got, want):
        assert err(g, x) < (1e-5 if dtype == "fp32" else 0.02)


def near_best(cfg, w, prompt, out):
    """Every generated token is, given the tokens before it, within rounding of
    the plain model's best."""
    lg = orc.forward(cfg, w, prompt + out[:-1])[len(prompt) - 1:]
    gap = lg.max(1).values - lg.gather(1, torch.tensor(out)[:, None]).squeeze(1)
    assert float((gap / lg.std(1)).max()) < 0.1


def greedy(cfg, w, prompt, n):
    x = list(prompt)
    for _ in range(n):
        x.append(int(orc.forward(cfg, w, x)[-1].argmax()))
    return x[len(prompt):]


@pytest.mark.parametrize("kw", [{}, {"num_microbatches": 2}, {"prefill_chunk": 7}, {"kv_tokens": 5 * PAGE}],
                         ids=["plain", "groups", "chunks", "few-pages"])
def test_greedy_generation(case, kw):
    """The engine's own entry point and scheduler, captured graphs replayed over
    several sessions: exactly the plain model's tokens in fp32, and in bf16
    tokens within rounding of the plain model's best."""
    from llm_sharding_demo_amd.config import SamplingParams

    dtype, path, cfg, w, _, _ = case
    eng = make_engine(path, dtype, **kw)
    prompts = [ids_of(n, cfg["vocab"], n) for n in (1, 70, 13, 64, 40)]
    sp = [SamplingParams(greedy=True, max_new_tokens=n) for n in (12, 5, 20, 3, 9)]
    want = [greedy(cfg, w, p, s.max_new_tokens) for p, s in zip(prompts, sp)] if dtype == "fp32" else None
    for _ in range(3):
        out = eng.generate_ids(prompts, sp)
        if dtype == "fp32":
            assert out == want
        for p, o in zip(prompts, out):
            near_best(cfg, w, p, o)
        assert eng.page_pools[0].available == eng.kv_pages
    assert eng.workers[0].captures > 0


def test_graphs_match_eager(case):
    """Same batches with and without captured graphs give the same tokens."""
    from llm_sharding_demo_amd.config import SamplingParams

    dtype, path, cfg, _, _, _ = case
    prompts = [ids_of(n, cfg["vocab"], n) for n in (30, 33, 31, 29)]
    sp = SamplingParams(temperature=0.8, top_k=20, seed=5, max_new_tokens=90)
    eager = make_engine(path, dtype, use_graphs=False).generate_ids(prompts, sp)
    eng = make_engine(path, dtype)
    for _ in range(3):
        assert eng.generate_ids(prompts, sp) == eager


@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
@pytest.mark.parametrize("kw", [{}, {"prefill_chunk": 16}], ids=["whole", "chunks"])
def test_two_stages(tmp_path, dtype, kw):
    """Two pipeline stages on one GPU (graph-captured transfers, padded residual
    rows, chunk graphs); the cut keeps shared caches together."""
    from llm_sharding_demo_amd.config import SamplingParams

    cfg = orc.config([orc.layer(), orc.layer(kv_from=0, window=9), orc.layer(rank=24), orc.layer(kv_from=2, rank=24)],
                     width=100)
    w = orc.random_weights(cfg, 5)
    if dtype == "bf16":
        for k in w:
            if k.endswith("correction"):
                w[k] = (3.0 * torch.arange(len(w[k]))).to(w[k].dtype)
    orc.save(str(tmp_path), cfg, w)
    eng = make_engine(str(tmp_path), dtype, num_stages=2, transport="devloop", **kw)
    assert eng.plan == [(0, 2), (2, 4)]
    prompts = [ids_of(n, cfg["vocab"], n) for n in (30, 5, 66, 32)]
    for _ in range(4):
        out = eng.generate_ids(prompts, SamplingParams(greedy=True, max_new_tokens=8))
        if dtype == "fp32":
            assert out == [greedy(cfg, w, p, 8) for p in prompts]
        for p, o in zip(prompts, out):
            near_best(cfg, w, p, o)
    lg = eng.forward_b(eng.forward_a(prompts[0]).cpu())
    check(lg.cpu(), orc.forward(cfg, w, prompts[0]), dtype)
    eng.shutdown()


def test_long_decoding(case):
    from llm_sharding_demo_amd.config import SamplingParams

    dtype, path, cfg, w, _, _ = case
    eng = make_engine(path, dtype)
    prompt = ids_of(3, cfg["vocab"], 1)
    near_best(cfg, w, prompt, eng.generate_ids([prompt], SamplingParams(greedy=True, max_new_tokens=250))[0])


def test_fp32_only_where_kernels_exist():
    from llm_sharding_demo_amd.config import EngineConfig
    from llm_sharding_demo_amd.runtime.engine import Engine

    with pytest.raises(ValueError, match="no fp32 kernels"):
        Engine(EngineConfig(model_id="gpt2-test", dtype="fp32", device=DEV, max_seq_len=64))
