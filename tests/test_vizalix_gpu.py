"""Vizalix kernels and whole models on the GPU against the plain model of
vizalix_oracle.py: bf16 kernels with inputs rounded to bf16 first, fp32 ones at
fp32 accuracy."""
from __future__ import annotations

import random

import numpy as np
import pytest
import torch

from llm_sharding_demo_amd.config import EngineConfig, SamplingParams
from llm_sharding_demo_amd.runtime.kv_cache import PAGE

from . import vizalix_oracle as orc

pytestmark = pytest.mark.gpu
F64 = torch.float64
BF, F32 = torch.bfloat16, torch.float32


@pytest.fixture(scope="module")
def C():
    from llm_sharding_demo_amd.ops.hip import _load

    return _load()


def cuda(t, dt=None):
    return t.to(device="cuda", dtype=dt if dt is not None else t.dtype).contiguous()


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device="cuda")


def err(got, want):
    """Largest difference over the wanted rows' root mean square."""
    want = want.double()
    return float((got.double().cpu() - want).abs().max() / want.pow(2).mean().sqrt())


def rounded(t, dt):
    return t.to(dt).double()


class Batch:
    """Ragged sequences of a launch: (slot, first position, tokens)."""

    def __init__(self, *seqs):
        self.seqs = seqs
        self.n = [s[2] for s in seqs]
        self.T = sum(self.n)
        self.cu_host = np.concatenate([[0], np.cumsum(self.n)]).tolist()
        self.slots, self.start, self.cu = i32([s[0] for s in seqs]), i32([s[1] for s in seqs]), i32(self.cu_host)
        self.tslot = i32([s[0] for s in seqs for _ in range(s[2])])
        self.tpos = i32([s[1] + j for s in seqs for j in range(s[2])])

    def tiles(self, rows):
        return i32([[i, o] for i, n in enumerate(self.n) for o in range(0, n, rows)]).reshape(-1, 2)

    def rows(self, i):
        return slice(self.cu_host[i], self.cu_host[i + 1])


# -- attention with mixed heads ---------------------------------------------------

def pools(k, v, dt, dp, vp, slots=3, seed=0):
    """Keys / values [slot][n, G, .] in shuffled pages of padded pools, and the table."""
    g = random.Random(seed)
    width = max(-(-len(x) // PAGE) for x in k.values()) + 1
    ids = list(range(slots * width))
    g.shuffle(ids)
    G = next(iter(k.values())).shape[1]
    K = torch.zeros(len(ids) + 1, G, PAGE, dp, dtype=dt)
    V = torch.zeros(len(ids) + 1, G, PAGE, vp, dtype=dt)
    table = torch.full((slots, width), len(ids), dtype=torch.int32)
    for s, kk in k.items():
        for j in range(-(-len(kk) // PAGE)):
            pg = ids.pop()
            table[s, j] = pg
            part = slice(j * PAGE, min(len(kk), (j + 1) * PAGE))
            n = part.stop - part.start
            K[pg, :, :n, : kk.shape[2]] = kk[part].transpose(0, 1).to(dt)
            V[pg, :, :n, : v[s].shape[2]] = v[s][part].transpose(0, 1).to(dt)
    return cuda(K), cuda(V), cuda(table)


def up(n, m):
    return -(-n // m) * m


SIZES = [(6, 2, 40, 24), (4, 4, 16, 20), (3, 1, 96, 72), (16, 4, 128, 128), (12, 12, 32, 64), (32, 8, 64, 128),
         (20, 5, 128, 48), (1, 1, 64, 16), (8, 1, 128, 128), (24, 3, 72, 96)]


def attention_case(H, G, D, V, dt, batch, window, cap=6.0, seed=0, stand_out=None):
    g = torch.Generator().manual_seed(seed)
    ends = {s: st + n for s, st, n in batch.seqs}
    k = {s: rounded(torch.randn(n, G, D, generator=g), dt) for s, n in ends.items()}
    v = {s: rounded(torch.randn(n, G, V, generator=g), dt) for s, n in ends.items()}
    q = rounded(torch.randn(batch.T, H, D, generator=g) * 1.5, dt)
    talk = rounded(torch.eye(H) + torch.randn(H, H, generator=g) * 0.5, BF)
    if stand_out:
        stand_out(k, v)
    want = [orc.talking_attention(q[batch.rows(i)], k[s], v[s], talk, D ** -0.5, cap, window, first=st)
            for i, (s, st, n) in enumerate(batch.seqs)]
    dp, vp = up(D, 32), up(V, 16)
    K, Vp, table = pools(k, v, dt, dp, vp)
    qp = torch.zeros(batch.T, H, dp, dtype=dt)
    qp[..., :D] = q.to(dt)
    out = torch.full((batch.T, up(H * vp, 64)), float("nan"), dtype=dt, device="cuda")
    return cuda(qp.reshape(batch.T, -1)), K, Vp, table, talk, torch.cat(want), out, D ** -0.5, cap


def unpad(out, H, V):
    vp = up(V, 16)
    assert not out[:, H * vp:].any()
    return out[:, : H * vp].reshape(-1, H, vp)[..., :V]


def frag(talk, hp):
    f = torch.zeros(hp, hp, dtype=torch.float16)
    f[: len(talk), : len(talk)] = talk.half()
    return cuda(f)


@pytest.mark.parametrize("H,G,D,V", SIZES)
@pytest.mark.parametrize("dt", [BF, F32])
def test_attention_plain(C, H, G, D, V, dt):
    b = Batch((1, 0, 3), (2, 70, 2), (0, 130, 1))
    q, K, Vp, table, talk, want, out, scale, cap = attention_case(H, G, D, V, dt, b, 67)
    C.talk_plain(q, K, Vp, table, b.tslot, b.tpos, cuda(talk, F32), 67, scale, cap, out)
    assert err(unpad(out, H, V), want) < (3e-2 if dt == BF else 2e-5)


@pytest.mark.parametrize("H,G,D,V", SIZES)
@pytest.mark.parametrize("window", [1 << 30, 67, 1, 32])
def test_attention_prefill(C, H, G, D, V, window):
    b = Batch((1, 0, 75), (2, 70, 2), (0, 130, 33))
    q, K, Vp, table, talk, want, out, scale, cap = attention_case(H, G, D, V, BF, b, window)
    hp = C.talk_heads(H, G, up(D, 32), up(V, 16), cap)
    C.talk_prefill(q, K, Vp, table, frag(talk, hp), b.tiles(C.talk_tile(hp)), b.slots, b.start, b.cu, window, scale, cap,
                   out)
    assert err(unpad(out, H, V), want) < 3e-2


@pytest.mark.parametrize("H,G,D,V", [s for s in SIZES if s[1] <= 8])
@pytest.mark.parametrize("window,splits", [(1 << 30, 1), (67, 1), (1, 1), (1 << 30, 3), (100, 2)])
def test_attention_decode(C, H, G, D, V, window, splits):
    b = Batch((1, 0, 1), (2, 63, 1), (0, 200, 1))
    q, K, Vp, table, talk, want, out, scale, cap = attention_case(H, G, D, V, BF, b, window)
    hd = max(16, C.talk_heads(H, G, up(D, 32), up(V, 16), cap), 32 if G > 4 else 0)
    C.talk_decode(q, K, Vp, table, frag(talk, hd), b.slots, b.tpos, window, scale, cap, splits, out)
    assert err(unpad(out, H, V), want) < 3e-2


@pytest.mark.parametrize("window", [1, 31, 32, 33, 64, 65, 100])
def test_attention_window_edges(C, window):
    """One key stands out for the heads that its group's scores are mixed into:
    it decides the output at the window's last place and not one further."""
    H, G, D, V = 8, 2, 32, 32
    for pos in (40, 63, 64, 127, 128, 150):
        for key in {max(0, pos - window + 1), pos - window, pos}:
            if key < 0:
                continue

            def stand_out(k, v, key=key):
                for s in k:
                    k[s][key] = 2.0
                    v[s][key] = 20.0
            b = Batch((1, pos, 1))
            args = attention_case(H, G, D, V, BF, b, window, cap=30.0, seed=pos, stand_out=stand_out)
            q, K, Vp, table, talk, want, out, scale, cap = args
            q.fill_(1.0)  # every head's score with that key is 2 sqrt(D) > 11, others are around zero
            eye = torch.eye(H, dtype=F64)
            k = {1: None}
            seen = key > pos - window
            hp = C.talk_heads(H, G, 32, 32, cap)
            outs = [out, out.clone(), out.clone()]
            C.talk_plain(q, K, Vp, table, b.tslot, b.tpos, cuda(eye, F32), window, scale, cap, outs[0])
            C.talk_prefill(q, K, Vp, table, frag(eye, hp), b.tiles(C.talk_tile(hp)), b.slots, b.start, b.cu, window,
                           scale, cap, outs[1])
            C.talk_decode(q, K, Vp, table, frag(eye, 16), b.slots, b.tpos, window, scale, cap, 2, outs[2])
            for o in outs:
                assert (float(o[0, : H * V].float().min()) > 10) == seen, (pos, key, window)


def test_attention_head_mixing(C):
    """The mixing matrix alone decides which heads see a key: a permutation
    sends head g's scores to head (g + 1) % H."""
    H, G, D, V = 16, 4, 64, 64
    b = Batch((1, 90, 20))
    q, K, Vp, table, _, _, out, scale, cap = attention_case(H, G, D, V, BF, b, 1 << 30)
    perm = torch.roll(torch.eye(H), 1, 0)
    hp = C.talk_heads(H, G, D, V, cap)
    rest = (b.slots, b.start, b.cu, 1 << 30, scale, cap)
    C.talk_prefill(q, K, Vp, table, frag(perm, hp), b.tiles(C.talk_tile(hp)), *rest, out)
    other = torch.empty_like(out)
    C.talk_plain(q, K, Vp, table, b.tslot, b.tpos, cuda(perm, F32), 1 << 30, scale, cap, other)
    plain = torch.empty_like(out)
    C.talk_plain(q, K, Vp, table, b.tslot, b.tpos, cuda(torch.eye(H), F32), 1 << 30, scale, cap, plain)
    assert err(out, other.double().cpu()) < 3e-2 and err(plain, other.double().cpu()) > 0.3


@pytest.mark.parametrize("H,G,D,V,rot", [(6, 2, 40, 24, 24), (4, 4, 64, 64, 64), (3, 1, 96, 72, 0), (16, 4, 128, 128, 64)])
@pytest.mark.parametrize("dt", [BF, F32])
def test_rope_append(C, H, G, D, V, rot, dt):
    from llm_sharding_demo_amd.config import RopeScaling, RopeSpec
    from llm_sharding_demo_amd.ops.hip import rope_spec_table

    g = torch.Generator().manual_seed(3)
    b = Batch((1, 60, 9), (0, 1000, 1), (2, 0, 3))
    dp, vp, gain = up(D, 32), up(V, 16), 1.25
    x = {n: rounded(torch.randn(b.T, h, d, generator=g), dt) for n, h, d in (("q", H, D), ("k", G, D), ("v", G, V))}
    y = torch.cat([torch.nn.functional.pad(x[n], (0, p - x[n].shape[2])).reshape(b.T, -1)
                   for n, p in (("q", dp), ("k", dp), ("v", vp))], 1)
    y = torch.nn.functional.pad(y, (0, up(y.shape[1], 64) - y.shape[1]))
    spec = {"dims": rot, "base": 500.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 128}}
    table = torch.randperm(3 * 16, generator=g).to(torch.int32).reshape(3, 16)
    K = torch.zeros(49, G, PAGE, dp, dtype=dt, device="cuda")
    Vp = torch.zeros(49, G, PAGE, vp, dtype=dt, device="cuda")
    rope = rope_spec_table(RopeSpec(rot, 500.0, RopeScaling(4.0, 1.0, 4.0, 128)), 1024, "cuda") if rot else None
    q = C.rope_append(cuda(y, dt), H, K, Vp, cuda(table), b.tslot, b.tpos, rope, gain)
    pos = b.tpos.cpu().tolist()
    turn = lambda t: orc.rotate(t * gain, pos, spec) if rot else t * gain  # noqa: E731
    tol = 3e-2 if dt == BF else 1e-5
    assert err(q.reshape(b.T, H, dp)[..., :D], turn(x["q"])) < tol
    wk = turn(x["k"])
    for t, (s, p) in enumerate(zip(b.tslot.cpu().tolist(), pos)):
        pg = int(table[s, p // PAGE])
        assert err(K[pg, :, p % PAGE, :D], wk[t]) < tol and err(Vp[pg, :, p % PAGE, :V], x["v"][t] * gain) < tol
    assert int((Vp.abs().sum((1, 3)) > 0).sum()) == b.T
