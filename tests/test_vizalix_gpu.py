"""Vizalix kernels and whole models on the GPU against the plain model of
vizalix_oracle.py: bf16 kernels with inputs rounded to bf16 first, fp32 ones at
fp32 accuracy."""
from __future__ import annotations

import numpy as np
import pytest
import torch

from llm_sharding_demo_amd.config import EngineConfig, SamplingParams
from llm_sharding_demo_amd.runtime.kv_cache import PAGE

from . import vizalix_oracle as orc
from .paged_helpers import (BF, F32, Batch, cuda, err, i32, ids_of, logit_err, pools, portion_steps, portions, rounded,
                            run_steps, up)

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def C():
    from llm_sharding_demo_amd.ops.hip import _load

    return _load()


# -- attention with mixed heads ---------------------------------------------------

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
@pytest.mark.parametrize("window,splits", [(1 << 30, 1), (67, 1), (1, 1), (32, 1), (1 << 30, 3), (67, 2), (5, 4)])
def test_attention_prefill(C, H, G, D, V, window, splits):
    b = Batch((1, 0, 75), (2, 70, 2), (0, 130, 33))
    q, K, Vp, table, talk, want, out, scale, cap = attention_case(H, G, D, V, BF, b, window)
    hp = C.talk_heads(H, G, up(D, 32), up(V, 16), cap)
    C.talk_prefill(q, K, Vp, table, frag(talk, hp), b.tiles(C.talk_tile(hp)), b.slots, b.start, b.cu, window, scale, cap,
                   splits, out)
    assert err(unpad(out, H, V), want) < 3e-2


@pytest.mark.parametrize("H,G,D,V", [s for s in SIZES if s[1] <= 8])
@pytest.mark.parametrize("window,splits", [(1 << 30, 1), (67, 1), (1, 1), (1 << 30, 3), (100, 2), (1 << 30, 17)])
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
            q, K, Vp, table, _, _, out, scale, cap = args
            q.fill_(1.0)  # every head's score with that key is 2 sqrt(D) > 11, others are around zero
            eye = torch.eye(H)
            seen = key > pos - window
            hp = C.talk_heads(H, G, 32, 32, cap)
            outs = [out, out.clone(), out.clone()]
            C.talk_plain(q, K, Vp, table, b.tslot, b.tpos, cuda(eye, F32), window, scale, cap, outs[0])
            C.talk_prefill(q, K, Vp, table, frag(eye, hp), b.tiles(C.talk_tile(hp)), b.slots, b.start, b.cu, window,
                           scale, cap, 2, outs[1])
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
    rest = (b.slots, b.start, b.cu, 1 << 30, scale, cap, 1)
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


# -- recurrences ------------------------------------------------------------------

DELTA = [(2, 2, 8, 8, 1), (4, 2, 24, 20, 3), (3, 3, 64, 64, 4), (2, 1, 128, 128, 4), (4, 4, 32, 100, 2), (2, 2, 96, 40, 4)]


class DeltaCase:
    """In-projection and low-rank rows of one sequence, and what comes out of it."""

    def __init__(self, C, H, G, D, V, n, T, dt, seed=0, decay=1.0, strong=0.0):
        self.C, self.dims, self.dt = C, (H, G, D, V), dt
        g = torch.Generator().manual_seed(seed)
        R = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
        self.ch = 2 * G * D + H * V
        self.c0, self.gain, self.eps = 64, 0.75, 1e-5
        x, b = rounded(R(T, self.ch), dt), rounded(R(T, H), dt)
        lowd, gate = rounded(R(T, H * D), dt), rounded(R(T, H * V), dt)
        taps, A = R(self.ch, n) / n ** 0.5, R(H)
        dtb, norm = R(H * D) - 2, 1 + 0.2 * R(V)
        A = -torch.exp(A) * decay
        if strong:  # some key channels forget nearly everything at every step
            dtb[torch.rand(H * D, generator=g) < 0.2] += strong
        self.y = torch.zeros(T, up(self.c0 + self.ch + H, 64), dtype=dt)
        self.y[:, self.c0: self.c0 + self.ch], self.y[:, self.c0 + self.ch: self.c0 + self.ch + H] = x, b
        self.nl = up(max(H * D, H * V), 16)
        self.low = torch.zeros(T, 2 * self.nl, dtype=dt)
        self.low[:, : H * D], self.low[:, self.nl: self.nl + H * V] = lowd, gate
        self.par = [cuda(t, F32) for t in (taps, A, dtb, norm)]
        A, taps, dtb, norm = A.double(), taps.double(), dtb.double(), norm.double()
        q, k, v = torch.split(orc.silu(orc.short_conv(x * self.gain, taps)), [G * D, G * D, H * V], 1)
        of = [h // (H // G) for h in range(H)]
        q, k = (orc.unit(t.reshape(T, G, D))[:, of] for t in (q, k))
        decays = torch.exp(A[:, None] * orc.softplus(lowd * self.gain + dtb).reshape(T, H, D))
        o, self.S = orc.delta_rule(q * D ** -0.5, k, v.reshape(T, H, V), decays, orc.sigmoid(b * self.gain))
        o = orc.rms(o, self.eps) * norm
        self.want = o.reshape(T, H * V) * orc.sigmoid(gate * self.gain)
        self.state = torch.full((3, H, D, up(V, 4)), float("nan"), device="cuda")
        self.ring = torch.full((3, n, self.ch), float("nan"), dtype=dt, device="cuda")

    def run(self, parts, chunked, slot=1):
        H, G, D, V = self.dims
        taps, A, dtb, norm = self.par
        outs = []
        for a, b in parts:
            out = torch.full((b - a, up(H * V, 64)), float("nan"), dtype=self.dt, device="cuda")
            single = b - a == 1 and not chunked
            self.C.delta_seq(cuda(self.y[a:b]), self.c0, self.c0 + self.ch, cuda(self.low[a:b]), self.nl, i32([slot]),
                             i32([a]), i32([0, b - a]), H, G, D, V, taps, self.ring, self.state, A, dtb, norm, self.gain,
                             self.eps, out, single, chunked)
            assert not out[:, H * V:].any()
            outs.append(out[:, : H * V])
        return torch.cat(outs)


SPLITS = [[100], [1] * 100, [2] * 50, [16, 16, 1, 31, 2, 3, 5], [7, 33, 1, 1, 58]]


@pytest.mark.parametrize("H,G,D,V,n", DELTA + [(2, 1, 200, 300, 5)])
@pytest.mark.parametrize("sizes", SPLITS)
@pytest.mark.parametrize("dt", [BF, F32])
def test_delta_rule_by_tokens(C, H, G, D, V, n, sizes, dt):
    c = DeltaCase(C, H, G, D, V, n, 60, dt)
    out = c.run(portions(60, sizes), False)
    assert err(out, c.want) < (3e-2 if dt == BF else 3e-5)
    assert err(c.state[1, ..., :V], c.S) < 2e-5  # the state is fp32 in both


@pytest.mark.parametrize("H,G,D,V,n", DELTA)
@pytest.mark.parametrize("sizes", SPLITS)
@pytest.mark.parametrize("decay,strong", [(1.0, 0.0), (0.01, 0.0), (8.0, 0.0), (4.0, 12.0)])
def test_delta_rule_in_chunks(C, H, G, D, V, n, sizes, decay, strong):
    """Slow decays, and some that outrun the range of a chunk's factors."""
    c = DeltaCase(C, H, G, D, V, n, 100, BF, decay=decay, strong=strong)
    out = c.run(portions(100, sizes), True)
    assert err(out, c.want) < 8e-2
    assert err(c.state[1, ..., :V], c.S) < 3e-2  # q, k and v are bf16 behind the convolution


def test_delta_rule_chunks_between_tokens(C):
    """A state passed between the two forms."""
    c = DeltaCase(C, 3, 3, 64, 64, 4, 90, BF)
    out = torch.cat([c.run([(0, 40)], True), c.run([(i, i + 1) for i in range(40, 60)], False), c.run([(60, 90)], True)])
    assert err(out, c.want) < 8e-2


SSM = [(2, 8, 8, 1, 1, 1), (6, 12, 20, 2, 3, 4), (4, 64, 128, 1, 1, 4), (3, 128, 64, 3, 3, 2), (8, 32, 16, 2, 4, 3),
       (2, 100, 36, 1, 2, 4), (20, 64, 16, 1, 1, 4)]


class SsmCase:
    def __init__(self, C, H, V, N, G, NG, n, T, dt, seed=0, decay=1.0):
        self.C, self.dims, self.dt = C, (H, V, N, G, NG), dt
        g = torch.Generator().manual_seed(seed)
        R = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
        inner, self.gain, self.eps = H * V, 0.75, 1e-5
        ch = inner + 2 * G * N
        z, x, d = rounded(R(T, inner), dt), rounded(R(T, ch), dt), rounded(R(T, H), dt)
        taps, bias, A = R(ch, n) / n ** 0.5, 0.3 * R(ch), R(H)
        dtb, skip, norm = R(H) - 1, 1 + 0.3 * R(H), 1 + 0.2 * R(inner)
        A = A + float(np.log(decay))
        self.y = torch.nn.functional.pad(torch.cat([z, x, d], 1), (0, up(inner + ch + H, 64) - inner - ch - H)).to(dt)
        self.par = [cuda(t, F32) for t in (taps, bias, -torch.exp(A), dtb, skip, norm)]
        taps, bias, A, dtb, skip, norm = (t.double() for t in (taps, bias, A, dtb, skip, norm))
        xbc = orc.silu(orc.short_conv(x * self.gain, taps, bias))
        u, B, Cc = torch.split(xbc, [inner, G * N, G * N], 1)
        of = [h // (H // G) for h in range(H)]
        yy, self.S = orc.ssd(u.reshape(T, H, V), B.reshape(T, G, N)[:, of], Cc.reshape(T, G, N)[:, of],
                             orc.softplus(d * self.gain + dtb), A, skip)
        yy = yy.reshape(T, inner) * orc.silu(z * self.gain)
        self.want = orc.rms(yy.reshape(T, NG, -1), self.eps).reshape(T, inner) * norm
        self.state = torch.full((3, H, N, up(V, 4)), float("nan"), device="cuda")
        self.ring = torch.full((3, n, ch), float("nan"), dtype=dt, device="cuda")

    def run(self, parts, chunked, slot=1):
        H, V, N, G, NG = self.dims
        taps, bias, A, dtb, skip, norm = self.par
        outs = []
        for a, b in parts:
            out = torch.full((b - a, up(H * V, 64)), float("nan"), dtype=self.dt, device="cuda")
            self.C.ssm_seq(cuda(self.y[a:b]), i32([slot]), i32([a]), i32([0, b - a]), H, G, N, V, NG, taps, bias, self.ring,
                           self.state, A, dtb, skip, norm, self.gain, self.eps, out, b - a == 1 and not chunked, chunked)
            assert not out[:, H * V:].any()
            outs.append(out[:, : H * V])
        return torch.cat(outs)


@pytest.mark.parametrize("H,V,N,G,NG,n", SSM + [(2, 200, 300, 1, 1, 5), (3, 10, 8, 1, 2, 2)])
@pytest.mark.parametrize("sizes", SPLITS)
@pytest.mark.parametrize("dt", [BF, F32])
def test_mamba2_by_tokens(C, H, V, N, G, NG, n, sizes, dt):
    c = SsmCase(C, H, V, N, G, NG, n, 60, dt)
    out = c.run(portions(60, sizes), False)
    assert err(out, c.want) < (3e-2 if dt == BF else 3e-5)
    assert err(c.state[1, ..., :V], c.S) < 2e-5


@pytest.mark.parametrize("H,V,N,G,NG,n", SSM)
@pytest.mark.parametrize("sizes", SPLITS)
@pytest.mark.parametrize("decay", [1.0, 0.01, 30.0])
def test_mamba2_in_chunks(C, H, V, N, G, NG, n, sizes, decay):
    c = SsmCase(C, H, V, N, G, NG, n, 100, BF, decay=decay)
    out = c.run(portions(100, sizes), True)
    assert err(out, c.want) < 8e-2
    assert err(c.state[1, ..., :V], c.S) < 3e-2


def test_recurrences_of_many_sequences(C):
    """Unequal sequences of one launch keep to their own slots."""
    c = SsmCase(C, 4, 16, 32, 2, 2, 4, 70, BF)
    H, V, N, G, NG = c.dims
    taps, bias, A, dtb, skip, norm = c.par
    lens, slots = [70, 3, 33, 1], [2, 0, 3, 1]
    y = torch.cat([c.y[:n] for n in lens])
    state = torch.full((4, H, N, V), float("nan"), device="cuda")
    ring = torch.full((4, 4, H * V + 2 * G * N), float("nan"), dtype=BF, device="cuda")
    out = torch.empty(sum(lens), H * V, dtype=BF, device="cuda")
    cu = np.concatenate([[0], np.cumsum(lens)]).tolist()
    C.ssm_seq(cuda(y), i32(slots), i32([0] * 4), i32(cu), H, G, N, V, NG, taps, bias, ring, state, A, dtb, skip, norm, c.gain,
              c.eps, out, False, True)
    for a, n in zip(cu, lens):
        assert err(out[a: a + n], c.want[:n]) < 6e-2
    assert err(state[2], c.S) < 3e-2
    # one token each: all four sequences step together from there
    pos = [n - 1 for n in lens]  # repeats each sequence's last token: other states, same for equal ones
    out2 = torch.empty(4, H * V, dtype=BF, device="cuda")
    before = state.clone()
    C.ssm_seq(cuda(torch.stack([c.y[p] for p in pos])), i32(slots), i32(lens), i32([0, 1, 2, 3, 4]), H, G, N, V, NG, taps,
              bias, ring, state, A, dtb, skip, norm, c.gain, c.eps, out2, True, False)
    assert all(float((state[s] - before[s]).abs().max()) > 0 for s in slots)


def test_gated_gemm_epilogue(C):
    """gelu(s g) (s u) and the SiLU form, split-K, tiled and GEMV rows."""
    from llm_sharding_demo_amd.ops.hip import HipBackend, interleave_experts

    be = HipBackend()
    be._counters = torch.zeros(8, 1 << 16, dtype=torch.int32, device="cuda")
    g = torch.Generator().manual_seed(0)
    for M in (1, 3, 8, 40, 200, 700):
        h, w = rounded(torch.randn(M, 128, generator=g), BF), rounded(torch.randn(2 * 192, 128, generator=g) * 0.1, BF)
        want = orc.gelu_tanh(h @ w[:192].T * 0.6) * (h @ w[192:].T * 0.6)
        buf = torch.full((M, 256), 7.0, dtype=BF, device="cuda")
        be.decode = M <= 200
        be.linear(cuda(h, BF), interleave_experts(cuda(w, BF), 192, 128), act="gelu_mul", out=buf[:, 64:], scale=0.6)
        assert err(buf[:, 64:], want) < 3e-2 and bool((buf[:, :64] == 7).all())
    y = torch.randn(5, 64, generator=g)
    out = torch.empty(5, 32, device="cuda")
    C.glu_f32(cuda(y), out, 1, 1.5)
    gate, up_ = (torch.cat([y[:, i: i + 16], y[:, i + 32: i + 48]], 1).double() * 1.5 for i in (0, 16))
    assert err(out, orc.gelu_tanh(gate) * up_) < 1e-5


# -- whole models ------------------------------------------------------------------

def odd_sizes():
    """Every mixer twice, nothing a multiple of a tile, one layer without a feed-forward."""
    return orc.config([orc.delta(), orc.attn(), orc.ssm(),
                       orc.delta(heads=3, kv_heads=3, dim=8, vdim=16, conv=1, ff=0, ranks=(3, 70)),
                       orc.attn(heads=3, kv_heads=1, dim=16, vdim=20, window=9, rot=16, scaling=None, ff=24),
                       orc.ssm(heads=2, vdim=24, state=5, groups=1, norm_groups=1, conv=2)], loop=(1, 3, 2))


def tile_sizes():
    """Sizes of the fused paths, GEMM-aligned width, the loop in front."""
    return orc.config([orc.delta(heads=2, kv_heads=1, dim=64, vdim=128, conv=4, ff=128, ranks=(32, 16)),
                       orc.ssm(heads=4, vdim=32, state=64, groups=2, norm_groups=4, ff=192),
                       orc.attn(heads=16, kv_heads=4, dim=64, vdim=64, window=100, scale=0.125, rot=32, ff=128),
                       orc.attn(heads=10, kv_heads=10, dim=32, vdim=16, window=33, rot=8, ff=64)],
                      width=128, vocab=320, loop=(0, 2, 3))


def open_model(tmp_path, cfg, dtype, seed=0, **kw):
    from llm_sharding_demo_amd.runtime.engine import Engine

    w = orc.random_weights(cfg, seed)
    orc.save(str(tmp_path), cfg, w)
    kw = {"max_batch": 4, "max_seq_len": 640, "kv_tokens": 1280, **kw}
    return w, Engine(EngineConfig(model_id=str(tmp_path), weights=str(tmp_path), dtype=dtype, device="cuda", **kw))


LIMIT = {"bf16": 0.08, "fp32": 5e-5}


@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
@pytest.mark.parametrize("make", [odd_sizes, tile_sizes])
def test_model_portions(tmp_path, dtype, make):
    """Whole prompts, pairs, single tokens and uneven portions give the same logits."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    cfg = make()
    w, eng = open_model(tmp_path, cfg, dtype)
    ses, ids = TraceSession(eng), ids_of(150)
    want = orc.forward(cfg, w, ids)
    for sizes in ([150], [2] * 75, [1] * 150, [63, 1, 2, 60, 24], [7, 130, 13], [16, 17, 32, 33, 3, 5]):
        got = run_steps(ses, {"a": ids}, portion_steps("a", 150, sizes))["a"]
        assert logit_err(got, want) < LIMIT[dtype], sizes
    assert eng.slots.available == 4 and eng.page_pools[0].available == 20


@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
@pytest.mark.parametrize("make", [odd_sizes, tile_sizes])
def test_model_mixed_batches(tmp_path, dtype, make):
    """Unequal requests in one batch; pages and slots are freed and used again."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    cfg = make()
    w, eng = open_model(tmp_path, cfg, dtype, kv_tokens=6 * PAGE)
    ses = TraceSession(eng)
    seqs = {k: ids_of(n, seed=n) for k, n in (("a", 100), ("b", 5), ("c", 131), ("d", 66))}
    want = {k: orc.forward(cfg, w, v) for k, v in seqs.items()}
    steps = [[("a", 70), ("b", 1)], [("a", 1), ("b", 3), ("c", 2)], [("b", 1), ("c", 61), ("a", 1)],
             [("c", 1), ("a", 28), ("d", 60)], [("d", 1), ("c", 2)], [("c", 65), ("d", 5)]]
    for _ in range(3):
        got = run_steps(ses, seqs, steps)
        for k in seqs:
            assert logit_err(got[k], want[k]) < LIMIT[dtype], k
        assert not ses.live and eng.page_pools[0].available == 6 and eng.slots.available == 4


@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
def test_model_long_sequence(tmp_path, dtype):
    """Several windows and pages of prompt, then long decoding past them."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    cfg = tile_sizes()
    w, eng = open_model(tmp_path, cfg, dtype, seed=4)
    ids = ids_of(420, vocab=320, seed=9)
    got = run_steps(TraceSession(eng), {"a": ids}, portion_steps("a", 420, [270]))["a"]
    assert logit_err(got, orc.forward(cfg, w, ids)) < LIMIT[dtype]


@pytest.mark.parametrize("make", [odd_sizes, tile_sizes])
def test_model_layers(tmp_path, make):
    """The residual after every layer run, in fp32."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    cfg = make()
    w, eng = open_model(tmp_path, cfg, "fp32")
    st, rows, want = eng.stages[0], [], []
    fwd = st.forward
    st.forward = lambda *a, **k: fwd(*a, residuals=rows, **k)
    ids = ids_of(40)
    TraceSession(eng).step([{"id": "a", "tokens": ids, "want": [39]}], ["a"])
    orc.forward(cfg, w, ids, want)
    assert len(rows) == len(want) == len(orc.passes(cfg))
    for got, x in zip(rows, want):
        assert err(got, x) < 2e-5


def near_greedy(cfg, w, prompt, out, tol):
    """Every generated token is the plain model's best behind what came before, up to `tol` of the logits' spread."""
    lg = orc.forward(cfg, w, prompt + out[:-1])[len(prompt) - 1:]
    best, got = lg.max(-1).values, lg[torch.arange(len(out)), torch.tensor(out)]
    return float((best - got).max()) <= tol * float(lg.std())


@pytest.mark.parametrize("dtype,tol", [("bf16", 0.15), ("fp32", 1e-3)])
@pytest.mark.parametrize("kw", [{}, {"num_microbatches": 2, "prefill_chunk": 20}, {"use_graphs": False},
                                {"kv_tokens": 5 * PAGE, "max_batch": 3}])
def test_model_greedy_generation(tmp_path, dtype, tol, kw):
    """Through the scheduler, with captured decode graphs, sessions repeated in
    used slots and pages."""
    cfg = odd_sizes()
    w, eng = open_model(tmp_path, cfg, dtype, **kw)
    prompts = [ids_of(n, seed=n) for n in (1, 70, 13, 64, 40)]
    sp = [SamplingParams(greedy=True, max_new_tokens=n) for n in (12, 5, 40, 3, 9)]
    first = None
    for _ in range(3):
        out = eng.generate_ids(prompts, sp)
        assert [len(o) for o in out] == [s.max_new_tokens for s in sp]
        assert all(near_greedy(cfg, w, p, o, tol) for p, o in zip(prompts, out))
        if dtype == "fp32":
            assert first is None or out == first
            first = out
        assert eng.page_pools[0].available == eng.kv_pages and eng.slots.available == eng.kv_slots


@pytest.mark.parametrize("transport", ["loopback", "devloop"])
def test_model_two_stages(tmp_path, transport):
    """A boundary between the loop's passes, and the compat forwards across it."""
    cfg = odd_sizes()
    w, eng = open_model(tmp_path, cfg, "bf16", num_stages=2, split_points=[3], transport=transport)
    prompts = [ids_of(n, seed=n) for n in (30, 5, 66)]
    for _ in range(2):
        out = eng.generate_ids(prompts, SamplingParams(greedy=True, max_new_tokens=8))
        assert all(len(o) == 8 and near_greedy(cfg, w, p, o, 0.15) for p, o in zip(prompts, out))
    hid = eng.forward_a(prompts[0])
    assert hid.shape == (30, 2 * 88)
    assert logit_err(eng.forward_b(hid).cpu(), orc.forward(cfg, w, prompts[0])) < LIMIT["bf16"]
    eng.shutdown()


def test_mixed_step_of_the_scheduler(tmp_path):
    """Decode rows and joining prompts in one forward."""
    cfg = odd_sizes()
    w, eng = open_model(tmp_path, cfg, "bf16", join_min=1)
    eng.workers[0].mixed_steps = True
    prompts = [ids_of(n, seed=n) for n in (30, 5, 66, 17, 40, 3)]
    sp = [SamplingParams(greedy=True, max_new_tokens=n) for n in (3, 12, 6, 20, 9, 15)]
    out = eng.generate_ids(prompts, sp)
    assert eng.workers[0].mixed_items > 0
    assert all(len(o) == s.max_new_tokens and near_greedy(cfg, w, p, o, 0.15) for p, s, o in zip(prompts, sp, out))


def test_fp32_refusals_stay(tmp_path):
    from llm_sharding_demo_amd.runtime.engine import Engine

    with pytest.raises(ValueError, match="fp32"):
        Engine(EngineConfig(model_id="gpt2-test", dtype="fp32", device="cuda", max_batch=1, max_seq_len=64))
