"""Fagunex kernels and whole models on the GPU against the plain model of
fagunex_oracle.py: bf16 kernels with inputs rounded to bf16 first, fp32 ones at
fp32 accuracy."""
from __future__ import annotations

import pytest
import torch

from llm_sharding_demo_amd.config import EngineConfig, SamplingParams
from llm_sharding_demo_amd.runtime.kv_cache import PAGE

from . import fagunex_oracle as orc
from .paged_helpers import BF, F32, Batch, cuda, err, i32, ids_of, logit_err, portion_steps, portions, rounded, run_steps, up

pytestmark = pytest.mark.gpu
ALL = 1 << 30
DTYPES = pytest.mark.parametrize("dt", [BF, F32], ids=["bf16", "fp32"])


@pytest.fixture(scope="module")
def C():
    from llm_sharding_demo_amd.ops.hip import _load

    return _load()


def randn(g, *shape, dt=F32):
    return rounded(torch.randn(*shape, generator=g), dt)


# -- elementwise norms -----------------------------------------------------------------

@pytest.mark.parametrize("width", [88, 104, 256, 1000, 2048, 4096])
@DTYPES
def test_norms_around_a_sublayer(C, width, dt):
    g = torch.Generator().manual_seed(width)
    H, f32, tol = up(width, 64), dt == F32, 2e-2 if dt == BF else 1e-5
    dev = lambda t, dt=dt: cuda(torch.nn.functional.pad(t, (0, H - width)), dt)  # noqa: E731
    vec = lambda: randn(g, width, dt=dt)  # noqa: E731
    for T, S, sdt in ((1, 0, None), (3, 1, F32), (70, 1, dt), (5, 4, dt), (2, 7, dt), (1100, 2, dt), (1030, 5, dt), (1025, 1, F32)):
        x = randn(g, T, width) * torch.linspace(0.01, 4, width)  # also where tanh is nearly linear
        (w1, b1, w2, b2), want, args = (vec() for _ in range(4)), x, (None, 0.0, None, None)
        if S:
            s = randn(g, S, T, width, dt=sdt)
            want = x + orc.dynamic_tanh(s.sum(0), 0.6, w1, b1)
            args = (dev(s, sdt), 0.6, dev(w1), dev(b1))
        xd = dev(x, F32)
        out = C.tanh_step(xd, *args, True, 0.9, dev(w2), dev(b2), None, f32)
        assert err(xd[:, :width], want) < 1e-5 and not xd[:, width:].any()
        assert err(out[:, :width], orc.dynamic_tanh(want, 0.9, w2, b2)) < tol and not out[:, width:].any()
        xd = dev(x, F32)
        out = C.tanh_step(xd, *args, True, 0.0, None, None, None, f32)  # the residual as it is
        assert err(out[:, :width], want) < tol and err(xd[:, :width], want) < 1e-5
        if S:
            xd = dev(x, F32)
            assert C.tanh_step(xd, *args, False, 0.0, None, None, None, f32) is None
            assert err(xd[:, :width], want) < 1e-5
        rows = [T - 1, 0]
        out = C.tanh_step(dev(x, F32), None, 0.0, None, None, True, 0.9, dev(w2), dev(b2), i32(rows), f32)
        assert err(out[:, :width], orc.dynamic_tanh(x[rows], 0.9, w2, b2)) < tol


class ShiftCase:
    """One sequence's residual rows and side slabs, run in portions beside others."""

    def __init__(self, n, width, dt, S, seed=0):
        g = torch.Generator().manual_seed(seed)
        self.dt, self.width, self.H, self.S, self.eps = dt, width, up(width, 64), S, 1e-3
        self.x = randn(g, n, width)
        self.slab = randn(g, max(S, 1), n, width, dt=dt)
        g = torch.Generator().manual_seed(100)
        self.ws, self.w, self.b, self.mix = (randn(g, width, dt=dt) for _ in range(4))
        self.want_x = self.x + (orc.rms(self.slab.sum(0), self.eps) * self.ws if S else 0)
        self.want = orc.token_shift(orc.dynamic_tanh(self.want_x, 0.7, self.w, self.b), self.mix)


def run_shift(C, cases, steps):
    """steps: [(case = slot, first, tokens), ...] each; last rows start as garbage."""
    c0 = cases[0]
    dev = lambda t, dt: cuda(torch.nn.functional.pad(t, (0, c0.H - c0.width)), dt)  # noqa: E731
    last = torch.full((len(cases), c0.H), float("nan"), device="cuda")
    f32, out = c0.dt == F32, {i: [] for i in range(len(cases))}
    for step in steps:
        b = Batch(*step)
        x = dev(torch.cat([cases[s].x[a:a + n] for s, a, n in step]), F32)
        slab = dev(torch.cat([cases[s].slab[:, a:a + n] for s, a, n in step], 1), c0.dt) if c0.S else None
        norm = (0.7, dev(c0.w, c0.dt), dev(c0.b, c0.dt))
        x_new, h = C.shift_norm(x, slab, dev(c0.ws, c0.dt) if c0.S else None, c0.width, c0.eps, *norm, dev(c0.mix, c0.dt), last,
                                b.tslot, b.tpos, f32)
        if any(n > 1 for _, _, n in step):
            C.shift_tail(x_new, *norm, last, b.tslot, b.cu[1:] - 1, f32)
        for i, (s, a, n) in enumerate(step):
            out[s].append(h[b.rows(i)])
            assert err(x_new[b.rows(i), : c0.width], cases[s].want_x[a:a + n]) < 1e-5
    for s, c in enumerate(cases):
        got = torch.cat(out[s])
        assert err(got[:, : c.width], c.want) < (2e-2 if c.dt == BF else 1e-5)
        assert not got[:, c.width:].any()


@pytest.mark.parametrize("width,S", [(88, 1), (104, 0), (256, 3), (2048, 1), (4096, 2)])
@DTYPES
def test_token_shift(C, width, S, dt):
    """Whole, in uneven portions down to two tokens, token by token, and beside others."""
    for sizes in ([60], [1] * 60, [2] * 30, [23, 1, 2, 30, 4]):
        run_shift(C, [ShiftCase(60, width, dt, S)], [[(0, a, b - a)] for a, b in portions(60, sizes)])
    cases = [ShiftCase(n, width, dt, S, seed=n) for n in (9, 2600, 30)]
    run_shift(C, cases, [[(0, 0, 1), (1, 0, 1300), (2, 0, 3)], [(2, 3, 2), (1, 1300, 1), (0, 1, 1)],
                         [(1, 1301, 2), (0, 2, 7), (2, 5, 25)], [(1, 1303, 1297)]])


def test_token_shift_of_long_prompts(C):
    """Runs of rows: portions that begin and end anywhere in them."""
    cases = [ShiftCase(n, 64, BF, 1, seed=n) for n in (17000, 5, 16, 1)]
    run_shift(C, cases, [[(0, 0, 6), (2, 0, 13), (1, 0, 5), (0 + 3, 0, 1)], [(2, 13, 3), (0, 6, 16994)]])


# -- routing, experts, token rows ----------------------------------------------------------

@pytest.mark.parametrize("E,top,shared", [(6, 2, True), (1, 1, False), (70, 5, True), (16, 16, False), (300, 3, True)])
def test_softmax_routing(C, E, top, shared):
    z = randn(torch.Generator().manual_seed(E), 37, up(E + 1, 64)) * 3
    ids, wts, sh = C.route_softmax(cuda(z, F32), E, top, shared)
    for t in range(37):
        order, w = orc.route(torch.ones(1, dtype=z.dtype), z[t, :E, None], top)
        assert ids[t].tolist() == order and err(wts[t], w) < 1e-5
    assert err(sh, orc.sigmoid(z[:, E])) < 1e-5 if shared else sh.numel() == 0


@pytest.mark.parametrize("T,K,N", [(1, 64, 16), (16, 128, 32), (17, 512, 64), (130, 2048, 64), (40, 4160, 48)])
def test_narrow_projections(C, T, K, N):
    """Router and token-side gate in one launch each, rows and K shared among the waves."""
    g = torch.Generator().manual_seed(T)
    a, w = randn(g, T, K, dt=BF), rounded(torch.randn(N, K, generator=g) * 2 / K ** 0.5, BF)
    z, tickets = a @ w.T, i32([0] * 16)
    for E, top, shared in ((N, 1, False), (N - 1, 3, True), (5, 5, True)):
        for splits in (1, 2, 5, 16):
            ids, wts, sh = C.router(cuda(a, BF), cuda(w, BF), E, top, shared, splits, tickets)
            for t in range(T):
                order, want = orc.route(torch.ones(1, dtype=z.dtype), z[t, :E, None], top)
                assert ids[t].tolist() == order and err(wts[t], want) < 1e-4
            assert not shared or err(sh, orc.sigmoid(z[:, E])) < 1e-4
            assert not tickets.any()
    table, ids = randn(g, 11, N, dt=BF), [(7 * i) % 11 for i in range(T)]
    out = C.side_gate(cuda(a, BF), cuda(w, BF), i32(ids), cuda(table, BF))
    assert err(out, orc.gelu_tanh(z) * table[ids]) < 1e-2


@pytest.mark.parametrize("T,E,top,ff,shared", [(1, 4, 2, 40, 24), (3, 6, 1, 64, 0), (4, 5, 5, 24, 72), (9, 4, 2, 40, 24),
                                               (70, 6, 3, 64, 96), (300, 5, 2, 48, 0), (700, 8, 2, 64, 40)])
@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
def test_silu_experts(tmp_path, T, E, top, ff, shared, dtype):
    """Streamed and grouped experts through the backend, the shared one weighed per token."""
    from llm_sharding_demo_amd.ops import Residual

    cfg = orc.config([orc.forget(experts=E, top=top, ff=ff, shared=shared)], side=0)
    w, eng = open_model(tmp_path, cfg, dtype)
    st, dt = eng.stages[0], BF if dtype == "bf16" else F32
    h = randn(torch.Generator().manual_seed(T), T, 88, dt=dt)
    want = orc.experts(h, cfg["layers"][0]["mlp"], lambda n: w["l0.mlp." + n].double())
    r = Residual(torch.zeros(T, 128, device="cuda"))
    st.backend.decode = False
    st.backend.experts_tanh(cuda(torch.nn.functional.pad(h, (0, 40)), dt), lambda n: st.w["layers.0." + n],
                            st.cfg.layers[0].mlp, lambda n: st.w["layers.0.norm2b" + n], r)
    assert err(r.post.slab.double().sum(0)[:, :88], want) < (3e-2 if dt == BF else 2e-5)
    eng.shutdown()


@DTYPES
def test_token_rows(C, dt):
    g = torch.Generator().manual_seed(0)
    a, table = randn(g, 30, 64, dt=dt), randn(g, 11, 64, dt=dt)
    ids = [(7 * i) % 11 for i in range(30)]
    out = C.side_mul(cuda(a, dt), i32(ids), cuda(table, dt))
    assert err(out, (a if dt == BF else orc.gelu_tanh(a)) * table[ids]) < (1e-2 if dt == BF else 1e-5)


# -- in front of the scores ----------------------------------------------------------------

@pytest.mark.parametrize("H,dim,rot,rank,gate", [(3, 24, 8, 40, 60), (5, 12, 20, 28, 0), (1, 1, 2, 3, 4), (16, 128, 64, 512, 64),
                                                 (2, 64, 0, 64, 0)])
@pytest.mark.parametrize("q_rank", [None, 36])
@DTYPES
def test_latent_rows(C, H, dim, rot, rank, gate, q_rank, dt):
    """Queries turned or normed, the latent normed and cached, the key part turned
    behind it -- in the order that brings interleaved pairs side by side."""
    from llm_sharding_demo_amd.config import RopeSpec
    from llm_sharding_demo_amd.ops.hip import rope_spec_table

    T, dp, cols, f32 = 9, up(dim + rot, 64), up(rank + rot, 64), dt == F32
    nq = H * dp if q_rank is None else up(q_rank, 64)
    g = torch.Generator().manual_seed(H)
    y = randn(g, T, up(nq + gate + rank + rot, 4)) * 2
    gain, qgain = randn(g, rank), randn(g, q_rank or 1)
    pos = [0, 63, 64, 65, 127, 128, 190, 191, 1]
    table = i32([[5, 5, 5], [2, 4, 0]])
    cache = torch.zeros(6, PAGE, cols, dtype=dt, device="cuda")
    rope = rope_spec_table(RopeSpec(rot, 100.0), 192, "cuda") if rot else None
    where = (i32([1] * T), i32(pos))
    turn = dict(rope=rope, q_head=dp, q_rot=dim)
    q = C.latent_post(cuda(y, F32), nq, True, f32, cache, rank, cuda(gain, F32), 1e-3, table, *where, None, 0, c_off=nq + gate,
                      q_gain=None if q_rank is None else cuda(qgain, F32), **turn)[0]
    tol = 1e-2 if dt == BF else 1e-5

    def heads(x):
        x = x.reshape(T, H, dp).clone()
        if rot:
            x[..., dim:dim + rot] = orc.rotate(x[..., dim:dim + rot], pos, 100.0, False)
        return x.reshape(T, -1)
    if q_rank is None:
        assert err(q, heads(y[:, :nq])) < tol
    else:
        assert err(q[:, :q_rank], orc.rms(y[:, :q_rank], 1e-3) * qgain) < tol and not q[:, q_rank:].any()
        z = randn(g, T, H * dp)
        q = C.latent_post(cuda(z, F32), H * dp, True, f32, None, 0, None, 1e-3, None, *where, None, 0, **turn)[0]
        assert err(q, heads(z)) < tol
    c = y[:, nq + gate:]
    want = torch.cat([orc.rms(c[:, :rank], 1e-3) * gain, orc.rotate(c[:, rank:rank + rot], pos, 100.0, False)], 1)
    got = torch.stack([cache[int(table[1, p // PAGE]), p % PAGE] for p in pos])
    assert err(got[:, : rank + rot], want) < tol and not got[:, rank + rot:].any()


# -- attention in the latent space ------------------------------------------------------------

class LatentCase:
    """Cached rows of some sequences in shuffled pages full of other values, and queries."""

    def __init__(self, C, H, rank, rot, dt, batch, window, sink, seed=0, stand_out=None):
        self.C, self.H, self.rank, self.batch, self.dt = C, H, rank, batch, dt
        g = torch.Generator().manual_seed(seed)
        cols = self.cols = up(rank + rot, 64)
        ends = {s: st + n for s, st, n in batch.seqs}
        c = {s: randn(g, n, rank + rot, dt=dt) for s, n in ends.items()}
        q = randn(g, batch.T, H, rank + rot, dt=dt)
        if stand_out:
            stand_out(q, c)
        self.window, self.scale = window or ALL, 2.0 * (rank + rot) ** -0.5
        s = torch.linspace(-2.0, 5.0, H).double() if sink else None
        self.sink = None if s is None else cuda(s, F32)
        width = max(-(-n // PAGE) for n in ends.values()) + 1
        order = torch.randperm(3 * width + 1, generator=g).tolist()
        pool = randn(g, len(order), PAGE, cols) * 4
        self.table = torch.tensor(order[:-1], dtype=torch.int32).reshape(3, width)
        for k, rows in c.items():
            for j in range(len(rows)):
                pool[self.table[k, j // PAGE], j % PAGE] = 0
                pool[self.table[k, j // PAGE], j % PAGE, : rank + rot] = rows[j]
        self.pool, self.table = cuda(pool, dt), self.table.cuda()
        self.q = cuda(torch.nn.functional.pad(q, (0, cols - rank - rot)).reshape(batch.T, -1), dt)
        self.want = torch.cat([orc.attend(q[batch.rows(i)], c[k][:, None].expand(-1, H, -1), c[k][:, None, :rank].expand(-1, H, -1),
                                          self.scale, window, s, first=st) for i, (k, st, n) in enumerate(batch.seqs)])

    def decode(self, splits=1):
        b = self.batch
        return self.C.latent_decode(self.q, self.pool, self.table, b.tslot, b.tpos, self.H, self.window, self.scale, splits,
                                    self.rank, self.sink)

    def prefill(self):
        from llm_sharding_demo_amd.ops.hip import latent_tiles

        b = self.batch
        b.host_qlens = b.n
        tiles = latent_tiles(b, self.H, self.C.latent_tile_rows(self.cols)).cuda()
        return self.C.latent_prefill(self.q, self.pool, self.table, tiles, b.slots, b.start, b.cu, self.H, self.window,
                                     self.scale, self.rank, self.sink)

    def err(self, o):
        return err(o.reshape(self.batch.T, self.H, -1)[..., : self.rank], self.want)


@pytest.mark.parametrize("H,rank,rot", [(17, 40, 8), (3, 28, 20), (16, 96, 32), (5, 120, 64), (32, 128, 128), (16, 200, 64),
                                        (4, 250, 64), (20, 320, 64), (8, 384, 32), (33, 512, 64), (1, 64, 2), (2, 600, 64)])
@pytest.mark.parametrize("window,sink", [(None, False), (61, True), (1, True), (None, True)])
def test_latent_attention(C, H, rank, rot, window, sink):
    """Prompt and decode kernels on every number of cached columns, values all of
    them but the last or fewer; beyond those the kernel without MFMA."""
    c = LatentCase(C, H, rank, rot, BF, Batch((1, 30, 9), (0, 0, 70), (2, 129, 2)), window, sink)
    if C.latent_tile_rows(c.cols):
        assert c.err(c.prefill()) < 3e-2
    c = LatentCase(C, H, rank, rot, BF, Batch((1, 0, 1), (0, 150, 1), (2, 63, 1)), window, sink, seed=1)
    for splits in (1, 2, 4):
        assert c.err(c.decode(splits)) < 3e-2
    c = LatentCase(C, H, rank, rot, F32, Batch((1, 30, 3), (0, 64, 2)), window, sink, seed=2)
    assert c.err(c.decode()) < 1e-5


@pytest.mark.parametrize("rank,rot", [(40, 8), (128, 64), (512, 64)])
def test_latent_attention_edges(C, rank, rot):
    """One key stands out, by its latent or by its turned part: it decides the output
    at the window's last place and not one further, near and far."""
    H = 4
    for window in (1, 33, 64, 65, 100, None):
        for pos in (40, 64, 127, 128, 150, 700):
            edge = 0 if window is None else pos - window
            for key in {edge, edge + 1, pos, pos // 2}:
                if not 0 <= key <= pos:
                    continue

                def stand_out(q, c, key=key):
                    q.fill_(1.0)
                    for k in c:
                        c[k][:] *= 0.1
                        c[k][key, :rank] = 2.0
                        c[k][key, rank:] = 2.0
                seen = orc.visible(pos, key, window)
                for b in (Batch((1, pos, 1)), Batch((1, max(0, pos - 5), pos - max(0, pos - 5) + 1))):
                    c = LatentCase(C, H, rank, rot, BF, b, window, False, seed=pos, stand_out=stand_out)
                    outs = [c.prefill()] + ([c.decode(1), c.decode(3)] if b.T == 1 else [])
                    for o in outs:
                        o = o.reshape(b.T, H, -1)[-1, :, :rank].float()
                        assert (float(o.min()) > 1.0) == seen, (window, pos, key)


def test_latent_sinks(C):
    """A sink far above and far below every score, in each kernel."""
    for b in (Batch((1, 90, 1)), Batch((1, 0, 1)), Batch((1, 60, 40))):
        c = LatentCase(C, 4, 56, 8, BF, b, None, True)
        for value in (-1e4, -60.0, 0.0, 60.0, 1e4):
            s = torch.full((4,), value)
            c.sink = cuda(s, F32)
            outs = [c.prefill()] + ([c.decode(1), c.decode(2)] if b.T == 1 else [])
            for o in outs:
                assert torch.isfinite(o.float()).all()
                if value < 0:
                    c.sink = None
                    assert err(o, c.prefill().double().cpu()) < 2e-2
                    c.sink = cuda(s, F32)
                elif value > 0:
                    assert float(o.float().abs().max()) < 1e-3


@pytest.mark.parametrize("H,dim,vdim", [(2, 64, 64), (3, 128, 48), (4, 192, 128), (1, 192, 32), (5, 64, 128)])
@pytest.mark.parametrize("window", [None, 100, 1])
def test_expanded_attention(C, H, dim, vdim, window):
    """Per-head keys and values of the rows in reach, sinks and output gates."""
    g = torch.Generator().manual_seed(dim)
    seqs = [(37, 200), (0, 130), (300, 3)]  # (first position, queries)
    lo = [0 if window is None else max(0, st - window + 1) for st, _ in seqs]
    n = [st + q - a for (st, q), a in zip(seqs, lo)]
    cu_q, cu_k = [0], [0]
    for (_, q), k in zip(seqs, n):
        cu_q.append(cu_q[-1] + q)
        cu_k.append(cu_k[-1] + k)
    T, scale = cu_q[-1], dim ** -0.5
    q, k, v = randn(g, T, H, dim, dt=BF), randn(g, cu_k[-1], H, dim, dt=BF), randn(g, cu_k[-1], H, vdim, dt=BF)
    sink, gate = torch.linspace(-1, 3, H).double(), randn(g, T, H * vdim + 8)
    tiles = i32([[i, o] for i, (_, m) in enumerate(seqs) for o in range(0, m, 128)])
    flat = lambda t: cuda(t.reshape(t.shape[0], -1), BF)  # noqa: E731
    out = C.latent_expanded(flat(q), flat(k), flat(v), tiles, i32(cu_q), i32([s for s, _ in seqs]), i32(lo), i32(cu_k), H,
                            window or ALL, scale, cuda(sink, F32), cuda(gate, F32)[:, 8:])
    for i, (st, m) in enumerate(seqs):
        a, b = slice(cu_q[i], cu_q[i + 1]), slice(cu_k[i], cu_k[i + 1])
        want = orc.attend(q[a], k[b], v[b], scale, window, sink, first=st - lo[i]).reshape(m, -1)
        assert err(out[a], want * orc.sigmoid(gate[a, 8:])) < 3e-2


# -- recurrence with forget gates ----------------------------------------------------------------

class ForgetCase:
    def __init__(self, C, H, D, V, dt, n, fast=2.0, seed=0):
        self.C, self.dims, self.dt, self.n, self.eps = C, (H, D, V), dt, n, 1e-4
        g = torch.Generator().manual_seed(seed)
        self.y = randn(g, n, H * (2 * D + V), dt=dt)
        self.bias = torch.linspace(-fast, 9, H * D)[torch.randperm(H * D, generator=g)].double()
        self.lower = torch.rand(H * D, generator=g).double() * 0.9 * (torch.rand(H * D, generator=g) < 0.5)
        self.norm = randn(g, V)
        q, z, v = self.y.split([H * D, H * D, H * V], 1)
        f = orc.forget_gates(z + self.bias, self.lower)
        o, self.S = orc.recurrence(orc.silu(q).reshape(n, H, D), f.reshape(n, H, D), v.reshape(n, H, V))
        self.want = (orc.rms(o, self.eps) * self.norm).reshape(n, -1)

    def state(self, slots=3):
        H, D, V = self.dims
        return torch.full((slots, H, D, up(V, 4)), float("nan"), device="cuda")

    def consts(self):
        H, D, V = self.dims
        return (H, D, V, *(cuda(t, F32) for t in (self.bias, self.lower, self.norm)), self.eps)

    def run(self, parts, segs=1, slot=1, chunked=True):
        H, D, V = self.dims
        S, out = self.state(), []
        for a, b in parts:
            y = cuda(torch.nn.functional.pad(self.y[a:b], (0, up(self.y.shape[1], 8) - self.y.shape[1])), self.dt)
            o = torch.full((b - a, up(H * V, 64)), float("nan"), dtype=self.dt, device="cuda")
            self.C.forget_seq(y, i32([slot]), i32([a]), i32([0, b - a]), *self.consts(), S, o, chunked and b - a > 1, segs)
            assert not o[:, H * V:].any()
            out.append(o[:, : H * V])
        return torch.cat(out), S[slot, ..., :V]


@pytest.mark.parametrize("H,D,V", [(2, 24, 20), (1, 32, 64), (3, 16, 36), (2, 64, 128), (2, 128, 64), (1, 128, 128), (1, 2, 4),
                                   (1, 7, 5), (1, 40, 200), (1, 200, 24)])
@DTYPES
def test_recurrence(C, H, D, V, dt):
    """Token by token and in chunks, in portions down to two tokens, in segments."""
    n = 150
    c = ForgetCase(C, H, D, V, dt, n)
    tol = 2e-2 if dt == BF else 3e-5
    ok = dt == BF and C.forget_ok(D, V)
    for sizes in ([n], [1] * n, [63, 1, 2, 60, 24], [2] * 75, [33, 32, 31, 54]):
        for chunked in ((False, True) if ok else (False,)):
            if chunked or len(sizes) < 70:
                o, S = c.run(portions(n, sizes), chunked=chunked)
                assert err(o, c.want) < tol and err(S, c.S) < (2e-3 if chunked else 3e-5), (sizes, chunked)
    if ok:
        for segs in (2, 3, 5, 16):
            for sizes in ([n], [40, 110], [100, 2, 48]):
                o, S = c.run(portions(n, sizes), segs)
                assert err(o, c.want) < tol and err(S, c.S) < 2e-3, (segs, sizes)


@pytest.mark.parametrize("fast", [2.0, 12.0, 40.0, 120.0])
def test_recurrence_that_forgets_fast(C, fast):
    """Gates that fall by more than a chunk's range take shorter chunks."""
    c = ForgetCase(C, 2, 64, 64, BF, 100, fast=fast)
    c.lower *= 0
    H, D, V = c.dims
    q, z, v = c.y.split([H * D, H * D, H * V], 1)
    o, S = orc.recurrence(orc.silu(q).reshape(-1, H, D), orc.sigmoid(z + c.bias).reshape(-1, H, D), v.reshape(-1, H, V))
    want = (orc.rms(o, c.eps) * c.norm).reshape(100, -1)
    for segs in (1, 3):
        got, s = c.run([(0, 100)], segs)
        assert err(got, want) < 2e-2 and err(s, S) < 2e-3


def test_recurrence_of_a_mixed_batch(C):
    """Ragged sequences in one launch, continued in their slots, also in segments."""
    cases = [ForgetCase(C, 2, 32, 32, BF, n, seed=n) for n in (100, 7, 260)]
    for c in cases[1:]:  # one set of constants
        c.bias, c.lower, c.norm = cases[0].bias, cases[0].lower, cases[0].norm
    H, D, V = 2, 32, 32
    for segs in (1, 4):
        S, out = cases[0].state(), [[], [], []]
        for step in ([(2, 0, 201), (0, 0, 64), (1, 0, 3)], [(0, 64, 36), (2, 201, 59), (1, 3, 4)]):
            b = Batch(*step)
            y = cuda(torch.cat([cases[s].y[a:a + n] for s, a, n in step]), BF)
            o = torch.empty(b.T, H * V, dtype=BF, device="cuda")
            C.forget_seq(y, b.slots, b.start, b.cu, *cases[0].consts(), S, o, True, segs)
            for i, (s, _, _) in enumerate(step):
                out[s].append(o[b.rows(i)])
        for s, c in enumerate(cases):
            q, z, v = c.y.split([H * D, H * D, H * V], 1)
            f = orc.forget_gates(z + c.bias, c.lower)
            o, _ = orc.recurrence(orc.silu(q).reshape(-1, H, D), f.reshape(-1, H, D), v.reshape(-1, H, V))
            assert err(torch.cat(out[s]), (orc.rms(o, c.eps) * c.norm).reshape(len(o), -1)) < 2e-2


# -- whole models ------------------------------------------------------------------

def odd_sizes():
    """Nothing a multiple of a tile, every mixer, layers of several shapes, one
    without a feed-forward, one without a shared expert."""
    return orc.config([orc.forget(), orc.full(), orc.windowed(), orc.forget(heads=1, dim=15, vdim=37, experts=0),
                       orc.full(heads=1, dim=10, rot_dim=2, vdim=7, kv_rank=21, experts=3, top=3, shared=0),
                       orc.windowed(heads=4, dim=8, rot_dim=16, vdim=12, kv_rank=24, q_rank=27, size=9, base=50.0)],
                      loop=(1, 3, 2))


def tile_sizes():
    """Sizes of the fused paths, GEMM-aligned width."""
    return orc.config([orc.windowed(heads=16, dim=64, rot_dim=64, vdim=64, kv_rank=192, q_rank=128, scale=0.09, size=100,
                                    experts=8, top=2, ff=128, shared=64),
                       orc.forget(heads=4, dim=64, vdim=64, experts=4, top=2, ff=64, shared=128),
                       orc.full(heads=8, dim=32, rot_dim=32, vdim=32, kv_rank=64, scale=0.125, experts=8, top=4, ff=64,
                                shared=64),
                       orc.forget(heads=2, dim=128, vdim=128, experts=8, top=1, ff=64, shared=64)],
                      width=128, vocab=320, side=64, loop=(0, 2, 2))


def large_heads():
    """Sizes beyond the MFMA kernels: latents over 576 columns, states over 128, expanded heads over 192."""
    return orc.config([orc.full(heads=2, dim=200, rot_dim=24, vdim=140, kv_rank=600, scale=0.07, experts=70, top=2, ff=16),
                       orc.forget(heads=2, dim=136, vdim=140, experts=2, top=1),
                       orc.windowed(heads=35, dim=6, rot_dim=2, vdim=4, kv_rank=580, q_rank=200, size=64)], width=72, side=70)


def open_model(tmp_path, cfg, dtype, seed=0, **kw):
    from llm_sharding_demo_amd.runtime.engine import Engine

    w = orc.random_weights(cfg, seed)
    orc.save(str(tmp_path), cfg, w)
    kw = {"max_batch": 4, "max_seq_len": 640, "kv_tokens": 1280, **kw}
    return w, Engine(EngineConfig(model_id=str(tmp_path), weights=str(tmp_path), dtype=dtype, device="cuda", **kw))


LIMIT = {"bf16": 0.1, "fp32": 2e-4}


def check_logits(got, want, dtype):
    """Nearly all rows are within rounding; a router's close call may move a few of a bf16 model's."""
    d = got.double() - want
    e = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()
    if dtype == "fp32":
        assert float(e.max()) < LIMIT[dtype]
    else:
        assert float((e > LIMIT[dtype]).double().mean()) < 0.06 and float(e.median()) < 0.5 * LIMIT[dtype], e.topk(8)


@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
@pytest.mark.parametrize("make", [odd_sizes, tile_sizes, large_heads])
def test_model_portions(tmp_path, dtype, make):
    """Whole prompts, pairs, single tokens and uneven portions give the same logits."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    cfg = make()
    w, eng = open_model(tmp_path, cfg, dtype)
    ses, ids = TraceSession(eng), ids_of(150)
    want = orc.forward(cfg, w, ids)
    for sizes in ([150], [2] * 75, [1] * 150, [63, 1, 2, 60, 24], [7, 130, 13], [16, 17, 32, 33, 3, 5]):
        check_logits(run_steps(ses, {"a": ids}, portion_steps("a", 150, sizes))["a"], want, dtype)
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
        check_logits(torch.cat([got[k] for k in seqs]), torch.cat([want[k] for k in seqs]), dtype)
        assert not ses.live and eng.page_pools[0].available == 6 and eng.slots.available == 4


@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
def test_model_long_sequence(tmp_path, dtype):
    """Several windows and pages of prompt, then long decoding past them."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    cfg = tile_sizes()
    w, eng = open_model(tmp_path, cfg, dtype, seed=4)
    ids = ids_of(520, vocab=320, seed=9)
    got = run_steps(TraceSession(eng), {"a": ids}, portion_steps("a", 520, [370]))["a"]
    check_logits(got, orc.forward(cfg, w, ids), dtype)


@pytest.mark.parametrize("make", [odd_sizes, tile_sizes, large_heads])
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
    assert len(rows) == len(want) == len(orc.runs(cfg))
    for got, x in zip(rows, want):
        assert err(got, x) < 2e-4


def near_greedy(cfg, w, prompt, out, tol):
    """Every generated token is the plain model's best behind what came before, up to `tol` of the logits' spread."""
    lg = orc.forward(cfg, w, prompt + out[:-1])[len(prompt) - 1:]
    best, got = lg.max(-1).values, lg[torch.arange(len(out)), torch.tensor(out)]
    return float((best - got).max()) <= tol * float(lg.std())


@pytest.mark.parametrize("dtype,tol", [("bf16", 0.3), ("fp32", 1e-3)])
@pytest.mark.parametrize("make,kw", [(odd_sizes, {}), (odd_sizes, {"num_microbatches": 2, "prefill_chunk": 20}),
                                     (odd_sizes, {"use_graphs": False}), (odd_sizes, {"kv_tokens": 5 * PAGE, "max_batch": 3}),
                                     (tile_sizes, {}), (large_heads, {})])
def test_model_greedy_generation(tmp_path, dtype, tol, make, kw):
    """Through the scheduler, with captured decode graphs, sessions repeated in
    used slots and pages."""
    cfg = make()
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


@pytest.mark.parametrize("split", [2, 5])
@pytest.mark.parametrize("transport", ["loopback", "devloop"])
def test_model_two_stages(tmp_path, transport, split):
    """Boundaries inside and behind the loop, and the compat forwards across them."""
    cfg = odd_sizes()
    w, eng = open_model(tmp_path, cfg, "bf16", num_stages=2, split_points=[split], transport=transport)
    prompts = [ids_of(n, seed=n) for n in (30, 5, 66)]
    for _ in range(2):
        out = eng.generate_ids(prompts, SamplingParams(greedy=True, max_new_tokens=8))
        assert all(len(o) == 8 and near_greedy(cfg, w, p, o, 0.3) for p, o in zip(prompts, out))
    hid = eng.forward_a(prompts[0])
    assert hid.shape == (30, 88 + 3)
    check_logits(eng.forward_b(hid).cpu(), orc.forward(cfg, w, prompts[0]), "bf16")
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
    assert all(len(o) == s.max_new_tokens and near_greedy(cfg, w, p, o, 0.3) for p, s, o in zip(prompts, sp, out))
