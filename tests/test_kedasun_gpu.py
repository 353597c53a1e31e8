"""Kedasun kernels and whole models on the GPU against the plain model of
kedasun_oracle.py: bf16 kernels with inputs rounded to bf16 first, fp32 ones at
fp32 accuracy."""
from __future__ import annotations

import pytest
import torch

from llm_sharding_demo_amd.config import EngineConfig, SamplingParams
from llm_sharding_demo_amd.runtime.kv_cache import PAGE

from . import kedasun_oracle as orc
from .paged_helpers import (BF, F32, Batch, cuda, err, i32, ids_of, logit_err, pools, portion_steps, portions, rounded,
                            run_steps, up)

pytestmark = pytest.mark.gpu
ALL = 1 << 30


@pytest.fixture(scope="module")
def C():
    from llm_sharding_demo_amd.ops.hip import _load

    return _load()


# -- grouped norms -----------------------------------------------------------------

@pytest.mark.parametrize("width,groups", [(88, 4), (88, 1), (90, 6), (96, 3), (256, 4), (1024, 1), (2048, 4), (3000, 2),
                                          (4096, 4), (4096, 1), (8192, 1), (96, 96)])
@pytest.mark.parametrize("dt", [BF, F32])
def test_norms_around_a_sublayer(C, width, groups, dt):
    g = torch.Generator().manual_seed(width + groups)
    H, eps, tol = up(width, 64), 1e-3, 2e-2 if dt == BF else 1e-5
    f32 = dt == F32

    def vec():
        return rounded(torch.randn(width, generator=g), dt)

    def dev(t, dt=dt):
        return cuda(torch.nn.functional.pad(t, (0, H - width)), dt)
    for T, S, sdt in ((1, 0, None), (3, 1, F32), (70, 1, dt), (5, 4, dt), (2, 7, dt), (700, 2, dt), (9, 9, F32)):
        x = rounded(torch.randn(T, width, generator=g) * torch.linspace(0.2, 4, width), F32)
        w1, w2, b = vec(), vec(), vec()
        args, want = (None, None, None), x
        if S:
            s = rounded(torch.randn(S, T, width, generator=g), sdt)
            bias = b if T % 2 else None
            want = x + orc.group_norm(s.sum(0) + (bias if bias is not None else 0), w1, groups, eps)
            args = (dev(s, sdt), None if bias is None else dev(bias), dev(w1))
        xd = dev(x, F32)
        out = C.group_norm(xd, groups, width, eps, *args, dev(w2), None, f32)
        assert err(xd[:, :width], want) < 1e-5 and not xd[:, width:].any()
        assert err(out[:, :width], orc.group_norm(want, w2, groups, eps)) < tol and not out[:, width:].any()
        if S:  # the residual alone
            xd = dev(x, F32)
            assert C.group_norm(xd, groups, width, eps, *args, None, None, f32) is None
            assert err(xd[:, :width], want) < 1e-5
        rows = [T - 1, 0]
        out = C.group_norm(dev(x, F32), groups, width, eps, None, None, None, dev(w2), i32(rows), f32)
        assert err(out[:, :width], orc.group_norm(x[rows], w2, groups, eps)) < tol


# -- in front of the scores ----------------------------------------------------------

HEADS = [(6, 2, 40, 24), (4, 4, 16, 20), (3, 1, 96, 72), (16, 4, 128, 128), (2, 2, 64, 256), (1, 1, 200, 16)]


class AppendCase:
    """In-projection rows of one sequence (shuffled pages), and what should become of them."""

    def __init__(self, C, H, G, D, V, dt, T, taps=0, norm=False, rot=0, lam=None, seed=0):
        self.C, self.dims, self.dt, self.n = C, (H, G, D, V), dt, taps
        g = torch.Generator().manual_seed(seed)
        R = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
        dp, vp = up(D, 32), up(V, 16)
        self.dp, self.vp, self.eps, self.lam = dp, vp, 1e-3 if norm else -1.0, lam
        x = {n: rounded(R(T, h, d), dt) for n, h, d in (("q", H, D), ("k", G, D), ("v", G, V))}
        pads = {"q": dp, "k": dp, "v": vp}
        pad = lambda n, t: torch.nn.functional.pad(t, (0, pads[n] - t.shape[-1]))  # noqa: E731
        y = torch.cat([pad(n, x[n]).reshape(T, -1) for n in "qkv"], 1)
        self.ch = y.shape[1]
        self.y = torch.nn.functional.pad(y, (0, up(self.ch + H, 64) - self.ch)).to(dt)
        w = {n: rounded(R(x[n].shape[1], x[n].shape[2], taps), F32) for n in "qkv"} if taps else None
        if taps:
            x = {n: orc.short_conv(x[n].reshape(T, -1), w[n].reshape(-1, taps)).reshape(x[n].shape) for n in "qkv"}
            self.taps = cuda(torch.cat([pad(n, w[n].transpose(1, 2)).transpose(1, 2).reshape(-1, taps) for n in "qkv"]).T, F32)
            self.ring = torch.full((3, taps, self.ch), float("nan"), dtype=dt, device="cuda")
        if norm:
            x["q"], x["k"] = orc.rms(x["q"], self.eps), orc.rms(x["k"], self.eps)
        self.rope = None
        if rot:  # the kernels turn pairs (i, i + rot / 2): order the oracle's dimensions so
            from llm_sharding_demo_amd.config import RopeSpec
            from llm_sharding_demo_amd.ops.hip import rope_spec_table, split_pairs

            order = split_pairs(D, rot)
            back = torch.argsort(order)
            for n in "qk":
                x[n] = orc.rotate(x[n][..., back], range(T), rot, 500.0)[..., order]
            self.rope = rope_spec_table(RopeSpec(rot, 500.0), 1024, "cuda")
        self.own = x["v"]
        if lam is not None:
            first = rounded(R(T, G, V), dt)
            x["v"] = orc.mix_values(x["v"], first, lam)
            self.first = pad("v", first).reshape(T, -1).to(dt)
        self.want = x
        self.table = torch.randperm(3 * 16, generator=g).to(torch.int32).reshape(3, 16)
        self.K = torch.zeros(49, G, PAGE, dp, dtype=dt, device="cuda")
        self.V = torch.zeros(49, G, PAGE, vp, dtype=dt, device="cuda")

    def run(self, parts, slot=1):
        H, G, D, V = self.dims
        qs, vs = [], []
        for a, b in parts:
            y, seq = cuda(self.y[a:b]), (i32([slot]), i32([a]), i32([0, b - a]))
            single = b - a == 1
            vout = torch.empty(b - a, G * self.vp, dtype=self.dt, device="cuda")
            first = cuda(self.first[a:b]) if self.lam is not None else None
            q = self.C.rope_append(y, H, self.K, self.V, cuda(self.table), i32([slot] * (b - a)), i32(list(range(a, b))),
                                   self.rope, 1.0, self.taps if self.n else None, self.ring if self.n else None, single,
                                   self.eps, D, first, self.lam or 0.0, vout)
            if self.n and not single:
                self.C.conv_tail(y, self.ring, *seq)
            qs.append(q.reshape(-1, H, self.dp))
            vs.append(vout.reshape(-1, G, self.vp))
        return torch.cat(qs), torch.cat(vs)

    def check(self, q, v, slot=1):
        H, G, D, V = self.dims
        T, tol = q.shape[0], 3e-2 if self.dt == BF else 2e-5
        pos = torch.arange(T)
        pg = self.table[slot, pos // PAGE].long().cuda()
        k, vv = (p[pg, :, pos.cuda() % PAGE] for p in (self.K, self.V))
        for got, want, d in ((q, self.want["q"], D), (k, self.want["k"], D), (vv, self.want["v"], V), (v, self.own, V)):
            assert err(got[..., :d], want) < tol
            assert not got[..., d:].any()


@pytest.mark.parametrize("H,G,D,V", HEADS)
@pytest.mark.parametrize("taps,norm,lam", [(4, True, 0.3), (3, True, None), (1, False, 0.7), (2, True, 0.5), (6, True, 0.4)])
@pytest.mark.parametrize("dt", [BF, F32])
def test_convolution_norm_and_append(C, H, G, D, V, taps, norm, lam, dt):
    """Whole, in uneven portions down to two tokens, and token by token."""
    for sizes in ([100], [1] * 100, [2] * 50, [63, 1, 2, 30, 4], [3, 5, 1, 1, 90]):
        c = AppendCase(C, H, G, D, V, dt, 100, taps, norm, lam=lam)
        c.check(*c.run(portions(100, sizes)))


@pytest.mark.parametrize("H,G,D,V", HEADS)
@pytest.mark.parametrize("rot,lam", [(8, None), (16, 0.3)])
@pytest.mark.parametrize("dt", [BF, F32])
def test_rotation_value_mixing_and_append(C, H, G, D, V, rot, lam, dt):
    c = AppendCase(C, H, G, D, V, dt, 70, rot=rot, lam=lam)
    c.check(*c.run([(0, 66), (66, 67), (67, 70)]))


def test_convolution_of_a_mixed_batch(C):
    """Decoded rows of some sequences in front of portions of others; long runs of rows."""
    H, G, D, V, taps = 4, 2, 64, 64, 4
    cases = [AppendCase(C, H, G, D, V, BF, n, taps, True, seed=s) for s, n in enumerate((41, 9, 5000))]
    K, Vp, ring = torch.zeros(100, G, PAGE, D, dtype=BF, device="cuda"), torch.zeros(100, G, PAGE, V, dtype=BF, device="cuda"), \
        torch.full((3, taps, cases[0].ch), float("nan"), dtype=BF, device="cuda")
    table = torch.randperm(99).to(torch.int32)[:3 * 33].reshape(3, 33)
    table = torch.cat([table, torch.full((3, 60), 99, dtype=torch.int32)], 1)
    table[2, :80] = torch.arange(80, dtype=torch.int32)
    table[0, :1], table[1, :1] = 90, 91
    w = cases[0].taps
    out = [[], [], []]
    for step in ([(0, 0, 40), (1, 0, 7)], [(0, 40, 1), (2, 0, 4990), (1, 7, 2)], [(2, 4990, 10)]):
        b = Batch(*step)
        y = cuda(torch.cat([cases[s].y[a:a + n] for s, a, n in step]))
        q = C.rope_append(y, H, K, Vp, cuda(table), b.tslot, b.tpos, None, 1.0, w, ring, False, 1e-3, D, None, 0.0, None)
        C.conv_tail(y, ring, b.slots, b.start, b.cu)
        for i, (s, _, _) in enumerate(step):
            out[s].append(q[b.rows(i)])
    for s, c in enumerate(cases):
        x = c.y[:, : H * D].double()
        want = orc.rms(orc.short_conv(x, w[:, : H * D].T.double().cpu()).reshape(-1, H, D), 1e-3)
        assert err(torch.cat(out[s]).reshape(-1, H, D), want) < 3e-2


# -- attention ---------------------------------------------------------------------

SIZES = [(6, 2, 40, 24), (4, 4, 16, 20), (3, 1, 96, 72), (16, 4, 128, 128), (12, 12, 32, 64), (32, 8, 64, 128),
         (20, 5, 128, 48), (1, 1, 64, 16), (8, 1, 128, 128), (24, 3, 72, 96)]
WINDOWS = [(None, 0), (67, 5), (1, 0), (32, 70), (5, 200), (64, 64)]


class AttentionCase:
    def __init__(self, C, H, G, D, V, dt, batch, window, keep, talk=True, biased=True, gated=True, seed=0, stand_out=None):
        self.C, self.batch, self.dims, self.dt = C, batch, (H, G, D, V), dt
        g = torch.Generator().manual_seed(seed)
        ends = {s: st + n for s, st, n in batch.seqs}
        k = {s: rounded(torch.randn(n, G, D, generator=g), dt) for s, n in ends.items()}
        v = {s: rounded(torch.randn(n, G, V, generator=g), dt) for s, n in ends.items()}
        q = rounded(torch.randn(batch.T, H, D, generator=g) * 2.0, dt)
        t = rounded(torch.eye(H) + torch.randn(H, H, generator=g) * 0.5, BF) if talk else None
        if stand_out:
            stand_out(q, k, v)
        slope = orc.slopes(H) if biased else None
        logits = rounded(torch.randn(batch.T, H, generator=g), dt)
        self.want = torch.cat([orc.attend(q[batch.rows(i)], k[s], v[s], D ** -0.5, window, keep, slope, t, first=st)
                               for i, (s, st, n) in enumerate(batch.seqs)])
        if gated:
            self.want = self.want * orc.sigmoid(logits)[:, :, None]
        dp, vp = up(D, 32), up(V, 16)
        K, Vp, table = pools(k, v, dt, dp, vp)
        qp = torch.zeros(batch.T, H, dp, dtype=dt)
        qp[..., :D] = q.to(dt)
        self.at = (cuda(qp.reshape(batch.T, -1)), K, Vp, table)
        self.window, self.scale, self.keep = window or ALL, D ** -0.5, keep
        self.slopes = cuda(torch.tensor(slope), F32) if biased else None
        wide = torch.zeros(batch.T, 64 + H, dtype=dt)  # gate logits behind other columns
        wide[:, 64:] = logits.to(dt)
        self.gate = cuda(wide)[:, 64:] if gated else None
        self.talk = None if t is None else cuda(t, F32)

    def out(self):
        H, _, _, V = self.dims
        return torch.full((self.batch.T, up(H * up(V, 16), 64)), float("nan"), dtype=self.dt, device="cuda")

    def err(self, out):
        H, _, _, V = self.dims
        vp = up(V, 16)
        assert not out[:, H * vp:].any()
        return err(out[:, : H * vp].reshape(-1, H, vp)[..., :V], self.want)

    @property
    def beside(self):
        return self.keep, self.slopes, self.gate

    def plain(self):
        b, out = self.batch, self.out()
        self.C.talk_plain(*self.at, b.tslot, b.tpos, self.talk, self.window, self.scale, 0.0, out, *self.beside,
                          self.talk is not None)
        return out

    def prefill(self, qt, splits=1):
        b, out, C = self.batch, self.out(), self.C
        seqs = (b.slots, b.start, b.cu)
        head = (b.tiles(64 * qt), qt, *seqs, self.window, self.scale, *self.beside, out)
        if self.talk is None:
            C.paged_prefill(*self.at, *head)
            return out
        H, G, _, _ = self.dims
        lse = torch.full((b.T, H), float("nan"), device="cuda")
        C.paged_prefill(*self.at, *head, lse)
        hp = C.talk_heads(H, G, self.at[1].shape[3], self.at[2].shape[3], -1.0)
        frag = torch.zeros(hp, hp, dtype=torch.float16, device="cuda")
        frag[:H, :H] = self.talk.half()
        C.mix_prefill(*self.at, frag, b.tiles(C.talk_tile(hp)), *seqs, self.window, self.scale, *self.beside, lse, splits,
                      out)
        return out

    def decode(self, splits):
        b, out = self.batch, self.out()
        if self.talk is None:
            self.C.paged_decode(*self.at, b.slots, b.tpos, self.window, self.scale, *self.beside, splits, out)
        else:
            self.C.mix_decode(*self.at, self.talk, b.slots, b.tpos, self.window, self.scale, *self.beside, splits, out)
        return out


@pytest.mark.parametrize("H,G,D,V", SIZES)
@pytest.mark.parametrize("window,keep", WINDOWS)
@pytest.mark.parametrize("talk", [False, True])
def test_attention_plain(C, H, G, D, V, window, keep, talk):
    b = Batch((1, 0, 3), (2, 70, 2), (0, 130, 1))
    for dt, tol in ((BF, 3e-2), (F32, 2e-5)):
        c = AttentionCase(C, H, G, D, V, dt, b, window, keep, talk)
        assert c.err(c.plain()) < tol


@pytest.mark.parametrize("H,G,D,V", SIZES)
@pytest.mark.parametrize("window,keep", WINDOWS)
@pytest.mark.parametrize("talk", [False, True])
def test_attention_prefill(C, H, G, D, V, window, keep, talk):
    b = Batch((1, 0, 140), (2, 70, 2), (0, 130, 33))
    c = AttentionCase(C, H, G, D, V, BF, b, window, keep, talk)
    for qt, splits in ((1, 1), (2, 3)):
        assert c.err(c.prefill(qt, splits)) < 3e-2


@pytest.mark.parametrize("H,G,D,V", SIZES)
@pytest.mark.parametrize("window,keep", WINDOWS)
@pytest.mark.parametrize("talk", [False, True])
def test_attention_decode(C, H, G, D, V, window, keep, talk):
    if talk and not C.mix_decode_ok(H, G):
        pytest.skip("decoded by the prompt kernels")
    b = Batch((1, 0, 1), (2, 63, 1), (0, 300, 1))
    c = AttentionCase(C, H, G, D, V, BF, b, window, keep, talk)
    for splits in (1, 2, 3, 17):
        assert c.err(c.decode(splits)) < 3e-2


def test_attention_without_bias_and_gate(C):
    for talk in (False, True):
        c = AttentionCase(C, 8, 2, 64, 64, BF, Batch((1, 0, 90), (0, 70, 5)), 40, 3, talk, biased=False, gated=False)
        assert c.err(c.plain()) < 3e-2 and c.err(c.prefill(1)) < 3e-2
        c = AttentionCase(C, 8, 2, 64, 64, BF, Batch((1, 90, 1)), 40, 3, talk, biased=False, gated=False)
        assert c.err(c.decode(2)) < 3e-2


@pytest.mark.parametrize("talk", [False, True])
def test_attention_edges(C, talk):
    """One key stands out: it decides the output at the window's last place and not
    one further, among the kept tokens and not one behind them, near and far."""
    H, G, D, V = 8, 2, 32, 32
    for window, keep in ((1, 0), (33, 3), (64, 1), (65, 64), (100, 65)):
        for pos in (40, 64, 127, 128, 150, 700):
            for key in {pos - window, pos - window + 1, keep - 1, keep, pos, pos // 2}:
                if not 0 <= key <= pos:
                    continue

                def stand_out(q, k, v, key=key):
                    q.fill_(1.0)  # every head's score with that key is 2 sqrt(D) > 11, others are around zero
                    for s in k:
                        k[s][key] = 2.0
                        v[s][key] = 20.0
                c = AttentionCase(C, H, G, D, V, BF, Batch((1, pos, 1)), window, keep, False, biased=False, gated=False,
                                  seed=pos, stand_out=stand_out)
                if talk:  # mixing that changes nothing
                    c.talk = torch.eye(H, device="cuda")
                seen = orc.visible(pos, key, window, keep)
                for o in (c.plain(), c.prefill(1), c.decode(1), c.decode(3)):
                    assert (float(o[0, : H * V].float().min()) > 10) == seen, (pos, key, window, keep)
                    assert c.err(o) < 3e-2


def test_attention_weight_mixing(C):
    """A permutation of the heads sends head g's weights to head g + 1, on the values
    of that head's own group."""
    H, G, D, V = 16, 4, 64, 64
    for b in (Batch((1, 90, 20)), Batch((1, 90, 1))):
        c = AttentionCase(C, H, G, D, V, BF, b, None, 0, True, gated=False)
        c.talk = torch.roll(torch.eye(H), 1, 0).cuda()
        outs = [c.plain(), c.prefill(1)] + ([c.decode(2)] if b.T == 1 else [])
        for o in outs[1:]:
            assert err(o, outs[0].double().cpu()) < 3e-2
        c.talk = torch.eye(H, device="cuda")
        assert err(c.plain(), outs[0].double().cpu()) > 0.3


def test_clamped_gate(C):
    """Split-K, tiled and GEMV rows, and the fp32 kernel."""
    from llm_sharding_demo_amd.ops.hip import HipBackend, interleave_experts

    be = HipBackend()
    be._counters = torch.zeros(8, 1 << 16, dtype=torch.int32, device="cuda")
    g = torch.Generator().manual_seed(0)
    for M in (1, 3, 8, 40, 200, 700):
        h, w = rounded(torch.randn(M, 128, generator=g), BF), rounded(torch.randn(2 * 192, 128, generator=g) * 0.2, BF)
        t = {"gate": w[:192], "up": w[192:], "down": torch.eye(192, dtype=torch.float64)}
        want = orc.feed_forward(h, lambda n: t[n], 1.25)
        be.decode = M <= 200
        be.fp32 = False
        assert err(be.clamped_glu(cuda(h, BF), interleave_experts(cuda(w, BF), 192, 128), 1.25), want) < 3e-2
        be.fp32 = True
        assert err(be.clamped_glu(cuda(h, F32), interleave_experts(cuda(w, F32), 192, 128), 1.25), want) < 1e-5


# -- whole models ------------------------------------------------------------------

def odd_sizes():
    """Nothing a multiple of a tile, both mixers, layers of several shapes, one
    without a feed-forward, one that keeps its own values."""
    mixed = dict(kv_heads=2, vdim=24)
    return orc.config([orc.full(v_mix=False, heads=3, kv_heads=1, dim=16, vdim=20, rot=6), orc.windowed(**mixed),
                       orc.full(**mixed), orc.windowed(heads=4, dim=16, conv=1, size=9, keep=0, ff=0, **mixed),
                       orc.full(heads=2, dim=8, rot=0, ff=24, limit=7.0, **mixed),
                       orc.windowed(v_mix=False, heads=3, kv_heads=3, dim=8, vdim=12, conv=5, size=33, keep=70)])


def tile_sizes():
    """Sizes of the fused paths, GEMM-aligned width."""
    mixed = dict(kv_heads=4, vdim=64)
    return orc.config([orc.windowed(heads=16, dim=64, conv=4, size=100, keep=4, ff=128, scale=0.125, **mixed),
                       orc.full(heads=8, dim=128, rot=64, scale=0.09, ff=192, **mixed),
                       orc.windowed(heads=20, dim=32, conv=2, size=64, keep=65, ff=64, **mixed),
                       orc.full(heads=4, dim=64, rot=64, scale=0.125, v_mix=False, kv_heads=4, vdim=16, ff=128)],
                      width=128, vocab=320, groups=2)


def many_heads():
    """Head counts beyond the MFMA kernels of mixed weights (decode, prompts), and
    more than 16 query heads per K / V head."""
    return orc.config([orc.windowed(heads=20, kv_heads=20, dim=16, vdim=16, scale=0.25, v_mix=False),
                       orc.windowed(heads=40, kv_heads=8, dim=16, vdim=16, scale=0.25, v_mix=False),
                       orc.full(heads=20, kv_heads=1, dim=16, vdim=16, rot=8, scale=0.25, v_mix=False),
                       orc.windowed(heads=2, kv_heads=1, dim=144, vdim=136, scale=0.1, v_mix=False),
                       orc.full(heads=2, kv_heads=1, dim=144, vdim=136, scale=0.1, v_mix=False)], groups=1)


def open_model(tmp_path, cfg, dtype, seed=0, **kw):
    from llm_sharding_demo_amd.runtime.engine import Engine

    w = orc.random_weights(cfg, seed)
    orc.save(str(tmp_path), cfg, w)
    kw = {"max_batch": 4, "max_seq_len": 640, "kv_tokens": 1280, **kw}
    return w, Engine(EngineConfig(model_id=str(tmp_path), weights=str(tmp_path), dtype=dtype, device="cuda", **kw))


LIMIT = {"bf16": 0.08, "fp32": 5e-5}


@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
@pytest.mark.parametrize("make", [odd_sizes, tile_sizes, many_heads])
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
    """The residual after every layer, in fp32."""
    from llm_sharding_demo_amd.runtime.trace import TraceSession

    cfg = make()
    w, eng = open_model(tmp_path, cfg, "fp32")
    st, rows, want = eng.stages[0], [], []
    fwd = st.forward
    st.forward = lambda *a, **k: fwd(*a, residuals=rows, **k)
    ids = ids_of(40)
    TraceSession(eng).step([{"id": "a", "tokens": ids, "want": [39]}], ["a"])
    orc.forward(cfg, w, ids, want)
    assert len(rows) == len(want) == len(cfg["layers"])
    for got, x in zip(rows, want):
        assert err(got, x) < 2e-5


def near_greedy(cfg, w, prompt, out, tol):
    """Every generated token is the plain model's best behind what came before, up to `tol` of the logits' spread."""
    lg = orc.forward(cfg, w, prompt + out[:-1])[len(prompt) - 1:]
    best, got = lg.max(-1).values, lg[torch.arange(len(out)), torch.tensor(out)]
    return float((best - got).max()) <= tol * float(lg.std())


@pytest.mark.parametrize("dtype,tol", [("bf16", 0.15), ("fp32", 1e-3)])
@pytest.mark.parametrize("make,kw", [(odd_sizes, {}), (odd_sizes, {"num_microbatches": 2, "prefill_chunk": 20}),
                                     (odd_sizes, {"use_graphs": False}), (odd_sizes, {"kv_tokens": 5 * PAGE, "max_batch": 3}),
                                     (tile_sizes, {}), (many_heads, {})])
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


@pytest.mark.parametrize("split", [1, 3])
@pytest.mark.parametrize("transport", ["loopback", "devloop"])
def test_model_two_stages(tmp_path, transport, split):
    """Boundaries in front of and behind the layer whose values others mix in, and
    the compat forwards across them."""
    cfg = odd_sizes()
    w, eng = open_model(tmp_path, cfg, "bf16", num_stages=2, split_points=[split], transport=transport)
    prompts = [ids_of(n, seed=n) for n in (30, 5, 66)]
    for _ in range(2):
        out = eng.generate_ids(prompts, SamplingParams(greedy=True, max_new_tokens=8))
        assert all(len(o) == 8 and near_greedy(cfg, w, p, o, 0.15) for p, o in zip(prompts, out))
    hid = eng.forward_a(prompts[0])
    assert hid.shape == (30, 88 + 2 * 24)
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
