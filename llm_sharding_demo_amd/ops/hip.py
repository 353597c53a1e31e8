"""HIP backend: the engine ops on the hand-written gfx950 kernels (_C.so).

There is no fallback: constructing `HipBackend` without the built extension
raises, so a GPU run can never silently execute eager PyTorch math.

Device weight layout (set up once per stage by `prepare_stage`):
  * lm_head rows padded to a multiple of 64 (50257 -> 50304) so the logits
    GEMM tiles evenly; padded logits are never sampled (sampler scans < V).
  * Llama q/k projection rows re-ordered per head so RoPE pairs (i, i+hd/2)
    become adjacent columns (2i, 2i+1): the QKV epilogue then rotates with one
    lane exchange.  Q.K is invariant to a common permutation of head dims, so
    q and the K cache simply live in that order.
  * Llama gate/up rows interleaved in 16-row blocks so one wave holds the gate
    and up value of the same output column (silu(gate)*up fused epilogue).
  * Timisun, Vizalix, Kedasun, Fagunex: every width padded with zeros to what the
    MFMA tiles want, so a model of any sizes runs (see _prepare_timisun,
    _prepare_vizalix, _prepare_kedasun and _prepare_fagunex); fp32 or bf16.
"""
from __future__ import annotations

import math
import os
from typing import Optional

import numpy as np
import torch

from ..config import AttentionSpec, ChannelDeltaSpec, ForgetSpec, LatentAttentionSpec, RopeSpec, SSMSpec
from ..runtime.kv_cache import layer_cache
from . import GLU_ALPHA, Backend, PostNorm, Residual
from .routing import Routing

_C = None
_ERR: Optional[BaseException] = None


def _load():
    global _C, _ERR
    if _C is not None:
        return _C
    try:
        from .. import _C as ext  # built in-tree by ops/build.py
    except ImportError as e:  # pragma: no cover
        _ERR = e
        raise RuntimeError(
            "llm_sharding_demo_amd._C (the gfx950 HIP kernels) is not built or failed to load; "
            "run `python -m llm_sharding_demo_amd.ops.build` (or __graft_entry__.build())") from e
    _C = ext
    return _C


def extension_loaded() -> bool:
    try:
        _load()
        return True
    except Exception:
        return False


def rope_pair_permutation(n_heads: int, hd: int) -> torch.Tensor:
    half = hd // 2
    per = []
    for i in range(half):
        per += [i, i + half]
    idx = torch.tensor(per)
    return torch.cat([h * hd + idx for h in range(n_heads)])


def interleave_gate_up(w: torch.Tensor, f: int, blk: int = 16) -> torch.Tensor:
    gate, up = w[:f], w[f:]
    h = w.shape[1]
    return torch.stack([gate.reshape(f // blk, blk, h), up.reshape(f // blk, blk, h)], 1).reshape(2 * f, h)


def _up(n: int, m: int) -> int:
    return -(-n // m) * m


def pad_to(t: torch.Tensor, *shape: int) -> torch.Tensor:
    """Zero-padded copy of t (contiguous)."""
    if tuple(t.shape) == shape:
        return t.contiguous()
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def interleave_experts(w: torch.Tensor, fp: int, hp: int, blk: int = 16) -> torch.Tensor:
    """[..., 2F, H] gate rows | up rows -> [..., 2 fp, hp] in 16-row blocks."""
    lead, f, h = w.shape[:-2], w.shape[-2] // 2, w.shape[-1]
    out = torch.zeros(*lead, fp // blk, 2, blk, hp, dtype=w.dtype, device=w.device)
    for j in range(2):
        part = w[..., j * f:(j + 1) * f, :]
        out[..., j, :, :h] = pad_to(part, *lead, fp, h).reshape(*lead, fp // blk, blk, h)
    return out.reshape(*lead, 2 * fp, hp)


def split_pairs(dim: int, dims: int) -> torch.Tensor:
    """Order of a head's dimensions that brings interleaved pairs (2i, 2i + 1) of
    the first `dims` to places i and i + dims / 2."""
    return torch.cat([torch.arange(0, dims, 2), torch.arange(1, dims, 2), torch.arange(dims, dim)])


def latent_tiles(meta, heads: int, rows: int) -> torch.Tensor:
    """(sequence, first (token, head) row) of every prefill attention tile."""
    n = np.asarray(meta.host_qlens, dtype=np.int64) * heads
    k = -(-n // rows)
    seq = np.repeat(np.arange(len(n)), k)
    first = np.arange(int(k.sum())) - np.repeat(np.cumsum(k) - k, k)
    return torch.from_numpy(np.stack([seq, first * rows], 1).astype(np.int32))


def rope_table(max_pos: int, hd: int, theta: float, device) -> torch.Tensor:
    inv = 1.0 / (theta ** (torch.arange(0, hd, 2, dtype=torch.float64) / hd))
    ang = torch.arange(max_pos, dtype=torch.float64)[:, None] * inv[None, :]
    return torch.stack([ang.cos(), ang.sin()], -1).float().contiguous().to(device)


def rope_spec_table(rope: RopeSpec, max_pos: int, device) -> torch.Tensor:
    """[max_pos, dims / 2, 2] cos, sin of a partial rotation, angles in fp64."""
    ang = torch.arange(max_pos, dtype=torch.float64)[:, None] * torch.tensor(rope.frequencies(), dtype=torch.float64)
    return torch.stack([ang.cos(), ang.sin()], -1).float().contiguous().to(device)


def prefill_tiles(meta) -> torch.Tensor:
    """(sequence, query offset) of every 64-query tile of a packed batch."""
    qlens = meta.host_qlens
    tiles = [(i, off) for i, n in enumerate(qlens) for off in range(0, n, 64)]
    return torch.tensor(tiles, dtype=torch.int32).reshape(-1, 2)


class LazyNorm:
    """A norm whose output has not been materialised: at M <= GEMV_NORM_MAX_M
    rows the consuming GEMV (csrc/kernels/gemv.hip) normalises the fp32
    residual rows itself, so the separate norm launch disappears.  Any other
    consumer materialises it through the norm kernel."""

    __slots__ = ("x", "w", "b", "eps", "rms")

    def __init__(self, x, w, b, eps, rms):
        self.x, self.w, self.b, self.eps, self.rms = x, w, b, eps, rms

    @property
    def shape(self):
        return self.x.shape

    @property
    def code(self) -> int:  # gemv norm code: 1 LayerNorm, 2 RMSNorm
        return 2 if self.rms else 1


# gemv epilogue codes (csrc/kernels/gemm.hip Epi)
_EPI = {"none": 0, "gelu": 1, "silu_mul": 2}
_GLU = {"silu_mul": 0, "gelu_mul": 1, "clamped_glu": 2}  # gated activations (common.h Glu)
EPI_F32, EPI_RESID, EPI_QKV = 3, 4, 6
# longest row the sampler loads once into registers (sample.hip: CH x NT x 4)
SAMPLER_ONE_LOAD = 13 * 1024 * 4


class HipBackend(Backend):
    """The engine ops on the gfx950 kernels.  Every routing decision (which
    kernel, how many K splits) comes from one table, `R` (ops/routing.py;
    `LSD_ROUTING=field=value,...` overrides fields for A/B runs)."""

    name = "hip"
    R: Routing = Routing.from_env()

    def __init__(self):
        self.C = _load()
        R = self.R
        self.C.gemm_set_sk_rows(R.sk_rows)
        self.C.gemm_set_big_min(R.big_min_blocks)
        self.C.gemm_set_nw2_rows(1 << 30)
        self.C.gemm_set_tiled3_max(R.tiled3_max)
        self.C.gemm_set_ring_slots(R.ring_slots)
        self.C.gemm_set_ring_tn(R.ring_tn)
        self.C.gemm_set_ring_fill(R.ring_fill)
        self.C.gemm_set_ring_m96(0)
        self.C.gemm_set_d256_slots(R.d256_slots)
        self.C.gemm_set_ring8(R.ring8)
        self.C.gemm_set_ring8_flags(0)
        self.C.norm_set_wave_min(R.norm_wave_min)
        self.C.norm_set_wave_narrow_min(R.norm_wave_narrow_min)
        self.C.attn_set_max_wg(R.attn_max_wg)
        self.C.gemv_set_nt(R.gemv_nt)
        self.C.moe_set_group_rows(R.moe_group_rows)
        self.C.attn_set_small_waves(R.attn_small_waves)
        self.C.attn_set_small_waves128(R.attn_small_waves128)
        self.C.attn_set_large_waves(64, R.attn_large_waves)
        self.C.attn_set_large_waves(128, R.attn_large_waves)
        self.counters = None
        self.fp32 = False  # the stage's element type (prepare_stage)
        self._rope = None
        self.lane = 0  # microbatch lane (stream) currently being issued; see pipeline.py
        self.concurrency = 1  # microbatch lanes running at once (set per round by the pipeline)

    # ------------------------------------------------------------------
    def prepare_stage(self, stage) -> None:
        cfg, w, dev = stage.cfg, stage.w, stage.device
        self.fp32 = stage.dtype == torch.float32
        if self.fp32 and not cfg.layers:
            raise ValueError(f"{cfg.arch} has no fp32 kernels: serve it in bf16")
        if cfg.arch == "timisun":
            self._prepare_timisun(stage)
        elif cfg.arch == "vizalix":
            self._prepare_vizalix(stage)
        elif cfg.arch == "kedasun":
            self._prepare_kedasun(stage)
        elif cfg.arch == "fagunex":
            self._prepare_fagunex(stage)
        elif stage.last:
            # pad the head IN PLACE: the stage keeps one [vocab_padded, H]
            # tensor and its weight dict points at the first V rows (a
            # contiguous view -- the tied GPT-2 embedding of a 1-stage pipeline
            # reads the same rows), so the unpadded copy is freed
            key = "wte" if cfg.arch == "gpt2" else "lm_head"
            head = w[key]
            if head.shape[0] == cfg.vocab_padded:
                stage._lm_head_padded = head
            else:
                pad = torch.zeros(cfg.vocab_padded, cfg.hidden, dtype=head.dtype, device=dev)
                pad[: cfg.vocab_size] = head
                w[key] = pad[: cfg.vocab_size]
                del head
                stage._lm_head_padded = pad
        if cfg.arch == "llama":
            perm_q = rope_pair_permutation(cfg.n_heads, cfg.head_dim)
            perm_k = rope_pair_permutation(cfg.n_kv_heads, cfg.head_dim) + cfg.q_size
            keep = torch.arange(cfg.q_size + cfg.kv_size, cfg.qkv_size)
            perm = torch.cat([perm_q, perm_k, keep]).to(dev)
            for i in stage.layers:  # a boundary layer may hold only one half here
                p = f"layers.{i}."
                if p + "self_attn.qkv.weight" in w:
                    w[p + "self_attn.qkv.weight"] = w[p + "self_attn.qkv.weight"].index_select(0, perm).contiguous()
                if p + "mlp.gate_up.weight" in w:
                    w[p + "mlp.gate_up.weight"] = interleave_gate_up(w[p + "mlp.gate_up.weight"], cfg.ffn).contiguous()
            stage._rope = rope_table(stage.max_seq, cfg.head_dim, cfg.rope_theta, dev)
        else:
            stage._rope = None
        self._rope = getattr(stage, "_rope", None)
        # split-K ticket counters: zero at rest, re-armed by each tile's last
        # arriver; one row per microbatch lane so concurrent lanes never share one
        self._counters = torch.zeros(8, 1 << 16, dtype=torch.int32, device=dev)
        stage._hip_prepared = True

    # -- Timisun ---------------------------------------------------------------
    def row_width(self, mcfg) -> int:
        return _up(mcfg.hidden, 64) if mcfg.layers else mcfg.hidden

    def layer_cache(self, mixer, shift: int = 0):
        return layer_cache(mixer, _up, shift)

    def latent_width(self, rank: int) -> int:
        return _up(rank, 64)

    def _prepare_timisun(self, stage) -> None:
        """Device layout per layer (zero padding everywhere: the extra rows and
        columns compute zeros):
          attn.in    [q rows, dims of a head padded to 64 | latent | router] x H
          attn.uk    [heads][rank][dim]: queries into the latent space
          attn.uk_rows  [heads dim][rank]: latents to keys (expanded prefill)
          attn.uv    [heads][vdim][rank]: out of it; vdim padded so that all
                     heads together fill the out-projection's K tiles
          mlp.*      gate / up interleaved in 16-row blocks
        Norm gains keep their stored values; the latent gain and the router
        correction are fp32."""
        cfg, w = stage.cfg, stage.w
        hp = self.row_width(cfg)
        if "embed_tokens" in w:
            rows = cfg.vocab_padded if stage.last else cfg.vocab_size
            e = pad_to(w["embed_tokens"], rows, hp)
            w["embed_tokens"] = e[: cfg.vocab_size]
            if stage.last:
                stage._lm_head_padded = e
        if "norm.weight" in w:
            w["norm.weight"] = pad_to(w["norm.weight"], hp)
        for i in stage.layers:
            m, f, p = cfg.layers[i].mixer, cfg.layers[i].mlp, f"layers.{i}."
            t = lambda n: w.pop(p + n)  # noqa: E731
            rank, dp = self.latent_width(m.kv_rank), _up(m.dim, 64)
            vp = self._latent_vcols(m)
            w[p + "input_layernorm.weight"] = pad_to(w[p + "input_layernorm.weight"], hp)
            q = pad_to(t("attn.q.weight").reshape(m.heads, m.dim, -1), m.heads, dp, hp).reshape(m.heads * dp, hp)
            rows = [q]
            if m.kv_from is None:
                rows.append(pad_to(t("attn.dkv.weight"), m.kv_rank, hp))
                w[p + "attn.dkv_norm.weight"] = w[p + "attn.dkv_norm.weight"].float().contiguous()
            if f is not None:
                rows.append(pad_to(t("mlp.router.weight"), f.experts, hp))
                w[p + "mlp.correction"] = w[p + "mlp.correction"].float().contiguous()
                self._prepare_experts(w, p, f, hp)
            n = sum(x.shape[0] for x in rows)
            w[p + "attn.in.weight"] = pad_to(torch.cat(rows), _up(n, 64), hp)
            uk = t("attn.uk.weight").reshape(m.heads, m.dim, m.kv_rank)
            w[p + "attn.uk.weight"] = pad_to(uk.transpose(1, 2), m.heads, rank, dp)
            if not self.fp32:
                w[p + "attn.uk_rows.weight"] = pad_to(uk, m.heads, dp, rank).reshape(m.heads * dp, rank)
            w[p + "attn.uv.weight"] = pad_to(t("attn.uv.weight").reshape(m.heads, m.vdim, m.kv_rank), m.heads, vp, rank)
            o = t("attn.o.weight").reshape(-1, m.heads, m.vdim)
            w[p + "attn.o.weight"] = pad_to(o, hp, m.heads, vp).reshape(hp, m.heads * vp)

    @staticmethod
    def _latent_vcols(m) -> int:
        """Columns of a value head: padded so that all heads together fill the
        out-projection's K tiles."""
        vp = _up(m.vdim, 16)
        while m.heads * vp % 64:
            vp += 16
        return vp

    @staticmethod
    def _prepare_experts(w, p: str, f, hp: int) -> None:
        """Gate / up rows interleaved in 16-row blocks, widths padded."""
        t = lambda n: w.pop(p + n)  # noqa: E731
        w[p + "mlp.experts.gate_up.weight"] = interleave_experts(t("mlp.experts.gate_up.weight"), _up(f.expert.ff, 64), hp)
        w[p + "mlp.experts.down.weight"] = pad_to(t("mlp.experts.down.weight"), f.experts, hp, _up(f.expert.ff, 64))
        if f.shared is not None:
            w[p + "mlp.shared.gate_up.weight"] = interleave_experts(t("mlp.shared.gate_up.weight"), _up(f.shared.ff, 64), hp)
            w[p + "mlp.shared.down.weight"] = pad_to(t("mlp.shared.down.weight"), hp, _up(f.shared.ff, 64))

    def _prepare_fagunex(self, stage) -> None:
        """Device layout per layer (zero padding everywhere):
          attn.in      [queries, or their latent | output gate | latent | turned key part] x H;
                       heads padded, turned pairs (2i, 2i + 1) moved to (i, i + dims / 2) --
                       scores do not change under a common order of q and k
          attn.uq      queries from their latent
          attn.uk      [heads][rank + turned][dim + turned]: queries into the latent space,
                       the turned part passed on by an identity block
          attn.uk_rows [heads dim][rank + turned]: cached rows to keys (expanded prefill)
          attn.uv      [heads][vdim][value columns of the attention kernels]
          mixer.in     q | forget gate | v of a recurrence
          mlp.router   router rows, behind them the shared expert's gate
          side.*       width of the tokens' rows padded
        The norms' alphas stay on the host; gains of latents, gate biases and bounds,
        sinks and the recurrence's norm are fp32."""
        cfg, w, dev = stage.cfg, stage.w, stage.device
        hp = self.row_width(cfg)
        self._ropes = {}

        def norm(name: str) -> None:
            w[name + ".weight"], w[name + ".bias"] = (pad_to(w[name + s], hp) for s in (".weight", ".bias"))
            w[name + ".alpha"] = w[name + ".alpha"].float().cpu()

        if "embed_tokens" in w:
            w["embed_tokens"] = pad_to(w["embed_tokens"], cfg.vocab_size, hp)
        if "lm_head" in w:
            e = pad_to(w["lm_head"], cfg.vocab_padded, hp)
            w["lm_head"], stage._lm_head_padded = e[: cfg.vocab_size], e
            norm("norm")
        for j, i in {cfg.weight_layer(i): i for i in stage.layers}.items():
            m, f, p = cfg.layers[i].mixer, cfg.layers[i].mlp, f"layers.{j}."
            t = lambda n: w.pop(p + n)  # noqa: E731
            f32 = lambda n: w.__setitem__(p + n, w[p + n].float().contiguous())  # noqa: E731
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ()):
                norm(p + n)
            w[p + "shift"] = pad_to(w[p + "shift"], hp)
            if isinstance(m, ForgetSpec):
                rows = torch.cat([t("mixer.q"), t("mixer.f"), t("mixer.v")])
                w[p + "mixer.in.weight"] = pad_to(rows, _up(rows.shape[0], 64), hp)
                for n in ("mixer.f.b", "mixer.lower", "mixer.norm"):
                    f32(n)
                o = t("mixer.o")
                w[p + "mixer.o"] = pad_to(o, hp, _up(o.shape[1], 64))
            else:
                self._prepare_latent(stage, m, p, hp)
            if f is not None:
                rows = [t("mlp.router.weight")] + ([t("mlp.shared.sg")] if f.shared_gate else [])
                rows = torch.cat(rows)
                w[p + "mlp.router.weight"] = pad_to(rows, _up(rows.shape[0], 64), hp)
                self._prepare_experts(w, p, f, hp)
            if cfg.token_side:
                n = _up(cfg.token_side, 64)
                w[p + "side.embed"] = pad_to(w[p + "side.embed"], cfg.vocab_size, n)
                w[p + "side.gate"], w[p + "side.proj"] = pad_to(w[p + "side.gate"], n, hp), pad_to(w[p + "side.proj"], hp, n)
                w[p + "side.norm"] = pad_to(w[p + "side.norm"], hp)

    def _prepare_latent(self, stage, m, p: str, hp: int) -> None:
        """Latent attention with a turned part (the layout is _prepare_fagunex')."""
        w, dev = stage.w, stage.device
        t = lambda n: w.pop(p + n)  # noqa: E731
        rot, rank, H = m.rot_dim, m.kv_rank, m.heads
        dp, cols, vp = _up(m.q_dim, 64), self.latent_width(rank + rot), self._latent_vcols(m)
        order = torch.arange(rot, device=dev)
        if rot and m.rope.interleaved:
            order = split_pairs(rot, rot).to(dev)
        if rot and m.rope not in self._ropes:
            self._ropes[m.rope] = rope_spec_table(m.rope, _up(stage.max_seq, 64), dev)

        def q_rows(x):  # [H (dim + rot), n] -> padded heads
            x = x.reshape(H, m.q_dim, -1)
            x = torch.cat([x[:, : m.dim], x[:, m.dim:].index_select(1, order)], 1)
            return pad_to(x, H, dp, x.shape[2])

        rows = []
        if m.q_rank is None:
            q = q_rows(t("attn.q.weight"))
            rows.append(pad_to(q, H, dp, hp).reshape(H * dp, hp))
        else:
            qr = _up(m.q_rank, 64)
            rows.append(pad_to(t("attn.dq.weight"), qr, hp))
            q = q_rows(t("attn.uq.weight"))
            w[p + "attn.uq.weight"] = pad_to(q, H, dp, qr).reshape(H * dp, qr)
            w[p + "attn.dq_norm.weight"] = w[p + "attn.dq_norm.weight"].float().contiguous()
        if m.gate:
            g = t("attn.g.weight").reshape(H, m.vdim, -1)
            rows.append(pad_to(g, H, vp, hp).reshape(H * vp, hp))
        d = t("attn.dkv.weight")
        rows.append(pad_to(torch.cat([d[:rank], d[rank:].index_select(0, order)]), rank + rot, hp))
        n = sum(x.shape[0] for x in rows)
        w[p + "attn.in.weight"] = pad_to(torch.cat(rows), _up(n, 64), hp)
        w[p + "attn.dkv_norm.weight"] = w[p + "attn.dkv_norm.weight"].float().contiguous()
        uk = torch.zeros(H, cols, dp, dtype=stage.dtype, device=dev)
        uk[:, :rank, : m.dim] = t("attn.uk.weight").reshape(H, m.dim, rank).transpose(1, 2)
        uk[:, rank: rank + rot, m.dim: m.q_dim] = torch.eye(rot, dtype=stage.dtype, device=dev)
        w[p + "attn.uk.weight"] = uk
        if not self.fp32:
            w[p + "attn.uk_rows.weight"] = uk.transpose(1, 2).reshape(H * dp, cols).contiguous()
        vc = self.C.latent_value_cols(cols, rank)
        w[p + "attn.uv.weight"] = pad_to(t("attn.uv.weight").reshape(H, m.vdim, rank), H, vp, vc)
        o = t("attn.o.weight").reshape(-1, H, m.vdim)
        w[p + "attn.o.weight"] = pad_to(o, hp, H, vp).reshape(hp, H * vp)
        if m.sink:
            w[p + "attn.sink"] = w[p + "attn.sink"].float().contiguous()

    def _prepare_vizalix(self, stage) -> None:
        """Device layout per layer (zero padding everywhere):
          mixer.in     rows of one in-projection
                       attention   q | k | v, dims of a head padded
                       delta rule  a1 | g1 (each to the same 64-multiple) | q | k | v | b
                       Mamba-2     as stored: z | x | B | C | dt
          mixer.low    [2][heads dim | heads vdim][rank]: the delta rule's a2 and g2
          mixer.out    [W_o | W_down] side by side: one residual projection over
                       the mixer's output and the feed-forward's inner row
          mlp.gate_up  interleaved in 16-row blocks
        Norm gains (one number each) stay on the host: they are factors of the
        kernels behind the projections.  Decays, biases, taps and norm weights
        of the recurrences, and the head mixing, are fp32."""
        cfg, w, dev = stage.cfg, stage.w, stage.device
        hp = self.row_width(cfg)
        self._ones = torch.ones(hp, dtype=stage.dtype, device=dev)
        self._ropes = {}
        if "embed_tokens" in w:
            w["embed_tokens"] = pad_to(w["embed_tokens"], cfg.vocab_size, hp)
        if "lm_head" in w:
            e = pad_to(w["lm_head"], cfg.vocab_padded, hp)
            w["lm_head"], stage._lm_head_padded = e[: cfg.vocab_size], e
            w["norm.weight"] = w["norm.weight"].expand(hp).contiguous()
        if "loop.in" in w:
            li = torch.stack(w["loop.in"].split(cfg.hidden, 1), 1)  # [H, 2, H]
            w["loop.in"] = pad_to(li, hp, 2, hp).reshape(hp, 2 * hp)
            w["loop.step"] = pad_to(w["loop.step"].float(), cfg.loop_times, hp)
        for j, i in {cfg.weight_layer(i): i for i in stage.layers}.items():
            m, f, p = cfg.layers[i].mixer, cfg.layers[i].mlp, f"layers.{j}."
            t = lambda n: w.pop(p + n)  # noqa: E731
            f32 = lambda n: w.__setitem__(p + n, w[p + n].float().contiguous())  # noqa: E731
            w[p + "input_layernorm.weight"] = w[p + "input_layernorm.weight"].float().cpu()
            o = t("mixer.o")
            if isinstance(m, AttentionSpec):
                dp, vp = _up(m.dim, 32), _up(m.vdim, 16)
                rows = [pad_to(t(f"mixer.{n}").reshape(h, d, -1), h, dd, hp).reshape(h * dd, hp) for n, h, d, dd in (
                    ("q", m.heads, m.dim, dp), ("k", m.kv_heads, m.dim, dp), ("v", m.kv_heads, m.vdim, vp))]
                o = pad_to(o.reshape(-1, m.heads, m.vdim), o.shape[0], m.heads, vp).reshape(-1, m.heads * vp)
                talk = w[p + "mixer.talk"] if m.talking else torch.eye(m.heads, dtype=stage.dtype, device=dev)
                if m.talking:
                    f32("mixer.talk")
                hq = 0 if self.fp32 else self.C.talk_heads(m.heads, m.kv_heads, dp, vp, m.softcap or 0.0)
                if hq and float(talk.abs().max()) < 6e4:  # the mixing matrix in fp16, padded for each kernel
                    w[p + "mixer.talk_prefill"] = pad_to(talk, hq, hq).half()
                    hd = max(16, hq, 32 if m.kv_heads > 4 else 0)
                    if 4 * m.kv_heads <= hd:
                        w[p + "mixer.talk_decode"] = pad_to(talk, hd, hd).half()
                if m.rope is not None and m.rope.dims and m.rope not in self._ropes:
                    self._ropes[m.rope] = rope_spec_table(m.rope, _up(stage.max_seq, 64), dev)
            elif isinstance(m, ChannelDeltaSpec):
                kr, n = self._low_rank(m), self._low_cols(m)
                rows = [pad_to(t("mixer.a1"), kr, hp), pad_to(t("mixer.g1"), kr, hp)]
                rows += [pad_to(t(f"mixer.{x}"), s, hp) for x, s in (
                    ("q", m.kv_heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.heads * m.vdim), ("b", m.heads))]
                w[p + "mixer.low.weight"] = torch.stack([pad_to(t("mixer.a2"), n, kr), pad_to(t("mixer.g2"), n, kr)])
                w[p + "mixer.taps"] = torch.cat([t(f"mixer.{x}.conv") for x in "qkv"]).float().contiguous()
                w[p + "mixer.A"] = -torch.exp(t("mixer.A_log").float())
                f32("mixer.dt_bias")
                f32("mixer.norm")
            else:
                rows = [pad_to(t("mixer.in"), m.inner + m.conv_channels + m.heads, hp)]
                w[p + "mixer.taps"] = t("mixer.conv").float().contiguous()
                w[p + "mixer.A"] = -torch.exp(t("mixer.A_log").float())
                for n in ("conv.b", "dt_bias", "D", "norm"):
                    f32("mixer." + n)
            n = sum(x.shape[0] for x in rows)
            w[p + "mixer.in.weight"] = pad_to(torch.cat(rows), _up(n, 64), hp)
            oc = _up(o.shape[1], 64)
            out = [pad_to(o, hp, oc)]
            if f is not None:
                fp = _up(f.ff, 64)
                w[p + "post_attention_layernorm.weight"] = w[p + "post_attention_layernorm.weight"].float().cpu()
                w[p + "mlp.gate_up.weight"] = interleave_experts(t("mlp.gate_up.weight"), fp, hp)
                out.append(pad_to(t("mlp.down_proj.weight"), hp, fp))
            w[p + "mixer.out.weight"] = torch.cat(out, 1).contiguous()

    def _prepare_kedasun(self, stage) -> None:
        """Device layout per layer (zero padding everywhere):
          mixer.in     q | k | v | gate rows of one in-projection, dims of a head
                       padded, rotated pairs (2i, 2i + 1) moved to (i, i + dims / 2)
                       -- scores do not change under a common order of q and k --
                       with its bias
          mixer.taps   of q | k | v, fp32
          mixer.talk   fp32, and fp16 padded for the prompt kernel
          mlp.gate_up  interleaved in 16-row blocks
        The share of mixed-in values stays on the host."""
        cfg, w, dev = stage.cfg, stage.w, stage.device
        hp = self.row_width(cfg)
        self._ropes = {}
        if "embed_tokens" in w:
            w["embed_tokens"] = pad_to(w["embed_tokens"], cfg.vocab_size, hp)
        if "lm_head" in w:
            e = pad_to(w["lm_head"], cfg.vocab_padded, hp)
            w["lm_head"], stage._lm_head_padded = e[: cfg.vocab_size], e
            w["norm.weight"] = pad_to(w["norm.weight"], hp)
        for i in stage.layers:
            m, f, p = cfg.layers[i].mixer, cfg.layers[i].mlp, f"layers.{i}."
            t = lambda n: w.pop(p + n)  # noqa: E731
            dp, vp = _up(m.dim, 32), _up(m.vdim, 16)
            heads = {"q": (m.heads, m.dim, dp), "k": (m.kv_heads, m.dim, dp), "v": (m.kv_heads, m.vdim, vp)}
            order = None
            if m.rope is not None and m.rope.dims:
                order = split_pairs(m.dim, m.rope.dims).to(dev) if m.rope.interleaved else None
                if m.rope not in self._ropes:
                    self._ropes[m.rope] = rope_spec_table(m.rope, _up(stage.max_seq, 64), dev)

            def rows(suffix: str) -> torch.Tensor:
                """q | k | v rows, one per padded channel."""
                out = []
                for n, (h, d, pad) in heads.items():
                    x = t(f"mixer.{n}{suffix}").reshape(h, d, -1)
                    if order is not None and n != "v":
                        x = x.index_select(1, order)
                    out.append(pad_to(x, h, pad, x.shape[2]).reshape(h * pad, -1))
                return torch.cat(out)

            w_in = rows("")
            if m.head_gate:
                w_in = torch.cat([w_in, t("mixer.g")])
            n = _up(w_in.shape[0], 64)
            w[p + "mixer.in.weight"] = pad_to(w_in, n, hp)
            if m.bias:
                w[p + "mixer.in.bias"] = pad_to(rows(".b")[:, 0], n)
                w[p + "mixer.o.b"] = pad_to(w[p + "mixer.o.b"], hp)
            if m.conv:
                w[p + "mixer.taps"] = rows(".conv").float().t().contiguous()  # [taps][channels]
            if m.mix_values is not None:
                w[p + "mixer.vmix"] = w[p + "mixer.vmix"].float().cpu()
            if m.distance_bias:
                w[p + "mixer.slopes"] = torch.tensor(m.slopes(), dtype=torch.float32, device=dev)
            if m.talking:
                w[p + "mixer.talk"] = talk = w[p + "mixer.talk"].float().contiguous()
                hq = 0 if self.fp32 else self.C.talk_heads(m.heads, m.kv_heads, dp, vp, -1.0)
                if hq and float(talk.abs().max()) < 6e4:
                    w[p + "mixer.talk_prefill"] = pad_to(talk, hq, hq).half()
            o = t("mixer.o").reshape(-1, m.heads, m.vdim)
            w[p + "mixer.o"] = pad_to(pad_to(o, o.shape[0], m.heads, vp).reshape(o.shape[0], -1), hp, _up(m.heads * vp, 64))
            for name in ("input_layernorm", "mixer.out_norm") + (("post_attention_layernorm", "mlp.out_norm") if f else ()):
                w[p + name + ".weight"] = pad_to(w[p + name + ".weight"], hp)
            if f is not None:
                fp = _up(f.ff, 64)
                w[p + "mlp.gate_up.weight"] = interleave_experts(t("mlp.gate_up.weight"), fp, hp)
                w[p + "mlp.down_proj.weight"] = pad_to(w[p + "mlp.down_proj.weight"], hp, fp)

    def value_width(self, mixer) -> int:
        return _up(mixer.vdim, 16)

    @staticmethod
    def _low_rank(m) -> int:
        return _up(max(m.decay_rank, m.gate_rank), 64)

    @staticmethod
    def _low_cols(m) -> int:
        return _up(max(m.heads * m.dim, m.heads * m.vdim), 16)

    # -- mixers of models/stage.py _mixer_layer --------------------------------
    def loop_enter(self, r: Residual, x0, w_in, step, t: int) -> None:
        self.flush(r)
        self.linear_residual(self.C.loop_pack(r.x, x0, step[t], self.fp32), w_in, None, r)

    def unit_rmsnorm(self, r: Residual, mcfg):
        return self.rmsnorm(r, self._ones, mcfg.norm_eps, width=self.norm_width(mcfg))

    def _rows(self, h, w, b=None):
        """In-projection rows in the element type."""
        return self.C.linear_fp32(h, w, None, b) if self.fp32 else self.linear(h, w, b)

    def mix(self, h, w, spec, kv, entry, meta, eps):
        """Mixer output, and room for the feed-forward's inner row behind it:
        [T, out columns + ff columns], the operand of the residual projection."""
        m, gain = spec.mixer, float(w("input_layernorm.weight"))
        y = self._rows(h, w("mixer.in.weight"))
        buf = torch.empty(y.shape[0], w("mixer.out.weight").shape[1], dtype=y.dtype, device=y.device)
        ff = _up(spec.mlp.ff, 64) if spec.mlp is not None else 0
        out = buf[:, : buf.shape[1] - ff]
        fn = (self._attend if isinstance(m, AttentionSpec) else
              self._channel_delta if isinstance(m, ChannelDeltaSpec) else self._ssm)
        fn(y, w, m, gain, kv, entry, meta, eps, out)
        return buf

    def mixer_residual(self, buf, h, w, spec, r: Residual) -> None:
        if spec.mlp is not None:
            gain, gu = float(w("post_attention_layernorm.weight")), w("mlp.gate_up.weight")
            mid = buf[:, buf.shape[1] - gu.shape[0] // 2:]
            if self.fp32:
                self.C.glu_f32(self.C.linear_fp32(h, gu), mid, _GLU["gelu_mul"], gain)
            else:
                self.linear(h, gu, act="gelu_mul", out=mid, scale=gain)
        self.linear_residual(buf, w("mixer.out.weight"), None, r)

    def _attend(self, y, w, m, gain, kv, entry, meta, eps, out):
        k, v = entry
        q = self.C.rope_append(y, m.heads, k, v, kv.table, meta.token_slots, meta.token_pos, self._rope_of(m), gain)
        for s, mt in self._parts(meta):
            self._attention(q[s], w, m, k, v, kv, mt, None, out[s])

    def _rope_of(self, m):
        return self._ropes[m.rope] if m.rope is not None and m.rope.dims else None

    # -- layers with norms around each sublayer (models/stage.py _sandwich_layer) ----
    def group_norm(self, r: Residual, w, mcfg):
        slab, bias, w_post = (r.post.slab, r.post.bias, r.post.rms[0]) if r.post is not None else (None, None, None)
        r.post = None
        return self.C.group_norm(r.x, mcfg.norm_groups, mcfg.hidden, mcfg.norm_eps, slab, bias, w_post, w, None, self.fp32)

    def group_norm_rows(self, x, w, mcfg, rows=None):
        return self.C.group_norm(x, mcfg.norm_groups, mcfg.hidden, mcfg.norm_eps, None, None, None, w, rows, self.fp32)

    def linear_post_norm(self, a, w, b, norm_w, r: Residual, mcfg) -> None:
        """x += norm(a w^T + b), left to the next group_norm or flush as the
        projection's slabs."""
        r.post = PostNorm(self._slabs(a, w, r.x), b, rms=(norm_w, mcfg.norm_groups, mcfg.hidden, mcfg.norm_eps))

    def _slabs(self, a, w, x):
        """a w^T as slabs [S, T, H] (their sum); x: rows of the same shape."""
        (M, K), N = a.shape, w.shape[0]
        if self.fp32 or self._gemv_in(a, K, EPI_F32) is not None or (
                not self._tiled(M, N) and self._resid_splits(M, N, K) == 1):
            return self._linear_f32(a, w)[None]
        return self.C.linear_residual(a, w, None, x, self._resid_splits(M, N, K), self._tiled(M, N), self.counters, True, None)

    # -- layers with elementwise norms (models/stage.py _token_layer) ----------------
    @staticmethod
    def _tanh(n):
        return float(n(".alpha")), n(".weight"), n(".bias")

    def _tanh_step(self, r: Residual, out: bool, pre=(0.0, None, None), rows=None):
        """Folds a pending elementwise norm; with `out` the residual normed by
        `pre`, or in the element type."""
        post = r.post if r.post is not None and r.post.tanh else None
        if r.post is not None and post is None:
            self.flush(r)
        r.post = None
        slab, args = (post.slab, post.tanh) if post is not None else (None, (0.0, None, None))
        return self.C.tanh_step(r.x, slab, *args, out, *pre, rows, self.fp32)

    def tanh_norm(self, r: Residual, n):
        return self._tanh_step(r, True, self._tanh(n))

    def tanh_norm_rows(self, x, n, rows=None):
        return self._tanh_step(Residual(x), True, self._tanh(n), rows)

    def shift_norm(self, r: Residual, w, last, meta, mcfg):
        """The layer's first norm, its rows moved towards the previous token's by
        w("shift"); `last` [slots, H]: the previous portion's last row."""
        if r.post is not None and r.post.tanh:
            self.flush(r)
        slab, gain = (r.post.slab, r.post.rms[0]) if r.post is not None else (None, None)
        r.post = None
        norm = self._tanh(lambda n: w("norm1" + n))
        r.x, h = self.C.shift_norm(r.x, slab, gain, mcfg.hidden, mcfg.norm_eps, *norm, w("shift"), last, meta.token_slots,
                                   meta.token_pos, self.fp32)
        for s, mt in self._parts(meta):
            if not mt.is_decode:
                self.C.shift_tail(r.x[s], *norm, last, mt.token_slots, mt.last_idx, self.fp32)
        return h

    def linear_tanh(self, a, wt, n, r: Residual) -> None:
        """x += norm(a wt^T), left to the next norm as the projection's slabs."""
        r.post = PostNorm(self._slabs(a, wt, r.x), tanh=self._tanh(n))

    def experts_tanh(self, h, w, mlp, n, r: Residual) -> None:
        """x += norm(experts(h)), left to the next norm: one slab per choice and the
        shared expert's."""
        wr, (T, H) = w("mlp.router.weight"), h.shape
        args = (mlp.experts, mlp.top, mlp.shared_gate)
        if not self.fp32 and wr.shape[0] <= 64 and T <= self.R.rows_few_t:
            ids, wts, shared = self.C.router(h, wr, *args, self.R.router_splits(T, wr.shape[1]), self.counters)
        else:
            ids, wts, shared = self.C.route_softmax(self._linear_f32(h, wr), *args)
        shared = shared if mlp.shared_gate else None
        if not self.fp32 and T <= self.R.moe_few_t:
            slab = torch.empty(1, T, H, dtype=torch.float32, device=h.device)
            self._moe_few(h, ids, wts, w, mlp, slab[0], shared, False)
        else:
            slab = torch.empty(mlp.top + (mlp.shared is not None), T, H, dtype=h.dtype, device=h.device)
            self._moe(h, ids, wts, w, mlp, slab, shared)
        r.post = PostNorm(slab, tanh=self._tanh(n))

    def token_side(self, r: Residual, ids, w, mcfg) -> None:
        """x += rms(proj(gelu(gate x) * e)) * norm, e the tokens' rows of the layer's
        table; the norm is left to the next layer."""
        x = self._tanh_step(r, True)
        wg, e = w("side.gate"), w("side.embed")
        if not self.fp32 and x.shape[0] <= self.R.rows_few_t:
            g = self.C.side_gate(x, wg, ids, e)
        else:
            g = self.C.side_mul(self._linear_f32(x, wg) if self.fp32 else self.linear(x, wg, act="gelu"), ids, e)
        r.post = PostNorm(self._slabs(g, w("side.proj"), r.x), rms=(w("side.norm"), 1, mcfg.hidden, mcfg.norm_eps))

    def forget_mix(self, h, w, m, state, meta, eps):
        """Recurrence with forget gates in front of the out-projection (rows padded)."""
        y = self._rows(h, w("mixer.in.weight"))
        out = torch.empty(y.shape[0], w("mixer.o").shape[1], dtype=y.dtype, device=y.device)
        for s, mt in self._parts(meta):
            chunked = self._chunked(mt) and self.C.forget_ok(m.dim, m.vdim)
            segs = self.R.forget_segments(mt.num_seqs * m.heads, mt.max_q) if chunked else 1
            self.C.forget_seq(y[s], mt.seq_slots, mt.q_start, mt.cu_q, m.heads, m.dim, m.vdim, w("mixer.f.b"),
                              w("mixer.lower"), w("mixer.norm"), eps, state, out[s], chunked, segs)
        return out

    def clamped_glu(self, h, w, limit: float):
        if self.fp32:
            y = self.C.linear_fp32(h, w)
            out = torch.empty(y.shape[0], y.shape[1] // 2, dtype=y.dtype, device=y.device)
            self.C.glu_f32(y, out, _GLU["clamped_glu"], limit)
            return out
        return self.linear(h, w, act="clamped_glu", scale=limit)

    def attend(self, h, w, m, kv, entry, meta, eps, first_values, keep_values: bool = False):
        """Attention before the output projection (heads padded), and with
        keep_values this layer's values.  first_values: rows that are mixed into
        the values (None: they stay as they are)."""
        y = self._rows(h, w("mixer.in.weight"), w("mixer.in.bias", None))
        (k, v), ring = entry[:2], entry[2] if m.conv else None
        G, vp = v.shape[1], v.shape[3]
        values = torch.empty(y.shape[0], G * vp, dtype=y.dtype, device=y.device) if keep_values else None
        taps = w("mixer.taps", None)
        q = self.C.rope_append(y, m.heads, k, v, kv.table, meta.token_slots, meta.token_pos, self._rope_of(m), 1.0, taps,
                               ring, meta.is_decode, eps if m.qk_norm else -1.0, m.dim, first_values,
                               0.0 if first_values is None else float(w("mixer.vmix")), values)
        out = torch.empty(y.shape[0], w("mixer.o").shape[1], dtype=y.dtype, device=y.device)
        c = q.shape[1] + G * (k.shape[3] + vp)
        gate = y[:, c: c + m.heads] if m.head_gate else None
        for s, mt in self._parts(meta):
            if m.conv and not meta.is_decode:
                self.C.conv_tail(y[s], ring, mt.seq_slots, mt.q_start, mt.cu_q)
            self._attention(q[s], w, m, k, v, kv, mt, None if gate is None else gate[s], out[s])
        return out, values

    def _attention(self, q, w, m, k, v, kv, mt, gate, out) -> None:
        """One part of a step (decode rows or prompt chunks) over the cache."""
        C, R = self.C, self.R
        H, G, dp, vp = m.heads, k.shape[1], k.shape[3], v.shape[3]
        window, cap, keep, slopes = m.window or 1 << 30, m.softcap or 0.0, m.keep_first, w("mixer.slopes", None)
        ctx = min(window + keep, mt.max_ctx)
        tp = w("mixer.talk_prefill", None)
        rows, seqs = (mt.token_slots, mt.token_pos), (mt.seq_slots, mt.q_start, mt.cu_q)
        at = (q, k, v, kv.table)
        beside = (keep, slopes, gate)
        if m.talking and not m.talk_weights and tp is not None and not keep and slopes is None and gate is None:
            td = w("mixer.talk_decode", None)
            if mt.is_decode and td is not None:
                C.talk_decode(*at, td, *rows, window, m.scale, cap, R.talk_splits(mt.num_seqs, ctx), out)
            else:
                tiles = self._query_tiles(mt, C.talk_tile(tp.shape[0]), q.device)
                C.talk_prefill(*at, tp, tiles, *seqs, window, m.scale, cap, R.talk_prefill_splits(tiles.shape[0], ctx), out)
            return
        mfma = not self.fp32 and m.softcap is None and C.paged_ok(dp, vp)
        if mfma and m.talking and m.talk_weights and tp is not None:
            if mt.is_decode and C.mix_decode_ok(H, G):
                C.mix_decode(*at, w("mixer.talk"), *rows, window, m.scale, *beside, R.mix_splits(mt.num_seqs, ctx, H, G), out)
                return
            lse = torch.empty(q.shape[0], H, dtype=torch.float32, device=q.device)
            tiles, qt = self._paged_tiles(mt, H, q.device)
            C.paged_prefill(*at, tiles, qt, *seqs, window, m.scale, *beside, out, lse)
            tiles = self._query_tiles(mt, C.talk_tile(tp.shape[0]), q.device)
            C.mix_prefill(*at, tp, tiles, *seqs, window, m.scale, *beside, lse, R.talk_prefill_splits(tiles.shape[0], ctx),
                          out)
        elif mfma and not m.talking:
            if mt.is_decode and H // G <= 16:
                C.paged_decode(*at, *rows, window, m.scale, *beside, R.paged_splits(mt.num_seqs * G, ctx), out)
            else:
                tiles, qt = self._paged_tiles(mt, H, q.device)
                C.paged_prefill(*at, tiles, qt, *seqs, window, m.scale, *beside, out)
        else:
            C.talk_plain(*at, *rows, w("mixer.talk") if m.talking else None, window, m.scale, cap, out, *beside,
                         m.talk_weights)

    def _paged_tiles(self, meta, heads: int, device):
        """Query tiles of the per-head prompt kernel and their size in 64 queries."""
        qt = 2 if self._query_tiles(meta, 128, device).shape[0] * heads >= self.R.paged_tile_min else 1
        return self._query_tiles(meta, 64 * qt, device), qt

    @staticmethod
    def _query_tiles(meta, rows: int, device):
        """(sequence, first query) of every `rows`-query tile, kept on the batch."""
        cache = meta.__dict__.setdefault("_query_tiles", {})
        if rows not in cache:
            if meta.is_decode:  # one each; made on the device (a captured decode step may ask)
                first = torch.arange(meta.num_seqs, dtype=torch.int32, device=device)
                cache[rows] = torch.stack([first, torch.zeros_like(first)], 1)
            else:
                cache[rows] = latent_tiles(meta, 1, rows).to(device)
        return cache[rows]

    def _channel_delta(self, y, w, m, gain, kv, entry, meta, eps, out):
        low = self._batch_linear(y, w("mixer.low.weight"))
        c0, n = 2 * self._low_rank(m), self._low_cols(m)
        for s, mt in self._parts(meta):
            self.C.delta_seq(y[s], c0, c0 + m.conv_channels, low[s], n, mt.seq_slots, mt.q_start, mt.cu_q, m.heads,
                             m.kv_heads, m.dim, m.vdim, w("mixer.taps"), entry[1], entry[0], w("mixer.A"),
                             w("mixer.dt_bias"), w("mixer.norm"), gain, eps, out[s], mt.is_decode,
                             self._chunked(mt) and self.C.chunk_ok(True, m.dim, m.vdim, m.kv_heads, m.heads))

    def _chunked(self, meta) -> bool:
        """Prompts of bf16 models run in chunks (very short portions token by token)."""
        return not self.fp32 and not meta.is_decode and meta.num_tokens > self.R.chunk_min * meta.num_seqs

    def _ssm(self, y, w, m, gain, kv, entry, meta, eps, out):
        for s, mt in self._parts(meta):
            self.C.ssm_seq(y[s], mt.seq_slots, mt.q_start, mt.cu_q, m.heads, m.groups, m.state, m.vdim, m.norm_groups,
                           w("mixer.taps"), w("mixer.conv.b"), entry[1], entry[0], w("mixer.A"), w("mixer.dt_bias"),
                           w("mixer.D"), w("mixer.norm"), gain, eps, out[s], mt.is_decode,
                           self._chunked(mt) and self.C.chunk_ok(False, m.state, m.vdim, m.groups, m.heads))

    def _tm(self, rows: float) -> int:
        return 64 if self.fp32 else self.R.group_tm(rows)

    def _batch_linear(self, a, w, gate=None):
        return self.C.batch_linear(a, w, 64 if self.fp32 else self.R.batch_tm(a.shape[0], w.shape[0], w.shape[1]), gate)

    def latent_project(self, h, w, m, mlp, kv, pool, meta, eps):
        """Queries per head, turned; the output gate's logits; the routing of experts
        `mlp` that read the same rows."""
        y = self._linear_f32(h, w("attn.in.weight"))
        own, dp = m.kv_from is None, w("attn.uk.weight").shape[2]
        nq = m.heads * dp if m.q_rank is None else w("attn.uq.weight").shape[1]
        ng = m.heads * self._latent_vcols(m) if m.gate else 0
        rope = self._ropes[m.rope] if m.rot_dim else None
        where = (meta.token_slots, meta.token_pos)
        turn = dict(rope=rope, q_head=dp, q_rot=m.dim)
        gains = w("attn.dkv_norm.weight") if own else None
        keep = self.fp32 and rope is None and m.q_rank is None  # the queries are read where they are
        q, ids, wts = self.C.latent_post(
            y, nq, not keep, self.fp32, pool if own else None, m.kv_rank, gains, eps, kv.table, *where,
            w("mlp.correction") if mlp is not None else None, mlp.top if mlp is not None else 0, c_off=nq + ng,
            q_gain=None if m.q_rank is None else w("attn.dq_norm.weight"), **turn)
        if m.q_rank is not None:
            q = self._linear_f32(q, w("attn.uq.weight"))
            if rope is not None or not self.fp32:
                q = self.C.latent_post(q, m.heads * dp, True, self.fp32, None, 0, None, eps, None, *where, None, 0, **turn)[0]
        return (y if keep else q), (y[:, nq: nq + ng] if m.gate else None), (ids, wts)

    def latent_attention(self, q, gate, w, m, kv, pool, meta):
        o = [self._latent_part(q[s], None if gate is None else gate[s], w, m, kv, pool, mt) for s, mt in self._parts(meta)]
        return o[0] if len(o) == 1 else torch.cat(o)  # mixed step: each part its own kernel

    def _latent_part(self, q, gate, w, m, kv, pool, meta):
        window = m.window or 1 << 30
        beside = (m.kv_rank, w("attn.sink") if m.sink else None)
        uk, uv = w("attn.uk.weight"), w("attn.uv.weight")
        rows = self.C.latent_tile_rows(pool.shape[2])
        if not self.fp32 and not meta.is_decode and q.shape[0] >= self.R.latent_expand_t:
            reach = self._latent_reach(meta, m.window)
            if reach is not None and uk.shape[2] <= 192 and uv.shape[1] <= 128 and self.R.latent_expand(
                    q.shape[0], reach[3], reach[2], uk.shape[2], uv.shape[1], pool.shape[2]):
                return self._latent_expanded(q, gate, w, m, kv, pool, meta, window, reach)
        q = self._batch_linear(q, uk)
        if meta.is_decode or self.fp32 or rows == 0:
            # one query per sequence, or the kernel that takes any token alone
            splits = self.R.latent_splits(q.shape[0], m.heads, min(window, meta.max_ctx))
            o = self.C.latent_decode(q, pool, kv.table, meta.token_slots, meta.token_pos, m.heads, window, m.scale,
                                     splits, *beside)
        else:
            o = self.C.latent_prefill(q, pool, kv.table, self._latent_tiles(meta, m.heads, rows, q.device),
                                      meta.seq_slots, meta.q_start, meta.cu_q, m.heads, window, m.scale, *beside)
        return self._batch_linear(o, uv, gate)

    def _latent_expanded(self, q, gate, w, m, kv, pool, meta, window, reach):
        """Keys and values of every row in reach made once, then per-head attention."""
        k_lo, cu_k, rows, _ = reach
        c = self.C.latent_gather(pool, kv.table, meta.seq_slots, k_lo, cu_k, rows)
        k = self.linear(c, w("attn.uk_rows.weight"))
        uv = w("attn.uv.weight")
        v = self.linear(c[:, : uv.shape[2]], uv.reshape(-1, uv.shape[2]))
        return self.C.latent_expanded(q, k, v, self._latent_tiles(meta, 1, 128, q.device), meta.cu_q, meta.q_start,
                                      k_lo, cu_k, m.heads, window, m.scale, w("attn.sink") if m.sink else None, gate)

    @staticmethod
    def _latent_reach(meta, window):
        """(first key position, row offset) per sequence on the device, rows in
        all, and keys scored per query on average; None where the host does not
        know the positions (a chunk graph is captured once for any of them)."""
        if meta.host_starts is None:
            return None
        cache = meta.__dict__.setdefault("_latent_reaches", {})
        if window not in cache:
            st = np.asarray(meta.host_starts, dtype=np.int64)
            n = np.asarray(meta.host_qlens, dtype=np.int64)
            lo = np.zeros_like(st) if window is None else np.maximum(0, st - window + 1)
            cu = np.zeros(len(st) + 1, dtype=np.int64)
            np.cumsum(st + n - lo, out=cu[1:])
            keys = st + (n + 1) / 2  # mean context, capped by the window
            if window is not None:
                keys = np.minimum(keys, window)
            dev = meta.cu_q.device
            both = torch.from_numpy(np.concatenate([lo, cu]).astype(np.int32)).to(dev)
            cache[window] = (both[: len(st)].clone(), both[len(st):].clone(), int(cu[-1]),
                             float((keys * n).sum() / max(1, n.sum())))
        return cache[window]

    @staticmethod
    def _latent_tiles(meta, heads: int, rows: int, device):
        cache = meta.__dict__.setdefault("_latent_tiles", {})
        if heads not in cache:
            cache[heads] = latent_tiles(meta, heads, rows).to(device)
        return cache[heads]

    def prepare_prefill(self, meta, mcfg) -> None:
        if mcfg.arch in ("vizalix", "kedasun"):
            for rows in {self.C.talk_tile(hp) for hp in (8, 16, 32)} | {64, 128}:
                self._query_tiles(meta, rows, meta.cu_q.device)
            return
        if not mcfg.layers:
            meta._tiles = prefill_tiles(meta).to(meta.cu_q.device)
            return
        for heads in {l.mixer.heads for l in mcfg.layers if isinstance(l.mixer, LatentAttentionSpec)}:
            self._latent_tiles(meta, heads, 128, meta.cu_q.device)

    def parallel_residual(self, o, h, routing, w, mlp, r: Residual) -> None:
        """x += o W_o^T + experts(h).  Everything that is not added in place --
        split-K partials of the out-projection, one row set per chosen expert
        and the shared expert's -- is written to one slab for the next norm."""
        wo = w("attn.o.weight")
        if mlp is None:
            self.linear_residual(o, wo, None, r)
            return
        ids, wts = routing
        T, H = h.shape
        if not self.fp32 and T <= self.R.moe_few_t:
            self.linear_residual(o, wo, None, r)
            self._moe_few(h, ids, wts, w, mlp, r.x, None, True)
            return
        shared = mlp.shared is not None
        so = self._slab_splits(o, wo)
        if so and bool(self.C.gemm_slab_bf16()) != (h.dtype == torch.bfloat16):
            so = 0  # slabs of two element types: the out-projection keeps its own
        slab = torch.empty(so + mlp.top + shared, T, H, dtype=h.dtype, device=h.device)
        self.linear_residual(o, wo, None, r, slab[:so] if so else None)
        self._moe(h, ids, wts, w, mlp, slab[so:], None)
        r.pending.append((slab, None))

    def _moe_few(self, h, ids, wts, w, mlp, x, shared_wts, add: bool) -> None:
        """x (+)= experts of a few tokens, weights streamed."""
        sh = mlp.shared
        self.C.moe_few(h, ids, wts, w("mlp.experts.gate_up.weight"), w("mlp.experts.down.weight"), mlp.expert.limit or 0.0,
                       GLU_ALPHA, w("mlp.shared.gate_up.weight") if sh else None, w("mlp.shared.down.weight") if sh else None,
                       (sh.limit or 0.0) if sh else 0.0, x, shared_wts, add)

    def _moe(self, h, ids, wts, w, mlp, slab, shared_wts) -> None:
        """slab[k] = choice k's expert, slab[top] the shared one, weighed per token."""
        tm = self._tm(h.shape[0] * mlp.top / mlp.experts)
        shared = mlp.shared is not None
        perm, tiles = self.C.moe_group(ids, mlp.experts, tm)
        mid, mids = self.C.moe_up(h, perm, tiles, mlp.top, w("mlp.experts.gate_up.weight"), mlp.expert.limit or 0.0,
                                  GLU_ALPHA, w("mlp.shared.gate_up.weight") if shared else None,
                                  (mlp.shared.limit or 0.0) if shared else 0.0, tm)
        self.C.moe_down(mid, mids if shared else None, perm, tiles, wts, w("mlp.experts.down.weight"),
                        w("mlp.shared.down.weight") if shared else None, slab, tm, shared_wts)

    def _slab_splits(self, a, w) -> int:
        """Partial slabs linear_residual(a, w) leaves for the next norm (0: it
        adds into the residual)."""
        M, K = a.shape
        N = w.shape[0]
        if self.fp32 or self._gemv_in(a, K, EPI_RESID) is not None or self._tiled(M, N) or not self.R.defer_resid \
                or (self.R.blaslt_resid(M, K, self._decode) and a.is_contiguous()):
            return 0
        s = self._resid_splits(M, N, K)
        return s if s > 1 else 0

    def _linear_f32(self, a, w):
        """a w^T with fp32 output (no bias)."""
        if self.fp32:
            return self.C.linear_fp32(a, w)
        if self._gemv_in(a, w.shape[1], EPI_F32) is not None:
            return self.C.gemv(a, w, None, EPI_F32, 0, None, None, 0.0, None, None, None, None, None, 0, 0, 0, None)
        tiled, splits = self._gemm_kw(a.shape[0], w.shape[0], w.shape[1])
        return self.C.linear_f32(a, w, tiled, splits, self.counters)

    @property
    def counters(self):
        return None if self._counters is None else self._counters[self.lane % 8]

    @counters.setter
    def counters(self, value):
        self._counters = None if value is None else value.reshape(-1, 1 << 16)

    # ------------------------------------------------------------------
    # routing (ops/routing.py): this forward's phase and lane count applied
    @classmethod
    def _tiled(cls, M: int, N: int = 0) -> bool:
        return cls.R.tiled(M, N)

    @property
    def _decode(self) -> bool:
        return getattr(self, "decode", True)

    def _gemm_kw(self, M: int, N: int, K: int, nw: int = 1):
        return self.R.gemm_kw(M, N, K, self.concurrency, nw)

    def _resid_splits(self, M: int, N: int, K: int) -> int:
        return self.R.resid_splits(M, N, K, self._decode, getattr(self, "concurrency", 1))

    @classmethod
    def decode_attn_splits(cls, B: int, nh: int, n_kv: int, hd: int, max_ctx: int) -> int:
        return cls.R.attn_splits(B, nh, n_kv, hd, max_ctx)

    # ------------------------------------------------------------------
    def embed(self, ids, pos, wte, wpe, scale: float = 1.0):
        if self.fp32:
            return self.C.embed_fp32(ids, wte, scale)
        return self.C.embed(ids, pos, wte, wpe, scale)

    def _norm(self, r: Residual, w, b, eps, rms: bool, offset: float = 0.0, width: int = 0):
        if not self.fp32 and not offset and not width and not r.pending and r.x.shape[0] <= self.R.gemv_norm_max_m and r.x.shape[1] % 8 == 0:
            return LazyNorm(r.x, w, b, eps, rms)
        self._flush_extra(r)
        slab, pb = (r.pending[0] if r.pending else (None, None))
        if self.fp32:
            out = self.C.norm_fp32(r.x, slab, w, eps, None, True, width, offset)
        else:
            out = self.C.norm(r.x, slab, pb, w, b, eps, rms, None, True, width, offset)
        r.pending.clear()
        return out

    def _flush_extra(self, r: Residual) -> None:
        while len(r.pending) > 1:
            slab, pb = r.pending.pop(0)
            self._fold(r.x, slab, pb)

    def _fold(self, x, slab, pb) -> None:
        if self.fp32:
            self.C.norm_fp32(x, slab, None, 0.0, None, False, 0, 0.0)
        else:
            self.C.norm(x, slab, pb, None, None, 0.0, True, None, False)

    def flush(self, r: Residual):
        if r.post is not None and r.post.tanh:
            self._tanh_step(r, False)
        elif r.post is not None:
            post, r.post = r.post, None
            w_post, *parts = post.rms
            self.C.group_norm(r.x, *parts, post.slab, post.bias, w_post, None, None, self.fp32)
        for slab, pb in r.pending:
            self._fold(r.x, slab, pb)
        r.pending.clear()
        return r.x

    def layernorm(self, r, w, b, eps):
        return self._norm(r, w, b, eps, False)

    def rmsnorm(self, r, w, eps, offset: float = 0.0, width: int = 0):
        return self._norm(r, w, None, eps, True, offset, width)

    def norm_rows(self, x, w, b, eps, rms: bool, rows=None, offset: float = 0.0, width: int = 0):
        if self.fp32:
            return self.C.norm_fp32(x, None, w, eps, rows, True, width, offset)
        if offset or width:
            return self.C.norm(x, None, None, w, b, eps, rms, rows, True, width, offset)
        if rows is None and x.shape[0] <= self.R.gemv_norm_max_m and x.shape[1] % 8 == 0:
            return LazyNorm(x, w, b, eps, rms)
        return self.C.norm(x, None, None, w, b, eps, rms, rows, True)

    def materialize(self, xn):
        if isinstance(xn, LazyNorm):
            return self.C.norm(xn.x, None, None, xn.w, xn.b, xn.eps, xn.rms, None, True)
        return xn

    def _gemv_in(self, xn, K: int, epi: int):
        """(x, norm code, gamma, beta, eps) for a GEMV launch, or None when this
        GEMM does not run on the GEMV (the caller takes the MFMA path)."""
        M = xn.shape[0]
        if M > self.R.gemv_max_m:
            return None
        if isinstance(xn, LazyNorm):
            if self.C.gemv_ok(M, K, epi, xn.code):
                return xn.x, xn.code, xn.w, xn.b, xn.eps
            xn = self.materialize(xn)
        if self.C.gemv_ok(M, K, epi, 0):
            return xn, 0, None, None, 0.0
        return None

    def qkv_kv_append(self, xn, w, b, cache_k, cache_v, meta, mcfg):
        g = self._gemv_in(xn, w.shape[1], EPI_QKV)
        if g is not None:
            x, nc, gw, gb, eps = g
            return self.C.gemv(x, w, b, EPI_QKV, nc, gw, gb, eps, None, cache_k, cache_v,
                               meta.token_slots, meta.token_pos, mcfg.q_size, mcfg.kv_size,
                               mcfg.head_dim, self._rope)
        xn = self.materialize(xn)
        if self.R.blaslt_qkv(xn.shape[0], w.shape[1], getattr(self, "decode", False)) and xn.is_contiguous():
            y = self.C.blaslt_f32(xn, w, self.lane)
            if y is not None:
                return self.C.qkv_post(y, b, cache_k, cache_v, meta.token_slots, meta.token_pos,
                                       mcfg.q_size, mcfg.kv_size, mcfg.head_dim, self._rope)
        tiled, splits = self._gemm_kw(xn.shape[0], w.shape[0], w.shape[1])
        return self.C.linear_qkv(xn, w, b, cache_k, cache_v, meta.token_slots, meta.token_pos,
                                 mcfg.q_size, mcfg.kv_size, mcfg.head_dim, self._rope,
                                 tiled, splits, self.counters)

    def attention(self, q, cache_k, cache_v, meta):
        n_kv, hd = cache_k.shape[1], cache_k.shape[3]
        nh = q.shape[1] // hd
        if meta.is_decode:
            splits = self.decode_attn_splits(meta.num_seqs, nh, n_kv, hd, meta.max_ctx)
            return self.C.attn_decode(q, cache_k, cache_v, meta.seq_slots, meta.token_pos, nh, splits)
        tiles = getattr(meta, "_tiles", None)
        if tiles is None:
            tiles = prefill_tiles(meta).to(q.device)
            meta._tiles = tiles
        return self.C.attn_prefill(q, cache_k, cache_v, tiles, meta.seq_slots, meta.q_start,
                                   meta.cu_q, nh)

    def linear(self, a, w, b=None, act: str = "none", out=None, scale: float = 1.0):
        """act(a w^T + b) in bf16; out: the caller's rows; scale: common factor
        of a gated activation's halves, or the clamped one's limit."""
        if act in ("gelu_mul", "clamped_glu") or out is not None:
            return self._linear_into(a, w, act, out, scale)
        code = _EPI[act]
        g = self._gemv_in(a, w.shape[1], code)
        if g is not None:
            x, nc, gw, gb, eps = g
            return self.C.gemv(x, w, b, code, nc, gw, gb, eps, None, None, None, None, None,
                               0, 0, 0, None)
        a = self.materialize(a)
        dec = getattr(self, "decode", False)
        if code == 1 and self.R.blaslt_gelu(a.shape[0], dec) and a.is_contiguous():
            y = self.C.blaslt_linear(a, w, b, code, self.lane)
            if y is not None:
                return y
        if code == 2 and self.R.blaslt_silu(a.shape[0], w.shape[0], dec) and a.is_contiguous():
            y = self.C.blaslt_linear(a, w, b, 0, self.lane)
            if y is not None:
                return self.C.silu_mul(y)
        tiled, splits = self._gemm_kw(a.shape[0], w.shape[0], w.shape[1], 2 if code == 2 else 1)
        return self.C.linear(a, w, b, code, tiled, splits, self.counters)

    def _linear_into(self, a, w, act: str, out, scale: float):
        glu = _GLU.get(act)
        code = _EPI[act] if glu is None else _EPI["silu_mul"]
        g = self._gemv_in(a, w.shape[1], code)
        if g is not None:
            x, nc, gw, gb, eps = g
            return self.C.gemv_into(x, w, code, nc, gw, gb, eps, out, glu or 0, scale)
        a = self.materialize(a)
        tiled, splits = self._gemm_kw(a.shape[0], w.shape[0], w.shape[1], 2 if code == 2 else 1)
        return self.C.linear(a, w, None, code + (glu or 0), tiled, splits, self.counters, out, scale)

    def linear_residual(self, a, w, b, r: Residual, room=None) -> None:
        """x += a w^T + b; `room`: slab rows the caller owns and appends to
        r.pending itself (_slab_splits of them)."""
        M, K = a.shape
        N = w.shape[0]
        if self.fp32:
            self.C.linear_fp32(a, w, r.x)
            return
        if self._gemv_in(a, K, EPI_RESID) is not None:  # adds straight into r.x
            self.C.gemv(a, w, b, EPI_RESID, 0, None, None, 0.0, r.x, None, None, None, None,
                        0, 0, 0, None)
            return
        if self.R.blaslt_resid(M, K, self._decode) and a.is_contiguous() \
                and self.C.blaslt_residual(a, w, b, r.x, self.lane):
            return
        splits = self._resid_splits(M, N, K)
        tiled = self._tiled(M, N)
        # decode split-K: hand the S partial slabs to the next norm (which
        # reads the rows anyway) instead of a last-arriver reduce in the GEMM
        defer = bool(self.R.defer_resid) and not tiled and splits > 1
        slab = self.C.linear_residual(a, w, b, r.x, splits, tiled, self.counters, defer, room)
        if slab is not None and room is None:
            r.pending.append((slab, b))

    def logits(self, xn, w):
        if self.fp32:
            return self.C.linear_fp32(xn, w)
        g = self._gemv_in(xn, w.shape[1], EPI_F32)
        if g is not None:
            x, nc, gw, gb, eps = g
            if not (self.R.segmax and w.shape[0] % 8 == 0 and w.shape[0] > SAMPLER_ONE_LOAD):
                return self.C.gemv(x, w, None, EPI_F32, nc, gw, gb, eps, None, None, None, None,
                                   None, 0, 0, 0, None)
            # one GEMV workgroup = one 8-logit segment: its epilogue writes the
            # segment maxima too, so the single-stream sampler reads ~100
            # candidate segments instead of three passes over a row too long
            # for its one-load path (Llama-3's 128 K vocabulary: sampler 36.4 ->
            # 20.2 us; GPT-2's 50 K rows load once and stay faster without:
            # 15.5 vs 17.2 us; profiles/r6_*_b1_kernel_stats_v2.csv)
            seg = torch.empty(x.shape[0], w.shape[0] // 8, dtype=torch.float32, device=x.device)
            out = self.C.gemv_logits(x, w, nc, gw, gb, eps, seg)
            out._lsd_segmax = seg
            return out
        xn = self.materialize(xn)
        tiled, splits = self.R.logits_kw(xn.shape[0], w.shape[0], w.shape[1], self.concurrency)
        if not (self.R.segmax and tiled and w.shape[0] % 8 == 0):
            return self.C.linear_f32(xn, w, tiled, splits, self.counters)
        # the epilogue also writes each 8-logit segment's maximum; the sampler
        # derives its top-k threshold from them and reads only the segments
        # that reach it (attached to the logits: a slice drops it, and the
        # sampler then scans the full rows)
        seg = torch.empty(xn.shape[0], w.shape[0] // 8, dtype=torch.float32, device=xn.device)
        out = self.C.linear_f32(xn, w, tiled, splits, self.counters, seg)
        out._lsd_segmax = seg
        return out

    def sample(self, logits, samp, vocab: int):
        return self.C.sample(logits, vocab, samp.temperature, samp.top_k, samp.greedy,
                             samp.seeds, samp.step, getattr(logits, "_lsd_segmax", None))

    def sample_into(self, logits, samp, vocab: int, out, meta=None) -> None:
        # one kernel: draw into `out`, advance the per-row sampler counters
        # and (meta given) the decode batch's positions
        self.C.sample_into(logits, vocab, samp.temperature, samp.top_k, samp.greedy,
                           samp.seeds, samp.step, out, getattr(samp, "active", None),
                           meta.token_pos if meta is not None else None,
                           getattr(logits, "_lsd_segmax", None))

    def gather_rows(self, x, idx):
        return x.index_select(0, idx.long())
