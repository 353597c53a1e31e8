"""Op backends.

The model code (models/stage.py: the blocks of one pipeline stage) is written once against the `Backend` interface below.  Two implementations exist:

* `ReferenceBackend` -- plain PyTorch in fp32 (ops/reference.py).  Used on CPU
  (tests, golden numerics, the tiny-gpt2 reference config).
* `HipBackend` (ops/hip.py) -- the hand-written CDNA4 kernels in
  csrc/kernels/*.hip, routed by one table (ops/routing.py).  Used for every
  tensor on a GPU; hipBLASLt only runs when an A/B run asks for it
  (LSD_ROUTING=blaslt=1).  There is no silent fallback: if the extension is
  missing on a GPU box, `get_backend` raises.

Residual stream convention: the residual `x` is fp32 [T, H].  GEMMs whose
epilogue is "add into the residual" may split K across workgroups; their
fp32 partial slabs are parked in `Residual.pending` and folded into `x` by the
next norm (or `flush`).  This keeps the reduction deterministic and costs no
extra kernel launch.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import List, Optional, Tuple

import torch

from ..config import AttentionSpec, ChannelDeltaSpec
from ..runtime.kv_cache import LayerCache, layer_cache
from . import reference as ref


@dataclass
class Residual:
    x: torch.Tensor  # fp32 [T, H]
    pending: List[Tuple[torch.Tensor, Optional[torch.Tensor]]] = field(default_factory=list)
    # output of a sublayer that is normed before it is added, folded in by the
    # next norm or flush
    post: Optional["PostNorm"] = None


@dataclass
class PostNorm:
    """A sublayer's output [S, T, H] (split-K slabs) on its way through a norm
    into the residual: RMS in equal parts (weight, model config), or elementwise
    (alpha, weight, bias)."""

    slab: torch.Tensor
    bias: Optional[torch.Tensor] = None
    rms: Optional[tuple] = None   # (weight, parts, columns, eps)
    tanh: Optional[tuple] = None  # (alpha, weight, bias)


# sigmoid slope of the experts' gated activation (fixed by the design)
GLU_ALPHA = 1.702


class Backend:
    name = "abstract"

    def prepare_stage(self, stage) -> None:  # optional weight re-layout
        pass

    def row_width(self, mcfg) -> int:
        """Columns of the residual rows (>= hidden; the rest stays zero)."""
        return mcfg.hidden

    def latent_width(self, rank: int) -> int:
        """Columns of a cached latent row (>= rank; the rest stays zero)."""
        return rank

    def value_width(self, mixer) -> int:
        """Columns of a value head (>= vdim; the rest stays zero)."""
        return mixer.vdim

    def layer_cache(self, mixer, shift: int = 0) -> LayerCache:
        """What a layer keeps per page and per slot (runtime/kv_cache.py)."""
        return layer_cache(mixer, shift=shift)

    def norm_width(self, mcfg) -> int:
        """`width` argument of the norms: the true row width where rows are padded, else 0."""
        return mcfg.hidden if self.row_width(mcfg) != mcfg.hidden else 0

    @staticmethod
    def _parts(meta):
        """(rows, meta) of a step's decode rows and prompt chunks."""
        if getattr(meta, "dec", None) is not None:
            return [(slice(0, meta.b), meta.dec), (slice(meta.b, meta.num_tokens), meta.pf)]
        return [(slice(0, meta.num_tokens), meta)]

    def prepare_prefill(self, meta, mcfg) -> None:
        """Device-side helpers of a prefill batch, made before a graph capture."""


class ReferenceBackend(Backend):
    """fp32 PyTorch implementation of the engine ops (CPU golden path)."""

    name = "reference"

    def embed(self, ids, pos, wte, wpe, scale: float = 1.0):
        x = ref.embed(ids, pos, wte, wpe)
        return x if scale == 1.0 else x * scale

    def _combine(self, r: Residual) -> None:
        for slabs, bias in r.pending:
            r.x += slabs.sum(0)
            if bias is not None:
                r.x += bias.float()
        r.pending.clear()

    def flush(self, r: Residual) -> torch.Tensor:
        self._combine(r)
        return r.x

    def layernorm(self, r: Residual, w, b, eps):
        self._combine(r)
        return ref.layernorm(r.x, w, b, eps)

    def rmsnorm(self, r: Residual, w, eps, offset: float = 0.0, width: int = 0):
        self._combine(r)
        return ref.rmsnorm(r.x, w, eps, offset)

    def norm_rows(self, x, w, b, eps, rms: bool, rows=None, offset: float = 0.0, width: int = 0):
        if rows is not None:
            x = x.index_select(0, rows.long())
        return ref.rmsnorm(x, w, eps, offset) if rms else ref.layernorm(x, w, b, eps)

    # -- latent attention and experts (models/stage.py _parallel_layer) -------
    # `w(name)`: the layer's tensors; `pool`: its cache layer (kv.pools)
    def latent_project(self, h, w, m, mlp, kv, pool, meta, eps):
        """Queries [T, heads, rank + turned part] in the latent space, the output
        gate's logits (None: no gate) and, for experts `mlp` that read the same
        rows, the routing (ids, weights); a layer with its own latents appends
        them to the cache."""
        pos = meta.token_pos
        if m.kv_from is None:
            c, kr = ref.linear(h, w("attn.dkv.weight")).split([m.kv_rank, m.rot_dim], 1)
            c = torch.cat([ref.rmsnorm(c, w("attn.dkv_norm.weight"), eps), ref.partial_rope(kr[:, None], pos, m.rope)[:, 0]], 1)
            ref.latent_append(pool, kv.table, c, meta.token_slots, pos)
        if m.q_rank is None:
            q = ref.linear(h, w("attn.q.weight"))
        else:
            q = ref.linear(ref.rmsnorm(ref.linear(h, w("attn.dq.weight")), w("attn.dq_norm.weight"), eps), w("attn.uq.weight"))
        q, qr = q.reshape(-1, m.heads, m.q_dim).split([m.dim, m.rot_dim], 2)
        uk = w("attn.uk.weight").float().reshape(m.heads, m.dim, m.kv_rank)
        q = torch.matmul(q.transpose(0, 1), uk).transpose(0, 1)
        q = torch.cat([q, ref.partial_rope(qr, pos, m.rope)], 2)
        gate = ref.linear(h, w("attn.g.weight")) if m.gate else None
        routing = None
        if mlp is not None:
            z = ref.linear(h, w("mlp.router.weight"))
            routing = ref.route(z, w("mlp.correction"), mlp.top)
        return q, gate, routing

    def latent_attention(self, q, gate, w, m, kv, pool, meta):
        sink = w("attn.sink").float() if m.sink else None
        o = torch.cat([ref.latent_attention(q[s], pool, kv.table, mt.seq_slots, mt.q_start, mt.cu_q, m.scale, m.window,
                                            m.kv_rank, sink) for s, mt in self._parts(meta)])
        uv = w("attn.uv.weight").float().reshape(m.heads, m.vdim, m.kv_rank)
        o = torch.matmul(o.transpose(0, 1), uv.transpose(1, 2)).transpose(0, 1)
        o = o.reshape(o.shape[0], -1)
        return o if gate is None else o * torch.sigmoid(gate)

    def parallel_residual(self, o, h, routing, w, spec, r: Residual) -> None:
        """x += o W_o^T + experts(h): both halves of a parallel block."""
        self.linear_residual(o, w("attn.o.weight"), None, r)
        if spec is None:
            return
        r.x += self._experts(h, routing, w, spec)

    def _experts(self, h, routing, w, spec):
        ids, wts = routing
        y = ref.moe(h, ids, wts, w("mlp.experts.gate_up.weight"), w("mlp.experts.down.weight"), spec.expert.limit,
                    GLU_ALPHA)
        if spec.shared is not None:
            z = ref.expert(h, w("mlp.shared.gate_up.weight"), w("mlp.shared.down.weight"), spec.shared.limit, GLU_ALPHA)
            y = y + (z * torch.sigmoid(ref.linear(h, w("mlp.shared.sg"))) if spec.shared_gate else z)
        return y

    # -- layers with elementwise norms (models/stage.py _token_layer); a norm is
    # n(".weight"), n(".bias") and one number n(".alpha") --------------------------
    def tanh_norm(self, r: Residual, n):
        self._combine(r)
        return ref.tanh_norm(r.x, n(".alpha"), n(".weight"), n(".bias"))

    def tanh_norm_rows(self, x, n, rows=None):
        return self.tanh_norm(Residual(x if rows is None else x.index_select(0, rows.long())), n)

    def shift_norm(self, r: Residual, w, last, meta, mcfg):
        """The layer's first norm, its rows moved towards the previous token's by
        w("shift"); `last` [slots, hidden]: the previous portion's last row."""
        h = self.tanh_norm(r, lambda n: w("norm1" + n))
        return torch.cat([ref.token_shift(h[s], w("shift"), last, mt) for s, mt in self._parts(meta)])

    def linear_tanh(self, a, wt, n, r: Residual) -> None:
        """x += norm(a wt^T)."""
        self._combine(r)
        r.x += self.tanh_norm(Residual(ref.linear(a, wt)), n)

    def experts_tanh(self, h, w, mlp, n, r: Residual) -> None:
        """x += norm(experts(h))."""
        self._combine(r)
        routing = ref.route_softmax(ref.linear(h, w("mlp.router.weight")), mlp.top)
        r.x += self.tanh_norm(Residual(self._experts(h, routing, w, mlp)), n)

    def token_side(self, r: Residual, ids, w, mcfg) -> None:
        """x += rms(proj(gelu(gate x) * e)) * norm, e the tokens' rows of the layer's table."""
        self._combine(r)
        g = ref.gelu_new(ref.linear(r.x, w("side.gate"))) * w("side.embed").index_select(0, ids.long()).float()
        r.x += ref.rmsnorm(ref.linear(g, w("side.proj")), w("side.norm"), mcfg.norm_eps)

    def forget_mix(self, h, w, m, state, meta, eps):
        """Recurrence with forget gates before W_o [T, heads * vdim]."""
        T, H, D, V = h.shape[0], m.heads, m.dim, m.vdim
        q = torch.nn.functional.silu(ref.linear(h, w("mixer.q"))).view(T, H, D)
        # 1 - f, formed without cancellation where f is close to one
        k = (1 - w("mixer.lower").float()) * torch.sigmoid(-ref.linear(h, w("mixer.f"), w("mixer.f.b")))
        k, v = k.view(T, H, D), ref.linear(h, w("mixer.v")).view(T, H, V)
        o = torch.cat([ref.forget_rule(q[s], k[s], v[s], state, mt) for s, mt in self._parts(meta)])
        return ref.rmsnorm(o, w("mixer.norm"), eps).view(T, H * V)

    # -- mixers of models/stage.py _mixer_layer --------------------------------
    def loop_enter(self, r: Residual, x0, w_in, step, t: int) -> None:
        """x <- W_in [x; x0] + step[t]: a pass of the looped layers begins."""
        self._combine(r)
        r.x.copy_(ref.linear(torch.cat([r.x, x0], 1), w_in) + step[t].float())

    def unit_rmsnorm(self, r: Residual, mcfg):
        self._combine(r)
        return ref.rmsnorm(r.x, r.x.new_ones(r.x.shape[1]), mcfg.norm_eps)

    def mix(self, h, w, spec, kv, entry, meta, eps):
        """Mixer output before W_o [T, heads * vdim] fp32; `entry`: the layer's
        cache tensors (kv.entries)."""
        m = spec.mixer
        h = h * w("input_layernorm.weight").float()
        fn = (self._attend if isinstance(m, AttentionSpec) else
              self._channel_delta if isinstance(m, ChannelDeltaSpec) else self._ssm)
        return fn(h, w, m, kv, entry, meta, eps)

    def _attend(self, h, w, m, kv, entry, meta, eps):
        return self.attend(h, w, m, kv, entry, meta, eps, None)[0]

    def _channel_delta(self, h, w, m, kv, entry, meta, eps):
        T, H, G, D, V = h.shape[0], m.heads, m.kv_heads, m.dim, m.vdim
        x = torch.cat([ref.linear(h, w(f"mixer.{n}")) for n in "qkv"], 1)
        taps = torch.cat([w(f"mixer.{n}.conv") for n in "qkv"])
        dt = ref.linear(ref.linear(h, w("mixer.a1")), w("mixer.a2")) + w("mixer.dt_bias").float()
        g = torch.exp(-torch.exp(w("mixer.A_log").float())[:, None] * torch.nn.functional.softplus(dt).view(T, H, D))
        beta = torch.sigmoid(ref.linear(h, w("mixer.b")))
        o = torch.empty(T, H, V)
        for s, mt in self._parts(meta):
            y = torch.nn.functional.silu(ref.ring_conv(x[s], taps, None, entry[1], mt))
            q, k, v = y.split([G * D, G * D, H * V], 1)
            q, k = (ref.unit(u.reshape(-1, G, D)).repeat_interleave(H // G, 1) for u in (q, k))
            o[s] = ref.delta_rule(q * D ** -0.5, k, v.reshape(-1, H, V), g[s], beta[s], entry[0], mt)
        o = ref.rmsnorm(o, w("mixer.norm"), eps)
        return o.view(T, H * V) * torch.sigmoid(ref.linear(ref.linear(h, w("mixer.g1")), w("mixer.g2")))

    def _ssm(self, h, w, m, kv, entry, meta, eps):
        T, H, G, V, N = h.shape[0], m.heads, m.groups, m.vdim, m.state
        z, x, dt = ref.linear(h, w("mixer.in")).split([m.inner, m.conv_channels, H], 1)
        dt = torch.nn.functional.softplus(dt + w("mixer.dt_bias").float())
        decay = torch.exp(-torch.exp(w("mixer.A_log").float()) * dt)
        y = torch.empty(T, H, V)
        for s, mt in self._parts(meta):
            c = torch.nn.functional.silu(ref.ring_conv(x[s], w("mixer.conv"), w("mixer.conv.b"), entry[1], mt))
            u, B, C = c.split([m.inner, G * N, G * N], 1)
            B, C = (t.reshape(-1, G, N).repeat_interleave(H // G, 1) for t in (B, C))
            u = u.reshape(-1, H, V)
            y[s] = ref.ssd(u, B, C, dt[s], decay[s], entry[0], mt) + w("mixer.D").float()[:, None] * u
        y = (y.view(T, -1) * torch.nn.functional.silu(z)).view(T, m.norm_groups, -1)
        return ref.rmsnorm(y, y.new_ones(y.shape[-1]), eps).view(T, -1) * w("mixer.norm").float()

    # -- layers with norms around each sublayer (models/stage.py _sandwich_layer) ----
    def group_norm(self, r: Residual, w, mcfg):
        self._combine(r)
        return ref.group_rmsnorm(r.x, w, mcfg.norm_eps, mcfg.norm_groups)

    def group_norm_rows(self, x, w, mcfg, rows=None):
        x = x if rows is None else x.index_select(0, rows.long())
        return ref.group_rmsnorm(x, w, mcfg.norm_eps, mcfg.norm_groups)

    def linear_post_norm(self, a, w, b, norm_w, r: Residual, mcfg) -> None:
        """x += norm(a w^T + b)."""
        self._combine(r)
        r.x += ref.group_rmsnorm(ref.linear(a, w, b), norm_w, mcfg.norm_eps, mcfg.norm_groups)

    def clamped_glu(self, h, w, limit: float):
        y = ref.linear(h, w)
        f = y.shape[1] // 2
        return ref.clamped_glu(y[:, :f], y[:, f:], limit, GLU_ALPHA)

    def attend(self, h, w, m: AttentionSpec, kv, entry, meta, eps, first_values, keep_values: bool = False):
        """Attention before the output projection [T, heads * vdim], and with
        keep_values this layer's values [T, kv heads * vdim].  first_values: rows
        that are mixed into the values (None: they stay as they are)."""
        qkv = torch.cat([ref.linear(h, w(f"mixer.{n}"), w(f"mixer.{n}.b", None)) for n in "qkv"], 1)
        if m.conv:
            taps, x = torch.cat([w(f"mixer.{n}.conv") for n in "qkv"]), qkv
            qkv = torch.cat([ref.ring_conv(x[s], taps, None, entry[2], mt) for s, mt in self._parts(meta)])
        G, pos = m.kv_heads, meta.token_pos
        q, k, v = qkv.split([m.heads * m.dim, G * m.dim, G * m.vdim], 1)
        q, k = q.reshape(-1, m.heads, m.dim), k.reshape(-1, G, m.dim)
        if m.qk_norm:
            q, k = (ref.rmsnorm(t, t.new_ones(m.dim), eps) for t in (q, k))
        q, k = (ref.partial_rope(t, pos, m.rope) for t in (q, k))
        values = v.contiguous() if keep_values else None
        if first_values is not None:
            lam = w("mixer.vmix").float()
            v = (1 - lam) * v + lam * first_values.float()
        for pool, x in zip(entry, (k, v.reshape(-1, G, m.vdim))):
            ref.paged_append(pool, kv.table, x, meta.token_slots, pos)
        o = self._attention_parts(q, w, m, kv, entry, meta)
        if m.head_gate:
            o = o * torch.sigmoid(ref.linear(h, w("mixer.g")))[..., None]
        return o.reshape(o.shape[0], -1), values

    def _attention_parts(self, q, w, m, kv, entry, meta):
        talk = w("mixer.talk") if m.talking else None
        slopes = torch.tensor(m.slopes()) if m.distance_bias else None
        return torch.cat([ref.talking_attention(q[s], entry[0], entry[1], kv.table, mt.seq_slots, mt.q_start, mt.cu_q,
                                                talk, m.scale, m.softcap, m.window, m.talk_weights, slopes, m.keep_first)
                          for s, mt in self._parts(meta)])

    def mixer_residual(self, o, h, w, spec, r: Residual) -> None:
        """x += o W_o^T + feed-forward(h): both halves of a parallel block."""
        self.linear_residual(o, w("mixer.o"), None, r)
        if spec.mlp is not None:
            y = ref.linear(h * w("post_attention_layernorm.weight").float(), w("mlp.gate_up.weight"))
            f = y.shape[1] // 2
            self.linear_residual(ref.gelu_new(y[:, :f]) * y[:, f:], w("mlp.down_proj.weight"), None, r)

    def qkv_kv_append(self, xn, w, b, cache_k, cache_v, meta, mcfg):
        """QKV projection; K,V appended to the cache at (slot, pos); returns q [T, nh, hd]."""
        y = ref.linear(xn, w, b)
        T = y.shape[0]
        hd = mcfg.head_dim
        q = y[:, : mcfg.q_size].reshape(T, mcfg.n_heads, hd)
        k = y[:, mcfg.q_size: mcfg.q_size + mcfg.kv_size].reshape(T, mcfg.n_kv_heads, hd)
        v = y[:, mcfg.q_size + mcfg.kv_size:].reshape(T, mcfg.n_kv_heads, hd)
        if mcfg.arch == "llama":
            q = ref.apply_rope(q, meta.token_pos.cpu(), mcfg.rope_theta)
            k = ref.apply_rope(k, meta.token_pos.cpu(), mcfg.rope_theta)
        ref.kv_append(cache_k, cache_v, k, v, meta.token_slots, meta.token_pos)
        return q

    def attention(self, q, cache_k, cache_v, meta):
        o = ref.attention(q, cache_k, cache_v, meta.seq_slots, meta.q_start, meta.cu_q)
        return o.reshape(o.shape[0], -1)

    def linear(self, a, w, b=None, act: str = "none"):
        y = ref.linear(a, w, b)
        if act == "gelu":
            y = ref.gelu_new(y)
        elif act == "silu_mul":
            f = y.shape[1] // 2
            y = ref.silu_mul(y[:, :f], y[:, f:])
        return y

    def linear_residual(self, a, w, b, r: Residual) -> None:
        self._combine(r)
        r.x += ref.linear(a, w, b)

    def logits(self, xn, w):
        return ref.linear(xn, w)

    def sample(self, logits, samp, vocab: int):
        return ref.sample(logits, samp.temperature, samp.top_k, samp.greedy,
                          samp.uniforms(), vocab)

    def sample_into(self, logits, samp, vocab: int, out, meta=None) -> None:
        """Decode step: sampled ids into `out`, then the sampler counters (and,
        given the decode `meta`, its positions) advance."""
        out.copy_(self.sample(logits, samp, vocab))
        samp.advance()
        if meta is not None:
            meta.advance()

    def gather_rows(self, x, idx):
        return x.index_select(0, idx.long())


_REFERENCE = ReferenceBackend()


def hip_available() -> bool:
    try:
        from . import hip  # noqa: F401
        return hip.extension_loaded()
    except Exception:  # pragma: no cover - depends on build
        return False


def get_backend(device) -> Backend:
    dev = torch.device(device)
    if dev.type == "cpu":
        return _REFERENCE
    from .hip import HipBackend  # raises loudly if the extension is missing

    return HipBackend()  # one per stage: owns that stage's split-K counters / tables
