"""Pure-PyTorch reference implementations of every op the engine uses.

These are the *semantics* the hand-written HIP kernels in `csrc/kernels/`
must reproduce; they also run the whole engine on CPU (tests, golden
numerics).  They compute in fp32 regardless of input dtype.

Op semantics follow HF GPT-2, which the reference delegates to
(`/root/reference/server.py:79-102`; [tf5.15] models/gpt2/modeling_gpt2.py):
  * LayerNorm eps 1e-5, affine (K4)
  * Conv1D = x @ W + b, with W stored [in, out] by HF; we store W^T [out, in]
  * gelu_new = tanh-approximation GELU (K11, [tf5.15] activations.py:59-66)
  * causal softmax(QK^T / sqrt(hd)) V (K7) -- the causal mask is explicit here
    (the reference gets causality only implicitly through SDPA, quirk Q3).
Llama ops (RMSNorm, RoPE, SwiGLU, GQA) follow [tf5.15] models/llama.
"""
from __future__ import annotations

import math
from typing import Optional

import torch
import torch.nn.functional as F

UNIT_EPS = 1e-6  # inside the root of a unit vector's length (fixed by the design)
_GELU_C = math.sqrt(2.0 / math.pi)


def gelu_new(x: torch.Tensor) -> torch.Tensor:
    return 0.5 * x * (1.0 + torch.tanh(_GELU_C * (x + 0.044715 * torch.pow(x, 3.0))))


def embed(ids: torch.Tensor, pos: torch.Tensor, wte: torch.Tensor,
          wpe: Optional[torch.Tensor]) -> torch.Tensor:
    """x[t] = wte[ids[t]] + wpe[pos[t]]  -> fp32 [T, H]."""
    x = wte.index_select(0, ids.long()).float()
    if wpe is not None:
        x = x + wpe.index_select(0, pos.long()).float()
    return x


def layernorm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    return F.layer_norm(x.float(), (x.shape[-1],), w.float(), b.float(), eps)


def rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float, offset: float = 0.0) -> torch.Tensor:
    """offset 1: weights stored around zero (gain 1 + w)."""
    xf = x.float()
    var = xf.pow(2).mean(-1, keepdim=True)
    return xf * torch.rsqrt(var + eps) * (w.float() + offset)


def group_rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float, groups: int) -> torch.Tensor:
    """`groups` equal consecutive parts of a row, each over its own root mean square."""
    xf = x.float().view(*x.shape[:-1], groups, -1)
    return (xf * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps)).view(x.shape) * w.float()


def linear(a: torch.Tensor, w: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """a [T, K] @ w[N, K]^T (+ bias) in fp32."""
    out = a.float() @ w.float().t()
    if bias is not None:
        out = out + bias.float()
    return out


def silu_mul(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    g = gate.float()
    return g * torch.sigmoid(g) * up.float()


def rope_cos_sin(pos: torch.Tensor, head_dim: int, theta: float):
    inv = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float64) / head_dim))
    ang = pos.double()[:, None] * inv[None, :]
    return ang.cos().float(), ang.sin().float()  # [T, hd/2]


def apply_rope(x: torch.Tensor, pos: torch.Tensor, theta: float) -> torch.Tensor:
    """HF rotate_half convention: pairs (i, i + hd/2).  x: [T, nh, hd]."""
    hd = x.shape[-1]
    cos, sin = rope_cos_sin(pos.to(torch.float64), hd, theta)
    cos = cos.to(x.device)[:, None, :]
    sin = sin.to(x.device)[:, None, :]
    x1, x2 = x[..., : hd // 2].float(), x[..., hd // 2:].float()
    return torch.cat([x1 * cos - x2 * sin, x2 * cos + x1 * sin], dim=-1)


def kv_append(k_cache: torch.Tensor, v_cache: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
              slots: torch.Tensor, pos: torch.Tensor) -> None:
    """Cache layout [slots, n_kv, max_seq, hd]; k, v: [T, n_kv, hd]."""
    s, p = slots.long(), pos.long()
    k_cache[s, :, p, :] = k.to(k_cache.dtype)
    v_cache[s, :, p, :] = v.to(v_cache.dtype)


def attention(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
              seq_slots: torch.Tensor, q_start: torch.Tensor, cu_q: torch.Tensor) -> torch.Tensor:
    """Causal attention of packed queries over the KV cache.

    q: [T, nh, hd] packed; sequence i owns rows cu_q[i]:cu_q[i+1], whose
    positions are q_start[i] + j.  Keys/values for sequence i live at
    k_cache[seq_slots[i], :, 0:q_start[i]+len_i].  GQA: nh % n_kv == 0.
    Returns fp32 [T, nh, hd].
    """
    nh, hd = q.shape[1], q.shape[2]
    n_kv = k_cache.shape[1]
    grp = nh // n_kv
    out = torch.empty(q.shape, dtype=torch.float32, device=q.device)
    scale = 1.0 / math.sqrt(hd)
    for i in range(seq_slots.numel()):
        a, b = int(cu_q[i]), int(cu_q[i + 1])
        if b == a:
            continue
        st = int(q_start[i])
        L = st + (b - a)
        s = int(seq_slots[i])
        kk = k_cache[s, :, :L].float().repeat_interleave(grp, dim=0)  # [nh, L, hd]
        vv = v_cache[s, :, :L].float().repeat_interleave(grp, dim=0)
        qq = q[a:b].float().transpose(0, 1)  # [nh, Lq, hd]
        sc = torch.matmul(qq, kk.transpose(1, 2)) * scale  # [nh, Lq, L]
        qpos = torch.arange(st, L, device=q.device)[:, None]
        kpos = torch.arange(L, device=q.device)[None, :]
        sc = sc.masked_fill(kpos > qpos, float("-inf"))
        p = torch.softmax(sc, dim=-1)
        out[a:b] = torch.matmul(p, vv).transpose(0, 1)
    return out


def paged_rows(table: torch.Tensor, slots: torch.Tensor, pos: torch.Tensor, page: int) -> torch.Tensor:
    """Flat cache rows (page * page size + offset) of positions `pos` of `slots`."""
    s, p = slots.long(), pos.long()
    return table[s, p // page].long() * page + p % page


def latent_append(pool: torch.Tensor, table: torch.Tensor, c: torch.Tensor, slots, pos) -> None:
    """pool [pages, page, rank]; c [T, rank]."""
    rows = paged_rows(table, slots, pos, pool.shape[1])
    pool.view(-1, pool.shape[2])[rows] = c.to(pool.dtype)


def latent_attention(q: torch.Tensor, pool: torch.Tensor, table: torch.Tensor, seq_slots, q_start, cu_q,
                     scale: float, window: Optional[int], vdim: Optional[int] = None,
                     sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """q [T, heads, columns] in the latent space; the cached rows are keys of every
    head, their first vdim columns (None: all) the values.  Query at position i
    sees i - window < j <= i; sink [heads]: a further score without a value.
    Returns fp32 [T, heads, vdim]."""
    vdim = q.shape[2] if vdim is None else vdim
    out = torch.empty(*q.shape[:2], vdim, dtype=torch.float32, device=q.device)
    flat = pool.view(-1, pool.shape[2])
    for i in range(seq_slots.numel()):
        a, b = int(cu_q[i]), int(cu_q[i + 1])
        if b == a:
            continue
        st, end = int(q_start[i]), int(q_start[i]) + b - a
        lo = 0 if window is None else max(0, st - window + 1)
        kpos = torch.arange(lo, end, device=q.device)
        c = flat[paged_rows(table, seq_slots[i].expand_as(kpos), kpos, pool.shape[1])].float()[:, : q.shape[2]]
        s = torch.matmul(q[a:b].float().transpose(0, 1), c.t()) * scale  # [heads, Lq, keys]
        d = torch.arange(st, end, device=q.device)[:, None] - kpos[None, :]
        hide = d < 0 if window is None else (d < 0) | (d >= window)
        s = s.masked_fill(hide, float("-inf"))
        if sink is not None:
            s = torch.cat([s, sink[:, None, None].expand(-1, b - a, 1)], 2)
        p = torch.softmax(s, dim=-1)[..., : kpos.numel()]
        out[a:b] = torch.matmul(p, c[:, :vdim]).transpose(0, 1)
    return out


def partial_rope(x: torch.Tensor, pos: torch.Tensor, rope) -> torch.Tensor:
    """x [T, heads, dim]: pairs (i, i + dims / 2), or (2i, 2i + 1) where the
    layout is interleaved, of the first rope.dims dimensions turn."""
    if rope is None or rope.dims == 0:
        return x
    half = rope.dims // 2
    ang = pos.double()[:, None] * torch.tensor(rope.frequencies(), dtype=torch.float64, device=pos.device)
    cos, sin = ang.cos().float()[:, None], ang.sin().float()[:, None]
    if rope.interleaved:
        a, b = x[..., 0: 2 * half: 2].float(), x[..., 1: 2 * half: 2].float()
        turned = torch.stack([a * cos - b * sin, b * cos + a * sin], -1).flatten(-2)
        return torch.cat([turned, x[..., 2 * half:].float()], -1)
    a, b = x[..., :half].float(), x[..., half: 2 * half].float()
    return torch.cat([a * cos - b * sin, b * cos + a * sin, x[..., 2 * half:].float()], -1)


def paged_append(pool: torch.Tensor, table: torch.Tensor, x: torch.Tensor, slots, pos) -> None:
    """pool [pages, heads, page, dim]; x [T, heads, dim]."""
    page = pool.shape[2]
    pg = table[slots.long(), pos.long() // page].long()
    pool[pg, :, pos.long() % page] = x.to(pool.dtype)


def talking_attention(q, k_pool, v_pool, table, seq_slots, q_start, cu_q, talk, scale: float,
                      softcap: Optional[float], window: Optional[int], talk_weights: bool = False,
                      slopes: Optional[torch.Tensor] = None, keep_first: int = 0) -> torch.Tensor:
    """q [T, heads, dim] over paged keys and values [pages, kv heads, page, .]:
    scores are capped, lessened by slopes [heads] times the distance, mixed over
    the heads (talk [heads, heads]; talk_weights: behind the softmax) and
    softmaxed over i - window < j <= i and j < keep_first.  Returns fp32
    [T, heads, vdim]."""
    T, H, _ = q.shape
    page, grp = k_pool.shape[2], H // k_pool.shape[1]
    out = torch.empty(T, H, v_pool.shape[3], dtype=torch.float32, device=q.device)
    for i in range(seq_slots.numel()):
        a, b = int(cu_q[i]), int(cu_q[i + 1])
        if b == a:
            continue
        st, end = int(q_start[i]), int(q_start[i]) + b - a
        lo = 0 if window is None else max(0, st - window + 1)
        kpos = torch.arange(lo, end, device=q.device)
        kpos = torch.cat([torch.arange(min(lo, keep_first), device=q.device), kpos])
        pg = table[int(seq_slots[i]), kpos // page].long()
        k, v = (p[pg, :, kpos % page].float().transpose(0, 1).repeat_interleave(grp, 0) for p in (k_pool, v_pool))
        s = torch.matmul(q[a:b].float().transpose(0, 1), k.transpose(1, 2)) * scale  # [heads, Lq, keys]
        if softcap is not None:
            s = softcap * torch.tanh(s / softcap)
        d = torch.arange(st, end, device=q.device)[:, None] - kpos[None, :]
        if slopes is not None:
            s = s - slopes[:, None, None] * d
        mix = lambda x: x if talk is None else torch.matmul(talk.float(), x.reshape(H, -1)).view_as(x)  # noqa: E731
        if not talk_weights:
            s = mix(s)
        hide = d < 0 if window is None else (d < 0) | ((d >= window) & (kpos >= keep_first))
        p = torch.softmax(s.masked_fill(hide, float("-inf")), -1)
        out[a:b] = torch.matmul(mix(p) if talk_weights else p, v).transpose(0, 1)
    return out


def unit(x: torch.Tensor) -> torch.Tensor:
    return x * torch.rsqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def ring_conv(x: torch.Tensor, taps: torch.Tensor, bias, ring: torch.Tensor, meta) -> torch.Tensor:
    """Causal convolution per channel of packed rows x [T, channels] (last
    column of taps: the current token).  ring [slots, taps, channels] holds the
    inputs of positions p at p % taps and is brought up to date."""
    n = taps.shape[1]
    out = torch.empty_like(x, dtype=torch.float32)
    for i in range(meta.seq_slots.numel()):
        a, b, st, slot = int(meta.cu_q[i]), int(meta.cu_q[i + 1]), int(meta.q_start[i]), int(meta.seq_slots[i])
        past = [ring[slot, p % n].float() if p >= 0 else torch.zeros(x.shape[1]) for p in range(st - n + 1, st)]
        rows = torch.cat([torch.stack(past), x[a:b].float()]) if past else x[a:b].float()
        out[a:b] = sum(rows[j: j + b - a] * taps[:, j].float() for j in range(n))
        for p in range(max(st, st + b - a - n), st + b - a):
            ring[slot, p % n] = x[a + p - st].to(ring.dtype)
    return out if bias is None else out + bias.float()


def _scan(meta, state: torch.Tensor, step) -> None:
    """step(t, S) -> S over every token of every sequence; a sequence's state
    [heads, rows, vdim] starts at zero and is kept in state[slot]."""
    for i in range(meta.seq_slots.numel()):
        a, b, slot = int(meta.cu_q[i]), int(meta.cu_q[i + 1]), int(meta.seq_slots[i])
        S = state[slot].clone() if int(meta.q_start[i]) > 0 else torch.zeros_like(state[slot])
        for t in range(a, b):
            S = step(t, S)
        state[slot] = S


def delta_rule(q, k, v, g, beta, state, meta) -> torch.Tensor:
    """S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.
    q, k, g [T, H, D], v [T, H, V], beta [T, H], state [slots, H, D, V]."""
    out = torch.empty(v.shape, dtype=torch.float32)

    def step(t, S):
        S = g[t][..., None] * S
        u = beta[t][:, None] * (v[t] - torch.matmul(k[t][:, None], S)[:, 0])
        S = S + k[t][..., None] * u[:, None]
        out[t] = torch.matmul(q[t][:, None], S)[:, 0]
        return S
    _scan(meta, state, step)
    return out


def ssd(x, B, C, dt, decay, state, meta) -> torch.Tensor:
    """S <- decay S + dt B x^T; y = S^T C.  x [T, H, V], B, C [T, H, N]."""
    out = torch.empty(x.shape, dtype=torch.float32)

    def step(t, S):
        S = decay[t][:, None, None] * S + B[t][..., None] * (dt[t][:, None] * x[t])[:, None]
        out[t] = torch.matmul(C[t][:, None], S)[:, 0]
        return S
    _scan(meta, state, step)
    return out


def forget_rule(q, k, v, state, meta) -> torch.Tensor:
    """S <- diag(1 - k) S + k v^T; o = S^T q.  q, k [T, H, D], v [T, H, V],
    state [slots, H, D, V]."""
    out = torch.empty(v.shape, dtype=torch.float32)

    def step(t, S):
        S = S + k[t][..., None] * (v[t][:, None] - S)
        out[t] = torch.matmul(q[t][:, None], S)[:, 0]
        return S
    _scan(meta, state, step)
    return out


def tanh_norm(x: torch.Tensor, alpha: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """Dynamic tanh: no statistics of the row."""
    return torch.tanh(alpha.float() * x.float()) * w.float() + b.float()


def token_shift(h: torch.Tensor, amount: torch.Tensor, last: torch.Tensor, meta) -> torch.Tensor:
    """Packed rows, each moved towards its sequence's previous one by `amount` per
    column; last [slots, width] holds the row before a portion (zeros before
    position 0) and is brought up to date."""
    out = torch.empty_like(h)
    for i in range(meta.seq_slots.numel()):
        a, b, slot = int(meta.cu_q[i]), int(meta.cu_q[i + 1]), int(meta.seq_slots[i])
        if b == a:
            continue
        first = last[slot: slot + 1] if int(meta.q_start[i]) > 0 else torch.zeros_like(h[:1])
        before = torch.cat([first, h[a: b - 1]])
        out[a:b] = h[a:b] + (before - h[a:b]) * amount.float()
        last[slot] = h[b - 1]
    return out


def route_softmax(z: torch.Tensor, top: int):
    """Router logits [T, E] -> (expert ids [T, top], weights [T, top]): the largest
    logits choose, their softmax weighs."""
    z, ids = torch.topk(z.float(), top, dim=-1)
    return ids, torch.softmax(z, -1)


def route(z: torch.Tensor, correction: torch.Tensor, top: int):
    """Router logits [T, E] -> (expert ids [T, top], weights [T, top]): the
    corrected sigmoid scores choose, the plain ones weigh."""
    s = torch.sigmoid(z.float())
    ids = torch.topk(s + correction.float(), top, dim=-1).indices
    w = s.gather(1, ids)
    return ids, w / (w.sum(-1, keepdim=True) + 1e-20)


def clamped_glu(gate: torch.Tensor, up: torch.Tensor, limit: Optional[float], alpha: float) -> torch.Tensor:
    """limit None: plain SiLU(gate) * up."""
    if limit is None:
        return silu_mul(gate, up)
    g = gate.clamp(max=limit)
    return g * torch.sigmoid(alpha * g) * (up.clamp(-limit, limit) + 1)


def expert(h: torch.Tensor, gate_up: torch.Tensor, down: torch.Tensor, limit: Optional[float], alpha: float) -> torch.Tensor:
    y = linear(h, gate_up)
    f = y.shape[1] // 2
    return linear(clamped_glu(y[:, :f], y[:, f:], limit, alpha), down)


def moe(h: torch.Tensor, ids: torch.Tensor, w: torch.Tensor, gate_up: torch.Tensor, down: torch.Tensor,
        limit: Optional[float], alpha: float) -> torch.Tensor:
    out = torch.zeros(h.shape[0], down.shape[1], dtype=torch.float32, device=h.device)
    for e in ids.unique().tolist():
        t, k = (ids == e).nonzero(as_tuple=True)
        out.index_add_(0, t, expert(h[t], gate_up[e], down[e], limit, alpha) * w[t, k][:, None])
    return out


def sample(logits: torch.Tensor, temperature: torch.Tensor, top_k: torch.Tensor,
           greedy: torch.Tensor, uniforms: torch.Tensor, vocab: int) -> torch.Tensor:
    """Per-row sampler.  Reference semantics (server.py:187-206):
    logits/T -> topk(k) -> softmax over the k values -> draw -> map to vocab id.
    `uniforms` [B] in [0,1) drive the draw (inverse CDF over the top-k sorted
    descending), so the result is a deterministic function of its inputs.
    greedy rows return argmax (lowest index on ties).
    """
    B = logits.shape[0]
    lg = logits[:, :vocab].float()
    out = torch.empty(B, dtype=torch.int32, device=logits.device)
    for r in range(B):
        row = lg[r]
        if bool(greedy[r]):
            out[r] = int(torch.argmax(row))
            continue
        k = int(top_k[r])
        vals, idx = torch.topk(row / float(temperature[r]), k)
        # stable ordering for ties: by value desc then index asc
        order = sorted(range(k), key=lambda j: (-float(vals[j]), int(idx[j])))
        vals, idx = vals[order], idx[order]
        p = torch.softmax(vals, dim=-1)
        c = torch.cumsum(p, 0)
        u = float(uniforms[r]) * float(c[-1])
        j = int(torch.searchsorted(c, torch.tensor([u], dtype=c.dtype)).clamp(max=k - 1))
        out[r] = int(idx[j])
    return out
