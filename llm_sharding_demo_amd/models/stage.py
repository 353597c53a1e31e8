"""One pipeline stage of a GPT-2, Llama, Timisun, Vizalix, Kedasun or Fagunex model.

Generalises the reference's two hard-wired shards (`server.py:51-105`):
  * ShardA (`server.py:68-86`): wte + wpe + blocks[0:split]   -> stage 0
  * ShardB (`server.py:90-103`): blocks[split:] + ln_f + lm_head -> stage P-1
to P stages with an arbitrary layer range each.  Differences by design:
  * a stage materialises only its own layers (quirk Q4),
  * the causal mask is explicit in the attention op (quirk Q3),
  * K/V are appended to the shard-local cache, so decode processes one token
    per sequence (quirk Q5),
  * the last stage computes lm_head for the last position of each sequence
    only (quirk Q6) unless `all_logits` is requested (compat /forward_b),
  * a stage boundary may fall between the attention and the MLP half of a
    layer (`units`, parallel/partition.py): unit 2i = attention half of layer
    i, unit 2i+1 = its MLP half.  Only the residual stream crosses either kind
    of boundary; the KV cache of layer i lives with its attention half.
"""
from __future__ import annotations

import functools
from typing import Dict, Optional, Sequence, Tuple

import torch

from ..config import ID_DIGITS, ForgetSpec, ModelConfig
from ..ops import Residual, get_backend
from ..runtime.batch import BatchMeta
from ..runtime.kv_cache import KVCache, LatentCache, PagedCache
from .weights import layer_half, maybe_load, stage_tensor_shapes


class StageModel:
    def __init__(self, cfg: ModelConfig, layer_start: int, layer_end: int, first: bool,
                 last: bool, device="cpu", dtype: Optional[torch.dtype] = None, seed: int = 0,
                 weights_path: Optional[str] = None, max_slots: int = 8, max_seq: int = 1024,
                 weights: Optional[Dict[str, torch.Tensor]] = None,
                 units: Optional[Tuple[int, int]] = None, backend=None,
                 variants: Optional[Sequence[Tuple[int, int]]] = None,
                 pages: Optional[int] = None, reserved_slots: Sequence[int] = ()):
        """pages / reserved_slots: size of a paged cache's pool and the slots
        that own pages permanently (runtime/kv_cache.py LatentCache); pages
        None: every slot does."""
        self.cfg = cfg
        self.device = torch.device(device)
        if dtype is None:
            dtype = torch.float32 if self.device.type == "cpu" else torch.bfloat16
        self.dtype = dtype
        if units is None:
            units = (2 * layer_start, 2 * layer_end)
        ua, ub = units
        if not 0 <= ua <= ub <= 2 * cfg.n_layers:
            raise ValueError(f"unit range {units} outside [0, {2 * cfg.n_layers}]")
        self.unit_start, self.unit_end = ua, ub
        # alternating splits (parallel/partition.py make_alt_unit_plans): the
        # unit range run for even / odd microbatch groups, both inside `units`
        self.variants = [tuple(v) for v in variants] if variants else [(ua, ub)]
        if any(not (ua <= a <= b <= ub) for a, b in self.variants):
            raise ValueError(f"variant ranges {self.variants} outside the stage's units {units}")
        self.layer_start, self.layer_end = ua // 2, (ub + 1) // 2  # layers touched
        self.first, self.last = first, last
        self.layers = range(self.layer_start, self.layer_end)
        # layers whose attention half (and so whose KV cache) lives here
        self.kv_layers = [i for i in self.layers if ua <= 2 * i < ub]
        self._kv_index = {i: j for j, i in enumerate(self.kv_layers)}
        if weights is None:
            weights = maybe_load(cfg, weights_path, self.layers, first, last, seed, self.device, dtype,
                                 units=units)
        else:
            weights = {k: v.to(device=self.device, dtype=dtype).contiguous() for k, v in weights.items()
                       if self._owns(k)}
        self.w = weights
        self.max_seq = min(max_seq, cfg.max_positions)
        # `backend` overrides the device default: the fp32 golden model runs the
        # plain PyTorch ops (ops/reference.py) on the GPU (utils/golden.py)
        self.backend = backend if backend is not None else get_backend(self.device)
        # columns of the residual rows (hidden, or padded by the backend)
        self.row_width = self.backend.row_width(cfg)
        # rows that cross a stage boundary: the residual, beside it the embedding
        # output where a loop's passes read it again, the values that later layers
        # mix in, and the digits of the token ids where every layer looks them up;
        # (heads, columns of a head, the model's own of them) each
        self.wire_names = ["x"] + (["x0"] if cfg.loop_times else [])
        self.wire_parts = [(1, self.row_width, cfg.hidden)] * len(self.wire_names)
        m = cfg.mixed_values
        if m is not None:
            self.wire_names.append("values")
            self.wire_parts.append((m.kv_heads, self.backend.value_width(m), m.vdim))
        if cfg.token_side:
            self.wire_names.append("ids")
            self.wire_parts.append((1, 4, ID_DIGITS))
        self.wire_width = sum(n * c for n, c, _ in self.wire_parts)
        if cfg.whole_layers and (ua % 2 or ub % 2):
            raise ValueError(f"{cfg.name}: layers cannot be cut in half (units {units})")
        if cfg.paged_cache:
            own = cfg.cache_layers(self.kv_layers)
            self._pool_index = {i: k for k, i in enumerate(own)}
            for i in self.kv_layers:
                j = cfg.layers[i].mixer.kv_from
                if j is not None and j not in self._pool_index:
                    raise ValueError(f"layer {i} shares layer {j}'s cache: both must be on one stage")
            if pages is None:  # no page allocator in front: every slot owns its pages
                pages, reserved_slots = 0, range(max_slots)
            args = (max_slots, pages, self.max_seq, dtype, self.device, reserved_slots)
            if cfg.arch == "timisun":
                self.kv = LatentCache([self.backend.latent_width(cfg.layers[i].mixer.kv_rank) for i in own], *args)
            else:
                self.kv = PagedCache([self.backend.layer_cache(cfg.layers[i].mixer, cfg.shift_width) for i in own], *args)
        else:
            self.kv = KVCache(len(self.kv_layers), max_slots, cfg.n_kv_heads, self.max_seq,
                              cfg.head_dim, dtype, self.device)
        self.backend.prepare_stage(self)

    def _owns(self, name: str) -> bool:
        """Is tensor `name` used by this stage (its units, embeddings, head)?"""
        if self.cfg.arch in ("vizalix", "fagunex"):
            return name in stage_tensor_shapes(self.cfg, self.layers, self.first, self.last)
        lh = layer_half(name)
        if lh is None:
            emb = name in ("wte", "wpe", "embed_tokens")
            head = name in ("ln_f.weight", "ln_f.bias", "norm.weight", "lm_head") or (
                name in ("wte", "embed_tokens") and self.cfg.tie_embeddings)
            return (emb and self.first) or (head and self.last)
        return self.unit_start <= 2 * lh[0] + lh[1] < self.unit_end

    # ------------------------------------------------------------------
    def _lw(self, i: int, name: str, *default) -> torch.Tensor:
        p = "h." if self.cfg.arch == "gpt2" else "layers."
        return self.w.get(f"{p}{i}.{name}", *default) if default else self.w[f"{p}{i}.{name}"]

    # [tf5.15] modeling_gpt2.py:262-309 GPT2Block.forward, split at the residual
    def _gpt2_attn(self, li: int, i: int, r: Residual, meta: BatchMeta) -> None:
        be, c, w = self.backend, self.cfg, self._lw
        xn = be.layernorm(r, w(i, "ln_1.weight"), w(i, "ln_1.bias"), c.norm_eps)
        q = be.qkv_kv_append(xn, w(i, "attn.c_attn.weight"), w(i, "attn.c_attn.bias"),
                             self.kv.k(li), self.kv.v(li), meta, c)
        self._attn_out(q, li, meta, w(i, "attn.c_proj.weight"), w(i, "attn.c_proj.bias"), r)

    def _attn_out(self, q, li: int, meta: BatchMeta, wo, bo, r: Residual) -> None:
        """Attention + output projection + residual add: one fused launch when
        the backend has it for this shape (small decode batches), else two."""
        be = self.backend
        dec = getattr(meta, "dec", None)
        if dec is not None:  # mixed step (runtime/batch.py MixedMeta): each part its own kernel
            b = meta.b
            o = torch.cat([be.attention(q[:b], self.kv.k(li), self.kv.v(li), dec),
                           be.attention(q[b:], self.kv.k(li), self.kv.v(li), meta.pf)])
            be.linear_residual(o, wo, bo, r)
            return
        fused = getattr(be, "attention_oproj", None)
        if fused is not None and fused(q, self.kv.k(li), self.kv.v(li), meta, wo, bo, r):
            return
        o = be.attention(q, self.kv.k(li), self.kv.v(li), meta)
        be.linear_residual(o, wo, bo, r)

    def _gpt2_mlp(self, i: int, r: Residual) -> None:
        be, c, w = self.backend, self.cfg, self._lw
        xn = be.layernorm(r, w(i, "ln_2.weight"), w(i, "ln_2.bias"), c.norm_eps)
        h = be.linear(xn, w(i, "mlp.c_fc.weight"), w(i, "mlp.c_fc.bias"), act="gelu")
        be.linear_residual(h, w(i, "mlp.c_proj.weight"), w(i, "mlp.c_proj.bias"), r)

    def _llama_attn(self, li: int, i: int, r: Residual, meta: BatchMeta) -> None:
        be, c, w = self.backend, self.cfg, self._lw
        xn = be.rmsnorm(r, w(i, "input_layernorm.weight"), c.norm_eps)
        q = be.qkv_kv_append(xn, w(i, "self_attn.qkv.weight"), None,
                             self.kv.k(li), self.kv.v(li), meta, c)
        self._attn_out(q, li, meta, w(i, "self_attn.o_proj.weight"), None, r)

    def _llama_mlp(self, i: int, r: Residual) -> None:
        be, c, w = self.backend, self.cfg, self._lw
        xn = be.rmsnorm(r, w(i, "post_attention_layernorm.weight"), c.norm_eps)
        h = be.linear(xn, w(i, "mlp.gate_up.weight"), None, act="silu_mul")
        be.linear_residual(h, w(i, "mlp.down_proj.weight"), None, r)

    # Timisun: one norm, attention and experts both read it, both are added
    def _parallel_layer(self, i: int, r: Residual, meta: BatchMeta) -> None:
        be, c, spec = self.backend, self.cfg, self.cfg.layers[i]
        w = functools.partial(self._lw, i)
        m = spec.mixer
        pool = self.kv.pools[self._pool_index[i if m.kv_from is None else m.kv_from]]
        h = be.rmsnorm(r, w("input_layernorm.weight"), c.norm_eps, offset=1.0, width=c.hidden)
        q, gate, routing = be.latent_project(h, w, m, spec.mlp, self.kv, pool, meta, c.norm_eps)
        o = be.latent_attention(q, gate, w, m, self.kv, pool, meta)
        be.parallel_residual(o, h, routing, w, spec.mlp, r)

    # Vizalix: mixer and feed-forward of the same residual, each behind a norm
    # with one number for a gain -- applied after the projections that follow,
    # so both read the same normed rows
    def _mixer_layer(self, i: int, r: Residual, x0, meta: BatchMeta) -> None:
        be, c, spec = self.backend, self.cfg, self.cfg.layers[i]
        if spec.enter is not None:  # a pass of the loop begins: x <- W_in [x; x0] + step
            be.loop_enter(r, x0, self.w["loop.in"], self.w["loop.step"], spec.enter)
        w = functools.partial(self._lw, c.weight_layer(i))
        h = be.unit_rmsnorm(r, c)
        o = be.mix(h, w, spec, self.kv, self.kv.entries[self._pool_index[i]], meta, c.norm_eps)
        be.mixer_residual(o, h, w, spec, r)

    # Kedasun: attention, then a feed-forward, each between a norm of the
    # residual and a norm of its output
    def _sandwich_layer(self, i: int, r: Residual, side: dict, meta: BatchMeta) -> None:
        be, c, spec = self.backend, self.cfg, self.cfg.layers[i]
        w, m = functools.partial(self._lw, i), spec.mixer
        h = be.group_norm(r, w("input_layernorm.weight"), c)
        first = side.get("values") if m.mix_values is not None and m.mix_values != i else None
        o, values = be.attend(h, w, m, self.kv, self.kv.entries[self._pool_index[i]], meta, c.norm_eps, first,
                              keep_values=m.mix_values == i)
        if m.mix_values == i:
            side["values"] = values
        be.linear_post_norm(o, w("mixer.o"), w("mixer.o.b", None), w("mixer.out_norm.weight"), r, c)
        if spec.mlp is not None:
            h = be.group_norm(r, w("post_attention_layernorm.weight"), c)
            h = be.clamped_glu(h, w("mlp.gate_up.weight"), spec.mlp.limit)
            be.linear_post_norm(h, w("mlp.down_proj.weight"), None, w("mlp.out_norm.weight"), r, c)

    # Fagunex: the sandwich with elementwise norms; mixers read rows shifted towards
    # the previous token's, the feed-forward is a mixture of experts, and rows of the
    # tokens' own come last
    def _token_layer(self, i: int, r: Residual, side: dict, meta: BatchMeta) -> None:
        be, c, spec = self.backend, self.cfg, self.cfg.layers[i]
        w, m = functools.partial(self._lw, c.weight_layer(i)), spec.mixer
        entry = self.kv.entries[self._pool_index[i]]
        h = be.shift_norm(r, w, entry[-1], meta, c)
        if isinstance(m, ForgetSpec):
            o, out = be.forget_mix(h, w, m, entry[0], meta, c.norm_eps), "mixer.o"
        else:
            q, gate, _ = be.latent_project(h, w, m, None, self.kv, entry[0], meta, c.norm_eps)
            o, out = be.latent_attention(q, gate, w, m, self.kv, entry[0], meta), "attn.o.weight"
        be.linear_tanh(o, w(out), lambda n: w("norm1b" + n), r)
        if spec.mlp is not None:
            h = be.tanh_norm(r, lambda n: w("norm2" + n))
            be.experts_tanh(h, w, spec.mlp, lambda n: w("norm2b" + n), r)
        if c.token_side:
            be.token_side(r, side["ids"], w, c)

    # -- stage boundaries: the residual, and what travels beside it (wire_parts) --
    def _unpack(self, rows: torch.Tensor):
        """Residual rows and the side rows {"x0": ..., "values": ...}."""
        if len(self.wire_parts) == 1:
            return rows, {}
        parts = [p.contiguous() for p in rows.split([n * c for n, c, _ in self.wire_parts], 1)]
        side = dict(zip(self.wire_names, parts))
        if "values" in side:
            side["values"] = side["values"].to(self.dtype)
        if "ids" in side:
            d = side["ids"].to(torch.int32)
            side["ids"] = (d[:, 0] + 256 * d[:, 1] + 65536 * d[:, 2]).contiguous()
        return side.pop("x"), side

    def _pack(self, x: torch.Tensor, side: dict) -> torch.Tensor:
        if len(self.wire_parts) == 1:
            return x
        rows = [x]
        for name, (n, c, _) in list(zip(self.wire_names, self.wire_parts))[1:]:
            v = side.get(name)
            if name == "ids":
                rows.append(torch.stack([v % 256, v // 256 % 256, v // 65536, torch.zeros_like(v)], 1).float())
            else:  # None: the first layer that has them comes later
                rows.append(v.float() if v is not None else x.new_zeros(x.shape[0], n * c))
        return torch.cat(rows, 1)

    def boundary_rows(self, rows: torch.Tensor) -> torch.Tensor:
        """Rows as they leave the stage -> the model's own columns (compat forwards)."""
        parts = rows.split([n * c for n, c, _ in self.wire_parts], 1)
        return torch.cat([p.reshape(-1, n, c)[..., :own].reshape(-1, n * own)
                          for p, (n, c, own) in zip(parts, self.wire_parts)], 1)

    def wire_rows(self, rows: torch.Tensor) -> torch.Tensor:
        """Inverse of boundary_rows: padded as the backend wants them."""
        parts = rows.split([n * own for n, _, own in self.wire_parts], 1)
        pad = torch.nn.functional.pad
        return torch.cat([pad(p.reshape(-1, n, own), (0, c - own)).reshape(-1, n * c)
                          for p, (n, c, own) in zip(parts, self.wire_parts)], 1)

    # ------------------------------------------------------------------
    def embed(self, ids: torch.Tensor, meta: BatchMeta) -> torch.Tensor:
        if self.cfg.arch == "gpt2":
            return self.backend.embed(ids, meta.token_pos, self.w["wte"], self.w["wpe"])
        if self.cfg.embed_scale != 1.0:
            return self.backend.embed(ids, meta.token_pos, self.w["embed_tokens"], None, self.cfg.embed_scale)
        return self.backend.embed(ids, meta.token_pos, self.w["embed_tokens"], None)

    def forward(self, meta: BatchMeta, inp: torch.Tensor, all_logits: bool = False,
                head: bool = True, head_rows: Optional[torch.Tensor] = None,
                variant: int = 0, residuals: Optional[list] = None) -> torch.Tensor:
        """inp: token ids int32 [T] (first stage) or hidden fp32 [T, H].

        Returns hidden fp32 [T, H] (non-last stage, or `head=False`: a
        non-final prefill chunk only fills the KV cache) or fp32 logits
        [B, vocab_padded] for the last query of each sequence (last stage;
        [T, vocab_padded] with all_logits; the rows `head_rows` of the packed
        batch when given -- e.g. only the prompts whose final chunk this is).
        `variant`: which of the stage's unit ranges to run (the microbatch
        group's parity under alternating splits; 0 otherwise).  `residuals`
        collects the residual rows after every whole layer (debugging)."""
        side: dict = {}
        if self.first:
            x = self.embed(inp, meta)
            side["ids"] = inp
            if self.cfg.loop_times:
                side["x0"] = self.embed(inp, meta)  # the residual is updated in place
        else:
            x, side = self._unpack(inp)
        r = Residual(x)
        # decode-only routing rules (ops/hip.py); a mixed step's rows follow them up to 512
        self.backend.decode = getattr(meta, "routing_decode", meta.is_decode) and meta.num_tokens <= 512 \
            if getattr(meta, "dec", None) is not None else meta.is_decode
        gpt2 = self.cfg.arch == "gpt2"
        attn_fn = self._gpt2_attn if gpt2 else self._llama_attn
        mlp_fn = self._gpt2_mlp if gpt2 else self._llama_mlp
        ua, ub = self.variants[variant % len(self.variants)]
        for u in range(ua, ub):
            i = u >> 1
            if self.cfg.whole_layers:  # a whole layer: its second unit is empty
                if not u & 1:
                    if self.cfg.arch == "timisun":
                        self._parallel_layer(i, r, meta)
                    elif self.cfg.arch == "kedasun":
                        self._sandwich_layer(i, r, side, meta)
                    elif self.cfg.arch == "fagunex":
                        self._token_layer(i, r, side, meta)
                    else:
                        self._mixer_layer(i, r, side.get("x0"), meta)
                    if residuals is not None:
                        residuals.append(self.backend.flush(r)[:, : self.cfg.hidden].clone())
                continue
            if u & 1:
                mlp_fn(i, r)
            else:
                attn_fn(self._kv_index[i], i, r, meta)
        x = self.backend.flush(r)
        if not (self.last and head):
            return x if self.last else self._pack(x, side)
        return self.head(x, meta, all_logits, head_rows)

    def head(self, x: torch.Tensor, meta: BatchMeta, all_logits: bool = False,
             rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        be, c = self.backend, self.cfg
        if rows is None:
            rows = None if (all_logits or meta.is_decode) else meta.last_idx  # last query per sequence
        if c.arch == "timisun":
            xn = be.norm_rows(x, self.w["norm.weight"], None, c.norm_eps, True, rows, offset=1.0, width=c.hidden)
        elif c.arch == "vizalix":
            xn = be.norm_rows(x, self.w["norm.weight"], None, c.norm_eps, True, rows, width=be.norm_width(c))
        elif c.arch == "kedasun":
            xn = be.group_norm_rows(x, self.w["norm.weight"], c, rows)
        elif c.arch == "fagunex":
            xn = be.tanh_norm_rows(x, lambda n: self.w["norm" + n], rows)
        elif c.arch == "gpt2":
            xn = be.norm_rows(x, self.w["ln_f.weight"], self.w["ln_f.bias"], c.norm_eps, False, rows)
        else:
            xn = be.norm_rows(x, self.w["norm.weight"], None, c.norm_eps, True, rows)
        return be.logits(xn, self.lm_head_weight)

    @property
    def lm_head_weight(self) -> torch.Tensor:
        if hasattr(self, "_lm_head_padded"):
            return self._lm_head_padded
        return self.w[{"gpt2": "wte", "timisun": "embed_tokens"}.get(self.cfg.arch, "lm_head")]

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.w.values())
