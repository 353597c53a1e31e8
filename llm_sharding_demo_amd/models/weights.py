"""Stage-local weight materialisation.

Replaces the reference's "every pod loads the full model from the Hub"
(`server.py:40-42,108`, quirk Q4): a stage materialises ONLY its own layers,
plus the token embedding on the first stage and the final norm + lm_head on
the last stage (`wte` is tied to `lm_head` in GPT-2, so both ends hold a copy;
SURVEY.md §7.4 item 7).

Canonical layout: every projection weight is stored [out_features, in_features]
(K-contiguous), i.e. HF GPT-2 Conv1D weights ([in, out], [tf5.15]
pytorch_utils.py:106-121) are transposed once at load time.  That is the
layout the MFMA kernels want: the B-operand fragment of
`mfma_f32_16x16x32_bf16` is 8 consecutive K elements of one output column,
one 16-byte load.

Random init: each tensor gets its own seed derived from (seed, tensor name),
so any layer partition produces bit-identical weights (the property the
partition-invariance tests rely on).
"""
from __future__ import annotations

import os
import zlib
from typing import Dict, Iterable, Optional, Tuple

import torch

from ..config import ChannelDeltaSpec, ForgetSpec, ModelConfig, SSMSpec


def _seed(seed: int, name: str) -> int:
    return (zlib.crc32(f"{seed}:{name}".encode()) * 2654435761 + seed) % (2 ** 63 - 1)


def _randn(shape, std, seed, name, device, dtype):
    dev = torch.device(device)
    g = torch.Generator(device=dev)
    g.manual_seed(_seed(seed, name))
    t = torch.randn(shape, generator=g, device=dev, dtype=torch.float32) * std
    return t.to(dtype)


def gpt2_layer_names(i: int):
    return [f"h.{i}.{n}" for n in (
        "ln_1.weight", "ln_1.bias", "attn.c_attn.weight", "attn.c_attn.bias",
        "attn.c_proj.weight", "attn.c_proj.bias", "ln_2.weight", "ln_2.bias",
        "mlp.c_fc.weight", "mlp.c_fc.bias", "mlp.c_proj.weight", "mlp.c_proj.bias")]


def _gpt2_shapes(cfg: ModelConfig, i: int) -> Dict[str, tuple]:
    h, f = cfg.hidden, cfg.ffn
    p = f"h.{i}."
    return {
        p + "ln_1.weight": (h,), p + "ln_1.bias": (h,),
        p + "attn.c_attn.weight": (3 * h, h), p + "attn.c_attn.bias": (3 * h,),
        p + "attn.c_proj.weight": (h, h), p + "attn.c_proj.bias": (h,),
        p + "ln_2.weight": (h,), p + "ln_2.bias": (h,),
        p + "mlp.c_fc.weight": (f, h), p + "mlp.c_fc.bias": (f,),
        p + "mlp.c_proj.weight": (h, f), p + "mlp.c_proj.bias": (h,),
    }


def _llama_shapes(cfg: ModelConfig, i: int) -> Dict[str, tuple]:
    h, f = cfg.hidden, cfg.ffn
    p = f"layers.{i}."
    return {
        p + "input_layernorm.weight": (h,),
        p + "self_attn.qkv.weight": (cfg.qkv_size, h),  # q | k | v rows
        p + "self_attn.o_proj.weight": (h, cfg.q_size),
        p + "post_attention_layernorm.weight": (h,),
        p + "mlp.gate_up.weight": (2 * f, h),  # gate rows | up rows
        p + "mlp.down_proj.weight": (h, f),
    }


def _timisun_shapes(cfg: ModelConfig, i: int) -> Dict[str, tuple]:
    h, m, f = cfg.hidden, cfg.layers[i].mixer, cfg.layers[i].mlp
    p = f"layers.{i}."
    out = {p + "input_layernorm.weight": (h,),                  # stored around zero
           p + "attn.q.weight": (m.heads * m.dim, h),
           p + "attn.uk.weight": (m.heads * m.dim, m.kv_rank),
           p + "attn.uv.weight": (m.heads * m.vdim, m.kv_rank),
           p + "attn.o.weight": (h, m.heads * m.vdim)}
    if m.kv_from is None:
        out[p + "attn.dkv.weight"] = (m.kv_rank, h)
        out[p + "attn.dkv_norm.weight"] = (m.kv_rank,)
    if f is not None:
        out[p + "mlp.router.weight"] = (f.experts, h)
        out[p + "mlp.correction"] = (f.experts,)
        out[p + "mlp.experts.gate_up.weight"] = (f.experts, 2 * f.expert.ff, h)  # gate rows | up rows
        out[p + "mlp.experts.down.weight"] = (f.experts, h, f.expert.ff)
        if f.shared is not None:
            out[p + "mlp.shared.gate_up.weight"] = (2 * f.shared.ff, h)
            out[p + "mlp.shared.down.weight"] = (h, f.shared.ff)
    return out


def _vizalix_shapes(cfg: ModelConfig, i: int) -> Dict[str, tuple]:
    """Tensors of layer i (named by the layer that owns them)."""
    h, m, f = cfg.hidden, cfg.layers[i].mixer, cfg.layers[i].mlp
    p = f"layers.{cfg.weight_layer(i)}."
    out = {p + "input_layernorm.weight": ()}  # one number for all coordinates
    if isinstance(m, ChannelDeltaSpec):
        qk, v = m.kv_heads * m.dim, m.heads * m.vdim
        mix = {"q": (qk, h), "k": (qk, h), "v": (v, h), "q.conv": (qk, m.conv), "k.conv": (qk, m.conv),
               "v.conv": (v, m.conv), "b": (m.heads, h), "A_log": (m.heads,), "dt_bias": (m.heads * m.dim,),
               "a1": (m.decay_rank, h), "a2": (m.heads * m.dim, m.decay_rank), "g1": (m.gate_rank, h),
               "g2": (v, m.gate_rank), "norm": (m.vdim,), "o": (h, v)}
    elif isinstance(m, SSMSpec):
        mix = {"in": (m.inner + m.conv_channels + m.heads, h), "conv": (m.conv_channels, m.conv),
               "conv.b": (m.conv_channels,), "dt_bias": (m.heads,), "A_log": (m.heads,), "D": (m.heads,),
               "norm": (m.inner,), "o": (h, m.inner)}
    else:
        mix = {"q": (m.heads * m.dim, h), "k": (m.kv_heads * m.dim, h), "v": (m.kv_heads * m.vdim, h),
               "o": (h, m.heads * m.vdim)}
        if m.talking:
            mix["talk"] = (m.heads, m.heads)
    out.update((p + "mixer." + n, s) for n, s in mix.items())
    if f is not None:
        out[p + "post_attention_layernorm.weight"] = ()
        out[p + "mlp.gate_up.weight"] = (2 * f.ff, h)  # gate rows | up rows
        out[p + "mlp.down_proj.weight"] = (h, f.ff)
    return out


def _kedasun_shapes(cfg: ModelConfig, i: int) -> Dict[str, tuple]:
    h, m, f = cfg.hidden, cfg.layers[i].mixer, cfg.layers[i].mlp
    p = f"layers.{i}."
    rows = {"q": m.heads * m.dim, "k": m.kv_heads * m.dim, "v": m.kv_heads * m.vdim}
    mix: Dict[str, tuple] = {n: (r, h) for n, r in rows.items()}
    mix["o"] = (h, m.heads * m.vdim)
    if m.bias:
        mix.update((n + ".b", (r,)) for n, r in rows.items())
        mix["o.b"] = (h,)
    if m.conv:
        mix.update((n + ".conv", (r, m.conv)) for n, r in rows.items())
    if m.mix_values is not None:
        mix["vmix"] = ()
    if m.talking:
        mix["talk"] = (m.heads, m.heads)
    if m.head_gate:
        mix["g"] = (m.heads, h)
    out = {p + "input_layernorm.weight": (h,), p + "mixer.out_norm.weight": (h,)}
    out.update((p + "mixer." + n, s) for n, s in mix.items())
    if f is not None:
        out[p + "post_attention_layernorm.weight"] = out[p + "mlp.out_norm.weight"] = (h,)
        out[p + "mlp.gate_up.weight"] = (2 * f.ff, h)  # gate rows | up rows
        out[p + "mlp.down_proj.weight"] = (h, f.ff)
    return out


def _fagunex_shapes(cfg: ModelConfig, i: int) -> Dict[str, tuple]:
    """Tensors of layer i (named by the layer that owns them)."""
    h, m, f, n = cfg.hidden, cfg.layers[i].mixer, cfg.layers[i].mlp, cfg.token_side
    p = f"layers.{cfg.weight_layer(i)}."
    out: Dict[str, tuple] = {"shift": (h,)}
    for name in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ()):
        out.update({name + ".weight": (h,), name + ".bias": (h,), name + ".alpha": ()})
    if isinstance(m, ForgetSpec):
        d, v = m.heads * m.dim, m.heads * m.vdim
        out.update({"mixer.q": (d, h), "mixer.f": (d, h), "mixer.f.b": (d,), "mixer.lower": (d,), "mixer.v": (v, h),
                    "mixer.norm": (m.vdim,), "mixer.o": (h, v)})
    else:
        q, v = m.heads * m.q_dim, m.heads * m.vdim
        out.update({"attn.dkv.weight": (m.kv_rank + m.rot_dim, h), "attn.dkv_norm.weight": (m.kv_rank,),
                    "attn.uk.weight": (m.heads * m.dim, m.kv_rank), "attn.uv.weight": (v, m.kv_rank), "attn.o.weight": (h, v)})
        if m.q_rank is None:
            out["attn.q.weight"] = (q, h)
        else:
            out.update({"attn.dq.weight": (m.q_rank, h), "attn.dq_norm.weight": (m.q_rank,), "attn.uq.weight": (q, m.q_rank)})
        if m.sink:
            out["attn.sink"] = (m.heads,)
        if m.gate:
            out["attn.g.weight"] = (v, h)
    if f is not None:
        out.update({"mlp.router.weight": (f.experts, h),
                    "mlp.experts.gate_up.weight": (f.experts, 2 * f.expert.ff, h),  # gate rows | up rows
                    "mlp.experts.down.weight": (f.experts, h, f.expert.ff)})
        if f.shared is not None:
            out.update({"mlp.shared.gate_up.weight": (2 * f.shared.ff, h), "mlp.shared.down.weight": (h, f.shared.ff)})
            if f.shared_gate:
                out["mlp.shared.sg"] = (1, h)
    if n:
        out.update({"side.embed": (cfg.vocab_size, n), "side.gate": (n, h), "side.proj": (h, n), "side.norm": (h,)})
    return {p + k: s for k, s in out.items()}


_ATTN_PARTS = ("ln_1.", "attn.", "input_layernorm.", "self_attn.", "mixer.")
_MLP_PARTS = ("ln_2.", "mlp.", "post_attention_layernorm.")


def layer_half(name: str) -> Optional[Tuple[int, int]]:
    """(layer, 0 = attention half | 1 = MLP half) of a per-layer tensor name,
    None for embeddings / final norm / lm_head (parallel/partition.py units)."""
    for pre in ("h.", "layers."):
        if name.startswith(pre):
            idx, rest = name[len(pre):].split(".", 1)
            if rest.startswith(_ATTN_PARTS):
                return int(idx), 0
            if rest.startswith(_MLP_PARTS):
                return int(idx), 1
            raise ValueError(f"unknown per-layer tensor {name!r}")
    return None


def _filter_units(shapes: Dict[str, tuple], units: Optional[Tuple[int, int]]) -> Dict[str, tuple]:
    if units is None:
        return shapes
    ua, ub = units
    out = {}
    for n, s in shapes.items():
        lh = layer_half(n)
        if lh is None or ua <= 2 * lh[0] + lh[1] < ub:
            out[n] = s
    return out


def stage_tensor_shapes(cfg: ModelConfig, layers: Iterable[int], first: bool, last: bool,
                        units: Optional[Tuple[int, int]] = None):
    """Tensors a stage materialises; with `units` only the halves of the
    boundary layers that the stage runs."""
    if cfg.arch in ("vizalix", "fagunex"):  # whole layers, several of which may share their tensors
        return _stage_tensor_shapes(cfg, layers, first, last)
    return _filter_units(_stage_tensor_shapes(cfg, layers, first, last), units)


def _stage_tensor_shapes(cfg: ModelConfig, layers: Iterable[int], first: bool, last: bool):
    shapes: Dict[str, tuple] = {}
    if cfg.arch == "timisun":
        if first or last:
            shapes["embed_tokens"] = (cfg.vocab_size, cfg.hidden)  # tied head
        for i in layers:
            shapes.update(_timisun_shapes(cfg, i))
        if last:
            shapes["norm.weight"] = (cfg.hidden,)
    elif cfg.arch == "vizalix":
        if first:
            shapes["embed_tokens"] = (cfg.vocab_size, cfg.hidden)
        for i in layers:
            shapes.update(_vizalix_shapes(cfg, i))
            if cfg.layers[i].enter is not None:
                shapes["loop.in"] = (cfg.hidden, 2 * cfg.hidden)
                shapes["loop.step"] = (cfg.loop_times, cfg.hidden)
        if last:
            shapes["norm.weight"] = ()
            shapes["lm_head"] = (cfg.vocab_size, cfg.hidden)
    elif cfg.arch == "fagunex":
        if first:
            shapes["embed_tokens"] = (cfg.vocab_size, cfg.hidden)
        for i in layers:
            shapes.update(_fagunex_shapes(cfg, i))
        if last:
            shapes.update({"norm.weight": (cfg.hidden,), "norm.bias": (cfg.hidden,), "norm.alpha": ()})
            shapes["lm_head"] = (cfg.vocab_size, cfg.hidden)
    elif cfg.arch == "kedasun":
        if first:
            shapes["embed_tokens"] = (cfg.vocab_size, cfg.hidden)
        for i in layers:
            shapes.update(_kedasun_shapes(cfg, i))
        if last:
            shapes["norm.weight"] = (cfg.hidden,)
            shapes["lm_head"] = (cfg.vocab_size, cfg.hidden)
    elif cfg.arch == "gpt2":
        if first:
            shapes["wte"] = (cfg.vocab_size, cfg.hidden)
            shapes["wpe"] = (cfg.max_positions, cfg.hidden)
        for i in layers:
            shapes.update(_gpt2_shapes(cfg, i))
        if last:
            shapes["ln_f.weight"] = (cfg.hidden,)
            shapes["ln_f.bias"] = (cfg.hidden,)
            shapes["wte"] = (cfg.vocab_size, cfg.hidden)  # tied lm_head
    else:
        if first:
            shapes["embed_tokens"] = (cfg.vocab_size, cfg.hidden)
        for i in layers:
            shapes.update(_llama_shapes(cfg, i))
        if last:
            shapes["norm.weight"] = (cfg.hidden,)
            shapes["lm_head"] = (cfg.vocab_size, cfg.hidden)
    return shapes


def _init_one(cfg: ModelConfig, name: str, shape, seed: int, device, dtype) -> torch.Tensor:
    base = name.rsplit(".", 1)[-1]
    if cfg.arch == "timisun":
        return _timisun_init(cfg, name, shape, seed, device, dtype)
    if cfg.arch == "vizalix":
        return _vizalix_init(cfg, name, shape, seed, device, dtype)
    if cfg.arch == "kedasun":
        return _kedasun_init(name, shape, seed, device, dtype)
    if cfg.arch == "fagunex":
        return _fagunex_init(name, shape, seed, device, dtype)
    if name == "embed_tokens":
        # untied (Llama) input embeddings at unit scale (the T5 / muP
        # convention: the residual stream enters at the RMS its norms produce).
        # With HF's 0.02 the first layers' outputs dwarf the stream and random
        # -init depth amplifies bf16 rounding: fp32 vs bf16-emulated logits at
        # 32 layers, H = 2048: 6.6 % -> 1.1 % of the logit std; H = 1024: 3.3 %
        # -> 0.7 % (profiles/r3_llama_init_depth.log).  Residual projections
        # below are depth-scaled (0.02 / sqrt(2L)) as in GPT-2 / Llama training.
        return _randn(shape, 1.0, seed, name, device, dtype)
    if name in ("wte", "lm_head"):
        return _randn(shape, 0.02, seed, name, device, dtype)
    if name == "wpe":
        return _randn(shape, 0.01, seed, name, device, dtype)
    if "norm" in name or "ln_" in name:
        if base == "weight":
            return (1.0 + _randn(shape, 0.05, seed, name, device, torch.float32)).to(dtype)
        return _randn(shape, 0.02, seed, name, device, dtype)
    if base == "bias":
        return _randn(shape, 0.02, seed, name, device, dtype)
    std = 0.02
    if name.endswith("c_proj.weight") or name.endswith("o_proj.weight") or name.endswith("down_proj.weight"):
        std = 0.02 / (2 * cfg.n_layers) ** 0.5
    return _randn(shape, std, seed, name, device, dtype)


def _timisun_init(cfg: ModelConfig, name: str, shape, seed: int, device, dtype) -> torch.Tensor:
    """Unit-variance projections (std 1 / sqrt(fan-in)); the two residual
    projections of a layer are depth-scaled."""
    if name == "embed_tokens":
        return _randn(shape, cfg.hidden ** -0.5, seed, name, device, dtype)
    if name.endswith("dkv_norm.weight"):
        return (1.0 + _randn(shape, 0.05, seed, name, device, torch.float32)).to(dtype)
    if name.endswith(("norm.weight", "layernorm.weight")):
        return _randn(shape, 0.05, seed, name, device, dtype)
    if name.endswith("correction"):
        return _randn(shape, 0.02, seed, name, device, dtype)
    std = shape[-1] ** -0.5
    if name.endswith(("attn.o.weight", "down.weight")):
        std /= (2 * cfg.n_layers) ** 0.5
    if len(shape) == 3:
        return _stacked(shape, std, seed, name, device, dtype)
    return _randn(shape, std, seed, name, device, dtype)


def _stacked(shape, std: float, seed: int, name: str, device, dtype) -> torch.Tensor:
    """Experts one by one: no fp32 image of the whole stack."""
    out = torch.empty(shape, device=device, dtype=dtype)
    for e in range(shape[0]):
        out[e] = _randn(shape[1:], std, seed, f"{name}.{e}", device, dtype)
    return out


def _vizalix_init(cfg: ModelConfig, name: str, shape, seed: int, device, dtype) -> torch.Tensor:
    """Unit-variance projections, depth-scaled residual ones; decays between
    slow and fast, head mixing near the identity."""
    def around(mean, std):
        return (mean + _randn(shape, std, seed, name, device, torch.float32)).to(dtype)

    leaf = name.split(".", 2)[-1] if name.startswith("layers.") else name
    if leaf == "embed_tokens":
        return _randn(shape, 1.0, seed, name, device, dtype)
    if leaf.endswith(("norm.weight", "layernorm.weight", "mixer.norm", "mixer.D")):
        return around(1.0, 0.05)
    if leaf == "mixer.A_log":
        return around(0.5, 0.7)
    if leaf == "mixer.dt_bias":
        return around(-3.0, 1.0)
    if leaf == "mixer.talk":
        return (torch.eye(shape[0], device=device) + _randn(shape, 0.3 * shape[0] ** -0.5, seed, name, device,
                                                            torch.float32)).to(dtype)
    if leaf in ("mixer.conv.b", "loop.step"):
        return _randn(shape, 0.1, seed, name, device, dtype)
    std = shape[-1] ** -0.5
    if leaf in ("mixer.o", "mlp.down_proj.weight"):
        std /= (2 * cfg.n_layers) ** 0.5
    return _randn(shape, std, seed, name, device, dtype)


def _kedasun_init(name: str, shape, seed: int, device, dtype) -> torch.Tensor:
    """Unit-variance projections (the norms behind them set the residual's
    scale), short convolutions that mostly pass the current token, head mixing
    near the identity, half of the values mixed in."""
    def around(mean, std):
        return (mean + _randn(shape, std, seed, name, device, torch.float32)).to(dtype)

    leaf = name.split(".", 2)[-1] if name.startswith("layers.") else name
    if leaf == "embed_tokens":
        return _randn(shape, 1.0, seed, name, device, dtype)
    if leaf.endswith("norm.weight"):
        return around(1.0, 0.05)
    if leaf == "mixer.vmix":
        return around(0.5, 0.05)
    if leaf == "mixer.talk":
        return around(torch.eye(shape[0], device=device), 0.3 * shape[0] ** -0.5)
    if leaf.endswith(".conv"):
        return around((torch.arange(shape[1], device=device) == shape[1] - 1).float(), 0.2)
    if leaf.endswith(".b"):
        return _randn(shape, 0.1, seed, name, device, dtype)
    return _randn(shape, shape[-1] ** -0.5, seed, name, device, dtype)


def _fagunex_init(name: str, shape, seed: int, device, dtype) -> torch.Tensor:
    """Unit-variance projections (the norms behind them bound what enters the
    residual), forget gates between short and long memory, sinks near the
    scores, half a token's shift."""
    def around(mean, std):
        return (mean + _randn(shape, std, seed, name, device, torch.float32)).to(dtype)

    leaf = name.split(".", 2)[-1] if name.startswith("layers.") else name
    if leaf == "embed_tokens" or leaf == "side.embed":
        return _randn(shape, 1.0, seed, name, device, dtype)
    if leaf.endswith("alpha") or leaf == "shift":
        return around(0.5, 0.05)
    if leaf.endswith(".bias"):
        return _randn(shape, 0.02, seed, name, device, dtype)
    if leaf.endswith(("norm.weight", "norm")) or (leaf.startswith("norm") and leaf.endswith("weight")):
        return around(1.0, 0.05)
    if leaf == "mixer.lower":
        return around(0.0, 0.3).clamp(0.0, 0.9)
    if leaf == "mixer.f.b":
        return around(3.0, 1.5)
    if leaf == "attn.sink":
        return around(0.0, 1.0)
    if len(shape) == 3:
        return _stacked(shape, shape[-1] ** -0.5, seed, name, device, dtype)
    return _randn(shape, shape[-1] ** -0.5, seed, name, device, dtype)


def init_stage_weights(cfg: ModelConfig, layers, first: bool, last: bool, seed: int,
                       device, dtype, units=None) -> Dict[str, torch.Tensor]:
    shapes = stage_tensor_shapes(cfg, layers, first, last, units)
    return {n: _init_one(cfg, n, s, seed, device, dtype) for n, s in shapes.items()}


# ---------------------------------------------------------------------------
# Checkpoint loading (safetensors / torch weights_only) -- stage-local slices
# ---------------------------------------------------------------------------

_GPT2_CONV1D = ("attn.c_attn.weight", "attn.c_proj.weight", "mlp.c_fc.weight", "mlp.c_proj.weight")


def _open_checkpoint(path: str):
    """(name -> tensor, the names, (name, a, b) -> columns a .. b - 1 of a tensor);
    reads lazily where possible."""
    files = []
    if os.path.isdir(path):
        for fn in sorted(os.listdir(path)):
            if fn.endswith(".safetensors"):
                files.append(os.path.join(path, fn))
        if not files:
            for fn in ("pytorch_model.bin", "model.pt"):
                if os.path.isfile(os.path.join(path, fn)):
                    files.append(os.path.join(path, fn))
    else:
        files = [path]
    if not files:
        raise FileNotFoundError(f"no checkpoint files in {path}")
    if files[0].endswith(".safetensors"):
        from safetensors import safe_open

        index = {}
        handles = [safe_open(f, framework="pt") for f in files]
        for h in handles:
            for k in h.keys():
                index[k] = h
        return lambda k: index[k].get_tensor(k), set(index), lambda k, a, b: index[k].get_slice(k)[:, a:b]
    sd = {}
    for f in files:
        sd.update(torch.load(f, map_location="cpu", weights_only=True))  # never unpickles code
    return lambda k: sd[k], set(sd), lambda k, a, b: sd[k][:, a:b]


def _stack_experts(p: str, rest: str, experts: int, get) -> torch.Tensor:
    """Expert tensors of the layer with checkpoint prefix p: gate and up joined,
    routed experts stacked."""
    def part(prefix: str) -> torch.Tensor:
        if rest.endswith("gate_up.weight"):
            return torch.cat([get(prefix + "gate"), get(prefix + "up")], 0)
        return get(prefix + "down")

    if rest.startswith("mlp.shared."):
        return part(p + "mlp.shared.")
    return torch.stack([part(f"{p}mlp.e{e}.") for e in range(experts)])


def _timisun_tensor(cfg: ModelConfig, name: str, get) -> torch.Tensor:
    """One canonical tensor from a checkpoint in the design's own names
    (l<i>.mix.*, l<i>.mlp.e<k>.*); experts are stacked, gate and up joined."""
    if name == "embed_tokens":
        return get("embed")
    if name == "norm.weight":
        return get("final.norm")
    _, i, rest = name.split(".", 2)
    p = f"l{i}."
    if rest == "input_layernorm.weight":
        return get(p + "norm1")
    if rest.startswith("attn."):
        leaf = rest.split(".")[1]
        return get(p + "mix." + {"dkv_norm": "dkv.norm"}.get(leaf, leaf))
    if rest in ("mlp.router.weight", "mlp.correction"):
        return get(p + "mlp." + rest.split(".")[1])
    return _stack_experts(p, rest, cfg.layers[int(i)].mlp.experts, get)


def _vizalix_tensor(name: str, get) -> torch.Tensor:
    """One canonical tensor from a checkpoint in the design's own names."""
    top = {"embed_tokens": "embed", "norm.weight": "final.norm", "lm_head": "head", "loop.in": "loop.in",
           "loop.step": "loop.step"}
    if name in top:
        return get(top[name])
    _, i, rest = name.split(".", 2)
    if rest.startswith("mixer."):
        return get(f"l{i}.mix." + rest[len("mixer."):])
    if rest == "mlp.gate_up.weight":
        return torch.cat([get(f"l{i}.mlp.gate"), get(f"l{i}.mlp.up")], 0)
    return get(f"l{i}." + {"input_layernorm.weight": "norm1", "post_attention_layernorm.weight": "norm2",
                           "mlp.down_proj.weight": "mlp.down"}[rest])


def _kedasun_tensor(name: str, get) -> torch.Tensor:
    """One canonical tensor from a checkpoint in the design's own names."""
    top = {"embed_tokens": "embed", "norm.weight": "final.norm", "lm_head": "head"}
    if name in top:
        return get(top[name])
    _, i, rest = name.split(".", 2)
    own = {"input_layernorm.weight": "norm1", "mixer.out_norm.weight": "norm1b",
           "post_attention_layernorm.weight": "norm2", "mlp.out_norm.weight": "norm2b", "mlp.down_proj.weight": "mlp.down"}
    if rest in own:
        return get(f"l{i}.{own[rest]}")
    if rest == "mlp.gate_up.weight":
        return torch.cat([get(f"l{i}.mlp.gate"), get(f"l{i}.mlp.up")], 0)
    return get(f"l{i}.mix." + rest[len("mixer."):])


def _fagunex_tensor(cfg: ModelConfig, name: str, get, get_columns) -> torch.Tensor:
    """One canonical tensor from a checkpoint in the design's own names;
    get_columns(name, a, b) reads some columns of a tensor."""
    norm = {"weight": "", "bias": ".b", "alpha": ".alpha"}
    top = {"embed_tokens": "embed", "lm_head": "head"}
    if name in top:
        return get(top[name])
    if name.startswith("norm."):
        return get("final.norm" + norm[name.split(".")[1]])
    _, i, rest = name.split(".", 2)
    p = f"l{i}."
    if rest.startswith("norm"):
        n, leaf = rest.split(".")
        return get(p + n + norm[leaf])
    if rest == "side.embed":  # one table for all layers, a layer's columns side by side
        n = cfg.token_side
        return get_columns("side.embed", int(i) * n, int(i) * n + n)
    if rest.startswith(("side.", "shift")):
        return get(p + rest)
    if rest.startswith("mixer."):
        return get(p + "mix." + rest[len("mixer."):])
    if rest.startswith("attn."):
        leaf = rest.split(".")[1]
        return get(p + "mix." + {"dkv_norm": "dkv.norm", "dq_norm": "dq.norm"}.get(leaf, leaf))
    if rest in ("mlp.router.weight", "mlp.shared.sg"):
        return get(p + rest.removesuffix(".weight"))
    run = next(l for j, l in enumerate(cfg.layers) if cfg.weight_layer(j) == int(i))
    return _stack_experts(p, rest, run.mlp.experts, get)


def load_stage_weights(cfg: ModelConfig, path: str, layers, first: bool, last: bool,
                       device, dtype, units=None) -> Dict[str, torch.Tensor]:
    get, keys, get_columns = _open_checkpoint(path)
    out: Dict[str, torch.Tensor] = {}
    want = stage_tensor_shapes(cfg, layers, first, last, units)

    def find(name):
        for pre in ("", "transformer.", "model."):
            if pre + name in keys:
                return get(pre + name)
        raise KeyError(name)

    for name, shape in want.items():
        if cfg.arch == "timisun":
            t = _timisun_tensor(cfg, name, get)
        elif cfg.arch == "vizalix":
            t = _vizalix_tensor(name, get)
        elif cfg.arch == "kedasun":
            t = _kedasun_tensor(name, get)
        elif cfg.arch == "fagunex":
            t = _fagunex_tensor(cfg, name, get, get_columns)
        elif cfg.arch == "gpt2":
            src = {"wte": "wte.weight", "wpe": "wpe.weight"}.get(name, name)
            t = find(src)
            if any(name.endswith(c) for c in _GPT2_CONV1D):
                t = t.t()  # Conv1D [in, out] -> [out, in]
        else:
            if name.endswith("self_attn.qkv.weight"):
                p = name[: -len("qkv.weight")]
                t = torch.cat([find(p + "q_proj.weight"), find(p + "k_proj.weight"),
                               find(p + "v_proj.weight")], 0)
            elif name.endswith("mlp.gate_up.weight"):
                p = name[: -len("gate_up.weight")]
                t = torch.cat([find(p + "gate_proj.weight"), find(p + "up_proj.weight")], 0)
            elif name == "embed_tokens":
                t = find("embed_tokens.weight")
            elif name == "lm_head":
                t = get("lm_head.weight") if "lm_head.weight" in keys else find("embed_tokens.weight")
            else:
                t = find(name)
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"{name}: checkpoint shape {tuple(t.shape)} != expected {shape}")
        out[name] = t.to(device=device, dtype=dtype).contiguous()
    return out


def hf_state_dict_to_canonical(cfg: ModelConfig, sd: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    """Full HF GPT2LMHeadModel/LlamaForCausalLM state dict -> canonical names (all layers)."""
    import tempfile

    from safetensors.torch import save_file

    with tempfile.TemporaryDirectory() as d:
        tensors = {k: v.detach().contiguous().clone() for k, v in sd.items()}
        if "lm_head.weight" in tensors and cfg.tie_embeddings:
            tensors.pop("lm_head.weight")
        save_file(tensors, os.path.join(d, "model.safetensors"))
        return load_stage_weights(cfg, d, range(cfg.n_layers), True, True, "cpu", torch.float32)


def canonical_to_hf_gpt2(cfg: ModelConfig, w: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    """Canonical (all layers) -> HF GPT2LMHeadModel state dict (for golden tests)."""
    sd = {"transformer.wte.weight": w["wte"], "transformer.wpe.weight": w["wpe"],
          "transformer.ln_f.weight": w["ln_f.weight"], "transformer.ln_f.bias": w["ln_f.bias"],
          "lm_head.weight": w["wte"]}
    for i in range(cfg.n_layers):
        for n in gpt2_layer_names(i):
            t = w[n]
            if any(n.endswith(c) for c in _GPT2_CONV1D):
                t = t.t()
            sd["transformer." + n] = t.contiguous()
    return sd


def canonical_to_hf_llama(cfg: ModelConfig, w: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    sd = {"model.embed_tokens.weight": w["embed_tokens"], "model.norm.weight": w["norm.weight"],
          "lm_head.weight": w["lm_head"]}
    q, kv, f = cfg.q_size, cfg.kv_size, cfg.ffn
    for i in range(cfg.n_layers):
        p = f"layers.{i}."
        qkv = w[p + "self_attn.qkv.weight"]
        sd["model." + p + "self_attn.q_proj.weight"] = qkv[:q]
        sd["model." + p + "self_attn.k_proj.weight"] = qkv[q:q + kv]
        sd["model." + p + "self_attn.v_proj.weight"] = qkv[q + kv:]
        sd["model." + p + "self_attn.o_proj.weight"] = w[p + "self_attn.o_proj.weight"]
        gu = w[p + "mlp.gate_up.weight"]
        sd["model." + p + "mlp.gate_proj.weight"] = gu[:f]
        sd["model." + p + "mlp.up_proj.weight"] = gu[f:]
        sd["model." + p + "mlp.down_proj.weight"] = w[p + "mlp.down_proj.weight"]
        sd["model." + p + "input_layernorm.weight"] = w[p + "input_layernorm.weight"]
        sd["model." + p + "post_attention_layernorm.weight"] = w[p + "post_attention_layernorm.weight"]
    return {k: v.contiguous() for k, v in sd.items()}


def maybe_load(cfg: ModelConfig, weights: Optional[str], layers, first, last, seed, device, dtype,
               units=None):
    if weights:
        return load_stage_weights(cfg, weights, layers, first, last, device, dtype, units)
    return init_stage_weights(cfg, layers, first, last, seed, device, dtype, units)
