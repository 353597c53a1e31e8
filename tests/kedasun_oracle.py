"""Plain, slow Kedasun model for the tests: one function per mechanism.

Written from the design's equations in float64, with no cache, no batching and
nothing in common with the product code: `cfg` is the parsed config.json
dictionary and `w` maps tensor names to tensors, both in the checkpoint's own
layout.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, weight, groups: int, eps: float):
    """Consecutive parts of equal size, each over its own root mean square."""
    n = x.shape[-1] // groups
    return torch.cat([rms(x[..., g * n:(g + 1) * n], eps) for g in range(groups)], -1) * weight


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def short_conv(x, taps):
    """x [T, channels]; the last column of taps [channels, n] weighs the
    current token, zeros stand before the start."""
    n = taps.shape[1]
    y = torch.zeros_like(x)
    for back in range(min(n, x.shape[0])):
        y[back:] += taps[:, n - 1 - back] * x[: x.shape[0] - back]
    return y


def rotate(x, positions, dims: int, base: float):
    """x [T, heads, dim]: dimensions 2i and 2i + 1 of the first `dims` turn together."""
    out = x.clone()
    p = torch.as_tensor(positions, dtype=F64)[:, None]
    for i in range(dims // 2):
        a = p * base ** (-2 * i / dims)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def visible(i: int, j: int, window: Optional[int], keep: int = 0) -> bool:
    return j <= i and (window is None or i - j < window or j < keep)


def slopes(heads: int) -> List[float]:
    return [2.0 ** (-8 * (h + 1) / heads) for h in range(heads)]


def softmax(s):
    p = torch.exp(s - s.max(-1, keepdim=True).values)
    return p / p.sum(-1, keepdim=True)


def attend(q, k, v, scale: float, window: Optional[int] = None, keep: int = 0, slope: Optional[List[float]] = None,
           talk=None, first: int = 0):
    """q [T, H, dim] at positions first .. over k / v [n, G, .] of positions
    0 .. n - 1: scores less a distance bias, softmax, then the heads' weights
    are mixed by talk [H, H]."""
    T, H = q.shape[:2]
    n, G = k.shape[:2]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    of = [h // (H // G) for h in range(H)]
    k, v = k[:, of], v[:, of]
    for t in range(T):
        i = first + t
        keys = [j for j in range(n) if visible(i, j, window, keep)]
        s = (k[keys] * q[t]).sum(-1).T * scale  # [H, keys]
        if slope is not None:
            s = s - torch.tensor(slope, dtype=s.dtype)[:, None] * torch.tensor([i - j for j in keys], dtype=s.dtype)
        p = softmax(s)
        if talk is not None:
            p = talk @ p
        out[t] = (p.T[:, :, None] * v[keys]).sum(0)
    return out


def mix_values(v, v_first, lam):
    return v if v_first is None else (1 - lam) * v + lam * v_first


def attention(h, m: dict, w, v_first):
    """Output rows and this layer's values (before mixing)."""
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    turn = lambda x: rotate(x, range(T), rot["dims"], rot["base"])  # noqa: E731
    q, k = turn((h @ w("q").T).reshape(T, H, D)), turn((h @ w("k").T).reshape(T, G, D))
    v = (h @ w("v").T).reshape(T, G, V)
    o = attend(q, k, mix_values(v, v_first, w("vmix") if v_first is not None else None), m["scale"])
    return o.reshape(T, H * V) @ w("o").T, v


def attention_2(h, m: dict, w, v_first, eps: float):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ w(n).T + w(n + ".b"), w(n + ".conv")) for n in "qkv")
    q, k, v = rms(q.reshape(T, H, D), eps), rms(k.reshape(T, G, D), eps), v.reshape(T, G, V)
    mixed = mix_values(v, v_first, w("vmix") if v_first is not None else None)
    o = attend(q, k, mixed, m["scale"], m["mask"]["size"], m["mask"]["keep_first"], slopes(H), w("talk"))
    o = o * sigmoid(h @ w("g").T)[:, :, None]
    return o.reshape(T, H * V) @ w("o").T + w("o.b"), v


def feed_forward(h, w, limit: float):
    g = torch.clamp(h @ w("gate").T, max=limit)
    u = torch.clamp(h @ w("up").T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1)) @ w("down").T


def layer(x, spec: dict, w, norm: dict, v_first):
    """w: name -> tensor of the layer ('norm1', 'mix.q', ...).  v_first: values
    of the first layer that mixes them, None up to that one."""
    n = lambda t, name: group_norm(t, w(name), norm["groups"], norm["eps"])  # noqa: E731
    mix = lambda name: w("mix." + name)  # noqa: E731
    m = spec["mixer"]
    of = v_first if m.get("v_mix") else None
    if spec["type"] == "attention_2":
        y, v = attention_2(n(x, "norm1"), m, mix, of, norm["eps"])
    else:
        y, v = attention(n(x, "norm1"), m, mix, of)
    x = x + n(y, "norm1b")
    if spec.get("mlp"):
        y = feed_forward(n(x, "norm2"), lambda name: w("mlp." + name), spec["mlp"]["limit"])
        x = x + n(y, "norm2b")
    return x, v if m.get("v_mix") and v_first is None else v_first


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], layers: Optional[list] = None):
    """Logits [T, vocab] of one whole sequence; `layers` collects the residual
    stream after every layer."""
    w = {k: v.to(F64) for k, v in w.items()}
    x, v_first = w["embed"][list(tokens)] * cfg["embedding"]["scale"], None
    for i, spec in enumerate(cfg["layers"]):
        x, v_first = layer(x, spec, lambda n, i=i: w[f"l{i}.{n}"], cfg["norm"], v_first)
        if layers is not None:
            layers.append(x)
    return group_norm(x, w["final.norm"], cfg["norm"]["groups"], cfg["norm"]["eps"]) @ w["head"].T


def is_greedy(cfg: dict, w, prompt: List[int], out: List[int]) -> bool:
    """Is every token of `out` the likeliest one behind the prompt and those before it?"""
    best = forward(cfg, w, prompt + out[:-1])[len(prompt) - 1:].argmax(-1)
    return best.tolist() == out


# ---------------------------------------------------------------------------
# Random models of any sizes
# ---------------------------------------------------------------------------

def full(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.2, rot=24, base=1000.0, v_mix=True, ff=40, limit=1.5):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
             "rot": {"dims": rot, "base": base}, "v_mix": v_mix}
    return {"type": "attention", "mixer": mixer, "mlp": _mlp(ff, limit)}


def windowed(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.3, conv=3, size=70, keep=5, v_mix=True, ff=40, limit=0.8):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "conv": conv,
             "mask": {"size": size, "keep_first": keep}, "v_mix": v_mix}
    return {"type": "attention_2", "mixer": mixer, "mlp": _mlp(ff, limit)}


def _mlp(ff, limit):
    return {"ff": ff, "kind": "dense", "limit": limit} if ff else None


def config(layers, vocab=200, width=88, groups=4, eps=1e-5, scale=0.7) -> dict:
    return {"architecture": "Kedasun", "vocab": vocab, "width": width, "embedding": {"scale": scale},
            "norm": {"eps": eps, "groups": groups}, "layers": layers}


def mixer_shapes(layer: dict, width: int) -> Dict[str, tuple]:
    m, d = layer["mixer"], width
    H, G, o = m["heads"], m["kv_heads"], m["heads"] * m["vdim"]
    n = {"q": H * m["dim"], "k": G * m["dim"], "v": G * m["vdim"]}
    out = {k: (s, d) for k, s in n.items()}
    out["o"] = (d, o)
    if m.get("v_mix"):
        out["vmix"] = ()
    if layer["type"] == "attention_2":
        for k, s in n.items():
            out[k + ".b"], out[k + ".conv"] = (s,), (s, m["conv"])
        out.update({"talk": (H, H), "g": (H, d), "o.b": (d,)})
    return out


def shapes(cfg: dict) -> Dict[str, tuple]:
    d = cfg["width"]
    out = {"embed": (cfg["vocab"], d), "final.norm": (d,), "head": (cfg["vocab"], d)}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        out.update({p + "norm1": (d,), p + "norm1b": (d,)})
        out.update((p + "mix." + n, s) for n, s in mixer_shapes(layer, d).items())
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out.update({p + "norm2": (d,), p + "norm2b": (d,), p + "mlp.gate": (ff, d), p + "mlp.up": (ff, d),
                        p + "mlp.down": (d, ff)})
    return out


def random_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """bfloat16-exact random tensors; projections at unit output scale, gates
    and ups that reach the clamp, uneven head mixing."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if "norm" in last:
            t = 1 + 0.3 * t
        elif last == "vmix":
            t = 0.4 + 0.1 * t
        elif last == "talk":
            t = torch.eye(shape[0]) + t * 0.4
        elif last == "conv":
            t = t / math.sqrt(shape[1]) + (torch.arange(shape[1]) == shape[1] - 1)
        elif last == "b":
            t = 0.4 * t
        elif name != "embed":
            t = t / math.sqrt(shape[-1]) * 1.2
        out[name] = t.to(torch.bfloat16)
    return out


def save(path: str, cfg: dict, w: Dict[str, torch.Tensor]) -> None:
    import json
    import os

    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
