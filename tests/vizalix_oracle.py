"""Plain, slow Vizalix model for the tests: one function per mechanism.

Written from the design's equations in float64 (one token at a time where
something recurs), with no cache, no batching and nothing in common with the
product code: `cfg` is the parsed config.json dictionary and `w` maps tensor
names to tensors, both in the checkpoint's own layout.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, gain, eps):
    """One number scales every coordinate."""
    return rms(x, eps) * gain


def silu(z):
    return z / (1 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def short_conv(x, taps, bias=None):
    """x [T, channels]; the last column of taps [channels, n] weighs the
    current token, zeros stand before the start."""
    n = taps.shape[1]
    y = torch.zeros_like(x)
    for back in range(min(n, x.shape[0])):
        y[back:] += taps[:, n - 1 - back] * x[: x.shape[0] - back]
    return y if bias is None else y + bias


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k [T, H, dim], v [T, H, vdim], g [T, H, dim] decays in (0, 1), beta
    [T, H] -> outputs [T, H, vdim] and the last state [H, dim, vdim]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    read = lambda vec: (S * vec[:, :, None]).sum(1)  # noqa: E731  S^T vec per head
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - read(k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = read(q[t])
    return out, S


def channel_delta(h, m: dict, w, eps: float):
    """w: name -> tensor of the mixer ('q', 'q.conv', ...)."""
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(short_conv(h @ w("q").T, w("q.conv"))).reshape(T, G, D)
    k = silu(short_conv(h @ w("k").T, w("k.conv"))).reshape(T, G, D)
    v = silu(short_conv(h @ w("v").T, w("v.conv"))).reshape(T, H, V)
    q, k = unit(q) * D ** -0.5, unit(k)
    of = [i // (H // G) for i in range(H)]
    dt = softplus(h @ w("a1").T @ w("a2").T + w("dt_bias")).reshape(T, H, D)
    g = torch.exp(-torch.exp(w("A_log"))[None, :, None] * dt)
    o, _ = delta_rule(q[:, of], k[:, of], v, g, sigmoid(h @ w("b").T))
    o = rms(o, eps) * w("norm") * sigmoid(h @ w("g1").T @ w("g2").T).reshape(T, H, V)
    return o.reshape(T, H * V) @ w("o").T


def frequencies(rot: dict) -> List[float]:
    out = []
    n = rot["dims"]
    sc = rot.get("scaling")
    for i in range(n // 2):
        f = rot["base"] ** (-2 * i / n)
        if sc:
            length = 2 * math.pi / f
            if length > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif length >= sc["original"] / sc["high"]:
                s = (sc["original"] / length - sc["low"]) / (sc["high"] - sc["low"])
                f = (1 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate(x, positions, rot: dict):
    """x [T, heads, dim]: the first rot['dims'] dimensions turn in pairs (i, i + dims / 2)."""
    half = rot["dims"] // 2
    a = torch.outer(torch.as_tensor(positions, dtype=F64), torch.tensor(frequencies(rot), dtype=F64))[:, None]
    u, v = x[..., :half], x[..., half: 2 * half]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a), x[..., 2 * half:]], -1)


def visible(i: int, j: int, window: Optional[int]) -> bool:
    return j <= i and (window is None or i - j < window)


def talking_attention(q, k, v, talk, scale: float, softcap: Optional[float], window: Optional[int], first: int = 0):
    """q [T, H, dim] at positions first .. over k / v [n, G, .] of positions
    0 .. n - 1: capped scores are mixed over the heads, then softmax."""
    T, H = q.shape[:2]
    n, G = k.shape[:2]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    of = [h // (H // G) for h in range(H)]
    k, v = k[:, of], v[:, of]
    for t in range(T):
        keys = [j for j in range(n) if visible(first + t, j, window)]
        s = (k[keys] * q[t]).sum(-1).T * scale  # [H, keys]
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        s = talk @ s
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        p = p / p.sum(-1, keepdim=True)
        out[t] = (p.T[:, :, None] * v[keys]).sum(0)
    return out


def attention(h, m: dict, w, first: int = 0):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = list(range(first, first + T))
    q = rotate((h @ w("q").T).reshape(T, H, D), pos, m["rot"])
    k = rotate((h @ w("k").T).reshape(T, G, D), pos, m["rot"])
    v = (h @ w("v").T).reshape(T, G, V)
    o = talking_attention(q, k, v, w("talk"), m["scale"], m.get("softcap"), (m.get("mask") or {}).get("size"))
    return o.reshape(T, H * V) @ w("o").T


def ssd(x, B, C, dt, A_log, D):
    """x [T, H, vdim], B / C [T, H, N], dt [T, H] -> y and the last state [H, N, vdim]."""
    T, H, V = x.shape
    S = torch.zeros(H, B.shape[2], V, dtype=x.dtype)
    y = torch.zeros_like(x)
    for t in range(T):
        decay = torch.exp(-torch.exp(A_log) * dt[t])
        S = decay[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        y[t] = (S * C[t][:, :, None]).sum(1) + D[:, None] * x[t]
    return y, S


def mamba2(h, m: dict, w, eps: float):
    T, H, V, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    z, xbc, dt = torch.split(h @ w("in").T, [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(short_conv(xbc, w("conv"), w("conv.b")))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=-1)
    of = [i // (H // G) for i in range(H)]
    y, _ = ssd(x.reshape(T, H, V), B.reshape(T, G, N)[:, of], C.reshape(T, G, N)[:, of],
               softplus(dt + w("dt_bias")), w("A_log"), w("D"))
    y = y.reshape(T, inner) * silu(z)
    y = rms(y.reshape(T, m["norm_groups"], -1), eps).reshape(T, inner) * w("norm")
    return y @ w("o").T


def feed_forward(h, w):
    return (gelu_tanh(h @ w("gate").T) * (h @ w("up").T)) @ w("down").T


def layer(x, spec: dict, w, eps: float):
    """w: name -> tensor of the layer ('norm1', 'mix.q', ...)."""
    h = norm(x, w("norm1"), eps)
    mix = lambda n: w("mix." + n)  # noqa: E731
    if spec["type"] == "channel_delta":
        y = channel_delta(h, spec["mixer"], mix, eps)
    elif spec["type"] == "mamba2":
        y = mamba2(h, spec["mixer"], mix, eps)
    else:
        y = attention(h, spec["mixer"], mix)
    if spec.get("mlp"):
        y = y + feed_forward(norm(x, w("norm2"), eps), lambda n: w("mlp." + n))
    return x + y


def passes(cfg: dict):
    """(layer, number of the pass if it starts one) in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], layers: Optional[list] = None):
    """Logits [T, vocab] of one whole sequence; `layers` collects the residual
    stream after every layer run."""
    w = {k: v.to(F64) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = x0 = torch.stack([w["embed"][t] for t in tokens])
    for i, t in passes(cfg):
        if t is not None:
            x = torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][t]
        x = layer(x, cfg["layers"][i], lambda n, i=i: w[f"l{i}.{n}"], eps)
        if layers is not None:
            layers.append(x)
    return norm(x, w["final.norm"], eps) @ w["head"].T


def is_greedy(cfg: dict, w, prompt: List[int], out: List[int]) -> bool:
    """Is every token of `out` the likeliest one behind the prompt and those before it?"""
    best = forward(cfg, w, prompt + out[:-1])[len(prompt) - 1:].argmax(-1)
    return best.tolist() == out


# ---------------------------------------------------------------------------
# Random models of any sizes
# ---------------------------------------------------------------------------

def delta(heads=4, kv_heads=2, dim=24, vdim=20, conv=3, ff=40, ranks=(10, 6)):
    """`ranks` (inner widths of the decay and gate projections) only shape the tensors."""
    return {"type": "channel_delta", "ranks": ranks, "mlp": _mlp(ff),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def attn(heads=6, kv_heads=2, dim=40, vdim=24, window=70, scale=0.2, softcap=6.0, rot=24, base=10000.0,
         scaling=(4.0, 1.0, 4.0, 96), ff=40):
    s = dict(zip(("factor", "low", "high", "original"), scaling)) if scaling else None
    return {"type": "attention", "mlp": _mlp(ff),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap,
                      "mask": {"size": window}, "rot": {"dims": rot, "base": base, "scaling": s}}}


def ssm(heads=6, vdim=12, state=20, groups=2, norm_groups=3, conv=4, ff=40):
    return {"type": "mamba2", "mlp": _mlp(ff),
            "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups,
                      "conv": conv}}


def _mlp(ff):
    return {"ff": ff, "kind": "dense"} if ff else None


def config(layers, vocab=200, width=88, eps=1e-5, loop=None) -> dict:
    out = {"architecture": "Vizalix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def mixer_shapes(layer: dict, width: int) -> Dict[str, tuple]:
    m, d = layer["mixer"], width
    H = m["heads"]
    if layer["type"] == "channel_delta":
        qk, v, (ra, rg) = m["kv_heads"] * m["dim"], H * m["vdim"], layer["ranks"]
        return {"q": (qk, d), "k": (qk, d), "v": (v, d), "q.conv": (qk, m["conv"]), "k.conv": (qk, m["conv"]),
                "v.conv": (v, m["conv"]), "b": (H, d), "A_log": (H,), "dt_bias": (H * m["dim"],), "a1": (ra, d),
                "a2": (H * m["dim"], ra), "g1": (rg, d), "g2": (v, rg), "norm": (m["vdim"],), "o": (d, v)}
    if layer["type"] == "mamba2":
        inner = H * m["vdim"]
        ch = inner + 2 * m["groups"] * m["state"]
        return {"in": (inner + ch + H, d), "conv": (ch, m["conv"]), "conv.b": (ch,), "dt_bias": (H,), "A_log": (H,),
                "D": (H,), "norm": (inner,), "o": (d, inner)}
    G = m["kv_heads"]
    return {"q": (H * m["dim"], d), "k": (G * m["dim"], d), "v": (G * m["vdim"], d), "talk": (H, H),
            "o": (d, H * m["vdim"])}


def shapes(cfg: dict) -> Dict[str, tuple]:
    d = cfg["width"]
    out = {"embed": (cfg["vocab"], d), "final.norm": (), "head": (cfg["vocab"], d)}
    if cfg.get("loop"):
        out["loop.in"], out["loop.step"] = (d, 2 * d), (cfg["loop"]["times"], d)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        out[p + "norm1"] = ()
        out.update((p + "mix." + n, s) for n, s in mixer_shapes(layer, d).items())
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out.update({p + "norm2": (), p + "mlp.gate": (ff, d), p + "mlp.up": (ff, d), p + "mlp.down": (d, ff)})
    return out


def random_weights(cfg: dict, seed: int = 0, gain: float = 1.5) -> Dict[str, torch.Tensor]:
    """bfloat16-exact random tensors; projections at unit output scale times
    `gain`, decays between slow and fast, scores that reach the cap."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            t = 1 + 0.3 * t
        elif name.endswith(("mix.norm", "mix.D")):
            t = 1 + 0.2 * t
        elif last == "A_log":
            t = 0.3 + 0.8 * t
        elif last == "dt_bias":
            t = -3 + t
        elif last == "talk":
            t = torch.eye(shape[0]) + t * 0.4
        elif last == "conv":
            t = t / math.sqrt(shape[1])
        elif name.endswith("conv.b") or name == "loop.step":
            t = 0.3 * t
        elif name == "embed":
            t = 1.5 * t
        elif last in ("o", "down"):
            t = t / math.sqrt(shape[1]) * 0.7
        else:
            t = t / math.sqrt(shape[-1]) * gain
        out[name] = t.to(torch.bfloat16)
    return out


def save(path: str, cfg: dict, w: Dict[str, torch.Tensor]) -> None:
    import json
    import os

    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump({**cfg, "layers": [{k: v for k, v in l.items() if k != "ranks"} for l in cfg["layers"]]}, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
