"""Plain, slow Fagunex model for the tests: one function per mechanism.

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


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps: float):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def dynamic_tanh(x, alpha, weight, bias):
    return torch.tanh(alpha * x) * weight + bias


def token_shift(h, amount):
    """h [T, width]: every row moves towards the one before it (zeros in front)."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * amount


def token_side(x, e, gate, proj, weight, eps: float):
    """x [T, width], e [T, dim]: the tokens' own rows, gated by the residual."""
    return x + rms((gelu_tanh(x @ gate.T) * e) @ proj.T, eps) * weight


def rotate(x, positions, base: float, interleaved: bool):
    """x [T, ..., dims], all of it turned: dimensions 2i and 2i + 1 together, or i and i + dims / 2."""
    n = x.shape[-1]
    out = x.clone()
    p = torch.as_tensor(positions, dtype=F64).reshape([-1] + [1] * (x.dim() - 2))
    for i in range(n // 2):
        a = p * base ** (-2 * i / n)
        a0, a1 = (2 * i, 2 * i + 1) if interleaved else (i, i + n // 2)
        u, v = x[..., a0], x[..., a1]
        out[..., a0] = u * torch.cos(a) - v * torch.sin(a)
        out[..., a1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def visible(i: int, j: int, window: Optional[int]) -> bool:
    return j <= i and (window is None or i - j < window)


def softmax_sink(s, sink=None):
    """Weights over the last axis; sink [heads]: one more term of the denominator per row."""
    top = s.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink[:, None])
    p = torch.exp(s - top)
    rest = p.sum(-1, keepdim=True)
    return p / (rest if sink is None else rest + torch.exp(sink[:, None] - top))


def attend(q, k, v, scale: float, window: Optional[int] = None, sink=None, first: int = 0):
    """q [T, H, dim] at positions first .. over k, v [n, H, .] of positions 0 .. n - 1."""
    out = torch.zeros(q.shape[0], q.shape[1], v.shape[2], dtype=q.dtype)
    for t in range(q.shape[0]):
        keys = [j for j in range(k.shape[0]) if visible(first + t, j, window)]
        p = softmax_sink((k[keys] * q[t]).sum(-1).T * scale, sink)  # [H, keys]
        out[t] = (p.T[:, :, None] * v[keys]).sum(0)
    return out


def latent_attention(h, m: dict, w, eps: float, kind: str):
    """Both kinds of attention; w: name -> tensor of the mixer."""
    T, H, D, R, V, K = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    windowed = kind == "latent_attention"
    if windowed:
        q = (rms(h @ w("dq").T, eps) * w("dq.norm")) @ w("uq").T
    else:
        q = h @ w("q").T
    q = q.reshape(T, H, D + R)
    ckr = h @ w("dkv").T
    c, kr = rms(ckr[:, :K], eps) * w("dkv.norm"), ckr[:, K:]
    turn = lambda x: rotate(x, range(T), m["rot"]["base"], windowed)  # noqa: E731
    q = torch.cat([q[..., :D], turn(q[..., D:])], -1)
    k = torch.cat([(c @ w("uk").T).reshape(T, H, D), turn(kr)[:, None].expand(T, H, R)], -1)
    v = (c @ w("uv").T).reshape(T, H, V)
    o = attend(q, k, v, m["scale"], m["mask"]["size"] if windowed else None, w("sink") if windowed else None)
    o = o.reshape(T, H * V)
    return (o * sigmoid(h @ w("g").T) if windowed else o) @ w("o").T


def forget_gates(z, lower):
    return lower + (1 - lower) * sigmoid(z)


def recurrence(q, f, v, state=None):
    """q, f [T, H, D], v [T, H, V]: outputs [T, H, V] and the last state [H, D, V]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            S[h] = f[t, h][:, None] * S[h] + (1 - f[t, h])[:, None] * v[t, h][None, :]
            out[t, h] = S[h].T @ q[t, h]
    return out, S


def hgrn2(h, m: dict, w, eps: float):
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    f = forget_gates(h @ w("f").T + w("f.b"), w("lower"))
    o, _ = recurrence(silu(h @ w("q").T).reshape(T, H, D), f.reshape(T, H, D), (h @ w("v").T).reshape(T, H, V))
    return (rms(o, eps) * w("norm")).reshape(T, H * V) @ w("o").T


def route(h_t, router, top: int):
    """One token's experts and their weights."""
    z = router @ h_t
    ids = sorted(range(len(z)), key=lambda e: -float(z[e]))[:top]
    e = torch.exp(z[ids] - z[ids].max())
    return ids, e / e.sum()


def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def experts(h, f: dict, w):
    """w: name -> tensor of the feed-forward ('router', 'e0.gate', 'shared.up', ...)."""
    part = lambda x, name: expert(x, w(name + ".gate"), w(name + ".up"), w(name + ".down"))  # noqa: E731
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        ids, wt = route(h[t], w("router"), f["router"]["top"])
        for e, g in zip(ids, wt):
            out[t] += g * part(h[t: t + 1], f"e{e}")[0]
    if f.get("shared"):
        out = out + sigmoid(h @ w("shared.sg").T) * part(h, "shared")
    return out


def layer(x, spec: dict, w, eps: float, e=None):
    """w: name -> tensor of the layer ('norm1', 'mix.q', ...); e [T, dim]: its rows of the token-side table."""
    norm = lambda t, n: dynamic_tanh(t, w(n + ".alpha"), w(n), w(n + ".b"))  # noqa: E731
    mix = lambda name: w("mix." + name)  # noqa: E731
    h = token_shift(norm(x, "norm1"), w("shift"))
    if spec["type"] == "hgrn2":
        y = hgrn2(h, spec["mixer"], mix, eps)
    else:
        y = latent_attention(h, spec["mixer"], mix, eps, spec["type"])
    x = x + norm(y, "norm1b")
    if spec.get("mlp"):
        x = x + norm(experts(norm(x, "norm2"), spec["mlp"], lambda n: w("mlp." + n)), "norm2b")
    return x if e is None else token_side(x, e, w("side.gate"), w("side.proj"), w("side.norm"), eps)


def runs(cfg: dict) -> List[int]:
    """The layer of every run, in order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], layers: Optional[list] = None):
    """Logits [T, vocab] of one whole sequence; `layers` collects the residual
    stream after every layer run."""
    w = {k: v.to(F64) for k, v in w.items()}
    x, eps = w["embed"][list(tokens)], cfg["norm"]["eps"]
    n = (cfg.get("token_side") or {}).get("dim")
    for i in runs(cfg):
        e = w["side.embed"][list(tokens)][:, i * n:(i + 1) * n] if n else None
        x = layer(x, cfg["layers"][i], lambda name, i=i: w[f"l{i}.{name}"], eps, e)
        if layers is not None:
            layers.append(x)
    return dynamic_tanh(x, w["final.norm.alpha"], w["final.norm"], w["final.norm.b"]) @ w["head"].T


def is_greedy(cfg: dict, w, prompt: List[int], out: List[int]) -> bool:
    """Is every token of `out` the likeliest one behind the prompt and those before it?"""
    best = forward(cfg, w, prompt + out[:-1])[len(prompt) - 1:].argmax(-1)
    return best.tolist() == out


# ---------------------------------------------------------------------------
# Random models of any sizes
# ---------------------------------------------------------------------------

def _mlp(experts, top, ff, shared):
    if not experts:
        return None
    out = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    return {**out, "shared": {"ff": shared}} if shared else out


def _latent(kind, heads, dim, rot_dim, vdim, kv_rank, scale, base, mlp, **more):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
             "rot": {"base": base, "dims": rot_dim}, **more}
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def windowed(heads=3, dim=24, rot_dim=8, vdim=20, kv_rank=40, q_rank=36, scale=0.25, size=70, base=500.0, experts=5,
             top=2, ff=24, shared=40):
    return _latent("latent_attention", heads, dim, rot_dim, vdim, kv_rank, scale, base, _mlp(experts, top, ff, shared),
                   q_rank=q_rank, mask={"size": size})


def full(heads=5, dim=12, rot_dim=20, vdim=16, kv_rank=28, scale=0.3, base=900.0, experts=4, top=3, ff=40, shared=24):
    return _latent("latent_attention_2", heads, dim, rot_dim, vdim, kv_rank, scale, base, _mlp(experts, top, ff, shared))


def forget(heads=3, dim=24, vdim=20, experts=6, top=1, ff=32, shared=16):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}, "mlp": _mlp(experts, top, ff, shared)}


def config(layers, vocab=200, width=88, eps=1e-5, side=12, loop=None) -> dict:
    out = {"architecture": "Fagunex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if side:
        out["token_side"] = {"dim": side}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def mixer_shapes(layer: dict, d: int) -> Dict[str, tuple]:
    m = layer["mixer"]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    if layer["type"] == "hgrn2":
        n = H * D
        return {"q": (n, d), "f": (n, d), "f.b": (n,), "lower": (n,), "v": (H * V, d), "norm": (V,), "o": (d, H * V)}
    R, K = m["rot_dim"], m["kv_rank"]
    out = {"dkv": (K + R, d), "dkv.norm": (K,), "uk": (H * D, K), "uv": (H * V, K), "o": (d, H * V)}
    if layer["type"] == "latent_attention":
        Q = m["q_rank"]
        out.update({"dq": (Q, d), "dq.norm": (Q,), "uq": (H * (D + R), Q), "sink": (H,), "g": (H * V, d)})
    else:
        out["q"] = (H * (D + R), d)
    return out


def shapes(cfg: dict) -> Dict[str, tuple]:
    d, n = cfg["width"], (cfg.get("token_side") or {}).get("dim")
    norm = lambda name: {name: (d,), name + ".b": (d,), name + ".alpha": ()}  # noqa: E731
    out = {"embed": (cfg["vocab"], d), **norm("final.norm"), "head": (cfg["vocab"], d)}
    if n:
        out["side.embed"] = (cfg["vocab"], n * len(cfg["layers"]))
    for i, layer in enumerate(cfg["layers"]):
        p, f = f"l{i}.", layer["mlp"]
        out.update({**norm(p + "norm1"), **norm(p + "norm1b"), p + "shift": (d,)})
        out.update((p + "mix." + k, s) for k, s in mixer_shapes(layer, d).items())
        if f:
            out.update({**norm(p + "norm2"), **norm(p + "norm2b"), p + "mlp.router": (f["router"]["experts"], d)})
            parts = {f"e{e}": f["expert"]["ff"] for e in range(f["router"]["experts"])}
            if f.get("shared"):
                parts["shared"] = f["shared"]["ff"]
                out[p + "mlp.shared.sg"] = (1, d)
            for k, ff in parts.items():
                out.update({f"{p}mlp.{k}.gate": (ff, d), f"{p}mlp.{k}.up": (ff, d), f"{p}mlp.{k}.down": (d, ff)})
        if n:
            out.update({p + "side.gate": (n, d), p + "side.proj": (d, n), p + "side.norm": (d,)})
    return out


def random_weights(cfg: dict, seed: int = 0, gates: float = 2.0) -> Dict[str, torch.Tensor]:
    """bfloat16-exact random tensors: projections at unit output scale, forget
    gates from near their lower bound to near one (their bias spread over
    -+2 gates), routers whose choices are clear."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last == "alpha":
            t = 0.7 + 0.1 * t
        elif last == "shift":
            t = 0.5 + 0.3 * t
        elif last == "lower":
            t = 0.8 * torch.rand(shape, generator=g) * (torch.rand(shape, generator=g) < 0.8)
        elif name.endswith(".f.b"):
            t = 1.0 + gates * t
        elif name.endswith("norm") or last.startswith("norm"):
            t = 1 + 0.3 * t
        elif last == "b":
            t = 0.2 * t
        elif last == "sink":
            t = 1.0 + t
        elif last == "router":
            t = t * 4 / math.sqrt(shape[-1])
        elif name not in ("embed", "side.embed"):
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
