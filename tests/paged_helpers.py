"""What the GPU tests of models over a paged cache share: ragged batches, shuffled
pages, error measures, and steps of token ids through a trace session."""
from __future__ import annotations

import random

import numpy as np
import torch

from llm_sharding_demo_amd.runtime.kv_cache import PAGE

BF, F32 = torch.bfloat16, torch.float32


def cuda(t, dt=None):
    return t.to(device="cuda", dtype=dt if dt is not None else t.dtype).contiguous()


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device="cuda")


def err(got, want):
    """Largest difference, relative to the wanted value plus the root mean square of all."""
    want = want.double()
    return float(((got.double().cpu() - want).abs() / (want.pow(2).mean().sqrt() + want.abs())).max())


def rounded(t, dt):
    return t.to(dt).double()


class Batch:
    """Ragged sequences of a launch: (slot, first position, tokens)."""

    def __init__(self, *seqs):
        self.seqs = seqs
        self.n = [s[2] for s in seqs]
        self.T = sum(self.n)
        self.cu_host = np.concatenate([[0], np.cumsum(self.n)]).tolist()
        self.slots, self.start, self.cu = i32([s[0] for s in seqs]), i32([s[1] for s in seqs]), i32(self.cu_host)
        self.tslot = i32([s[0] for s in seqs for _ in range(s[2])])
        self.tpos = i32([s[1] + j for s in seqs for j in range(s[2])])

    def tiles(self, rows):
        return i32([[i, o] for i, n in enumerate(self.n) for o in range(0, n, rows)]).reshape(-1, 2)

    def rows(self, i):
        return slice(self.cu_host[i], self.cu_host[i + 1])


def pools(k, v, dt, dp, vp, slots=3, seed=0):
    """Keys / values [slot][n, G, .] in shuffled pages of padded pools, and the table."""
    g = random.Random(seed)
    width = max(-(-len(x) // PAGE) for x in k.values()) + 1
    ids = list(range(slots * width))
    g.shuffle(ids)
    G = next(iter(k.values())).shape[1]
    K = torch.zeros(len(ids) + 1, G, PAGE, dp, dtype=dt)
    V = torch.zeros(len(ids) + 1, G, PAGE, vp, dtype=dt)
    table = torch.full((slots, width), len(ids), dtype=torch.int32)
    for s, kk in k.items():
        for j in range(-(-len(kk) // PAGE)):
            pg = ids.pop()
            table[s, j] = pg
            part = slice(j * PAGE, min(len(kk), (j + 1) * PAGE))
            n = part.stop - part.start
            K[pg, :, :n, : kk.shape[2]] = kk[part].transpose(0, 1).to(dt)
            V[pg, :, :n, : v[s].shape[2]] = v[s][part].transpose(0, 1).to(dt)
    return cuda(K), cuda(V), cuda(table)


def up(n, m):
    return -(-n // m) * m


def portions(n, sizes):
    out, at = [], 0
    for s in sizes:
        if at < n:
            out.append((at, min(n, at + s)))
            at += s
    return out + ([(at, n)] if at < n else [])


def ids_of(n, vocab=200, seed=0):
    r = random.Random(seed)
    return [r.randrange(vocab) for _ in range(n)]


def logit_err(got, want):
    """Worst row's root mean square difference over the logits' own."""
    d = got.double() - want
    return float((d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt().max() / want.std())


def run_steps(ses, seqs, steps):
    """steps: [[(id, tokens), ...], ...] -> {id: logits of all its tokens}."""
    at, out = dict.fromkeys(seqs, 0), {k: [] for k in seqs}
    for st in steps:
        ent = [{"id": k, "tokens": seqs[k][at[k]: at[k] + n], "want": list(range(n))} for k, n in st]
        for k, n in st:
            at[k] += n
        got = ses.step(ent, [k for k, _ in st if at[k] == len(seqs[k])])
        for k, n in st:
            out[k].append(got[:n])
            got = got[n:]
    return {k: torch.cat(v) for k, v in out.items() if v}


def portion_steps(rid, n, sizes):
    return [[(rid, b - a)] for a, b in portions(n, list(sizes) + [1] * n)]
