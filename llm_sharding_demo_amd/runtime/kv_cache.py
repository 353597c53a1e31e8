"""Shard-local KV cache + slot allocator.

The reference has no KV cache: every decode step re-sends and recomputes the
whole sequence on both shards (`server.py:169-181`, quirk Q5).  Here each
pipeline stage owns the K/V of ITS layers only, so the only thing that
crosses the inter-stage link per decode step is the boundary hidden state.

Layout (one allocation per stage):
    buf[layer, 0|1 (K|V), slot, kv_head, position, head_dim]   bf16 on GPU
Each (slot, head) row-block is contiguous over positions, so the decode
attention kernel streams K and V for one sequence/head as one linear 1 KiB-
per-wave-instruction read.  Sized for MI355X's 288 GB HBM: the engine asks
`plan_slots` for the slot count that fits the free-memory budget after the
stage's weights (runtime/engine.py `_kv_slots`, reported on /health and
/metrics); two extra slots hold decode pad rows and compat forwards.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, List, Sequence, Tuple

import torch

from ..config import AttentionSpec, ChannelDeltaSpec, ForgetSpec, SSMSpec

PAGE = 64  # tokens per page of a paged cache (csrc/kernels/attention_latent.hip)


class KVCache:
    def __init__(self, n_layers: int, slots: int, n_kv: int, max_seq: int, head_dim: int,
                 dtype: torch.dtype, device):
        self.n_layers, self.slots, self.n_kv = n_layers, slots, n_kv
        self.max_seq, self.head_dim = max_seq, head_dim
        shape = (max(n_layers, 1), 2, slots, n_kv, max_seq, head_dim)
        self.buf = torch.zeros(shape, dtype=dtype, device=device)

    def k(self, layer: int) -> torch.Tensor:
        return self.buf[layer, 0]

    def v(self, layer: int) -> torch.Tensor:
        return self.buf[layer, 1]

    @property
    def nbytes(self) -> int:
        return self.buf.numel() * self.buf.element_size()

    @staticmethod
    def bytes_per_slot(n_layers: int, n_kv: int, max_seq: int, head_dim: int, elt: int = 2) -> int:
        return n_layers * 2 * n_kv * max_seq * head_dim * elt


def pad_up(n: int, m: int) -> int:
    return -(-n // m) * m


def pages_for(tokens: int) -> int:
    return -(-int(tokens) // PAGE)


@dataclass(frozen=True)
class LayerCache:
    """What one layer keeps of a sequence: tensors of its PAGE-token pages
    (their shapes), and tensors of its slot -- recurrent state in fp32, the
    last inputs of a short convolution in the model's element type."""

    pages: Tuple[tuple, ...] = ()
    state: Tuple[tuple, ...] = ()   # fp32, per slot
    ring: Tuple[tuple, ...] = ()    # element type, per slot

    def page_bytes(self, elt: int = 2) -> int:
        return elt * sum(torch.Size(s).numel() for s in self.pages)

    def slot_bytes(self, elt: int = 2) -> int:
        return sum(4 * torch.Size(s).numel() for s in self.state) + sum(elt * torch.Size(s).numel() for s in self.ring)


def layer_cache(mixer, up: Callable[[int, int], int] = lambda n, m: n, shift: int = 0) -> LayerCache:
    """Cache of one layer; up(n, m): the backend's padding of n to a multiple of m.
    shift: columns of the last token's row that the layer keeps too, the last of its state.
      attention   K [kv head][token][dim], V [kv head][token][vdim] per page, and the
                  q | k | v rows of positions p % taps in front of a short convolution
      delta rule  S [heads][dim][vdim] and the conv inputs of positions p % taps
      Mamba-2     S [heads][state][vdim], and the same
      forget gate S [heads][dim][vdim]
      latent      one row per token: `rank` columns and the turned key part"""
    if shift:
        c = layer_cache(mixer, up)
        return LayerCache(c.pages, c.state + ((up(shift, 64),),), c.ring)
    if isinstance(mixer, AttentionSpec):
        g = mixer.kv_heads
        dp, vp = up(mixer.dim, 32), up(mixer.vdim, 16)
        ring = ((mixer.conv, (mixer.heads + g) * dp + g * vp),) if mixer.conv else ()
        return LayerCache(pages=((g, PAGE, dp), (g, PAGE, vp)), ring=ring)
    if isinstance(mixer, (ChannelDeltaSpec, SSMSpec)):
        rows = mixer.dim if isinstance(mixer, ChannelDeltaSpec) else mixer.state
        return LayerCache(state=((mixer.heads, rows, up(mixer.vdim, 4)),), ring=((mixer.conv, mixer.conv_channels),))
    if isinstance(mixer, ForgetSpec):
        return LayerCache(state=((mixer.heads, mixer.dim, up(mixer.vdim, 4)),))
    return LayerCache(pages=((PAGE, up(mixer.kv_rank + mixer.rot_dim, 64)),))


class PagedCache:
    """Per-layer caches of models with per-layer specs: entries[k] holds layer
    k's tensors, a pool of PAGE-token pages ([page, ...]) per LayerCache.pages
    and per-slot tensors ([slot, ...]) per LayerCache.state / .ring, and one
    page table serves all of them, table[slot, position // PAGE].  Pages
    belong to sequences, not to slots: the host's page allocator hands them out
    (the scheduler at admission, runtime/trace.py as a sequence grows) and
    `assign` writes a slot's table row.  Table entries without a page point at
    the scratch page, which pad rows also write to.  A slot's state needs no
    clearing: whoever runs position 0 starts from zero.  `reserved` further
    slots own a full row of pages each (compat forwards)."""

    def __init__(self, layers: Sequence[LayerCache], slots: int, pages: int, max_seq: int, dtype: torch.dtype, device,
                 reserved: Sequence[int] = ()):
        self.slots, self.pages, self.max_seq = slots, pages, max_seq
        self.width = pages_for(max_seq)
        extra = len(reserved) * self.width
        self.scratch = pages + extra
        # zeros: a masked key of a page's unused tail must be a finite number
        z = lambda n, s, dt: torch.zeros(n, *s, dtype=dt, device=device)  # noqa: E731
        self.entries = [[z(pages + extra + 1, s, dtype) for s in l.pages] + [z(slots, s, torch.float32) for s in l.state] +
                        [z(slots, s, dtype) for s in l.ring] for l in layers]
        self.table = torch.full((slots, self.width), self.scratch, dtype=torch.int32, device=device)
        for k, s in enumerate(reserved):
            self.table[s] = torch.arange(pages + k * self.width, pages + (k + 1) * self.width, dtype=torch.int32,
                                         device=device)

    def rows(self, assignments):
        """(slots int64 [n], table rows int32 [n, width]) on the host for
        assignments = [(slot, pages), ...]."""
        import numpy as np

        out = np.full((len(assignments), self.width), self.scratch, dtype=np.int32)
        for k, (_, pages) in enumerate(assignments):
            if len(pages) > self.width:
                raise ValueError(f"{len(pages)} pages exceed the table width {self.width}")
            out[k, : len(pages)] = pages
        return np.asarray([s for s, _ in assignments], dtype=np.int64), out

    def assign(self, assignments) -> None:
        slots, rows = self.rows(assignments)
        dev = self.table.device
        self.table.index_copy_(0, torch.from_numpy(slots).to(dev), torch.from_numpy(rows).to(dev))

    @property
    def nbytes(self) -> int:
        return sum(p.numel() * p.element_size() for e in self.entries for p in e) + self.table.numel() * 4


class LatentCache(PagedCache):
    """Paged cache of latent rows (latent attention): pools[k][page, token, rank]
    per layer that owns latents."""

    def __init__(self, ranks: Sequence[int], slots: int, pages: int, max_seq: int, dtype: torch.dtype, device,
                 reserved: Sequence[int] = ()):
        super().__init__([LayerCache(pages=((PAGE, r),)) for r in ranks], slots, pages, max_seq, dtype, device, reserved)
        self.pools = [e[0] for e in self.entries]

    @staticmethod
    def bytes_per_page(ranks: Sequence[int], elt: int = 2) -> int:
        return PAGE * sum(ranks) * elt


def plan_pages(requested: int, per_page: int, device, fraction: float = 0.85, reserve: int = 0,
               mem_get_info=None) -> int:
    """Pages of `per_page` bytes <= requested that fit `fraction` of the free
    device memory left after `reserve` bytes (cf. plan_slots)."""
    dev = torch.device(device)
    if per_page == 0 or (dev.type != "cuda" and mem_get_info is None):
        return requested
    free, _ = (mem_get_info or torch.cuda.mem_get_info)(dev)
    return max(0, min(requested, int(max(0, free - reserve) * fraction) // per_page))


def plan_slots(requested: int, n_layers: int, n_kv: int, max_seq: int, head_dim: int,
               device, fraction: float = 0.85, elt: int = 2, reserve: int = 0,
               mem_get_info=None) -> int:
    """Largest slot count <= requested whose KV fits `fraction` of the free
    device memory left after `reserve` bytes (the stage's weights, loaded
    after this is decided).  `mem_get_info` is injectable for tests."""
    dev = torch.device(device)
    if dev.type != "cuda" and mem_get_info is None:
        return requested
    free, _ = (mem_get_info or torch.cuda.mem_get_info)(dev)
    per = KVCache.bytes_per_slot(n_layers, n_kv, max_seq, head_dim, elt)
    if per == 0:  # a stage without attention halves holds no KV
        return requested
    fit = int(max(0, free - reserve) * fraction) // per
    if fit < 1:
        raise MemoryError(f"KV cache: one slot needs {per / 2**30:.2f} GiB, free {free / 2**30:.2f} GiB")
    return min(requested, fit)


class SlotAllocator:
    """Host-side free list of KV slots (native version: SlotAllocator in
    csrc/runtime/runtime.cpp)."""

    def __init__(self, n: int):
        self._free: List[int] = list(range(n - 1, -1, -1))
        self.capacity = n

    def alloc(self, k: int = 1) -> List[int]:
        if k > len(self._free):
            raise RuntimeError(f"out of KV slots: want {k}, have {len(self._free)}")
        return [self._free.pop() for _ in range(k)]

    def free(self, slots) -> None:
        for s in slots:
            self._free.append(int(s))

    @property
    def available(self) -> int:
        return len(self._free)
