"""Paged cache pools and the per-step metadata every model's forward reads.

A block id names the same 16-token page in every pool of a model, so the scheduler and its block
manager (csrc/runtime) know nothing of what a page holds:

  KVCache        per-head keys and values (Llama)
  LatentKVCache  one latent row per token for all heads (latent attention), one pool per layer RUN:
                 a layer that a looped stack runs several times has a pool for each pass, and
                 layers of different widths have pools of their own widths
  HybridCache    per layer run, per-head keys and values with their pooled blocks, latent rows (a run may
                 read another's), or the state slots of a recurrent layer, which belong to sequences
                 (the scheduler hands them out) and not to pages
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Sequence

import torch


@dataclass
class StepMeta:
    """Device views of one step's metadata (layout from the native scheduler)."""
    input_ids: torch.Tensor
    positions: torch.Tensor
    slots: torch.Tensor
    q_start: torch.Tensor
    q_len: torch.Tensor
    ctx_len: torch.Tensor
    block_table: torch.Tensor
    items: torch.Tensor
    n_items: torch.Tensor
    att_counters: torch.Tensor  # persistent zeroed workspace (partition tickets), not step data
    logit_rows: torch.Tensor
    num_seqs: int = 0  # host-side count, used only by the CPU reference path
    part_size: Optional[torch.Tensor] = None  # device int[1]: decode partition size of the step
    # recurrent layers: each sequence's state slot and first scan item, the step's scan items
    state_slot: Optional[torch.Tensor] = None
    scan_first: Optional[torch.Tensor] = None
    scan_items: Optional[torch.Tensor] = None
    n_scan: Optional[torch.Tensor] = None


class KVCache:
    """Per-layer paged pools (bf16): K [NB, KV, 128/8, 16, 8] fragment-major,
    V^T [NB, KV, 128, 16] (layouts: csrc/ops/rope_cache.hip)."""

    def __init__(self, num_layers: int, num_blocks: int, kv_heads: int, device, dtype=torch.bfloat16,
                 block_size: int = 16):
        self.num_blocks = num_blocks
        self.block_size = block_size
        self.k = torch.zeros(num_layers, num_blocks, kv_heads, 16, block_size, 8, dtype=dtype, device=device)
        self.v = torch.zeros(num_layers, num_blocks, kv_heads, 128, block_size, dtype=dtype, device=device)

    def nbytes(self) -> int:
        return self.k.numel() * self.k.element_size() + self.v.numel() * self.v.element_size()

    @staticmethod
    def bytes_per_block(num_layers: int, kv_heads: int, block_size: int = 16) -> int:
        return 2 * num_layers * kv_heads * block_size * 128 * 2


class LatentKVCache:
    """Pools [blocks, D/8, 16, 8] of the given widths D (one per layer run): fragment-major rows
    (csrc/ops/latent_cache.hip)."""

    def __init__(self, widths: Sequence[int], num_blocks: int, device, dtype=torch.bfloat16, block_size: int = 16):
        if block_size != 16:
            raise ValueError("latent pages hold 16 tokens")
        self.num_blocks = num_blocks
        self.block_size = block_size
        self.pages: List[torch.Tensor] = [
            torch.zeros(num_blocks, d // 8, block_size, 8, dtype=dtype, device=device) for d in widths]

    @staticmethod
    def bytes_per_block(widths: Sequence[int], itemsize: int, block_size: int = 16) -> int:
        return sum(widths) * block_size * itemsize

    def nbytes(self) -> int:
        return sum(p.numel() * p.element_size() for p in self.pages)


class HybridCache:
    """`layers` has a list per layer run, an entry for each of its mixers. Attention has (keys [blocks, G, DK/8, 16,
    8], values alike, pooled keys [blocks, per page, G, DK], pooled values): a pooled block lies with the page of
    its last token (csrc/ops/paged_kv.hip); several key heads may share a value head. A state space has (state
    fp32 [slots, H, V, N], ring of the convolution's inputs [slots, rows, channels]), a matrix memory (state fp32
    [slots, H, V, N], its running maximum at every row [slots, H, V]), linear attention (state fp32 [slots, H, V, N]); a
    sequence that starts overwrites what its slot held. Latent attention has (rows [blocks, D/8, 16, 8],), as LatentKVCache;
    ("same", j) is the entry of run j."""

    def __init__(self, kinds: Sequence[Sequence[tuple]], num_blocks: int, slots: int, device, dtype=torch.bfloat16,
                 block_size: int = 16):
        if block_size != 16:
            raise ValueError("pages hold 16 tokens")
        self.num_blocks, self.slots, self.block_size = num_blocks, slots, block_size
        zeros = lambda dt, *s: torch.zeros(*s, dtype=dt, device=device)  # noqa: E731

        def pools(kind, *n):
            if kind == "same":
                return self.layers[n[0]][0]
            if kind == "latent":
                return zeros(dtype, num_blocks, n[0] // 8, 16, 8),
            if kind == "attention":
                G, dk, dv, per, gv = n
                return (zeros(dtype, num_blocks, G, dk // 8, 16, 8), zeros(dtype, num_blocks, gv, dv // 8, 16, 8),
                        zeros(dtype, num_blocks if per else 0, per, G, dk), zeros(dtype, num_blocks if per else 0, per, gv, dv))
            H, V, N = n[:3]
            state = zeros(torch.float32, slots, H, V, N)
            if kind == "linear":
                return state,
            return state, zeros(torch.float32, slots, H, V) if kind == "memory" else zeros(dtype, slots, *n[3:])
        self.layers: List[List[tuple]] = []
        for run in kinds:
            self.layers.append([pools(*k) for k in run])

    @staticmethod
    def bytes_per_block(kinds: Sequence[Sequence[tuple]], itemsize: int, block_size: int = 16) -> int:
        each = {"attention": lambda G, dk, dv, per, gv: (G * dk + gv * dv) * (block_size + per),
                "latent": lambda D: D * block_size}
        return itemsize * sum(each[kind](*n) for run in kinds for kind, *n in run if kind in each)

    @staticmethod
    def bytes_per_slot(kinds: Sequence[Sequence[tuple]], itemsize: int) -> int:
        each = {"state": lambda H, V, N, rows, ch: 4 * H * V * N + rows * ch * itemsize,
                "memory": lambda H, V, N: 4 * H * V * (N + 1), "linear": lambda H, V, N: 4 * H * V * N}
        return sum(each[kind](*n) for run in kinds for kind, *n in run if kind in each)

    def nbytes(self) -> int:
        pools = {id(t): t for run in self.layers for ts in run for t in ts}
        return sum(t.numel() * t.element_size() for t in pools.values())
