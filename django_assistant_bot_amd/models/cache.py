"""Per-forward batch description and the paged caches of the decoder families.

One native block manager (csrc/runtime/kv_manager.h) hands out block ids; every cache is indexed by the
same ids, so scheduling, block tables and prefix reuse do not depend on what a block holds: per-head keys
and values (``KVCache``) or one latent per token (``LatentCache``).  ``HybridCache`` adds what recurrent
layers carry: a state slot per sequence, handed out by the same manager.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import NamedTuple

import torch

from .. import ops


@dataclass
class AttnMeta:
    """Per-forward batch description (device tensors, fixed shapes in decode graphs)."""

    decode: bool
    positions: torch.Tensor  # int32 [T]
    slots: torch.Tensor  # int64 [T] cache slot of each token (<0 = padding)
    block_tables: torch.Tensor  # int32 [B, max_blocks]
    ctx_lens: torch.Tensor  # int32 [B] total tokens in cache after this step
    cu_q: torch.Tensor | None = None  # int32 [B+1] (prefill)
    max_q: int = 1
    workspace: ops.DecodeWorkspace | None = None
    part_size: int = 512
    # mixed step: the LAST n_decode tokens are single-token decode rows (one per sequence) with their
    # own block tables / context lengths; the tokens before them are prefill chunks described above
    n_decode: int = 0
    dec_block_tables: torch.Tensor | None = None
    dec_ctx_lens: torch.Tensor | None = None
    order: torch.Tensor | None = None  # int32 [B] decode attention dispatch order (longest context first;
    # of the decode rows in a mixed step)
    # host copies of the prefill chunks' (query tokens, context length), for families that size work by them
    chunk_lens: list | None = None
    max_len: int | None = None  # longest context any decode row of the engine can reach
    # models with recurrent layers: int32 state slot of every prefill chunk (of every row when ``decode``), and of the
    # decode rows of a mixed step
    state_slots: torch.Tensor | None = None
    dec_state_slots: torch.Tensor | None = None


class KVCache:
    """Paged KV cache: per layer [num_blocks, Hkv_local, block_size, D] for K and for V."""

    def __init__(self, layers, num_blocks, kv_heads, block_size, head_dim, device, dtype=torch.bfloat16):
        self.num_blocks, self.block_size = num_blocks, block_size
        self.k = torch.zeros((layers, num_blocks, kv_heads, block_size, head_dim), device=device, dtype=dtype)
        self.v = torch.zeros_like(self.k)

    @staticmethod
    def bytes_per_block(layers, kv_heads, block_size, head_dim, dtype=torch.bfloat16):
        return 2 * layers * kv_heads * block_size * head_dim * torch.finfo(dtype).bits // 8


class LatentCache:
    """Paged latents: one [num_blocks, block_size, width] tensor per layer that computes a latent; a layer
    that reuses another layer's latent shares that layer's tensor.  ``widths``: row width of each layer's
    latent (padded); ``source``: for each layer, the layer whose latent it reads."""

    def __init__(self, widths, source, num_blocks, block_size, device, dtype=torch.bfloat16):
        self.num_blocks, self.block_size = num_blocks, block_size
        self.c = [torch.zeros((num_blocks, block_size, w), device=device, dtype=dtype) if src == i else None
                  for i, (w, src) in enumerate(zip(widths, source))]
        for i, src in enumerate(source):
            self.c[i] = self.c[src]

    @staticmethod
    def bytes_per_block(widths, source, block_size, dtype=torch.bfloat16):
        own = sum(w for i, w in enumerate(widths) if source[i] == i)
        return own * block_size * torch.finfo(dtype).bits // 8


class RunMemory(NamedTuple):
    """What one layer run keeps (None: nothing of the kind)."""

    kv: tuple | None = None  # per-head keys and values: (kv_heads, D)
    latent: int | None = None  # latent row: its padded width
    ring: tuple | None = None  # convolution inputs per slot: (taps, channels)
    state: tuple | None = None  # fp32 state per slot: its shape


class HybridCache:
    """Memory of a decoder whose layers mix attention and recurrence, one entry per layer RUN (a looped layer has
    its own in every pass).  Attention: paged K and V [num_blocks, kv_heads, block_size, D], or paged latent rows ``c``
    [num_blocks, block_size, width].  Recurrence: per slot the ring of the last ``taps`` convolution inputs [slots, taps,
    channels] and the fp32 state [slots, *shape].  The last slot takes the writes of padded decode rows."""

    def __init__(self, runs: list, num_blocks, block_size, slots, device, dtype=torch.bfloat16):
        self.num_blocks, self.block_size, self.slots = num_blocks, block_size, slots

        def z(on, *shape, dt=dtype):
            return None if on is None else torch.zeros(shape, device=device, dtype=dt)

        self.k, self.v, self.c, self.ring, self.state = [], [], [], [], []
        for m in runs:
            for c in (self.k, self.v):
                c.append(m.kv and z(m.kv, num_blocks, m.kv[0], block_size, m.kv[1]))
            self.c.append(z(m.latent, num_blocks, block_size, m.latent))
            self.ring.append(z(m.ring, slots, *(m.ring or ())))
            self.state.append(z(m.state, slots, *(m.state or ()), dt=torch.float32))

    @staticmethod
    def bytes_per_block(runs, block_size, dtype=torch.bfloat16):
        cells = sum(2 * m.kv[0] * m.kv[1] for m in runs if m.kv) + sum(m.latent for m in runs if m.latent)
        return cells * block_size * torch.finfo(dtype).bits // 8

    @staticmethod
    def bytes_per_slot(runs, dtype=torch.bfloat16):
        ring = sum(math.prod(m.ring) for m in runs if m.ring) * torch.finfo(dtype).bits // 8
        return ring + 4 * sum(math.prod(m.state) for m in runs if m.state)
