"""Per-forward batch description and the paged caches of the decoder families.

One native block manager (csrc/runtime/kv_manager.h) hands out block ids; every cache is indexed by the
same ids, so scheduling, block tables and prefix reuse do not depend on what a block holds: per-head keys
and values (``KVCache``) or one latent per token (``LatentCache``).  ``HybridCache`` adds what recurrent
layers carry: a state slot per sequence, handed out by the same manager.
"""
from __future__ import annotations

from dataclasses import dataclass

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


class HybridCache:
    """Memory of a decoder whose layers mix attention and recurrence, one entry per layer RUN (a looped layer has
    its own in every pass).  Attention: paged K and V [num_blocks, kv_heads, block_size, D].  Recurrence: per slot
    the ring of the last ``taps`` convolution inputs [slots, taps, channels] and the fp32 state [slots, heads, V,
    Dp].  The last slot takes the writes of padded decode rows.  ``specs``: per run (attention (kv_heads, D) or None,
    (taps, ``ops.RecurrentShape``))."""

    def __init__(self, specs, num_blocks, block_size, slots, device, dtype=torch.bfloat16):
        self.num_blocks, self.block_size, self.slots = num_blocks, block_size, slots
        z = lambda *shape, dt=dtype: torch.zeros(shape, device=device, dtype=dt)  # noqa: E731
        self.k, self.v, self.ring, self.state = [], [], [], []
        for attn, (taps, d) in specs:
            for c in (self.k, self.v):
                c.append(None if attn is None else z(num_blocks, attn[0], block_size, attn[1]))
            self.ring.append(z(slots, taps, d.C))
            self.state.append(z(slots, d.H, d.V, d.Dp, dt=torch.float32))

    @staticmethod
    def bytes_per_block(specs, block_size, dtype=torch.bfloat16):
        return sum(2 * a[0] * a[1] * block_size * torch.finfo(dtype).bits // 8 for a, _ in specs if a is not None)

    @staticmethod
    def bytes_per_slot(specs, dtype=torch.bfloat16):
        return sum(t * d.C * torch.finfo(dtype).bits // 8 + 4 * d.H * d.V * d.Dp for _, (t, d) in specs)
