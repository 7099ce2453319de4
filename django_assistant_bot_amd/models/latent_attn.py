"""Attention over a paged latent cache, shared by the families that have it.

Two exact forms of the same scores: prefill expands K and V of the visible context from the cached rows and runs the
windowed flash kernel; decode folds W_uk into the query and W_uv behind the softmax, so each cached row is read once for
all heads.  A rotated key part that the heads share is a part of the cached row.  ``absorb_w`` carries an identity block
for it; ``kv_w`` does too where it spans whole rows, and where it spans their latent part only the rotated part is copied
to the expanded keys.

A layer provides ``mixer`` (``configs.LatentMixer``), ``D`` (padded head width), ``R`` (padded row width), ``kv_w`` [K rows; V
rows], ``absorb_w`` (the K rows of every head transposed) and ``sink`` (or None).
"""
from __future__ import annotations

import numpy as np
import torch

from .. import ops
from ..ops.latent import FLASH_WINDOW_DIMS, decode_split
from .cache import AttnMeta


class PrefillPlan:
    """What the chunks of one forward see: per window, the packed context rows (cu_k), and the latents
    gathered for them (shared by the layers that read one cache)."""

    def __init__(self, meta: AttnMeta, device):
        self.meta, self.device = meta, device
        self._cu: dict = {}
        self._c: dict = {}

    def context(self, window: int):
        if window not in self._cu:
            n = [min(ctx, q + window - 1) if window else ctx for q, ctx in self.meta.chunk_lens]
            cu = torch.from_numpy(np.concatenate([[0], np.cumsum(n)]).astype(np.int32))
            if self.device.type == "cuda":
                cu = cu.pin_memory().to(self.device, non_blocking=True)
            self._cu[window] = (cu, int(sum(n)))
        return self._cu[window]

    def latents(self, src: int, window: int, cache):
        if (src, window) not in self._c:
            cu, total = self.context(window)
            # one source's rows stay live at a time: the layers that share them are neighbours
            self._c = {k: v for k, v in self._c.items() if k[0] == src}
            self._c[src, window] = ops.latent_gather(cache.c[src], self.meta.block_tables, cu, self.meta.ctx_lens, total)
        return self._c[src, window]


class LatentAttention:
    """The host class provides ``frag``, ``f32``, ``dtype`` and ``_proj``."""

    def _split(self, L, batch: int, max_len: int) -> tuple[int, int]:
        return decode_split(batch, L.mixer.heads, L.R, L.mixer.window, max_len) if self.frag else (1, 128)

    def _latent_workspace(self, layers, max_batch: int, max_len: int):
        rows = [(b * L.mixer.heads * self._split(L, b, max_len)[0], L.R) for L in layers for b in range(1, max_batch + 1)]
        return ops.LatentWorkspace(max(r for r, _ in rows), max(r * R for r, R in rows), self.device)

    def _latent_attend(self, L, q, src: int, meta: AttnMeta, kv, plan):
        """q [T, H, D] (written rows are in the cache ``kv.c[src]``) -> [T, H, D]."""
        m, T = L.mixer, q.shape[0]
        Tp = 0 if meta.decode else T - meta.n_decode
        if Tp == T:
            return self._latent_prefill(L, q, src, meta, kv, plan)
        if meta.decode:
            return self._latent_decode(L, q, kv.c[src], meta.block_tables, meta.ctx_lens, meta)
        out = torch.empty((T, m.heads, L.D), dtype=self.dtype, device=q.device)
        if Tp:
            self._latent_prefill(L, q[:Tp], src, meta, kv, plan, out[:Tp])
        self._latent_decode(L, q[Tp:], kv.c[src], meta.dec_block_tables, meta.dec_ctx_lens, meta, out[Tp:])
        return out

    def _latent_decode(self, L, q, cache, block_tables, ctx_lens, meta: AttnMeta, out=None):
        m = L.mixer
        qa = ops.head_gemm(q, L.absorb_w, L.R)
        parts, min_part = self._split(L, q.shape[0], meta.max_len) if meta.workspace is not None else (1, 128)
        oa = ops.latent_decode(qa, cache, block_tables, ctx_lens, m.scale, m.window, L.sink, parts, meta.workspace,
                               meta.order, min_part, values=L.kv_w.shape[1])
        return ops.head_gemm(oa[..., :L.kv_w.shape[1]], L.kv_w, L.D, row0=m.heads * L.D, out=out)

    def _latent_prefill(self, L, q, src: int, meta: AttnMeta, kv, plan, out=None):
        m, HD = L.mixer, L.mixer.heads * L.D
        if self.f32 or L.D not in FLASH_WINDOW_DIMS:
            oa = ops.latent_attention(ops.head_gemm(q, L.absorb_w, L.R), kv.c[src], meta.block_tables, meta.cu_q,
                                      meta.ctx_lens, m.scale, m.window, L.sink)
            return ops.head_gemm(oa[..., :L.kv_w.shape[1]], L.kv_w, L.D, row0=HD, out=out)
        cu_k, total = plan.context(m.window)
        rows, n = plan.latents(src, m.window, kv), L.kv_w.shape[1]
        kvx = self._proj(rows[:, :n], L.kv_w, False, name="kv").view(total, 2, m.heads, L.D)
        if n < L.R:
            ops.latent_key_fill(kvx[:, 0], rows, m.q_at, m.c_at, m.rot.dims)
        return ops.flash_attention_window(q, kvx[:, 0], kvx[:, 1], meta.cu_q, cu_k, meta.max_q, m.scale, m.window,
                                          L.sink, out=out)
