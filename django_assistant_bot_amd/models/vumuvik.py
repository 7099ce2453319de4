"""Vumuvik decoder on the native kernels: latent attention with a paged latent cache.

The same contract as ``LlamaModel``: one ``forward`` serves packed prefill chunks, decode rows and mixed
steps, every op enqueues on the current stream, and decode has fixed shapes so it is captured in a HIP
graph.  The residual stream is fp32; between two projections everything is one element-wise pass
(``ops.dyt_residual``), because Dynamic Tanh has no row statistic.

Per layer:  [q | latent] GEMM -> latent write (slab sum, RMS norm, cache) -> attention -> o GEMM ->
norm1b, ls1, residual, norm2 (one launch) -> gate|up GEMM (+ tanh-GELU GLU) -> down GEMM -> norm2b, ls2,
residual, next norm1 (one launch).

Attention is ``latent_attn.LatentAttention``.  Layers that share a latent (``kv_from``) read the owner's cache with
their own expansion, window and sink.

The 32-bit mode (``dtype=torch.float32``) runs the same steps with fp32 weights, activations and cache on
the fp32 MFMA GEMM and the absorbed attention kernel.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from .. import ops
from ..ops.latent import DytNorm
from .cache import AttnMeta, LatentCache
from .configs import LatentMixer, VumuvikConfig
from .latent_attn import LatentAttention, PrefillPlan
from .projections import FragmentProjections


@dataclass
class LatentDecoderLayer:
    mixer: LatentMixer
    D: int  # padded head width
    R: int  # padded latent width
    norm1: DytNorm
    norm1b: DytNorm
    ls1: torch.Tensor
    qd_w: torch.Tensor  # [q; latent] (own latent) or [q]
    latent_norm: torch.Tensor | None
    kv_w: torch.Tensor  # [W_uk; W_uv], the K / V expansion
    absorb_w: torch.Tensor  # W_uk^T per head
    sink: torch.Tensor
    o_w: torch.Tensor
    norm2: DytNorm | None = None
    norm2b: DytNorm | None = None
    ls2: torch.Tensor | None = None
    gate_up_w: torch.Tensor | None = None
    down_w: torch.Tensor | None = None


class VumuvikModel(LatentAttention, FragmentProjections):
    vocab_parallel = False
    custom_ar = None

    def __init__(self, cfg: VumuvikConfig, weights: dict, device, tp_group=None, tp_size: int = 1,
                 interleaved_mlp: bool = True, consume: bool = False, tp_rank: int | None = None):
        if tp_size != 1:
            raise ValueError("Vumuvik runs on one GPU per replica (tp_size 1)")
        self.cfg, self.device = cfg, torch.device(device)
        self.interleaved_mlp = interleaved_mlp
        self.vocab_local, self.vocab_start = cfg.vocab_size, 0
        take = weights.pop if consume else weights.__getitem__
        dtype = weights["embed"].dtype
        self.f32 = dtype == torch.float32
        gpu = self.device.type == "cuda"
        self.frag = gpu and not self.f32
        if self.frag and not interleaved_mlp:
            raise ValueError("bf16 Vumuvik on the GPU takes gate / up rows in 8-row groups (interleaved_mlp)")
        if gpu and self.f32 and interleaved_mlp:
            raise ValueError("32-bit Vumuvik takes stacked gate / up rows")
        self.proj_group = {}

        def mat(key, name=""):
            t = take(key).to(self.device)
            if not self.frag:
                return t
            g = self.PROJ_GROUPS.get(name, 1)
            g = g if t.shape[0] % (16 * g) == 0 and t.numel() * 2 < (1 << 31) else 1
            if self.proj_group.setdefault((name, *t.shape), g) != g:
                raise AssertionError("one grouping per projection shape")
            return ops.shuffle_weights(t, g)

        def norm(key):
            a, w, b = take(key)
            return DytNorm(a, w.to(self.device), b.to(self.device))

        self.embed = take("embed").to(self.device)
        self.lm_head = mat("lm_head")
        self.final_norm = norm("final_norm")
        self.source = [cfg.source(i) for i in range(cfg.layers)]
        self.layers = []
        for i, blk in enumerate(cfg.blocks):
            p, own = f"l{i}.", blk.mixer.kv_from is None
            L = LatentDecoderLayer(
                blk.mixer, cfg.padded_head(i), cfg.padded_rank(i), norm(p + "norm1"), norm(p + "norm1b"),
                take(p + "ls1").to(self.device), mat(p + "qd_w"),
                take(p + "latent_norm").to(self.device) if own else None, mat(p + "kv_w"), mat(p + "absorb_w"),
                take(p + "sink").to(self.device), mat(p + "o_w"))
            if blk.ff is not None:
                L.norm2, L.norm2b, L.ls2 = norm(p + "norm2"), norm(p + "norm2b"), take(p + "ls2").to(self.device)
                L.gate_up_w, L.down_w = mat(p + "gate_up_w", "gate_up"), mat(p + "down_w")
            self.layers.append(L)
        if gpu and consume:
            torch.cuda.empty_cache()
        self.layer_tap = None  # called as tap(layer, residual stream) after every layer (numerics tests)

    @property
    def dtype(self):
        return self.embed.dtype

    # ------------------------------------------------------------------ what the engine asks of a family
    def _widths(self):
        return [L.R for L in self.layers]

    def make_cache(self, num_blocks: int, block_size: int, slots: int = 0) -> LatentCache:
        return LatentCache(self._widths(), self.source, num_blocks, block_size, self.device, self.dtype)

    def cache_bytes_per_block(self, block_size: int) -> int:
        return LatentCache.bytes_per_block(self._widths(), self.source, block_size, self.dtype)

    def decode_part(self, batch: int, part_size: int) -> int:
        return part_size  # (the latent decode splits by partition count, ``_split``)

    def make_workspace(self, max_batch: int, max_len: int, part_size: int):
        return self._latent_workspace(self.layers, max_batch, max_len)

    # ------------------------------------------------------------------ forward
    def _proj(self, x, w, dec: bool, allow_slabs: bool = True, name: str = "", epilogue=ops.EPI_NONE):
        if x.is_cuda and not self.f32:
            self_group = self.proj_group.get((name, *w.shape), 1)
            return self._stream_or_tile(x, w, dec, allow_slabs, name, epilogue, self_group)
        if x.is_cuda:
            y = ops.gemm_f32(x, w)
            return ops.glu_f32(y) if epilogue != ops.EPI_NONE else y
        epi = epilogue if self.interleaved_mlp else ops.EPI_NONE
        y = ops.gemm_bt(x, w, epilogue=epi)
        return ops.glu_f32(y) if epilogue != epi else y

    def forward(self, ids: torch.Tensor, meta: AttnMeta, kv: LatentCache) -> torch.Tensor:
        """ids int32 [T] -> final hidden states [T, padded width] (after the last norm)."""
        T, nl = ids.numel(), len(self.layers)
        # decode-sized steps stream the weights through the split-K kernel, whose slabs the next
        # element-wise pass sums; short prefill steps do the same
        small_pf = not meta.decode and not meta.n_decode and T <= self.PREFILL_STREAM_MAX_M
        sk = self.frag and (meta.decode and T <= self.STREAM_MAX_M or small_pf)
        plan = None if meta.decode else PrefillPlan(meta, self.device)
        x, h = ops.embed_dyt(ids, self.embed, self.cfg.embed_scale, self.layers[0].norm1)
        for li, L in enumerate(self.layers):
            nxt = self.layers[li + 1].norm1 if li + 1 < nl else self.final_norm
            a = self._mixer(li, L, h, meta, kv, plan, sk)
            y = self._proj(a.reshape(T, -1), L.o_w, sk, name="o")
            h = ops.dyt_residual(x, y, L.norm1b, L.ls1, nxt if L.norm2 is None else L.norm2, self.dtype)
            if L.norm2 is not None:
                act = self._proj(h, L.gate_up_w, sk, name="gate_up", epilogue=ops.EPI_GEGLU8)
                h = ops.dyt_residual(x, self._proj(act, L.down_w, sk, name="down"), L.norm2b, L.ls2, nxt, self.dtype)
            if self.layer_tap is not None:
                self.layer_tap(li, x)
        return h

    def _mixer(self, li: int, L: LatentDecoderLayer, h, meta: AttnMeta, kv: LatentCache, plan, sk: bool):
        m, src = L.mixer, self.source[li]
        HD, T = m.heads * L.D, meta.positions.numel()
        own = src == li
        qd = self._proj(h, L.qd_w, sk, name="qd")
        q = ops.latent_write(qd, HD, L.latent_norm, kv.c[li] if own else None, meta.slots, m.rank, self.cfg.eps)
        q = q.unflatten(1, (m.heads, L.D))
        return self._latent_attend(L, q, src, meta, kv, plan)

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        """[n, padded width] -> [n, vocab]."""
        y = self._proj(h, self.lm_head, self.frag and h.shape[0] <= self.STREAM_MAX_M, False, name="lm_head")
        return y[:, :self.cfg.vocab_size]
