"""Dispatch of a decoder's projections: which GEMM kernel runs a weight at a given row count.

Shared by the decoder families.  The host class provides ``frag`` (weights in the
``ops.shuffle_weights`` fragment layout), ``proj_group`` (grouping of each projection's copy),
``interleaved_mlp`` and ``tp_size``.
"""
from __future__ import annotations

import torch

from .. import ops


class FragmentProjections:
    frag = False
    tp_size = 1
    interleaved_mlp = True
    recurrent = False  # the model keeps a state slot per sequence (``models.cache.HybridCache``)

    def state_bytes(self, slots: int) -> int:
        """Bytes of ``slots`` state slots (none: every layer's memory is paged)."""
        return 0

    def step_bytes(self, tokens: int) -> int:
        """Bytes that a step over ``tokens`` tokens keeps from its first layer to its last (nothing worth planning for)."""
        return 0

    # stream_gemm.hip configurations (shuffled weights): BN 128 rows per workgroup at M <= 64 (13)
    # and M <= 128 (10).  Whole-chip tilings at M 65..128: gate_up's 28672 rows / 112 make exactly
    # 256 workgroups where BN 128 left 32 of the 256 CUs idle (cfg 20: 54.9 -> 51.5 us cold); the LM
    # head uses 192-row tiles (cfg 28: 2/3 of the X staging per weight byte, 228.7 -> 221.3 us).
    # qkv at 96 rows x 4 K-slices (cfg 21) measured slower than BN 128 x 4 (17.1 vs 15.8 us).
    # Decode batches of 129..256 rows: 64-row tiles, 2 k-groups x 4 row groups (cfg 27; M = 256:
    # qkv 27.4 / o 18.6 / gate_up 98.7 / down 49.2 us against 32.4 / 25.8 / 104 / 55 for two
    # M = 128 passes, profiles/decode_round2.md).
    STREAM_CFG_M16, STREAM_CFG_M32, STREAM_CFG_M64, STREAM_CFG_M128, STREAM_CFG_M256 = 30, 31, 13, 10, 27
    STREAM_WIDE = {"gate_up": 20, "lm_head": 28}
    STREAM_MAX_M = ops.STREAM_MAX_M
    PREFILL_STREAM_MAX_M = 128  # prefill steps of at most this many tokens stream too (0: off)

    def _stream_cfg(self, name: str, M: int, N: int) -> int:
        nat = ops.native()
        if M > 128 and name == "gate_up":
            # decode batches of 129..256: gate_up (+SwiGLU8) on the mid-M GEMM, 67-72 us against 90-96
            # on the M <= 256 streaming tiles (profiles/small_prefill_r6.md); qkv / o / down stream
            return -1
        if M > 128:
            cfg = self.STREAM_CFG_M256
        elif M <= 16 and N % nat.stream_gemm_bn(self.STREAM_CFG_M16) == 0:
            cfg = self.STREAM_CFG_M16
        elif M <= 32 and N % nat.stream_gemm_bn(self.STREAM_CFG_M32) == 0:
            cfg = self.STREAM_CFG_M32
        elif M <= 64:
            cfg = self.STREAM_CFG_M64
        else:
            cfg = self.STREAM_WIDE.get(name)
            if cfg is None or N % nat.stream_gemm_bn(cfg):
                cfg = self.STREAM_CFG_M128
        return cfg if N % nat.stream_gemm_bn(cfg) == 0 else -1

    @staticmethod
    def _stream_splits(N: int, K: int, bn: int = 128) -> int:
        """K-slices for stream_gemm: the fewest that give >= 192 workgroups of ``bn`` weight rows."""
        tiles, best = N // bn, 1
        for s in (1, 2, 4, 8, 16):
            if K % (128 * s):
                break
            best = s
            if tiles * s >= 192:
                break
        return best

    def _stream_choice(self, name: str, M: int, N: int, K: int) -> tuple[int, int]:
        """(stream_gemm cfg, K-slices) of a decode projection; cfg -1 = not streamable.  (The tuning
        harness benchmarks/decode_ab.py overrides this in a subclass.)"""
        cfg = self._stream_cfg(name, M, N)
        if cfg < 0 or K % 128:
            return -1, 1
        return cfg, self._stream_splits(N, K, ops.native().stream_gemm_bn(cfg))

    # Projections held in the grouped fragment layout (shuffle_weights(w, G): the G row blocks of
    # each 16 G-row group adjacent per 32-deep k chunk), so the decode GEMM's waves (one block each)
    # stream neighbouring bytes; every GEMM reading a copy takes its group (``proj_group``).  gate_up
    # at 8: batch-128 decode step 7.31 -> 7.23 ms (profiles/decode_stream_layout_r6.md)
    PROJ_GROUPS = {"gate_up": 8}

    # Split-K slabs of the decode projections as bf16 (the partial sums rounded once, as the TP path
    # hands them to its all-reduce) instead of fp32: half the bytes the producer writes and the
    # RMSNorm / RoPE consumers read; batch-128 decode step 7.503 -> 7.351 ms (benchmarks/decode_ab.py
    # slab32,slab16; profiles/decode_slab_r6.md).  TP keeps fp32: its fused all-reduce + norm sums
    # fp32 slabs.
    slab_bf16 = True

    def _proj(self, x, w, dec: bool, allow_slabs: bool = True, name: str = "", epilogue=ops.EPI_NONE):
        """One projection.  Decode-sized batches (``dec``) stream the fragment-layout weights
        through stream_gemm, as fp32 split-K slabs when a consumer sums them (RMSNorm, the decode
        attention's RoPE prologue) and ``allow_slabs``; everything else runs the MFMA GEMM on the
        same copy (gemm256 for large token counts, the 128x128 kernel below that)."""
        if not x.is_cuda:
            if epilogue == ops.EPI_SWIGLU8 or (epilogue == ops.EPI_NONE and name == "gate_up"):
                y = ops.linear(x, w)
                return ops.silu_mul(y, group=8 if self.interleaved_mlp else 0)
            return ops.linear(x, w)
        return self._stream_or_tile(x, w, dec, allow_slabs, name, epilogue, self.proj_group.get(name, 1))

    def _stream_or_tile(self, x, w, dec: bool, allow_slabs: bool, name: str, epilogue, grp: int, out=None, glu_bias=None):
        """``out`` / ``glu_bias``: of a gated epilogue (a view to write, fp32 [gate | up])."""
        if dec and self.frag:
            cfg, s = self._stream_choice(name, x.shape[0], w.shape[0], w.shape[1])
            if cfg >= 0:
                if epilogue != ops.EPI_NONE:
                    return ops.stream_gemm(x, w, epilogue=epilogue, nt=True, cfg=cfg, w_group=grp, out=out,
                                           glu_bias=glu_bias)
                sd = torch.bfloat16 if (self.slab_bf16 and self.tp_size == 1) else torch.float32
                out = ops.stream_gemm(x, w, splits=s, cfg=cfg, nt=True, slab_dtype=sd, w_group=grp)
                return ops.slab_reduce(out) if (s > 1 and not allow_slabs) else out
        return ops.gemm_bt(x, w, epilogue=epilogue, shuffled=self.frag, b_group=grp, out=out, glu_bias=glu_bias)


class HybridProjections(FragmentProjections):
    """The projections of a decoder that runs in bf16 (fragment layout on the GPU) or, with ``f32``, in 32-bit."""

    f32 = False
    GLU8 = {"silu": ops.EPI_SWIGLU8, "gelu": ops.EPI_GEGLU8, "relu": ops.EPI_REGLU8}

    def _place(self, t, name: str = ""):
        """A projection's weights as its GEMMs read them."""
        if not self.frag:
            return t
        g = self.PROJ_GROUPS.get(name, 1)
        g = g if t.shape[0] % (16 * g) == 0 and t.numel() * 2 < (1 << 31) else 1
        if self.proj_group.setdefault((name, *t.shape), g) != g:
            raise AssertionError("one grouping per projection shape")
        return ops.shuffle_weights(t, g)

    def _proj(self, x, w, dec: bool, allow_slabs: bool = True, name: str = ""):
        if x.is_cuda and not self.f32:
            return self._stream_or_tile(x, w, dec, allow_slabs, name, ops.EPI_NONE, self.proj_group.get((name, *w.shape), 1))
        return ops.gemm_f32(x, w) if self.f32 else ops.gemm_bt(x, w)

    def _aux(self, h, w, dec: bool, wide: bool = False):
        """A projection whose result stays in 32 bits: decode-sized steps as split-K slabs; ``wide``: as many columns as
        the large ones."""
        if not (h.is_cuda and not self.f32):
            return ops.gemm_f32(h, w)
        if dec:
            cfg, _ = self._stream_choice("aux", h.shape[0], w.shape[0], w.shape[1])
            s = next((s for s in (16, 8, 4, 2) if w.shape[1] % (128 * s) == 0), 1)
            if cfg >= 0 and s > 1:
                return ops.stream_gemm(h, w, splits=s, cfg=cfg, nt=True)
        return ops.gemm_bt(h, w, out_f32=True, shuffled=True) if wide else ops.gemm_narrow(h, w)

    def _glu(self, h, w, act: str, dec: bool, out=None, bias=None):
        """act(gate) * up of a [gate | up] projection (``bias`` fp32 [gate | up])."""
        if h.is_cuda and not self.f32:
            return self._stream_or_tile(h, w, dec, False, "gate_up", self.GLU8[act],
                                        self.proj_group.get(("gate_up", *w.shape), 1), out=out, glu_bias=bias)
        if self.interleaved_mlp:
            y = ops.gemm_bt(h, w, epilogue=self.GLU8[act], glu_bias=bias)
            return y if out is None else out.copy_(y)
        return ops.glu_f32(ops.gemm_f32(h, w), act, bias=bias, out=out)
