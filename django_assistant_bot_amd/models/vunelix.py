"""Vunelix decoder on the native kernels: selective scans and rotary latent attention, dense MLPs and routed experts, a loop
over a stretch of layers, paged latents beside recurrent state slots.

The same contract as ``LlamaModel``: one ``forward`` serves packed prefill portions, decode rows and mixed steps, every
op enqueues on the current stream, and decode has fixed shapes so it is captured in a HIP graph.  The residual stream is
fp32.  A layer is a mixer and a feed-forward, each between two RMS norms; everything between two of a sublayer's
projections is one element-wise pass (``ops.rms_residual``: slab sum, norm after, residual, next norm before).

    scan:        h -> in_w [x | z] -> convolution -> x_w [step | B | C] (fp32) -> scan, silu gate -> o_w
    attention:   h -> in_w [q | latent, rotated key | gate] -> norm, rotation, cache write -> latent attention -> gate -> o_w
    dense:       h -> gate_up_w (ReLU-gated epilogue) -> down_w
    experts:     h -> router_w (fp32) -> route -> grouped GEMMs;  h -> shared gate_up_w -> down_w

A prompt portion expands its steps with a GEMM (``dt_w``) before the scan; a decoded token does it inside the state step.

Before each pass of the loop x <- W_in [x; embedding] + step.  The embedding's half of that product depends on the token
alone, so it is a table made at load time (``loop_table``); a pass costs the product with x only.

The 32-bit mode (``dtype=torch.float32``) runs the same steps with fp32 weights, activations and cache.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from .. import ops
from .cache import AttnMeta, HybridCache, RunMemory
from .configs import DenseMlp, LatentMixer, MoeMlp, SelectiveMixer, VunelixConfig
from .latent_attn import LatentAttention, PrefillPlan
from .projections import HybridProjections
from .weights import selective_layout


@dataclass
class VunelixLayer:
    mixer: SelectiveMixer | LatentMixer
    norm1: torch.Tensor
    norm1b: torch.Tensor
    in_w: torch.Tensor
    o_w: torch.Tensor
    # scan
    scan: ops.SelectiveShape | None = None
    narrow: int = 0  # columns of the narrow projection
    x_w: torch.Tensor | None = None
    dt_w: torch.Tensor | None = None
    dt_bias: torch.Tensor | None = None
    conv_w: torch.Tensor | None = None
    conv_b: torch.Tensor | None = None
    A: torch.Tensor | None = None
    skip: torch.Tensor | None = None
    # attention
    D: int = 0  # padded head width
    R: int = 0  # padded width of a cached row
    latent_norm: torch.Tensor | None = None
    turns: torch.Tensor | None = None
    kv_w: torch.Tensor | None = None
    absorb_w: torch.Tensor | None = None
    sink: torch.Tensor | None = None
    # feed-forward
    norm2: torch.Tensor | None = None
    norm2b: torch.Tensor | None = None
    act: str = "silu"
    gate_up_w: torch.Tensor | None = None  # dense, or the shared expert
    down_w: torch.Tensor | None = None
    moe: MoeMlp | None = None
    router_w: torch.Tensor | None = None
    expert_gate_up_w: torch.Tensor | None = None
    expert_down_w: torch.Tensor | None = None


class VunelixModel(LatentAttention, HybridProjections):
    vocab_parallel = False
    custom_ar = None
    recurrent = True

    def __init__(self, cfg: VunelixConfig, weights: dict, device, tp_group=None, tp_size: int = 1,
                 interleaved_mlp: bool = True, consume: bool = False, tp_rank: int | None = None):
        if tp_size != 1:
            raise ValueError("Vunelix runs on one GPU per replica (tp_size 1)")
        self.cfg, self.device = cfg, torch.device(device)
        self.interleaved_mlp = interleaved_mlp
        self.vocab_local, self.vocab_start = cfg.vocab_size, 0
        take = weights.pop if consume else weights.__getitem__
        self.f32 = weights["embed"].dtype == torch.float32
        gpu = self.device.type == "cuda"
        self.frag = gpu and not self.f32
        if self.frag and not interleaved_mlp:
            raise ValueError("bf16 Vunelix on the GPU takes gate / up rows in 8-row groups (interleaved_mlp)")
        if gpu and self.f32 and interleaved_mlp:
            raise ValueError("32-bit Vunelix takes stacked gate / up rows")
        self.proj_group = {}

        def mat(key, name=""):
            return self._place(take(key).to(self.device), name) if key in weights else None

        def vec(key):
            return take(key).to(self.device).contiguous() if key in weights else None

        self.embed = take("embed").to(self.device)
        self.lm_head = mat("lm_head")
        self.final_norm = vec("final_norm")
        self.runs = cfg.runs()
        if cfg.passes:
            own, again = take("loop_w").to(self.device)
            self.loop_w, self.loop_step = self._place(own.contiguous()), vec("loop_step")
            self.loop_table = ops.gemm_f32(self.embed, again.contiguous()) if self.f32 else ops.gemm_bt(self.embed, again.contiguous(), out_f32=True)
        self.layers = []
        for i, blk in enumerate(cfg.blocks):
            p, m, f = f"l{i}.", blk.mixer, blk.mlp
            L = VunelixLayer(m, vec(p + "norm1"), vec(p + "norm1b"), mat(p + "in_w"), mat(p + "o_w"), norm2=vec(p + "norm2"),
                             norm2b=vec(p + "norm2b"))
            if isinstance(m, SelectiveMixer):
                lay = selective_layout(m)
                L.scan = ops.SelectiveShape(lay.inner, lay.state, lay.rank, lay.b_col, lay.c_col, lay.inner)
                L.narrow = lay.narrow
                L.x_w, L.dt_w, L.dt_bias, L.A, L.skip = mat(p + "x_w"), mat(p + "dt_w"), vec(p + "dt_bias"), vec(p + "A"), vec(p + "skip")
                L.conv_w, L.conv_b = vec(p + "conv_w"), vec(p + "conv_b")
            else:
                L.D, L.R, L.latent_norm = m.padded_head(), m.padded_row(), vec(p + "latent_norm")
                L.kv_w, L.absorb_w = mat(p + "kv_w"), mat(p + "absorb_w")
                if m.rot is not None:
                    L.turns = ops.rope_turns(m.rot.dims, m.rot.base, self.device, m.rot.scaling)
            L.gate_up_w, L.down_w = mat(p + "gate_up_w", "gate_up"), mat(p + "down_w")
            if isinstance(f, DenseMlp):
                L.act = f.act
            elif f is not None:
                L.moe, L.router_w = f, mat(p + "router_w")
                L.expert_gate_up_w, L.expert_down_w = mat(p + "expert_gate_up_w"), mat(p + "expert_down_w")
            self.layers.append(L)
        if gpu and consume:
            torch.cuda.empty_cache()
        self.layer_tap = None  # called as tap(run, residual stream) after every layer run (numerics tests)

    @property
    def dtype(self):
        return self.embed.dtype

    # ------------------------------------------------------------------ what the engine asks of a family
    def _specs(self):
        L = [self.layers[li] for li, _ in self.runs]
        return [RunMemory(latent=x.R) if x.scan is None else
                RunMemory(ring=(x.conv_w.shape[0], x.scan.C), state=(x.scan.C, x.scan.Np)) for x in L]

    def make_cache(self, num_blocks: int, block_size: int, slots: int = 1) -> HybridCache:
        return HybridCache(self._specs(), num_blocks, block_size, slots, self.device, self.dtype)

    def cache_bytes_per_block(self, block_size: int) -> int:
        return max(1, HybridCache.bytes_per_block(self._specs(), block_size, self.dtype))

    def state_bytes(self, slots: int) -> int:
        return slots * HybridCache.bytes_per_slot(self._specs(), self.dtype)

    def decode_part(self, batch: int, part_size: int) -> int:
        return part_size  # (the latent decode splits by partition count, ``_split``)

    def make_workspace(self, max_batch: int, max_len: int, part_size: int):
        attn = [L for L in self.layers if L.scan is None]
        return self._latent_workspace(attn, max_batch, max_len) if attn else None

    # ------------------------------------------------------------------ forward
    def forward(self, ids: torch.Tensor, meta: AttnMeta, kv: HybridCache) -> torch.Tensor:
        """ids int32 [T] -> final hidden states [T, padded width] (after the last norm)."""
        T, n, W, eps = ids.numel(), len(self.runs), self.cfg.hidden, self.cfg.eps
        # decode-sized steps stream the weights through the split-K kernel, whose slabs the consumers sum; short
        # prefill steps do the same
        small_pf = not meta.decode and not meta.n_decode and T <= self.PREFILL_STREAM_MAX_M
        sk = self.frag and (meta.decode and T <= self.STREAM_MAX_M or small_pf)
        plan = None if meta.decode else PrefillPlan(meta, self.device)

        def entry(r):
            """What run ``r`` reads: its norm's gain, or the stream itself where a pass starts."""
            if r == n:
                return dict(gain=self.final_norm)
            li, start = self.runs[r]
            return dict(gain=None, raw=True) if start is not None else dict(gain=self.layers[li].norm1)

        x = torch.empty((T, self.embed.shape[1]), dtype=torch.float32, device=ids.device)
        h = ops.rms_residual(x, None, n=W, eps=eps, dtype=self.dtype, again=(ids, self.embed), fresh=True, **entry(0))
        for r, (li, start) in enumerate(self.runs):
            L = self.layers[li]
            if start is not None:  # x <- W_in [x; embedding] + step
                y = self._aux(h, self.loop_w, sk, wide=True)
                h = ops.rms_residual(x, y, L.norm1, W, eps, self.dtype, self.loop_step[start], again=(ids, self.loop_table),
                                     fresh=True)
            y = self._scan(r, L, h, meta, kv, sk) if L.scan is not None else self._attention(r, L, h, meta, kv, plan, sk)
            if L.norm2 is None:
                h = ops.rms_residual(x, y, n=W, eps=eps, dtype=self.dtype, post=L.norm1b, **entry(r + 1))
            else:
                h = ops.rms_residual(x, y, L.norm2, W, eps, self.dtype, post=L.norm1b)
                y, pairs = self._mlp(L, h, sk)
                h = ops.rms_residual(x, y, n=W, eps=eps, dtype=self.dtype, pairs=pairs, post=L.norm2b, **entry(r + 1))
            if self.layer_tap is not None:
                self.layer_tap(r, x)
        return h

    def _scan(self, r: int, L: VunelixLayer, h, meta: AttnMeta, kv: HybridCache, sk: bool):
        d, ring, state, pos = L.scan, kv.ring[r], kv.state[r], meta.positions
        T = pos.numel()
        Tp = 0 if meta.decode else T - meta.n_decode
        y = self._proj(h, L.in_w, sk, name="in")
        slot = meta.state_slots if meta.decode else meta.dec_state_slots
        if Tp:
            u = ops.short_conv(y, 0, L.conv_w, L.conv_b, ring, meta.state_slots, pos, meta.cu_q, meta.max_q)
        else:
            u = torch.empty((T, d.C), dtype=self.dtype, device=h.device)
        out = torch.empty_like(u)
        if Tp < T:  # the gate's rows wait in ``out``
            ops.short_conv_step(y, 0, L.conv_w, L.conv_b, ring, slot, pos, Tp, u, d.z_col, out)
        low, step = ops.narrow_rows(self._aux(u, L.x_w, sk), L.narrow, d.rank, T, self.dtype)
        if Tp:
            dt = self._aux(step[:Tp], L.dt_w, False, wide=True)
            ops.selective_scan(u, d, dt, low, y, L.A, L.dt_bias, L.skip, state, meta.state_slots, pos, meta.cu_q, meta.max_q, out)
        if Tp < T:
            ops.selective_step(u, d, L.dt_w, step, low, L.A, L.dt_bias, L.skip, state, slot, pos, Tp, out)
        return self._proj(out, L.o_w, sk, name="o")

    def _attention(self, r: int, L: VunelixLayer, h, meta: AttnMeta, kv: HybridCache, plan, sk: bool):
        m = L.mixer
        HD = m.heads * L.D
        y = self._proj(h, L.in_w, sk, name="in")
        rope = None
        if m.rot is not None:
            rope = ops.LatentRope(L.turns, m.rot.gain, m.rot.dims, L.D, m.q_at, m.c_at, meta.positions)
        q = ops.latent_write(y, HD, L.latent_norm, kv.c[r], meta.slots, m.rank, self.cfg.eps, rope)
        o = self._latent_attend(L, q.unflatten(1, (m.heads, L.D)), r, meta, kv, plan).flatten(1)
        if m.gate:
            o = ops.sigmoid_gate(y, HD + L.R, o)
        return self._proj(o, L.o_w, sk, name="o")

    def _mlp(self, L: VunelixLayer, h, sk: bool):
        """-> (output of the dense MLP or the shared expert, or None; the routed experts' rows or None)."""
        m, y, pairs = L.moe, None, None
        if m is not None:
            idx, wt = ops.moe_route(self._aux(h, L.router_w, sk), 0, m.experts, m.top, m.scale, h.shape[0], m.scores)
            pairs = ops.moe_experts(h, idx, wt, L.expert_gate_up_w, L.expert_down_w, m.experts, 8 if self.interleaved_mlp else 0,
                                    m.weigh)
        if L.gate_up_w is not None:
            y = self._proj(self._glu(h, L.gate_up_w, L.act, sk), L.down_w, sk, name="down")
        return y, pairs

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        """[n, padded width] -> [n, vocab]."""
        y = self._proj(h, self.lm_head, self.frag and h.shape[0] <= self.STREAM_MAX_M, False, name="lm_head")
        if self.cfg.softcap:
            y = ops.softcap(y, self.cfg.softcap)
        return y[:, :self.cfg.vocab_size]
