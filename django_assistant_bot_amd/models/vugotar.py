"""Vugotar decoder on the native kernels: hybrid layers of chunked attention, gated delta rule and Mamba-2 mixers with
dense or expert MLPs, a loop over a stretch of layers, paged K / V beside recurrent state slots.

The same contract as ``LlamaModel``: one ``forward`` serves packed prefill portions, decode rows and mixed steps, every
op enqueues on the current stream, and decode has fixed shapes so it is captured in a HIP graph.  The residual stream is
fp32.  Mixer and MLP of a layer read one norm and are summed, so a layer is two large GEMMs around its mixers:

    h -> in_w  [attention q | k | v, convolution channels, gates, shared expert gate | up]
    h -> aux_w [recurrence gates, router logits] (fp32)        h -> gate_up_w (SwiGLU + bias epilogue)
    attention (rotary + norm + cache write, then chunked softmax)    recurrence (convolution, state, gated norm)
    [MLP | attention | recurrence] -> out_w -> residual (+ bias + experts + embedding of the next pass), next norm

The mixers write their column blocks of one activation buffer, scaled in fp32, so the sum over sublayers happens inside
the output GEMM.  A prompt portion runs the token-parallel convolution and a scan; a decoded token runs one kernel per
recurrence.  Every layer run of a loop has its own cache and state.

The 32-bit mode (``dtype=torch.float32``) runs the same steps with fp32 weights, activations and cache.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from .. import ops
from .cache import AttnMeta, HybridCache, RunMemory
from .configs import ChunkedMixer, DenseMlp, MoeMlp, ParallelMixer, VugotarConfig
from .projections import HybridProjections
from .weights import HybridLayout, hybrid_layout


@dataclass
class HybridDecoderLayer:
    lay: HybridLayout
    attn: ChunkedMixer | None
    D: int  # padded attention head width
    attn_scale: float  # of the attention output
    rec: ops.RecurrentShape
    rec_scale: float
    norm_part: int  # channels of one group of the recurrence's output norm
    norm1: torch.Tensor
    in_w: torch.Tensor
    aux_w: torch.Tensor
    out_w: torch.Tensor
    conv_w: torch.Tensor
    A: torch.Tensor
    dt_bias: torch.Tensor
    rec_norm: torch.Tensor
    conv_b: torch.Tensor | None = None
    skip: torch.Tensor | None = None
    turns: torch.Tensor | None = None
    sink: torch.Tensor | None = None
    gate_up_w: torch.Tensor | None = None
    gate_up_b: torch.Tensor | None = None
    down_b: torch.Tensor | None = None
    moe: MoeMlp | None = None
    expert_gate_up_w: torch.Tensor | None = None
    expert_down_w: torch.Tensor | None = None


def _recurrent_shape(mixer, lay: HybridLayout) -> ops.RecurrentShape:
    a = lay.aux.at
    if isinstance(mixer, ParallelMixer):
        d = mixer.right
        n = d.kv_heads * d.dim
        return ops.RecurrentShape(True, d.heads, d.kv_heads, d.dim, d.vdim, lay.conv, 0, n, 2 * n, a["a"], a["b"])
    inner, n = mixer.heads * mixer.vdim, mixer.groups * mixer.state
    # x | B | C: values, keys, queries
    return ops.RecurrentShape(False, mixer.heads, mixer.groups, mixer.state, mixer.vdim, lay.conv, inner + n, inner, 0,
                              a["a"], 0)


class VugotarModel(HybridProjections):
    vocab_parallel = False
    custom_ar = None
    recurrent = True

    def __init__(self, cfg: VugotarConfig, weights: dict, device, tp_group=None, tp_size: int = 1,
                 interleaved_mlp: bool = True, consume: bool = False, tp_rank: int | None = None):
        if tp_size != 1:
            raise ValueError("Vugotar runs on one GPU per replica (tp_size 1)")
        self.cfg, self.device = cfg, torch.device(device)
        self.interleaved_mlp = interleaved_mlp
        self.vocab_local, self.vocab_start = cfg.vocab_size, 0
        take = weights.pop if consume else weights.__getitem__
        self.f32 = weights["embed"].dtype == torch.float32
        gpu = self.device.type == "cuda"
        self.frag = gpu and not self.f32
        if self.frag and not interleaved_mlp:
            raise ValueError("bf16 Vugotar on the GPU takes gate / up rows in 8-row groups (interleaved_mlp)")
        if gpu and self.f32 and interleaved_mlp:
            raise ValueError("32-bit Vugotar takes stacked gate / up rows")
        self.proj_group = {}

        def mat(key, name=""):
            return self._place(take(key).to(self.device), name)

        def vec(key):
            return take(key).to(self.device).contiguous() if key in weights else None

        self.embed = take("embed").to(self.device)
        self.lm_head = mat("lm_head")
        self.final_norm = vec("final_norm")
        self.runs = cfg.runs()
        self.layers = []
        for i, blk in enumerate(cfg.blocks):
            p, m, f, lay = f"l{i}.", blk.mixer, blk.mlp, hybrid_layout(cfg, i)
            par = isinstance(m, ParallelMixer)
            attn = m.left if par else None
            rec = _recurrent_shape(m, lay)
            L = HybridDecoderLayer(
                lay, attn, cfg.padded_head(attn) if par else 0, m.left_scale if par else 1.0, rec,
                m.right_scale if par else 1.0, rec.V if par else rec.H * rec.V // m.norm_groups, vec(p + "norm1"),
                mat(p + "in_w"), mat(p + "aux_w"), mat(p + "out_w"), vec(p + "conv_w"), vec(p + "A"), vec(p + "dt_bias"),
                vec(p + "rec_norm"), conv_b=vec(p + "conv_b"), skip=vec(p + "skip"))
            if par:
                L.turns = ops.rope_turns(attn.rot_dims, attn.rot_base, self.device)
                L.sink = torch.zeros(attn.heads, dtype=torch.float32, device=self.device)
            if isinstance(f, DenseMlp):
                L.gate_up_w, L.gate_up_b, L.down_b = mat(p + "gate_up_w", "gate_up"), vec(p + "gate_up_b"), vec(p + "down_b")
            elif f is not None:
                L.moe = f
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
        return [RunMemory(kv=(x.attn.kv_heads, x.D) if x.attn else None, ring=(x.conv_w.shape[0], x.rec.C),
                          state=(x.rec.H, x.rec.V, x.rec.Dp)) for x in L]

    def make_cache(self, num_blocks: int, block_size: int, slots: int = 1) -> HybridCache:
        return HybridCache(self._specs(), num_blocks, block_size, slots, self.device, self.dtype)

    def cache_bytes_per_block(self, block_size: int) -> int:
        return max(1, HybridCache.bytes_per_block(self._specs(), block_size, self.dtype))

    def state_bytes(self, slots: int) -> int:
        return slots * HybridCache.bytes_per_slot(self._specs(), self.dtype)

    long_part = 2048

    def decode_part(self, batch: int, part_size: int) -> int:
        heads = [L.attn.kv_heads for L in self.layers if L.attn]
        return max(part_size, self.long_part) if heads and batch * min(heads) >= 512 else part_size

    def make_workspace(self, max_batch: int, max_len: int, part_size: int):
        attn = [L for L in self.layers if L.attn]
        if not attn:
            return None
        span = max(min(L.attn.chunk or max_len, max_len) for L in attn) + 32
        return ops.DecodeWorkspace(max_batch, max(L.attn.heads for L in attn), max(L.D for L in attn), -(-span // part_size),
                                   self.device)

    # ------------------------------------------------------------------ forward
    def forward(self, ids: torch.Tensor, meta: AttnMeta, kv: HybridCache) -> torch.Tensor:
        """ids int32 [T] -> final hidden states [T, padded width] (after the last norm)."""
        T, cfg, n = ids.numel(), self.cfg, len(self.runs)
        # decode-sized steps stream the weights through the split-K kernel, whose slabs the consumers sum; short
        # prefill steps do the same
        small_pf = not meta.decode and not meta.n_decode and T <= self.PREFILL_STREAM_MAX_M
        sk = self.frag and (meta.decode and T <= self.STREAM_MAX_M or small_pf)
        x, h = ops.rms_embed(ids, self.embed, self.layers[self.runs[0][0]].norm1, cfg.hidden, cfg.eps)
        for r, (li, _) in enumerate(self.runs):
            L = self.layers[li]
            nxt, again = self.final_norm, None
            if r + 1 < n:
                nxt = self.layers[self.runs[r + 1][0]].norm1
                again = (ids, self.embed) if self.runs[r + 1][1] else None
            y, pairs = self._layer(r, L, h, meta, kv, sk)
            if self.layer_tap is not None and again is not None:  # the stream before the next pass's embedding
                ops.rms_residual(x, y, None, cfg.hidden, cfg.eps, self.dtype, L.down_b, pairs)
                self.layer_tap(r, x)
                h = ops.rms_residual(x, None, nxt, cfg.hidden, cfg.eps, self.dtype, again=again)
                continue
            h = ops.rms_residual(x, y, nxt, cfg.hidden, cfg.eps, self.dtype, L.down_b, pairs, again)
            if self.layer_tap is not None:
                self.layer_tap(r, x)
        return h

    def _layer(self, r: int, L: HybridDecoderLayer, h, meta: AttnMeta, kv: HybridCache, sk: bool):
        """-> (sublayer output of the fused projection, the routed experts' rows or None)."""
        T, lay = h.shape[0], L.lay
        y = self._proj(h, L.in_w, sk, name="in")
        z = self._aux(h, L.aux_w, sk)
        cat = torch.empty((T, lay.width), dtype=self.dtype, device=h.device)
        pairs = None
        if L.gate_up_w is not None:
            self._glu(h, L.gate_up_w, "silu", sk, cat[:, :lay.ff], L.gate_up_b)
        elif L.moe is not None:
            m = L.moe
            idx, wt = ops.moe_route(z, lay.aux.at["router"], m.experts, m.top, m.scale, T)
            pairs = ops.moe_experts(h, idx, wt, L.expert_gate_up_w, L.expert_down_w, m.experts, 8 if self.interleaved_mlp else 0)
            if m.shared:
                ops.shared_glu(y, lay.inp.at["shared"], lay.ff, z, lay.aux.at["sg"], cat[:, :lay.ff])
        if L.attn is not None:
            self._attention(r, L, y, meta, kv, cat[:, lay.ff:lay.mix])
        self._recurrence(r, L, y, z, meta, kv, cat[:, lay.mix:])
        return self._proj(cat, L.out_w, sk, name="out"), pairs

    def _attention(self, r: int, L: HybridDecoderLayer, y, meta: AttnMeta, kv: HybridCache, out) -> None:
        a, kc, vc = L.attn, kv.k[r], kv.v[r]
        q = ops.qk_rope_write(y, L.lay.inp.at["qkv"], a.heads, a.kv_heads, L.D, a.dim, a.rot_dims, L.turns, self.cfg.eps, True,
                              meta.positions, meta.slots, kc, vc)
        T = q.shape[0]
        Tp = 0 if meta.decode else T - meta.n_decode
        if Tp:
            ops.chunk_prefill(q[:Tp], kc, vc, meta.block_tables, meta.cu_q, meta.ctx_lens, meta.max_q, a.scale, a.chunk, L.sink,
                              out[:Tp], L.attn_scale)
        if Tp < T:
            bt, ctx = (meta.block_tables, meta.ctx_lens) if meta.decode else (meta.dec_block_tables, meta.dec_ctx_lens)
            ops.chunk_decode(q[Tp:], kc, vc, bt, ctx, a.scale, a.chunk, L.sink, out[Tp:], L.attn_scale, meta.part_size,
                             meta.workspace, meta.order)

    def _recurrence(self, r: int, L: HybridDecoderLayer, y, z, meta: AttnMeta, kv: HybridCache, out) -> None:
        d, at, eps = L.rec, L.lay.inp.at, self.cfg.eps
        ring, state, pos = kv.ring[r], kv.state[r], meta.positions
        T, n = pos.numel(), d.H * d.V
        pad = out.shape[1] - n
        Tp = 0 if meta.decode else T - meta.n_decode
        o = None
        if Tp:
            c = ops.short_conv(y, at["conv"], L.conv_w, L.conv_b, ring, meta.state_slots, pos, meta.cu_q, meta.max_q)
            o = ops.state_scan(c, d, z, L.A, L.dt_bias, L.skip, state, meta.state_slots, pos, meta.cu_q, meta.max_q)
        if Tp < T:
            slot = meta.state_slots if meta.decode else meta.dec_state_slots
            if d.delta:
                dst = out
            else:
                dst = o = torch.empty((T, n), dtype=self.dtype, device=y.device) if o is None else o
            ops.state_decode(y, at["conv"], L.conv_w, L.conv_b, ring, d, z, L.A, L.dt_bias, L.skip, state, slot, pos, Tp,
                             dst, at["gate"], L.rec_norm if d.delta else None, eps, L.rec_scale, pad)
        rows = Tp if d.delta else T
        if rows:
            ops.gated_norm(o, y, at["gate"], L.norm_part, L.rec_norm, eps, out, 0, rows, not d.delta, d.delta, L.rec_scale, pad)

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        """[n, padded width] -> [n, vocab]."""
        y = self._proj(h, self.lm_head, self.frag and h.shape[0] <= self.STREAM_MAX_M, False, name="lm_head")
        return y[:, :self.cfg.vocab_size]
