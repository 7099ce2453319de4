"""Bizetar decoder on the native kernels: softmax attention with sinks, whose positions are distance slopes and a query
temperature or short convolutions and a rotation, PolyNorm MLPs and experts with identity experts, a weighted sum over depth.

The same contract as ``LlamaModel``: one ``forward`` serves packed prefill portions, decode rows and mixed steps, every op
enqueues on the current stream, and decode has fixed shapes so it is captured in a HIP graph.  The residual stream is fp32
and sublayers read it as it is, so everything that reads a sublayer's input is one GEMM, the gate of its result included:

    attention:  h -> in_w [q | k | v, output gate, result gate] -> bias, convolution, norm, rotation / temperature, value mix,
                cache write -> attention (sink, slopes) -> output gate -> o_w
    dense:      h -> up_w [up | result gate] -> PolyNorm -> down_w
    experts:    h -> rg_w [result gate];  h -> router_w (fp32) -> route -> grouped GEMMs

What follows a sublayer's last projection is one pass (``ops.gated_residual``): slab or expert-row sum, identity experts,
gate, norm, residual and, at a layer's end, the sum over the results of all earlier layers.  Those results are kept for the
step in fp32 (``depth``); every few layers the sums of the next ones over all results so far are formed at once
(``ops.depth_ahead``), so a layer reads the newest results only.  What outlives a step beside the pages is the convolution's
past inputs, in state slots.

The 32-bit mode (``dtype=torch.float32``) runs the same steps with fp32 weights, activations and cache.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from .. import ops
from .cache import AttnMeta, HybridCache, RunMemory
from .configs import BizetarConfig, MoeMlp, SinkMixer
from .projections import HybridProjections
from .weights import Columns, bizetar_columns


@dataclass
class BizetarLayer:
    mixer: SinkMixer
    inputs: ops.AttnInputs
    cols: Columns
    in_w: torch.Tensor
    o_w: torch.Tensor
    sink: torch.Tensor
    norm1: torch.Tensor
    rg1_b: torch.Tensor
    depth: torch.Tensor  # weights over the embedding and the layers' results
    slopes: torch.Tensor | None = None
    vmix: float = 0.0
    # feed-forward
    norm2: torch.Tensor | None = None
    rg2_b: torch.Tensor | None = None
    up_w: torch.Tensor | None = None
    act: tuple = ()
    ff: int = 0
    down_w: torch.Tensor | None = None
    moe: MoeMlp | None = None
    rg_w: torch.Tensor | None = None
    router_w: torch.Tensor | None = None
    correction: torch.Tensor | None = None
    expert_gate_up_w: torch.Tensor | None = None
    expert_down_w: torch.Tensor | None = None


class BizetarModel(HybridProjections):
    vocab_parallel = False
    custom_ar = None

    def __init__(self, cfg: BizetarConfig, weights: dict, device, tp_group=None, tp_size: int = 1,
                 interleaved_mlp: bool = True, consume: bool = False, tp_rank: int | None = None):
        if tp_size != 1:
            raise ValueError("Bizetar runs on one GPU per replica (tp_size 1)")
        self.cfg, self.device = cfg, torch.device(device)
        self.interleaved_mlp = interleaved_mlp
        self.vocab_local, self.vocab_start = cfg.vocab_size, 0
        take = weights.pop if consume else weights.__getitem__
        self.f32 = weights["embed"].dtype == torch.float32
        gpu = self.device.type == "cuda"
        self.frag = gpu and not self.f32
        if self.frag and not interleaved_mlp:
            raise ValueError("bf16 Bizetar on the GPU takes gate / up rows in 8-row groups (interleaved_mlp)")
        if gpu and self.f32 and interleaved_mlp:
            raise ValueError("32-bit Bizetar takes stacked gate / up rows")
        self.proj_group = {}

        def mat(key, name=""):
            return self._place(take(key).to(self.device), name) if key in weights else None

        def vec(key):
            return take(key).to(self.device).contiguous() if key in weights else None

        self.embed, self.embed_norm = take("embed").to(self.device), vec("embed_norm")
        self.lm_head = mat("lm_head")
        self.final_norm = vec("final_norm")
        self.layers = []
        for i, blk in enumerate(cfg.blocks):
            p, m, f = f"l{i}.", blk.mixer, blk.mlp
            turns = None if m.rot is None else ops.rope_turns(m.rot.dims, m.rot.base, self.device, m.rot.scaling)
            inputs = ops.AttnInputs(
                m.heads, m.kv_heads, m.padded_head(), m.dim, m.vdim, cfg.eps, m.norm == "whole", vec(p + "qk_norm"), vec(p + "qkv_b"),
                vec(p + "conv_w"), turns, 1.0 if m.rot is None else m.rot.gain,
                *((0.0, 1) if m.temp is None else (m.temp.coef, m.temp.every)))
            L = BizetarLayer(m, inputs, bizetar_columns(cfg, i), mat(p + "in_w"), mat(p + "o_w"), vec(p + "sink"), vec(p + "norm1"),
                             vec(p + "rg1_b"), vec(p + "depth"), vec(p + "slopes"), take(p + "vmix") if m.v_mix else 0.0,
                             vec(p + "norm2"), vec(p + "rg2_b"))
            if isinstance(f, MoeMlp):
                L.moe, L.rg_w, L.router_w, L.correction = f, mat(p + "rg_w"), mat(p + "router_w"), vec(p + "correction")
                L.expert_gate_up_w, L.expert_down_w = mat(p + "expert_gate_up_w"), mat(p + "expert_down_w")
            elif f is not None:
                L.up_w, L.down_w, L.act, L.ff = mat(p + "up_w"), mat(p + "down_w"), take(p + "act"), f.ff
            self.layers.append(L)
        if gpu and consume:
            torch.cuda.empty_cache()
        # the weights of a block of layers over the results before it: [layers, results]
        self.ahead = {b: torch.stack([L.depth[:b + 1] for L in self.layers[b:b + ops.MAX_AHEAD]]).contiguous()
                      for b in range(ops.MAX_AHEAD, len(self.layers), ops.MAX_AHEAD)}
        self.recurrent = any(L.inputs.conv is not None for L in self.layers)
        self.layer_tap = None  # called as tap(layer, residual stream) after every layer (numerics tests)

    @property
    def dtype(self):
        return self.embed.dtype

    # ------------------------------------------------------------------ what the engine asks of a family
    def _specs(self):
        return [RunMemory(kv=(a.G, a.D), ring=None if a.conv is None else tuple(a.conv.shape)) for a in (L.inputs for L in self.layers)]

    def make_cache(self, num_blocks: int, block_size: int, slots: int = 1) -> HybridCache:
        return HybridCache(self._specs(), num_blocks, block_size, slots, self.device, self.dtype)

    def cache_bytes_per_block(self, block_size: int) -> int:
        return max(1, HybridCache.bytes_per_block(self._specs(), block_size, self.dtype))

    def state_bytes(self, slots: int) -> int:
        return slots * HybridCache.bytes_per_slot(self._specs(), self.dtype)

    def step_bytes(self, tokens: int) -> int:
        return 4 * tokens * (len(self.layers) + (ops.MAX_AHEAD if self.ahead else 0)) * self.embed.shape[1]  # (``depth``)

    long_part = 2048

    def decode_part(self, batch: int, part_size: int) -> int:
        return max(part_size, self.long_part) if batch * min(L.inputs.G for L in self.layers) >= 512 else part_size

    def make_workspace(self, max_batch: int, max_len: int, part_size: int):
        a = [L.inputs for L in self.layers]
        return ops.DecodeWorkspace(max_batch, max(x.H for x in a), max(x.D for x in a), -(-(max_len + 32) // part_size), self.device)

    # ------------------------------------------------------------------ forward
    def forward(self, ids: torch.Tensor, meta: AttnMeta, kv: HybridCache) -> torch.Tensor:
        """ids int32 [T] -> final hidden states [T, padded width] (after the last norm)."""
        T, n, W, eps = ids.numel(), len(self.layers), self.cfg.hidden, self.cfg.eps
        # decode-sized steps stream the weights through the split-K kernel, whose slabs the consumers sum; short
        # prefill steps do the same
        small_pf = not meta.decode and not meta.n_decode and T <= self.PREFILL_STREAM_MAX_M
        sk = self.frag and (meta.decode and T <= self.STREAM_MAX_M or small_pf)
        depth = torch.empty((n, T, self.embed.shape[1]), dtype=torch.float32, device=ids.device)
        sums = torch.empty((ops.MAX_AHEAD, *depth.shape[1:]), dtype=torch.float32, device=ids.device) if self.ahead else None
        h = ops.norm_embed(ids, self.embed, self.embed_norm, W, eps, depth[0])
        x, src, first = torch.empty_like(depth[0]), depth[0], None
        for i, L in enumerate(self.layers):
            b = i - i % ops.MAX_AHEAD  # the first layer of the block
            if i in self.ahead:
                ops.depth_ahead(depth, self.ahead[i], sums)
            ahead = (sums[i - b], b + 1) if b else (None, 0)
            close = dict(depth=(depth, L.depth, i + 1, *ahead), gain=self.final_norm if i + 1 == n else None)
            y, z, first = self._attention(i, L, h, meta, kv, sk, first)
            h = ops.gated_residual(src, x, z, (y, L.cols.at["rg"], L.rg1_b), L.norm1, W, eps, self.dtype,
                                   **(close if L.norm2 is None else {}))
            if L.norm2 is not None:
                y, at, z, own = self._mlp(L, h, sk)
                h = ops.gated_residual(x, x, z, (y, at, L.rg2_b), L.norm2, W, eps, self.dtype, own=own, **close)
            src = x
            if self.layer_tap is not None:
                self.layer_tap(i, x)
        return h

    def _attention(self, i: int, L: BizetarLayer, h, meta: AttnMeta, kv: HybridCache, sk: bool, first):
        """-> (input projection, mixer output, the values that later layers mix in)."""
        a, at, kc, vc = L.inputs, L.cols.at, kv.k[i], kv.v[i]
        T = h.shape[0]
        y = self._proj(h, L.in_w, sk, name="in")
        mix = None
        if L.mixer.v_mix:
            if first is None:
                first = torch.empty((T, a.G, a.first_width), dtype=self.dtype, device=h.device)
                mix = (first, None)
            else:
                mix = (first, L.vmix)
        Tp = 0 if meta.decode else T - meta.n_decode
        q = ops.attn_inputs(y, at["qkv"], a, meta.positions, meta.slots, kc, vc, kv.ring[i], meta.cu_q if Tp else None, meta.max_q,
                            meta.state_slots if Tp else None, meta.state_slots if meta.decode else meta.dec_state_slots, Tp, mix)
        per = a.D if L.mixer.gate == "head" else 1
        o = torch.empty((T, a.H * a.D), dtype=self.dtype, device=h.device)
        if Tp:
            ops.chunk_prefill(q[:Tp], kc, vc, meta.block_tables, meta.cu_q, meta.ctx_lens, meta.max_q, L.mixer.scale, 0, L.sink,
                              o[:Tp], slopes=L.slopes, gate=(y, at["g"], per))
        if Tp < T:  # (mixed steps have finished projections)
            bt, ctx = (meta.block_tables, meta.ctx_lens) if meta.decode else (meta.dec_block_tables, meta.dec_ctx_lens)
            ops.chunk_decode(q[Tp:], kc, vc, bt, ctx, L.mixer.scale, 0, L.sink, o[Tp:], 1.0, meta.part_size, meta.workspace,
                             meta.order, L.slopes, (y[Tp:] if Tp else y, at["g"], per))
        return y, self._proj(o, L.o_w, sk, name="o"), first

    def _mlp(self, L: BizetarLayer, h, sk: bool):
        """-> (projection with the result's gate, its column, MLP output or None, routed experts or None)."""
        if L.moe is None:
            y = self._proj(h, L.up_w, sk, name="up")
            F = L.down_w.shape[1]
            return y, F, self._proj(ops.poly_norm(y, h.shape[0], L.ff, F, L.act, self.cfg.eps, self.dtype), L.down_w, sk, name="down"), None
        m = L.moe
        idx, wt = ops.moe_route(self._aux(h, L.router_w, sk), 0, m.outputs, m.top, m.scale, h.shape[0], m.scores, L.correction)
        pairs = ops.moe_experts(h, idx, wt, L.expert_gate_up_w, L.expert_down_w, m.experts, 8 if self.interleaved_mlp else 0, m.weigh)
        return self._proj(h, L.rg_w, sk, name="rg"), 0, None, ops.RoutedRows(pairs, idx, wt, m.experts)

    def logits(self, h: torch.Tensor) -> torch.Tensor:
        """[n, padded width] -> [n, vocab]."""
        y = self._proj(h, self.lm_head, self.frag and h.shape[0] <= self.STREAM_MAX_M, False, name="lm_head")
        return y[:, :self.cfg.vocab_size]
