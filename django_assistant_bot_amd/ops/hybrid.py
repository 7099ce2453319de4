"""Wrappers of the RMS-stream, recurrent, chunked-attention and expert kernels (rms_stream.hip, recurrent.hip,
attention.hip / attention_any.hip, moe.hip and the grouped GEMMs).

Same rules as ``kernels.py``: shapes and dtypes are checked on the host before a launch, every op enqueues on the
current stream, CPU tensors run ``ops.reference_hybrid``.  Activations are bf16, or fp32 in the 32-bit mode; the
residual stream, norms, scores, gates, recurrent state and router are fp32 in both.  A projection argument is the
finished output [T, N] or its split-K slabs [S, T, N].
"""
from __future__ import annotations

import math
from typing import NamedTuple

import torch

from . import reference_hybrid as ref
from ._lib import expect, native, ptr, same_device, stream
from .kernels import _head_strides, _i32

_ACT = (torch.bfloat16, torch.float32)


def _proj(y: torch.Tensor, T: int, need: int, what: str = "projection"):
    """(pointer, fp32, slabs, slab stride, row stride) of a projection of >= ``need`` columns and >= ``T`` rows."""
    expect(y.dtype in _ACT and y.dim() in (2, 3) and y.stride(-1) == 1, f"{what}: bf16 / fp32 rows or slabs")
    expect(y.shape[-2] >= T and y.shape[-1] >= need, f"{what}: too small")
    if y.dim() == 3:
        expect(y.is_contiguous(), f"{what}: contiguous slabs")
        return ptr(y), int(y.dtype == torch.float32), y.shape[0], y.stride(0), y.stride(1)
    return ptr(y), int(y.dtype == torch.float32), 1, 0, y.stride(0)


def _f32v(n: int, *ts) -> None:
    for t in ts:
        if t is not None:
            expect(t.dtype == torch.float32 and t.is_contiguous() and t.numel() == n, f"fp32 vector of {n}")


def _rows(out: torch.Tensor, T: int, n: int, dtype) -> None:
    expect(out.dim() == 2 and out.shape[0] >= T and out.shape[1] >= n and out.stride(1) == 1 and out.dtype == dtype,
           "bad output rows")


# ----------------------------------------------------------------------------------------------
# RMS norms around an fp32 residual stream


def rms_embed(ids, table, gain, n: int, eps: float):
    """-> (x = table[ids], fp32 residual stream; h = x / rms(x) * gain in the table's type).  ``n``: true width."""
    x = torch.zeros((ids.numel(), table.shape[1]), dtype=torch.float32) if not ids.is_cuda else torch.empty(
        (ids.numel(), table.shape[1]), dtype=torch.float32, device=ids.device)
    return x, rms_residual(x, None, gain, n, eps, table.dtype, again=(ids, table), fresh=True)


def rms_residual(x, y, gain, n: int, eps: float, dtype=torch.bfloat16, bias=None, pairs=None, again=None, fresh=False,
                 post=None, raw=False):
    """x += y (rows or slabs) + bias + the token's expert rows (``pairs`` [T * top, C]) + table[ids] (``again`` = (ids,
    table)), in place (fp32 [T, C]; ``fresh``: x starts at zero); returns x / rms(x) * gain as ``dtype`` (None without
    ``gain``; ``raw``: x itself).  ``post``: y + bias + expert rows are divided by their root mean square and multiplied with
    it before they are added.  The mean squares are over the first ``n`` columns; the padded ones are zero.  The table may
    be fp32."""
    ids, table = again if again is not None else (None, None)
    expect(not (raw and gain is not None), "raw: without a gain")
    if not x.is_cuda:
        return ref.rms_residual(x, y, gain, n, eps, dtype, bias, pairs, ids, table, post, raw, fresh)
    rows, cols = x.shape
    expect(x.dtype == torch.float32 and x.is_contiguous() and cols % 8 == 0 and 1 <= n <= cols and cols <= 16384,
           "the residual stream is contiguous fp32, width % 8")
    expect(dtype in _ACT, "bf16 / fp32 output")
    py = (0, 0, 1, 0, 8)
    if y is not None:
        py = _proj(y, rows, cols, "sublayer output")
        expect(py[4] % 8 == 0 and (dtype == torch.bfloat16 or py[1] == 1), "sublayer output rows")
    _f32v(cols, gain, bias, post)
    expect(post is None or y is not None or pairs is not None, "post: of a sublayer's output")
    top = 0
    if pairs is not None:
        expect(pairs.dtype == dtype and pairs.is_contiguous() and pairs.shape[1] == cols and pairs.shape[0] % rows == 0,
               "expert rows")
        top = pairs.shape[0] // rows
    if ids is not None:
        _i32(ids)
        expect(ids.numel() == rows and table.dtype in (dtype, torch.float32) and table.is_contiguous() and table.shape[1] == cols, "embedding")
    same_device(x, y, gain, bias, pairs, ids, table, post)
    h = torch.empty((rows, cols), dtype=dtype, device=x.device) if gain is not None or raw else None
    native().rms_residual(ptr(x), ptr(h), int(dtype == torch.float32), py, ptr(bias), ptr(pairs), top, ptr(ids),
                          ptr(table), int(table is not None and table.dtype == torch.float32), ptr(post), ptr(gain), int(n), float(eps), rows, cols, int(fresh), stream(x))
    return h


# ----------------------------------------------------------------------------------------------
# attention in chunks, interleaved rotary positions


def rope_turns(dims: int, base: float, device, scaling=None) -> torch.Tensor:
    """fp64 turns per position of the ``dims / 2`` rotated pairs: base^(-2i / dims) / 2 pi.  ``scaling`` (``configs.Yarn``):
    pairs that turn less than ``slow`` times in ``original`` positions are slowed down by ``factor``, those that turn more
    than ``fast`` times are not, with a ramp over the pairs between."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    turns = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / max(dims, 1)) / (2 * torch.pi)
    if scaling is not None:
        def pair(times):  # the (fractional) pair that turns so often
            return dims * math.log(scaling.original / (2 * math.pi * times)) / (2 * math.log(base))

        lo = max(math.floor(pair(scaling.fast)), 0)
        hi = min(math.ceil(pair(scaling.slow)), dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        turns = turns / scaling.factor * ramp + turns * (1.0 - ramp)
    return turns.to(device)


def qk_rope_write(y, col0: int, H: int, G: int, D: int, dim: int, rot: int, turns, eps: float, norm: bool, positions,
                  slots, kc, vc):
    """Columns col0.. of a projection hold H query, G key and G value heads of D (``dim`` of them real).  Rotates the
    pairs (2i, 2i + 1) of the first ``rot`` dimensions of q and k, divides both by their root mean square over ``dim``
    (``norm``), writes k / v into the paged caches [blocks, G, block_size, D]; -> q [T, H, D]."""
    T, dtype = positions.numel(), kc.dtype
    if not y.is_cuda:
        return ref.qk_rope_write(y, col0, H, G, D, dim, rot, turns, eps, norm, positions, slots, kc, vc, dtype)
    py = _proj(y, T, col0 + (H + 2 * G) * D)
    _i32(positions)
    expect(dtype in _ACT and kc.is_contiguous() and vc.is_contiguous() and kc.shape == vc.shape and kc.shape[1] == G
           and kc.shape[3] == D and vc.dtype == dtype, "K / V caches [blocks, G, block_size, D]")
    expect(slots.dtype == torch.int64 and slots.is_contiguous() and slots.numel() == T, "slots: int64 [T]")
    expect(D % 4 == 0 and D <= 1024 and 1 <= dim <= D and rot % 2 == 0 and 0 <= rot <= dim and col0 % 4 == 0
           and py[4] % 4 == 0, "head sizes")
    expect(rot == 0 or (turns.dtype == torch.float64 and turns.numel() == rot // 2), "turns: fp64 [rot / 2]")
    expect(dtype == torch.bfloat16 or py[1] == 1, "an fp32 cache takes an fp32 projection")
    same_device(y, turns, positions, slots, kc)
    q = torch.empty((T, H, D), dtype=dtype, device=y.device)
    native().qk_rope_write(py, int(col0), H, G, D, int(dim), int(rot), ptr(turns), float(eps), int(norm), ptr(positions),
                           ptr(slots), ptr(q), ptr(kc), ptr(vc), int(dtype == torch.float32), kc.shape[2], T, stream(y))
    return q


CHUNK_FLASH_DIMS = (64, 128, 256)


def _any(q, kc, vc, bt, cu, ctx, B, scale, chunk, sink, out, out_scale, slopes):
    T, H, D = q.shape
    expect(D % 2 == 0 and D <= 1024, "head width")
    native().any_attention(ptr(q), ptr(kc), ptr(vc), int(q.dtype == torch.float32), ptr(bt), bt.shape[1], kc.shape[2],
                           ptr(cu), ptr(ctx), B, T, H, kc.shape[1], D, int(chunk), float(scale), ptr(sink), ptr(slopes), ptr(out),
                           out.stride(0), float(out_scale), stream(q))
    return out


def _check_attn(q, kc, vc, bt, ctx, B, sink, out, slopes=None):
    T, H, D = q.shape
    _i32(bt)
    _i32(ctx)
    expect(q.is_contiguous() and kc.is_contiguous() and vc.is_contiguous() and q.dtype == kc.dtype == vc.dtype
           and q.dtype in _ACT and kc.shape == vc.shape and kc.shape[3] == D and H % kc.shape[1] == 0, "q / cache shapes")
    expect(bt.shape[0] >= B and ctx.numel() >= B, "block table / ctx_lens rows < batch")
    _f32v(H, sink, slopes)
    expect(out.shape[0] >= T and out.stride(-1) == 1 and out.shape[1] >= H * D and out.dtype == q.dtype
           and out.stride(0) % 8 == 0, "output rows")
    same_device(q, kc, bt, ctx, sink, slopes, out)


_NO_GATE = (0, 0, 1, 0, 0, 0, 1)


def _output_gate(gate, T: int, n: int):
    """(projection, column, per) of a gate of [T, n] outputs as the kernels take it."""
    if gate is None:
        return _NO_GATE
    y, col, per = gate
    expect(per >= 1 and n % per == 0, "whole groups of gated columns")
    return (*_proj(y, T, col + n // per, "gate"), int(col), int(per))


def chunk_prefill(q, kc, vc, bt, cu, ctx, max_q: int, scale: float, chunk: int, sink, out, out_scale: float = 1.0,
                  slopes=None, gate=None):
    """Causal attention of prompt portions over the paged cache in which query i sees the keys of its own chunk,
    i // chunk * chunk .. i (0: all before it).  ``sink`` fp32 [H]: one more score in the denominator.  ``slopes`` fp32
    [H]: slope * (i - j) is taken off the score of key j.  Writes out_scale * result to ``out``, rows [T, >= H D]; with ``gate``
    = (projection, column, per) times the sigmoid of its columns, as ``sigmoid_gate``."""
    T, H, D = q.shape

    def gated():
        if gate is not None:
            sigmoid_gate(gate[0], gate[1], out[:T, :H * D], gate[2])
        return out

    if not q.is_cuda:
        out[:T, :H * D] = ref.chunk_attention(q, kc, vc, bt, cu, ctx, scale, chunk, sink, out_scale, slopes).view(T, -1).to(out.dtype)
        return gated()
    _i32(cu)
    B = cu.numel() - 1
    _check_attn(q, kc, vc, bt, ctx, B, sink, out, slopes)
    if q.dtype == torch.float32 or D not in CHUNK_FLASH_DIMS or kc.shape[2] % 64:
        _any(q, kc, vc, bt, cu, ctx, B, scale, chunk, sink, out, out_scale, slopes)
        return gated()
    og = _output_gate(gate, T, H * D)
    fused = (gate is not None and D == 128 and chunk == 0 and out_scale == 1.0 and scale > 0 and (sink is not None or slopes is not None)
             and gate[0].dtype == torch.bfloat16 and gate[0].dim() == 2 and gate[1] % 4 == 0 and og[4] % 4 == 0 and gate[2] in (1, D))
    qst, qsh = _head_strides(q)
    native().flash_attention_chunk(ptr(q), qst, qsh, ptr(kc), ptr(vc), ptr(bt), bt.shape[1], kc.shape[2], ptr(out),
                                   out.stride(0), D, ptr(cu), ptr(ctx), B, int(max_q), H, kc.shape[1], D, float(scale),
                                   int(chunk), ptr(sink), ptr(slopes), float(out_scale), og if fused else _NO_GATE, stream(q))
    return out if fused else gated()


def chunk_decode(q, kc, vc, bt, ctx, scale: float, chunk: int, sink, out, out_scale: float = 1.0, part_size: int = 512,
                 workspace=None, order=None, slopes=None, gate=None):
    """The same for one new token per sequence (split over key partitions counted from the chunk's start).  ``gate`` =
    (projection, column, per): the output times the sigmoid of its columns, as ``sigmoid_gate``."""
    B, H, D = q.shape
    if not q.is_cuda:
        out[:B, :H * D] = ref.chunk_attention(
            q, kc, vc, bt, None, ctx, scale, chunk, sink, out_scale, slopes).view(B, -1).to(out.dtype)
        if gate is not None:
            sigmoid_gate(gate[0], gate[1], out[:B, :H * D], gate[2])
        return out
    _check_attn(q, kc, vc, bt, ctx, B, sink, out, slopes)
    G, bs = kc.shape[1], kc.shape[2]
    if q.dtype == torch.float32 or D not in (64, 128) or H // G > 16 or bs % 32:
        _any(q, kc, vc, bt, None, ctx, B, scale, chunk, sink, out, out_scale, slopes)
        if gate is not None:
            sigmoid_gate(gate[0], gate[1], out[:B, :H * D], gate[2])
        return out
    expect(part_size % 128 == 0, "part_size must be a multiple of 128")
    parts = workspace.max_parts if workspace is not None else 1
    if workspace is None:
        part_size = max(part_size, -(-(bt.shape[1] * bs + 32) // 128) * 128)
        ws = (0, 0, 0, 0)
    else:
        expect(workspace.o.numel() >= B * H * parts * D and workspace.m.numel() >= B * H * parts
               and workspace.cnt.numel() >= B * G, "decode workspace too small")
        span = min(bt.shape[1] * bs, chunk) + 31 if chunk else bt.shape[1] * bs
        expect(parts * part_size >= span, "decode workspace: too few partitions")
        ws = (ptr(workspace.o), ptr(workspace.m), ptr(workspace.l), ptr(workspace.cnt))
    if order is not None:
        _i32(order)
        expect(order.numel() >= B, "decode order must hold the batch")
    native().paged_decode_attention(ptr(q), ptr(kc), ptr(vc), ptr(bt), bt.shape[1], bs, ptr(ctx), ptr(out), *ws, B, H, G,
                                    D, int(part_size), int(parts), float(scale), stream(q), ptr(order), chunk=int(chunk),
                                    sink=ptr(sink), out_scale=float(out_scale), o_stride=out.stride(0), slopes=ptr(slopes),
                                    gate=_output_gate(gate, B, H * D))
    return out


# ----------------------------------------------------------------------------------------------
# narrow fp32 projection


def gemm_narrow(x, w):
    """x [M, K] . w [N, K]^T for a few columns that stay in fp32 (router logits, recurrence gates): fp32 [M, N], or split-K
    slabs [S, M, N] where the row tiles alone would leave CUs idle.  bf16 on the GPU (``w`` a ``shuffle_weights`` copy)."""
    if not x.is_cuda:
        return x.float() @ w.float().t()
    M, K = x.shape
    N = w.shape[0]
    expect(x.dtype == w.dtype == torch.bfloat16 and x.stride(1) == 1 and w.is_contiguous() and w.shape[1] == K, "bf16 operands")
    expect(K % 64 == 0 and N % 16 == 0 and x.stride(0) % 8 == 0, "gemm_narrow: K % 64, N % 16")
    tall = M >= 2048 and N > 128  # several column tiles read the same rows
    tiles, S = -(-M // (128 if tall else 32)) * -(-N // 128), 1
    want = 384 if tall else 1024  # (a tall launch fills the chip sooner, and its slabs are many bytes)
    while S < 16 and tiles * S < want and K % (128 * S) == 0 and K // (2 * S) >= 256:
        S *= 2
    out = torch.empty((S, M, N) if S > 1 else (M, N), dtype=torch.float32, device=x.device)
    native().gemm_narrow(ptr(x), x.stride(0), ptr(w), ptr(out), M, N, K, S, int(tall), stream(x))
    return out


# ----------------------------------------------------------------------------------------------
# recurrent mixers


class RecurrentShape(NamedTuple):
    """A matrix-state mixer: ``delta`` (gated delta rule) or state-space duality; heads, q / k groups, state rows, value
    columns; its convolution channels and where q, k, v start among them; its columns of the gate projection."""

    delta: bool
    H: int
    G: int
    D: int
    V: int
    C: int
    q_col: int
    k_col: int
    v_col: int
    a_col: int
    b_col: int

    @property
    def Dp(self) -> int:
        """Width of a stored state column."""
        j = -(-self.D // 32)
        return 32 * (j if j <= 4 else 6 if j <= 6 else 8)

    def native(self):
        return (int(self.delta), self.H, self.G, self.D, self.Dp, self.V, self.C, self.q_col, self.k_col, self.v_col,
                self.a_col, self.b_col)


MAX_STATE_ROWS, MAX_TAPS = 256, 16


def _check_state(d: RecurrentShape, z, T, A, dt_bias, skip, state, slot, ring=None, taps=0):
    pz = _proj(z, T, max(d.a_col, d.b_col if d.delta else 0) + d.H, "gate projection")
    expect(pz[1] == 1, "the gates of a recurrence are fp32")
    expect(d.H % d.G == 0 and 1 <= d.D <= MAX_STATE_ROWS and d.V >= 1, "recurrent sizes")
    _f32v(d.H, A, dt_bias, skip)
    expect(state.dtype == torch.float32 and state.is_contiguous() and tuple(state.shape[1:]) == (d.H, d.V, d.Dp), "state slots")
    _i32(slot)
    if ring is not None:
        expect(ring.is_contiguous() and tuple(ring.shape) == (state.shape[0], taps, d.C) and ring.dtype in _ACT, "ring slots")
    return pz


def _conv_args(y, col0: int, w, bias, ring, rows: int):
    taps, C = w.shape
    py = _proj(y, rows, col0 + C)
    expect(w.dtype == torch.float32 and w.is_contiguous() and taps <= MAX_TAPS and C % 8 == 0 and col0 % 8 == 0
           and py[4] % 8 == 0, "convolution: fp32 taps, channels in eights")
    expect(ring.dtype in _ACT and ring.is_contiguous() and tuple(ring.shape[1:]) == (taps, C), "ring")
    expect(ring.dtype == torch.bfloat16 or py[1] == 1, "fp32 activations take an fp32 projection")
    if bias is not None:
        _f32v(C, bias)
    return py


def short_conv_step(y, col0: int, w, bias, ring, slot, pos, row0: int, out, z_col: int = 0, z_out=None):
    """``short_conv`` of one decoded token per sequence: rows row0.. of the projection, into the same rows of ``out``.  With
    ``z_out`` also the columns z_col .. z_col + C (a gate) as finished rows."""
    taps, C = w.shape
    B, dtype = slot.numel(), ring.dtype
    if not y.is_cuda:
        c = ref.short_conv(y, col0, C, w, bias, ring, slot, pos, ref._spans(None, B, row0), dtype)
        out[row0:row0 + B] = c[row0:row0 + B]
        if z_out is not None:
            z_out[row0:row0 + B] = ref.total(y)[row0:row0 + B, z_col:z_col + C].to(dtype)
        return out
    py = _conv_args(y, col0, w, bias, ring, row0 + B)
    if z_out is not None:
        _proj(y, row0 + B, z_col + C, "gate")
        expect(z_col % 8 == 0 and z_out.is_contiguous() and z_out.shape[1] == C, "gate columns / rows")
        _rows(z_out, row0 + B, C, dtype)
    _i32(slot), _i32(pos)
    expect(pos.numel() >= row0 + B and out.is_contiguous() and out.shape[1] == C, "positions / output rows")
    _rows(out, row0 + B, C, dtype)
    same_device(y, w, bias, ring, slot, pos, out)
    native().short_conv_step(py, int(col0), C, taps, ptr(w), ptr(bias), ptr(ring), ptr(slot), ptr(pos), int(row0), B, ptr(out),
                             int(z_col), ptr(z_out), int(dtype == torch.float32), stream(y))
    return out


def short_conv(y, col0: int, w, bias, ring, slot, pos, cu, max_q: int):
    """Causal convolution (``w`` fp32 [taps, C], last tap = the token) and silu of the portions ``cu`` of columns
    col0.. of a projection; inputs before a portion come from ``ring`` [slots, taps, C], which is brought up to
    date.  -> [T, C]."""
    taps, C = w.shape
    T, dtype = pos.numel(), ring.dtype
    if not y.is_cuda:
        return ref.short_conv(y, col0, C, w, bias, ring, slot, pos, ref._spans(cu, 0, 0), dtype)
    py = _conv_args(y, col0, w, bias, ring, T)
    _i32(slot), _i32(pos), _i32(cu)
    n = cu.numel() - 1
    expect(slot.numel() >= n, "state slots")
    same_device(y, w, bias, ring, slot, pos, cu)
    out = torch.empty((T, C), dtype=dtype, device=y.device)
    native().short_conv(py, int(col0), C, taps, ptr(w), ptr(bias), ptr(ring), ptr(slot), ptr(pos), ptr(cu), n, int(max_q),
                        ptr(out), int(dtype == torch.float32), stream(y))
    return out


CHUNK_MIN_TOKENS = 24  # portions shorter than this are scanned token by token


def state_scan(conv, d: RecurrentShape, z, A, dt_bias, skip, state, slot, pos, cu, max_q: int, chunked: bool | None = None,
               segments: int | None = None):
    """The recurrence over the portions ``cu`` (the longest of ``max_q`` tokens) of convolved channels; ``state`` [slots, H,
    V, Dp] goes on from where the sequence left it (zero at position 0).  -> read-outs [T, H V].  ``chunked``: 64 tokens at a
    time on MFMA (bf16; default: where the sizes allow and the portions are long enough) or token by token.  ``segments``: of
    1024 tokens that a long portion is cut into so that they run side by side (default: when the launch would be small)."""
    T = conv.shape[0]
    if not conv.is_cuda:
        return ref.state_scan(conv, d, z, A, dt_bias, skip, state, slot, pos, ref._spans(cu, 0, 0)).to(conv.dtype)
    pz = _check_state(d, z, T, A, dt_bias, skip, state, slot)
    _i32(pos), _i32(cu)
    expect(conv.is_contiguous() and conv.dtype in _ACT and conv.shape[1] == d.C and pos.numel() >= T, "convolved channels")
    same_device(conv, z, A, dt_bias, skip, state, slot, pos, cu)
    out = torch.empty((T, d.H * d.V), dtype=conv.dtype, device=conv.device)
    n, nat = cu.numel() - 1, native()
    expect(slot.numel() >= n, "state slots")
    fits = conv.dtype == torch.bfloat16 and nat.state_chunks_ok(d.native())
    if chunked is None:
        chunked = fits and max_q >= CHUNK_MIN_TOKENS
    if chunked:
        expect(fits, "chunked scan: bf16, state rows % 8, at most 128")
        segs = nat.state_chunks_segments(d.native(), n, int(max_q)) if segments is None else segments
        ws = torch.empty((nat.state_chunks_bytes(d.native(), T, n, segs),), dtype=torch.uint8, device=conv.device)
        nat.state_chunks(ptr(conv), d.native(), pz, ptr(A), ptr(dt_bias), ptr(skip), ptr(state), ptr(slot), ptr(pos), ptr(cu),
                         n, int(max_q), T, segs, ptr(out), ptr(ws), stream(conv))
        return out
    nat.state_scan(ptr(conv), int(conv.dtype == torch.float32), d.native(), pz, ptr(A), ptr(dt_bias), ptr(skip),
                        ptr(state), ptr(slot), ptr(pos), ptr(cu), cu.numel() - 1, ptr(out), stream(conv))
    return out


def state_decode(y, col0: int, w, bias, ring, d: RecurrentShape, z, A, dt_bias, skip, state, slot, pos, row0: int, out,
                 g_col: int = 0, norm=None, eps: float = 0.0, out_scale: float = 1.0, pad: int = 0):
    """One decoded token per sequence, rows row0.. of the projections: convolution, ring, gates, state update and
    read-out.  delta: also the per-head norm (``norm`` [V]) and the silu gate (columns g_col..), out_scale * result into
    ``out`` [T, >= H V + pad] (``pad`` zero columns behind it); ssd: the read-out into ``out`` [T, H V]."""
    B, taps, dtype = slot.numel(), w.shape[0], ring.dtype
    n = d.H * d.V
    if not y.is_cuda:
        spans = ref._spans(None, B, row0)
        c = ref.short_conv(y, col0, d.C, w, bias, ring, slot, pos, spans, dtype)
        o = ref.state_scan(c, d, z, A, dt_bias, skip, state, slot, pos, spans)
        if d.delta:
            o = ref.gated_norm(o, y, g_col, d.V, False, True, norm, eps, out_scale)
            out[row0:row0 + B, n:n + pad] = 0
        out[row0:row0 + B, :n] = o[row0:row0 + B].to(out.dtype)
        return out
    T = row0 + B
    py = _proj(y, T, max(col0 + d.C, g_col + n if d.delta else 0))
    pz = _check_state(d, z, T, A, dt_bias, skip, state, slot, ring, taps)
    _i32(pos)
    expect(w.dtype == torch.float32 and w.is_contiguous() and tuple(w.shape) == (taps, d.C) and taps <= MAX_TAPS, "taps")
    expect(dtype == torch.bfloat16 or py[1] == 1, "fp32 activations take an fp32 projection")
    expect(pos.numel() >= T, "positions")
    if bias is not None:
        _f32v(d.C, bias)
    if d.delta:
        _f32v(d.V, norm)
    _rows(out, T, n + (pad if d.delta else 0), dtype)
    same_device(y, z, w, bias, ring, state, slot, pos, out)
    native().state_decode(py, int(col0), taps, ptr(w), ptr(bias), ptr(ring), int(dtype == torch.float32), d.native(), pz,
                          ptr(A), ptr(dt_bias), ptr(skip), ptr(state), ptr(slot), ptr(pos), int(row0), B, int(g_col),
                          ptr(norm), float(eps), float(out_scale), ptr(out), out.stride(0), int(pad), stream(y))
    return out


def gated_norm(y, gate, g_col: int, part: int, w, eps: float, out, row0: int, T: int, gate_first: bool, per_head: bool,
               scale: float = 1.0, pad: int = 0):
    """Rows row0 .. row0 + T of y [*, n] in groups of ``part``: y / rms(y) * w * silu(gate) (or, ``gate_first``, the norm
    of y silu(gate), times w), times ``scale``, into ``out`` with ``pad`` zero columns behind.  ``per_head``: w has ``part``
    entries shared by the groups."""
    n = y.shape[1]
    if not y.is_cuda:
        o = ref.gated_norm(y, gate, g_col, part, gate_first, per_head, w, eps, scale)
        out[row0:row0 + T, :n] = o[row0:row0 + T].to(out.dtype)
        out[row0:row0 + T, n:n + pad] = 0
        return out
    pg = _proj(gate, row0 + T, g_col + n, "gate")
    expect(y.is_contiguous() and y.dtype in _ACT and y.shape[0] >= row0 + T and n % part == 0, "read-outs")
    _f32v(part if per_head else n, w)
    _rows(out, row0 + T, n + pad, y.dtype)
    expect(y.dtype == torch.bfloat16 or pg[1] == 1, "fp32 activations take an fp32 projection")
    same_device(y, gate, w, out)
    native().gated_norm(ptr(y), int(y.dtype == torch.float32), pg, int(g_col), n, int(part), int(gate_first), int(per_head),
                        ptr(w), float(eps), float(scale), ptr(out), out.stride(0), int(pad), int(row0), int(T), stream(y))
    return out


# ----------------------------------------------------------------------------------------------
# mixture of experts

MAX_EXPERTS, MAX_TOP = 1024, 64


MOE_SCORES = ("softmax", "sigmoid", "softmax_raw")


def moe_route(z, col0: int, E: int, top: int, scale: float, T: int, scores: str = "softmax", correction=None):
    """fp32 router logits (columns col0..) -> (experts int32 [T, top], weights fp32 [T, top]): softmax over all experts,
    the ``top`` largest, over their sum, times ``scale``; ``scores`` "sigmoid", "softmax_raw": the ``top`` largest sigmoids /
    softmax scores as they are, times ``scale``.  ``correction`` fp32 [E] joins the scores where the experts are chosen, not
    in the weights."""
    expect(scores in MOE_SCORES, f"scores: one of {MOE_SCORES}")
    _f32v(E, correction)
    if not z.is_cuda:
        idx, wt = ref.moe_route(z, col0, E, top, scale, scores, correction)
        return idx[:T].int(), wt[:T]
    pz = _proj(z, T, col0 + E, "router logits")
    expect(pz[1] == 1 and 1 <= top <= min(E, MAX_TOP) and E <= MAX_EXPERTS, "router: fp32 logits, top <= experts")
    idx = torch.empty((T, top), dtype=torch.int32, device=z.device)
    wt = torch.empty((T, top), dtype=torch.float32, device=z.device)
    native().moe_route(pz, int(col0), E, top, float(scale), MOE_SCORES.index(scores), ptr(correction), ptr(idx), ptr(wt), T, stream(z))
    return idx, wt


def moe_experts(h, idx, wt, gate_up, down, E: int, group: int, weigh: str = "output"):
    """Each token's chosen experts: ``gate_up`` [E * 2F, K] and ``down`` [E * W, F] hold the experts one after the other
    (bf16 on the GPU: ``shuffle_weights`` copies with gate / up in 8-row groups; fp32: row-major, stacked).  -> [T * top,
    W], row t * top + k = weight * expert output (``weigh`` "input": the expert of weight * h).  A choice of ``E`` or more is an
    identity expert: its row is not written."""
    T, top = idx.shape
    expect(weigh in ("output", "input"), "weigh: output or input")
    if not h.is_cuda:
        return ref.moe_experts(h, idx, wt, gate_up, down, E, group, weigh)
    win = int(weigh == "input")
    K, F2, W = h.shape[1], gate_up.shape[0] // E, down.shape[0] // E
    P = T * top
    expect(h.stride(1) == 1 and h.dtype in _ACT and gate_up.dtype == h.dtype == down.dtype, "one type")
    expect(gate_up.is_contiguous() and down.is_contiguous() and gate_up.shape[1] == K and down.shape[1] * 2 == F2
           and gate_up.shape[0] == E * F2 and down.shape[0] == E * W, "expert weights")
    _i32(idx)
    expect(wt.dtype == torch.float32 and wt.is_contiguous() and tuple(wt.shape) == (T, top), "expert weights per token")
    same_device(h, idx, wt, gate_up, down)
    f32 = h.dtype == torch.float32
    bm = 64 if f32 else 32 if P <= 48 * E else 128 if P <= 400 * E else 256  # rows of a tile, by the mean load
    n_tiles = min(P, E) + P // bm
    dev, s, nat = h.device, stream(h), native()
    perm = torch.empty((P,), dtype=torch.int32, device=dev)
    tiles = torch.empty((n_tiles, 4), dtype=torch.int32, device=dev)
    words = nat.moe_plan_words(P, E)
    ws = torch.empty((words,), dtype=torch.int32, device=dev) if words else None
    nat.moe_plan(ptr(idx), P, E, bm, ptr(perm), ptr(tiles), n_tiles, ptr(ws), s)
    act = torch.empty((P, F2 // 2), dtype=h.dtype, device=dev)
    out = torch.empty((P, W), dtype=h.dtype, device=dev)
    if f32:
        expect(K % 16 == 0 and (F2 // 2) % 16 == 0 and W % 4 == 0 and h.stride(0) % 4 == 0, "fp32 experts: K % 16, F % 16")
        gu = torch.empty((P, F2), dtype=h.dtype, device=dev)
        nat.gemm_f32_grouped(ptr(h), h.stride(0), ptr(gate_up), ptr(gu), F2, F2, K, ptr(perm), top, 0, ptr(tiles), n_tiles, s)
        nat.glu_f32(ptr(act), F2 // 2, ptr(gu), P, F2 // 2, 0, 0, ptr(wt), ptr(perm), win, s)
        nat.gemm_f32_grouped(ptr(act), F2 // 2, ptr(down), ptr(out), W, W, F2 // 2, ptr(perm), 0, 1, ptr(tiles), n_tiles, s)
        return out
    expect(group == 8 and K % 64 == 0 and F2 % 128 == 0 and W % 32 == 0 and h.stride(0) % 8 == 0, "experts: K % 64, F % 64, W % 32")
    nat.gemm_grouped(ptr(h), h.stride(0), ptr(gate_up), ptr(act), F2 // 2, F2, K, ptr(perm), top, 0, ptr(tiles), n_tiles, bm,
                     1, ptr(wt), win, s)
    nat.gemm_grouped(ptr(act), F2 // 2, ptr(down), ptr(out), W, W, F2 // 2, ptr(perm), 0, 1, ptr(tiles), n_tiles, bm, 0, 0, 0, s)
    return out


def shared_glu(y, col0: int, n: int, z, sg_col: int, out):
    """out[:, :n] = silu(gate) * up * sigmoid(z[:, sg_col]); gate / up = columns col0.. / col0 + n.. of ``y``."""
    T = z.shape[-2]
    if not y.is_cuda:
        out[:, :n] = ref.shared_glu(y, col0, n, z, sg_col).to(out.dtype)
        return out
    py, pz = _proj(y, T, col0 + 2 * n), _proj(z, T, sg_col + 1, "shared gate")
    expect(pz[1] == 1 and n % 8 == 0 and col0 % 8 == 0 and py[4] % 8 == 0 and out.stride(0) % 8 == 0, "shared expert columns")
    _rows(out, T, n, out.dtype)
    expect(out.dtype == torch.bfloat16 or py[1] == 1, "fp32 activations take an fp32 projection")
    same_device(y, z, out)
    native().shared_glu(py, int(col0), int(n), pz, int(sg_col), ptr(out), out.stride(0), int(out.dtype == torch.float32), T,
                        stream(y))
    return out


# ----------------------------------------------------------------------------------------------
# gates and caps


def sigmoid_gate(y, col0: int, x, per: int = 1):
    """x [T, n] *= sigmoid(columns col0 .. of a projection), in place; a column gates ``per`` neighbours of x."""
    T, n = x.shape
    expect(n % per == 0, "whole groups of columns")
    if not x.is_cuda:
        return x.copy_((x.float() * torch.sigmoid(ref.total(y)[:T, col0:col0 + n // per]).repeat_interleave(per, 1)).to(x.dtype))
    py = _proj(y, T, col0 + n // per, "gate")
    expect(x.dtype in _ACT and x.stride(1) == 1 and x.stride(0) % 8 == 0 and n % 8 == 0 and py[4] % 8 == 0
           and (per % 8 == 0 or per == 1 and col0 % 8 == 0), "rows and columns in eights")
    expect(x.dtype == torch.bfloat16 or py[1] == 1, "fp32 activations take an fp32 projection")
    same_device(y, x)
    native().sigmoid_gate(py, int(col0), int(per), ptr(x), x.stride(0), int(x.dtype == torch.float32), n, T, stream(x))
    return x


def softcap(y, cap: float):
    """cap * tanh(y / cap), fp32, of logits [T, n] or their slabs."""
    T, n = y.shape[-2:]
    if not y.is_cuda:
        return cap * torch.tanh(ref.total(y) / cap)
    py = _proj(y, T, n, "logits")
    expect(n % 8 == 0 and py[4] % 8 == 0 and cap > 0, "columns in eights, a positive cap")
    out = torch.empty((T, n), dtype=torch.float32, device=y.device)
    native().softcap(py, float(cap), ptr(out), n, T, stream(y))
    return out
