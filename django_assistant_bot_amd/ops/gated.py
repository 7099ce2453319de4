"""Wrappers of the gated-sublayer kernels (gated_stream.hip) and of the step between an input projection and its attention
(attn_inputs.hip).

Same rules as ``hybrid.py``: host checks before a launch, current stream, CPU tensors run ``ops.reference_gated``; the
residual stream, norms, gates, angles and weights over depth are fp32 in both modes; a projection argument is the finished
output [T, N] or its split-K slabs [S, T, N].
"""
from __future__ import annotations

from typing import NamedTuple

import torch

from . import reference_gated as ref
from ._lib import expect, native, ptr, same_device, stream
from .hybrid import _ACT, MAX_TAPS, _f32v, _proj
from .kernels import _i32

_NONE = (0, 0, 1, 0, 8)  # no projection


class RoutedRows(NamedTuple):
    """Routed experts' rows as ``moe_experts`` leaves them, with their choices and weights; ``experts``: how many of the
    choices are experts, those behind are identity experts."""

    rows: torch.Tensor
    idx: torch.Tensor
    wt: torch.Tensor
    experts: int


def norm_embed(ids, table, gain, n: int, eps: float, x):
    """x = table[ids] / rms * gain (fp32 [T, C], in place; rms over the first ``n`` columns) -> x in the table's type."""
    T, cols = x.shape
    if not x.is_cuda:
        return ref.norm_embed(ids, table, gain, n, eps, x)
    _i32(ids)
    _f32v(cols, gain)
    expect(ids.numel() == T and table.dtype in _ACT and table.is_contiguous() and table.shape[1] == cols and cols % 8 == 0
           and 1 <= n <= cols <= 16384 and x.dtype == torch.float32 and x.is_contiguous(), "embedding table / stream")
    same_device(ids, table, gain, x)
    h = torch.empty((T, cols), dtype=table.dtype, device=x.device)
    f32 = int(table.dtype == torch.float32)
    native().gated_residual(0, ptr(x), ptr(h), f32, (ptr(table), f32, 1, 0, cols), ptr(ids), (0, 0, 0, 0, 0), _NONE, 0, 0, ptr(gain),
                            (0, 0, 0, 0, 0, 0, 0), 0, int(n), float(eps), T, cols, stream(x))
    return h


def gated_residual(src, x, y, gate, post, n: int, eps: float, dtype=torch.bfloat16, own: RoutedRows | None = None, depth=None,
                   gain=None):
    """x = src + f' / rms(f') * post with f' = f * sigmoid(columns col.. of a projection + bias), ``gate`` = (projection, col,
    bias), and f = the sublayer output ``y`` (rows or slabs) or the token's expert rows (``own``), in which identity experts
    give weight * src.  ``depth`` = (results fp32 [N, T, C], weights [k + 1], k, ahead, n): x becomes result k (kept if k < N)
    and then the sum over j <= k of weights[j] * result j, the first ``n`` of which are in ``ahead`` [T, C] (``depth_ahead``;
    None: none, n = 0).  fp32 [T, C]; ``x`` may be ``src``.  -> x, or with ``gain`` x / rms(x) * gain, as
    ``dtype``.  Mean squares are over the first ``n`` columns; the padded ones are zero."""
    expect((y is None) != (own is None), "a sublayer output or expert rows")
    if not x.is_cuda:
        return ref.gated_residual(src, x, y, gate, post, n, eps, dtype, own, depth, gain)
    T, cols = x.shape
    expect(x.dtype == src.dtype == torch.float32 and x.is_contiguous() and src.is_contiguous() and src.shape == x.shape
           and cols % 8 == 0 and 1 <= n <= cols <= 16384 and dtype in _ACT, "the residual stream is contiguous fp32, width % 8")
    g, col, bias = gate
    pg = _proj(g, T, col + cols, "gate")
    expect(pg[4] % 8 == 0 and pg[3] % 8 == 0 and col % 8 == 0 and (dtype == torch.bfloat16 or pg[1] == 1), "gate columns")
    py = _NONE
    if y is not None:
        py = _proj(y, T, cols, "sublayer output")
        expect(py[4] % 8 == 0 and py[1] == pg[1], "sublayer output rows, of the gate's type")
    _f32v(cols, bias, post, gain)
    routed = (0, 0, 0, 0, 0)
    if own is not None:
        top = own.idx.shape[1]
        _i32(own.idx)
        expect(own.rows.dtype == dtype and own.rows.is_contiguous() and tuple(own.rows.shape) == (T * top, cols)
               and tuple(own.idx.shape) == tuple(own.wt.shape) == (T, top) and own.wt.dtype == torch.float32
               and own.wt.is_contiguous(), "expert rows")
        routed = (ptr(own.rows), ptr(own.idx), ptr(own.wt), top, int(own.experts))
    over, w, k, ahead, n_ahead = depth if depth is not None else (None, None, 0, None, 0)
    if depth is not None:
        expect(over.dtype == torch.float32 and over.is_contiguous() and over.dim() == 3 and tuple(over.shape[1:]) == (T, cols)
               and 1 <= k <= over.shape[0], "results over depth")
        _f32v(k + 1, w)
        _f32v(T * cols, ahead)
        expect(0 <= n_ahead <= k and (ahead is not None or n_ahead == 0), "results ahead")
        expect(x.data_ptr() != over.data_ptr(), "the stream is not a result")
    same_device(x, src, y, g, bias, post, over, w, gain)
    h = torch.empty((T, cols), dtype=dtype, device=x.device)
    native().gated_residual(ptr(src), ptr(x), ptr(h), int(dtype == torch.float32), py, 0, routed, pg, int(col), ptr(bias), ptr(post),
                            (ptr(over), ptr(w), T * cols, k, int(depth is not None and k < over.shape[0]), ptr(ahead), n_ahead), ptr(gain), int(n),
                            float(eps), T, cols, stream(x))
    return h


MAX_AHEAD = 8  # layers whose sums are formed at once


def depth_ahead(over, w, out):
    """out[m] = sum over j of w[m][j] * over[j]: results fp32 [n, T, C], weights fp32 [m, n], out fp32 [>= m, T, C]."""
    m, n = w.shape
    if not over.is_cuda:
        out[:m] = torch.einsum("mn,ntc->mtc", w, over[:n])
        return out
    expect(over.dtype == out.dtype == torch.float32 and over.is_contiguous() and out.is_contiguous() and over.shape[0] >= n
           and out.shape[0] >= m and over.shape[1:] == out.shape[1:] and over.shape[2] % 8 == 0 and 1 <= m <= MAX_AHEAD and n >= 1,
           "results and sums")
    _f32v(m * n, w)
    same_device(over, w, out)
    native().depth_ahead(ptr(over), over.shape[1] * over.shape[2], ptr(w), n, m, ptr(out), stream(over))
    return out


def poly_norm(y, T: int, n: int, cols: int, act, eps: float, dtype):
    """act[0] N(z) + act[1] N(z^2) + act[2] N(z^3) + act[3] of the first ``n`` columns z of a projection, element-wise powers and
    N(v) = v / rms(v); -> [T, cols], zeros behind the first ``n``."""
    if not y.is_cuda:
        return ref.poly_norm(y, n, cols, act, eps, dtype)
    py = _proj(y, T, cols, "poly_norm input")
    expect(1 <= n <= cols <= 65536 and cols % 8 == 0 and py[4] % 8 == 0 and py[3] % 8 == 0 and len(act) == 4 and dtype in _ACT
           and (dtype == torch.bfloat16 or py[1] == 1), "poly_norm columns")
    out = torch.empty((T, cols), dtype=dtype, device=y.device)
    native().poly_norm(py, int(n), int(cols), *(float(a) for a in act), float(eps), ptr(out), int(dtype == torch.float32), T, stream(y))
    return out


# ----------------------------------------------------------------------------------------------


class AttnInputs(NamedTuple):
    """What happens to a layer's q, k and v columns, H / G / G heads of D (``dim`` and ``vdim`` of them real), before attention."""

    H: int
    G: int
    D: int
    dim: int
    vdim: int
    eps: float
    whole: bool  # the RMS norm runs over all heads of q and of k at once, not over each
    gain: torch.Tensor  # fp32 [(H + G) D]
    bias: torch.Tensor | None = None  # fp32 [(H + 2 G) D]
    conv: torch.Tensor | None = None  # fp32 [taps, (H + 2 G) D]: causal convolution, the last tap meets the token itself
    turns: torch.Tensor | None = None  # fp64 turns per position of the rotated pairs (2i, 2i + 1)
    rot_mul: float = 1.0  # factor on cosine and sine
    t_coef: float = 0.0  # queries are multiplied by 1 + t_coef ln(floor((p + 1) / t_every) + 1)
    t_every: int = 1

    @property
    def rot(self) -> int:
        return 0 if self.turns is None else 2 * self.turns.numel()

    @property
    def first_width(self) -> int:
        """Row width of a value head that other layers mix in."""
        return -(-self.vdim // 8) * 8


def attn_inputs(y, col0: int, a: AttnInputs, positions, slots, kc, vc, ring, cu, max_q: int, chunk_slots, row_slots, row0: int, mix=None):
    """Columns col0.. of a projection -> bias, convolution, norm, rotation, temperature and value mix; k / v go into the paged
    caches [blocks, G, block_size, D]; -> q [T, H, D].  Rows before ``row0`` are the portions ``cu`` (the longest of ``max_q``
    tokens), those behind single decoded tokens; with a convolution their past inputs are in ``ring`` [state slots, taps, (H +
    2 G) D] at ``chunk_slots`` / ``row_slots``, which is brought up to date.  ``mix`` = (values [T, G, first_width], weight): v
    becomes (1 - weight) v + weight * values; weight None: the values are written there."""
    T, dtype = positions.numel(), kc.dtype
    C = (a.H + 2 * a.G) * a.D
    if not y.is_cuda:
        return ref.attn_inputs(y, col0, a, positions, slots, kc, vc, ring, cu, chunk_slots, row_slots, row0, mix, dtype)
    py = _proj(y, T, col0 + C)
    _i32(positions)
    expect(dtype in _ACT and kc.is_contiguous() and vc.is_contiguous() and kc.shape == vc.shape and kc.shape[1] == a.G
           and kc.shape[3] == a.D and vc.dtype == dtype, "K / V caches [blocks, G, block_size, D]")
    expect(slots.dtype == torch.int64 and slots.is_contiguous() and slots.numel() == T, "slots: int64 [T]")
    expect(a.D % 8 == 0 and a.D <= 1024 and 1 <= a.dim <= a.D and a.vdim <= a.D and a.rot <= a.dim and col0 % 8 == 0
           and py[4] % 8 == 0 and py[3] % 8 == 0 and a.t_every >= 1, "head sizes")
    expect(dtype == torch.bfloat16 or py[1] == 1, "an fp32 cache takes an fp32 projection")
    expect(a.turns is None or a.turns.dtype == torch.float64, "turns: fp64")
    _f32v((a.H + a.G) * a.D, a.gain)
    _f32v(C, a.bias)
    taps = 1
    if a.conv is not None:
        taps = a.conv.shape[0]
        expect(a.conv.dtype == torch.float32 and a.conv.is_contiguous() and tuple(a.conv.shape) == (taps, C) and taps <= MAX_TAPS, "taps")
        expect(ring.dtype == dtype and ring.is_contiguous() and tuple(ring.shape[1:]) == (taps, C), "ring")
    first, lam = mix if mix is not None else (None, 0.0)
    if first is not None:
        expect(first.dtype == dtype and first.is_contiguous() and tuple(first.shape) == (T, a.G, a.first_width), "values to mix")
    same_device(y, positions, slots, kc, ring, cu, a.gain, a.bias, a.conv, a.turns, first)
    q = torch.empty((T, a.H, a.D), dtype=dtype, device=y.device)

    def launch(cu, rows, at, slot):
        if a.conv is not None:
            _i32(slot)
            expect(slot.numel() >= rows, "state slots")
        native().attn_inputs(
            py, int(col0), (a.H, a.G, a.D, a.dim, int(a.whole)), float(a.eps), ptr(a.gain), ptr(a.bias),
            (taps, ptr(a.conv), ptr(ring) if a.conv is not None else 0, ptr(slot) if a.conv is not None else 0),
            (a.rot, ptr(a.turns), float(a.rot_mul)), (float(a.t_coef), int(a.t_every)), ptr(positions), ptr(slots), ptr(q),
            (ptr(kc), ptr(vc), kc.shape[2]),
            (ptr(first), a.first_width, 0 if first is None else 1 if lam is None else 2, float(lam or 0.0)), ptr(cu), at, rows,
            int(max_q), int(dtype == torch.float32), stream(y))

    if row0:
        _i32(cu)
        launch(cu, cu.numel() - 1, 0, chunk_slots)
    if row0 < T:
        launch(None, T - row0, int(row0), row_slots)
    return q
