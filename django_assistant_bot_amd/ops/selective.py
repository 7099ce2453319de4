"""Wrappers of the selective-scan kernels (selective_scan.hip).

Same rules as ``hybrid.py``: shapes and dtypes are checked on the host before a launch, every op enqueues on the current
stream, CPU tensors run ``ops.reference_hybrid``.  The scanned channels, the gate and the result are bf16, or fp32 in the
32-bit mode; step, input, read-out, decays and state are fp32 in both.
"""
from __future__ import annotations

from typing import NamedTuple

import torch

from . import reference_hybrid as ref
from ._lib import expect, native, ptr, same_device, stream
from .hybrid import _ACT, _f32v, _proj, _rows
from .kernels import _i32

MAX_STATE, MAX_STEP_RANK = 256, 2048


class SelectiveShape(NamedTuple):
    """Channels and stored state entries of a channel; columns of the narrow projection: the step's ``rank`` dimensions from
    0, input and read-out from ``b_col`` / ``c_col``; gate columns of the input projection from ``z_col``."""

    C: int
    Np: int
    rank: int
    b_col: int
    c_col: int
    z_col: int


def state_width(n: int) -> int:
    """Width at which a channel's ``n`` state entries are stored."""
    return -(-n // 16) * 16 if n <= 64 else 128 if n <= 128 else 256


def narrow_rows(z, n: int, low: int, T: int, dtype=torch.bfloat16):
    """The first ``n`` columns of an fp32 projection as finished rows [T, n], and its first ``low`` columns as ``dtype``
    (the operand of another projection)."""
    if not z.is_cuda or dtype == torch.float32:
        y = ref.total(z) if z.dim() == 3 else z
        return y[:, :n], y[:, :low].to(dtype)
    pz = _proj(z, T, n, "narrow projection")
    expect(pz[1] == 1 and n % 8 == 0 and low % 8 == 0 and low <= n and pz[4] % 4 == 0, "fp32, columns in eights")
    out = torch.empty((T, n), dtype=torch.float32, device=z.device)
    lo = torch.empty((T, low), dtype=torch.bfloat16, device=z.device)
    native().narrow_rows(pz, ptr(out), ptr(lo), int(n), int(low), T, stream(z))
    return out, lo


def _check(u, d: SelectiveShape, low, A, dt_bias, skip, state, slot, pos, out, rows: int):
    expect(u.dtype in _ACT and u.is_contiguous() and u.shape[0] >= rows and u.shape[1] == d.C and d.C % 8 == 0, "channels")
    expect(d.Np == state_width(d.Np) and d.Np <= MAX_STATE and d.b_col % 4 == d.c_col % 4 == d.z_col % 8 == 0, "selective sizes")
    expect(state.dtype == torch.float32 and state.is_contiguous() and tuple(state.shape[1:]) == (d.C, d.Np), "state slots")
    expect(A.dtype == torch.float32 and A.is_contiguous() and tuple(A.shape) == (d.C, d.Np), "decays [C, Np]")
    _f32v(d.C, dt_bias, skip)
    _i32(slot), _i32(pos)
    pl = _proj(low, rows, max(d.rank, d.b_col + d.Np, d.c_col + d.Np), "narrow projection")
    expect(pl[1] == 1 and pl[2] == 1 and pl[4] % 4 == 0, "finished fp32 rows")
    expect(pos.numel() >= rows and out.is_contiguous() and out.shape[1] == d.C, "positions / output rows")
    _rows(out, rows, d.C, u.dtype)
    same_device(u, low, A, dt_bias, skip, state, slot, pos, out)
    return pl


def selective_scan(u, d: SelectiveShape, dt, low, y, A, dt_bias, skip, state, slot, pos, cu, max_q: int, out, segments: int | None = None):
    """The recurrence over the portions ``cu`` of the convolved channels ``u``, read-out, skip and silu gate, into the same
    rows of ``out`` [T, C]; ``state`` [slots, C, Np] goes on from where the sequence left it (zero at position 0).  ``dt``
    fp32 [T, C]: the step before bias and softplus; ``A``: -exp(A_log) log2(e).  ``max_q``: the longest portion;
    ``segments`` it is cut into, which run side by side (default: when the launch would be small)."""
    if not u.is_cuda:
        spans = ref._spans(cu, 0, 0)
        n = spans[-1][1]
        out[:n] = ref.selective_scan(u[:n], d, dt[:n], low[:n], y[..., :n, :], A, dt_bias, skip, state, slot, pos, spans, out.dtype)
        return out
    _i32(cu)
    n = cu.numel() - 1
    pl = _check(u, d, low, A, dt_bias, skip, state, slot, pos, out, dt.shape[0])
    py = _proj(y, dt.shape[0], d.z_col + d.C, "gate")
    expect(py[4] % 8 == 0 and (u.dtype == torch.bfloat16 or py[1] == 1), "gate rows")
    same_device(u, y, dt, cu)
    expect(dt.dtype == torch.float32 and dt.dim() == 2 and dt.shape[1] == d.C and dt.stride(1) == 1 and dt.stride(0) % 4 == 0,
           "steps: fp32 [T, C]")
    expect(slot.numel() >= n, "state slots")
    segs = native().selective_segments(tuple(d), n, int(max_q)) if segments is None else int(segments)
    ws = torch.empty((n * segs * d.C * (d.Np + 1),), dtype=torch.float32, device=u.device) if segs > 1 else None
    native().selective_scan(ptr(u), int(u.dtype == torch.float32), tuple(d), _proj(dt, dt.shape[0], d.C), pl, py, ptr(A),
                            ptr(dt_bias), ptr(skip), ptr(state), ptr(slot), ptr(pos), ptr(cu), n, int(max_q), segs,
                            ptr(ws), ptr(out), stream(u))
    return out


def selective_step(u, d: SelectiveShape, dt_w, step, low, A, dt_bias, skip, state, slot, pos, row0: int, out):
    """The same for one decoded token per sequence, rows row0..; ``dt_w`` [C, rank] (bf16 on the GPU: a ``shuffle_weights``
    copy) is applied to ``step`` [*, rank] (``narrow_rows``) here.  The rows of ``out`` hold the gate on entry."""
    B = slot.numel()
    if not u.is_cuda:
        dt = step.float() @ dt_w.float().t()
        c = ref.selective_scan(u, d._replace(z_col=0), dt, low, out.float(), A, dt_bias, skip, state, slot, pos, ref._spans(None, B, row0), out.dtype)
        out[row0:row0 + B] = c[row0:row0 + B]
        return out
    pl = _check(u, d, low, A, dt_bias, skip, state, slot, pos, out, row0 + B)
    expect(d.C % 16 == 0 and d.rank % 32 == 0 and d.rank <= MAX_STEP_RANK and dt_w.dtype == u.dtype and dt_w.is_contiguous()
           and tuple(dt_w.shape) == (d.C, d.rank), "step weights [C, rank]")
    expect(step.dtype == u.dtype and step.shape[0] >= row0 + B and step.shape[1] == d.rank and step.stride(1) == 1
           and step.stride(0) == (d.rank if step.dtype == torch.bfloat16 else pl[4]), "low-rank steps")
    native().selective_step(ptr(u), int(u.dtype == torch.float32), tuple(d), ptr(dt_w), ptr(step), pl, ptr(A), ptr(dt_bias), ptr(skip),
                            ptr(state), ptr(slot), ptr(pos), int(row0), B, ptr(out), stream(u))
    return out
