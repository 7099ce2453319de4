"""Wrappers of the latent-attention and Dynamic-Tanh kernels (latent_attention.hip, dyt.hip,
gemm_f32.hip and the windowed form of the flash kernel).

Same rules as ``kernels.py``: shapes and dtypes are checked on the host before a launch, every op
enqueues on the current stream, CPU tensors run ``ops.reference``.  Activations are bf16, or fp32 in
the 32-bit mode; the residual stream, norms, scores and softmax are fp32 in both.
"""
from __future__ import annotations

from typing import NamedTuple

import torch

from . import reference as ref
from ._lib import expect, native, ptr, same_device, stream
from .kernels import _head_strides, _i32

_ACT = (torch.bfloat16, torch.float32)


class DytNorm(NamedTuple):
    """Dynamic Tanh: tanh(alpha x) w + b."""

    alpha: float
    w: torch.Tensor  # fp32 [cols]
    b: torch.Tensor  # fp32 [cols]


def _f32(cols: int, *ts) -> None:
    for t in ts:
        if t is not None:
            expect(t.dtype == torch.float32 and t.is_contiguous() and t.numel() == cols, "fp32 vector of the row width")


def _norm(n: DytNorm | None):
    return (0.0, 0, 0) if n is None else (float(n.alpha), ptr(n.w), ptr(n.b))


def embed_dyt(ids, table, scale: float, norm: DytNorm):
    """-> (x = table[ids] * scale, fp32 residual stream; h = DyT(x) in the table's type)."""
    if not ids.is_cuda:
        return ref.embed_dyt(ids, table, scale, norm)
    _i32(ids)
    expect(table.dtype in _ACT and table.is_contiguous(), "embedding table must be bf16 or fp32")
    cols = table.shape[1]
    _f32(cols, norm.w, norm.b)
    same_device(ids, table, norm.w, norm.b)
    expect(cols % 8 == 0, "width % 8")
    x = torch.empty((ids.numel(), cols), dtype=torch.float32, device=ids.device)
    h = torch.empty((ids.numel(), cols), dtype=table.dtype, device=ids.device)
    native().embed_dyt(ptr(x), ptr(h), ptr(ids), ptr(table), int(table.dtype == torch.float32), float(scale),
                       *_norm(norm), ids.numel(), cols, stream(ids))
    return x, h


def dyt_residual(x, y, post: DytNorm | None, ls, nxt: DytNorm | None, dtype=torch.bfloat16):
    """x += ls * DyT_post(y), in place (fp32 [T, C]); returns DyT_next(x) as ``dtype`` (None without
    ``nxt``).  ``y``: [T, C], or the producing projection's split-K slabs [S, T, C] (summed in fp32)."""
    if not x.is_cuda:
        return ref.dyt_residual(x, y, post, ls, nxt, dtype)
    rows, cols = x.shape
    expect(x.dtype == torch.float32 and x.is_contiguous(), "the residual stream is contiguous fp32")
    expect(y.dtype in _ACT and y.is_contiguous() and tuple(y.shape[-2:]) == (rows, cols), "bad sublayer output")
    expect(dtype in _ACT and cols % 8 == 0, "bf16 / fp32 output, width % 8")
    for n in (post, nxt):
        if n is not None:
            _f32(cols, n.w, n.b)
    _f32(cols, ls)
    same_device(x, y, ls)
    S = y.shape[0] if y.dim() == 3 else 1
    h = torch.empty((rows, cols), dtype=dtype, device=x.device) if nxt is not None else None
    native().dyt_residual(ptr(x), ptr(h), int(dtype == torch.float32), ptr(y), int(y.dtype == torch.float32), S,
                          rows * cols, *_norm(post), ptr(ls), *_norm(nxt), rows, cols, stream(x))
    return h


def glu_f32(x, act: str = "gelu", bias=None, out=None):
    """fp32 [T, 2F] = [gate | up] (+ ``bias`` [gate | up]) -> act(gate) * up [T, F] (``act``: gelu (tanh), silu, relu)."""
    F2 = x.shape[-1]
    if not x.is_cuda:
        x = x if bias is None else x + bias
        g, u = x[..., :F2 // 2].float(), x[..., F2 // 2:].float()
        y = (ref.glu_act(g, act) * u).to(x.dtype)
        return y if out is None else out.copy_(y)
    expect(x.dtype == torch.float32 and x.is_contiguous() and F2 % 8 == 0, "contiguous fp32 [T, 2F], F % 4")
    if bias is not None:
        _f32(F2, bias)
    out = torch.empty((x.shape[0], F2 // 2), dtype=torch.float32, device=x.device) if out is None else out
    expect(out.dtype == torch.float32 and tuple(out.shape) == (x.shape[0], F2 // 2) and out.stride(1) == 1
           and out.stride(0) % 4 == 0, "bad glu output")
    native().glu_f32(ptr(out), out.stride(0), ptr(x), x.shape[0], F2 // 2, ref.GLU_ACTS.index(act), ptr(bias), 0, 0, 0,
                     stream(x))
    return out


def gemm_f32(a, b):
    """fp32 a [M, K] . b [N, K]^T."""
    if not a.is_cuda:
        return ref.gemm_bt(a, b, out_f32=True)
    M, K = a.shape
    N = b.shape[0]
    expect(a.dtype == torch.float32 and b.dtype == torch.float32 and b.is_contiguous() and a.stride(1) == 1, "fp32 rows")
    expect(b.shape[1] == K and K % 16 == 0 and N % 4 == 0 and a.stride(0) % 4 == 0, "gemm_f32: K % 16, N % 4")
    expect(M <= 64 * 65535, "gemm_f32: too many rows")
    out = torch.empty((M, N), dtype=torch.float32, device=a.device)
    native().gemm_f32(ptr(a), a.stride(0), 0, ptr(b), K, 0, ptr(out), N, 0, M, N, K, 1, stream(a))
    return out


# ----------------------------------------------------------------------------------------------
# latent attention


class LatentRope(NamedTuple):
    """Rotary positions of ``latent_write``: the neighbours (2i, 2i + 1) of columns q_at .. q_at + dims of every D-wide query
    head and of columns c_at .. c_at + dims of the latent row are a pair; ``turns`` fp64 [dims / 2] per position, ``gain`` on
    cosine and sine."""

    turns: torch.Tensor
    gain: float
    dims: int
    D: int
    q_at: int
    c_at: int
    positions: torch.Tensor  # int32 [T]


def latent_write(y, q_cols: int, gain, cache, slots, rank: int, eps: float, rope: LatentRope | None = None):
    """``y``: the [q | latent] projection, [T, q_cols (+ R ..)] or its split-K slabs [S, T, ...].  Writes the
    RMS-normed latents (statistic over ``rank`` <= R columns) into ``cache`` [blocks, block_size, R] at
    ``slots`` (int64, < 0 skipped) unless ``cache`` is None, and returns the q rows [T, q_cols] (a view of
    ``y`` when there is nothing to sum or rotate).  ``rope``: rotates a part of every head and of the row, which then is
    [latent | rotated key]."""
    if not y.is_cuda:
        return ref.latent_write(y, q_cols, gain, cache, slots, rank, eps, rope)
    T, N = y.shape[-2:]
    slabs = y.dim() == 3
    expect(y.dtype in _ACT and y.is_contiguous() and N % 8 == 0 and q_cols % 8 == 0, "bad projection")
    expect(slots.dtype == torch.int64 and slots.is_contiguous() and slots.numel() == T, "slots: int64 [T]")
    if cache is None and not slabs:
        return y[:, :q_cols]
    R = 0
    if cache is not None:
        R = cache.shape[-1]
        expect(cache.is_contiguous() and cache.dtype in _ACT and N >= q_cols + R and 1 <= rank <= R and R % 8 == 0,
               "latent cache does not fit the projection")
        expect(cache.dtype == torch.bfloat16 or y.dtype == torch.float32, "an fp32 cache takes an fp32 projection")
        _f32(R, gain)
    else:
        expect(N == q_cols, "a projection without latents is q only")
    ro = (0, 0, 0, 8, 0, 0, 1.0)
    if rope is not None:
        expect(cache is not None and rope.dims % 2 == 0 and rope.dims >= 2 and rope.D % 8 == rope.q_at % 8 == rope.c_at % 8 == 0
               and rope.q_at + rope.dims <= rope.D and rank <= rope.c_at and rope.c_at + rope.dims <= R and q_cols % rope.D == 0,
               "rotated columns")
        expect(rope.turns.dtype == torch.float64 and rope.turns.numel() == rope.dims // 2, "turns: fp64 [dims / 2]")
        _i32(rope.positions)
        expect(rope.positions.numel() == T, "positions")
        same_device(y, rope.turns, rope.positions)
        ro = (ptr(rope.turns), ptr(rope.positions), rope.dims, rope.D, rope.q_at, rope.c_at, float(rope.gain))
    q = None
    if slabs or rope is not None:
        dt = torch.bfloat16 if cache is None else cache.dtype
        q = torch.empty((T, q_cols), dtype=dt, device=y.device)
    native().latent_write(ptr(y), int(y.dtype == torch.float32), y.shape[0] if slabs else 1, T * N, N, ptr(q), q_cols,
                          ptr(gain), ptr(cache), int(cache is not None and cache.dtype == torch.float32), ptr(slots), T,
                          R, int(rank), float(eps), ro, stream(y))
    return y[:, :q_cols] if q is None else q


def latent_gather(cache, block_tables, cu_k, ctx_lens, total: int):
    """Packed copy [total, R] of the last cu_k[b+1] - cu_k[b] cached latents of every sequence."""
    if not cache.is_cuda:
        return ref.latent_gather(cache, block_tables, cu_k, ctx_lens)
    _i32(block_tables)
    _i32(cu_k)
    _i32(ctx_lens)
    B, R = cu_k.numel() - 1, cache.shape[-1]
    expect(block_tables.shape[0] >= B and ctx_lens.numel() >= B and cache.is_contiguous(), "block table / ctx rows < batch")
    expect(R * cache.element_size() % 16 == 0, "latent rows must be 16-B multiples")
    out = torch.empty((total, R), dtype=cache.dtype, device=cache.device)
    native().latent_gather(ptr(out), ptr(cache), ptr(block_tables), block_tables.shape[1], cache.shape[1], ptr(cu_k),
                           ptr(ctx_lens), B, int(total), R * cache.element_size(), stream(cache))
    return out


def head_gemm(x, w, n: int, row0: int = 0, out=None):
    """Per-head product y[t, h] = W_h x[t, h] with W_h = rows row0 + h n .. + n of ``w`` [rows, K].  bf16 on
    the GPU: ``w`` in the ``shuffle_weights`` layout; fp32 and the CPU: row-major.  -> [T, H, n]."""
    T, H, K = x.shape
    if not x.is_cuda:
        y = ref.head_gemm(x, w, row0, n)
        return y if out is None else out.copy_(y)
    expect(w.is_contiguous() and w.shape[1] == K and w.dtype == x.dtype and w.shape[0] >= row0 + H * n, "bad head weights")
    xt, xh = _head_strides(x)
    if out is None:
        out = torch.empty((T, H, n), dtype=x.dtype, device=x.device)
    expect(tuple(out.shape) == (T, H, n) and out.dtype == x.dtype and out.stride(2) == 1, "bad head_gemm output")
    same_device(x, w, out)
    if x.dtype == torch.float32:
        expect(K % 16 == 0 and n % 4 == 0 and all(s % 4 == 0 for s in (xt, xh, out.stride(0), out.stride(1))),
               "fp32 head_gemm: K % 16, n % 4")
        native().gemm_f32(ptr(x), xt, xh, ptr(w) + 4 * row0 * K, K, n * K, ptr(out), out.stride(0), out.stride(1), T, n,
                          K, H, stream(x))
        return out
    expect(x.dtype == torch.bfloat16 and n % 16 == 0 and K % 32 == 0 and row0 % 16 == 0, "head_gemm: n % 16, K % 32")
    expect(xt % 8 == 0 and xh % 8 == 0 and out.stride(0) % 4 == 0 and out.stride(1) % 4 == 0, "head_gemm strides")
    native().head_gemm(ptr(out), out.stride(0), out.stride(1), ptr(x), xt, xh, ptr(w), int(row0), T, H, int(n), K,
                       stream(x))
    return out


def latent_key_fill(k, rows, q_at: int, c_at: int, dims: int):
    """Copies the rotated key part, columns c_at .. c_at + dims of the gathered ``rows`` [T, R], to columns q_at.. of every
    head of ``k`` [T, H, D] (heads adjacent), in place.  Columns up to the next multiple of 8 are copied along."""
    T, H, D = k.shape
    if not k.is_cuda:
        k[:, :, q_at:q_at + dims] = rows[:, None, c_at:c_at + dims]
        return k
    R = rows.shape[1]
    expect(k.dtype == rows.dtype == torch.bfloat16 and rows.is_contiguous() and rows.shape[0] == T and k.stride(2) == 1
           and k.stride(1) == D and k.stride(0) % 8 == 0, "bf16 rows, adjacent heads")
    expect(all(v % 8 == 0 for v in (D, R, q_at, c_at)) and dims >= 1 and q_at + -(-dims // 8) * 8 <= D
           and c_at + -(-dims // 8) * 8 <= R, "rotated columns")
    same_device(k, rows)
    native().latent_key_fill(ptr(k), k.stride(0), D, ptr(rows), R, int(q_at), int(c_at), int(dims), H, T, stream(k))
    return k


FLASH_WINDOW_DIMS = (64, 128, 256)


def flash_attention_window(q, k, v, cu_q, cu_k, max_seqlen_q: int, scale: float, window: int = 0, sink=None, out=None):
    """Causal packed attention with a sliding window (``window`` keys, self included; 0 = all) and a softmax
    sink (fp32 [H]).  q [Tq, H, D] (the tail of each sequence's keys), k / v [Tk, H, D] strided views."""
    if not q.is_cuda:
        o = ref.flash_attention_window(q, k, v, cu_q, cu_k, scale, window, sink)
        return o if out is None else out.copy_(o)
    _i32(cu_q)
    _i32(cu_k)
    T, H, D = q.shape
    expect(all(t.dtype == torch.bfloat16 for t in (q, k, v)) and D in FLASH_WINDOW_DIMS, "bf16, head dim 64 / 128 / 256")
    expect(k.shape == v.shape and k.stride() == v.stride() and k.shape[1:] == (H, D), "k / v shape")
    expect(cu_q.numel() == cu_k.numel(), "cu_q / cu_k")
    qst, qsh = _head_strides(q)
    kst, ksh = _head_strides(k)
    expect(all(s % 8 == 0 for s in (qst, qsh, kst, ksh)), "attention strides must be multiples of 8 elements (16 B)")
    if sink is not None:
        _f32(H, sink)
    out = torch.empty((T, H, D), dtype=q.dtype, device=q.device) if out is None else out
    expect(tuple(out.shape) == (T, H, D) and out.dtype == q.dtype and out.stride(2) == 1 and out.stride(0) % 4 == 0
           and out.stride(1) % 4 == 0, "bad attention output")
    native().flash_attention_window(ptr(q), qst, qsh, ptr(k), ptr(v), kst, ksh, ptr(out), out.stride(0), out.stride(1),
                                    ptr(cu_q), ptr(cu_k), cu_q.numel() - 1, int(max_seqlen_q), H, D, float(scale),
                                    int(window), ptr(sink), stream(q))
    return out


def decode_split(batch: int, heads: int, R: int, window: int, max_len: int, target: int = 512) -> tuple[int, int]:
    """(key partitions per sequence, fewest keys of a partition) of a decode step: about ``target``
    workgroups (two per CU).  A partition's fp32 output is as large as 64 keys of latents, so partitions stay
    at 128 keys or more unless the batch is too small to care."""
    wgs = batch * native().latent_decode_groups(heads, R)
    min_part = 64 if wgs <= 4 else 128
    keys = min(window, max_len) + 63 if window else max_len  # a sequence's first tile starts up to 63 keys early
    return max(1, min(-(-target // wgs), -(-keys // min_part))), min_part


class LatentWorkspace:
    """Partition outputs of the latent decode (graph-capture safe): ``rows`` = the largest sequences x heads x
    partitions of any launch, ``cells`` the largest rows x R."""

    def __init__(self, rows: int, cells: int, device):
        self.o = torch.empty((cells,), dtype=torch.float32, device=device)
        self.ml = torch.empty((2 * rows,), dtype=torch.float32, device=device)


def latent_decode(q, cache, block_tables, ctx_lens, scale: float, window: int = 0, sink=None, parts: int = 1,
                  workspace: LatentWorkspace | None = None, order=None, min_part: int = 128, values: int | None = None):
    """q [B, H, R] absorbed queries (one new token per sequence) over the paged latents -> [B, H, R], or
    at least the first ``values`` columns of it (rows that end with a rotated key).  Each sequence's visible keys are split into up to ``parts`` partitions of >= ``min_part`` keys (``decode_split``)."""
    if not q.is_cuda:
        return ref.latent_attention(q, cache, block_tables, None, ctx_lens, scale, window, sink)
    B, H, R = q.shape
    bs = cache.shape[1]
    if q.dtype == torch.float32 or not native().latent_decode_ok(R) or native().latent_decode_values(R) < (values or R) or bs % 64:
        return latent_attention(q, cache, block_tables, None, ctx_lens, scale, window, sink)
    _i32(block_tables)
    _i32(ctx_lens)
    expect(q.is_contiguous() and cache.is_contiguous() and q.dtype == cache.dtype == torch.bfloat16
           and cache.shape[-1] == R, "bf16 queries / latents of one width")
    expect(block_tables.shape[0] >= B and ctx_lens.numel() >= B, "block table / ctx_lens rows < batch")
    if sink is not None:
        _f32(H, sink)
    if order is not None:
        _i32(order)
        expect(order.numel() >= B, "decode order must hold the batch")
    expect(parts == 1 or (workspace is not None and workspace.o.numel() >= B * H * parts * R
                          and workspace.ml.numel() >= 2 * B * H * parts), "latent decode workspace too small")
    out = torch.empty((B, H, native().latent_decode_values(R)), dtype=q.dtype, device=q.device)
    ws = (ptr(workspace.o), ptr(workspace.ml)) if parts > 1 else (0, 0)
    native().latent_decode(ptr(q), ptr(cache), ptr(block_tables), block_tables.shape[1], bs, ptr(ctx_lens), ptr(sink),
                           ptr(out), *ws, B, H, R, int(window), int(parts), int(min_part), float(scale), ptr(order),
                           stream(q))
    return out


def latent_attention(q, cache, block_tables, cu_q, ctx_lens, scale: float, window: int = 0, sink=None):
    """Absorbed attention of any query layout, rank and type: q [T, H, R], query t of sequence b (``cu_q``;
    None: one query per sequence) sees the window that ends at its own cached position."""
    if not q.is_cuda:
        return ref.latent_attention(q, cache, block_tables, cu_q, ctx_lens, scale, window, sink)
    _i32(block_tables)
    _i32(ctx_lens)
    T, H, R = q.shape
    B = T
    if cu_q is not None:
        _i32(cu_q)
        B = cu_q.numel() - 1
    expect(q.is_contiguous() and cache.is_contiguous() and q.dtype == cache.dtype and q.dtype in _ACT
           and cache.shape[-1] == R and R % 4 == 0 and R <= 2048, "queries / latents of one type and width <= 2048")
    expect(block_tables.shape[0] >= B and ctx_lens.numel() >= B, "block table / ctx_lens rows < batch")
    if sink is not None:
        _f32(H, sink)
    out = torch.empty_like(q)
    native().latent_any(ptr(out), ptr(q), ptr(cache), int(q.dtype == torch.float32), ptr(block_tables),
                        block_tables.shape[1], cache.shape[1], ptr(cu_q), ptr(ctx_lens), B, ptr(sink), T, H, R,
                        int(window), float(scale), stream(q))
    return out
