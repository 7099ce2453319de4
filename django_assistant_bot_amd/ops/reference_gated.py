"""Plain-PyTorch references of ``ops.gated`` (gated sublayers, sums over depth, PolyNorm, attention inputs): what CPU tensors
run."""
from __future__ import annotations

import torch

from .reference_hybrid import _spans, total


def _unit(v, n, eps):
    return v * torch.rsqrt(v.pow(2).sum(-1, keepdim=True) / n + eps)


def norm_embed(ids, table, gain, n, eps, x):
    x.copy_(_unit(table[ids.long()].float(), n, eps) * gain)
    return x.to(table.dtype, copy=True)


def gated_residual(src, x, y, gate, post, n, eps, dtype, own, depth, gain):
    T, C = x.shape
    if own is not None:
        real = (own.idx < own.experts)[..., None]
        each = torch.where(real, own.rows.float().view(T, -1, C), own.wt[..., None] * src[:, None])
        f = each.sum(1)
    else:
        f = total(y)[:T, :C]
    g, col, bias = gate
    f = f * torch.sigmoid(total(g)[:T, col:col + C] + bias)
    out = src + _unit(f, n, eps) * post
    if depth is not None:
        over, w, k, ahead, n0 = depth
        if k < over.shape[0]:
            over[k] = out
        out = w[k] * out + (w[n0:k, None, None] * over[n0:k]).sum(0)
        if ahead is not None:
            out = out + ahead
    x.copy_(out)
    return (x if gain is None else _unit(x, n, eps) * gain).to(dtype, copy=True)


def poly_norm(y, n, cols, act, eps, dtype):
    z = total(y)[:, :n].to(dtype).float()
    out = torch.zeros(z.shape[0], cols)
    out[:, :n] = sum(c * _unit(z.pow(k + 1), n, eps) for k, c in enumerate(act[:3])) + act[3]
    return out.to(dtype)


def attn_inputs(y, col0, a, positions, slots, kc, vc, ring, cu, chunk_slots, row_slots, row0, mix, dtype):
    T, heads = positions.numel(), a.H + 2 * a.G
    C = heads * a.D
    u = total(y)[:T, col0:col0 + C]
    if a.bias is not None:
        u = u + a.bias
    u = u.to(dtype).float()
    x = u
    if a.conv is not None:
        taps = a.conv.shape[0]
        x = torch.zeros(T, C)
        spans = (list(zip(_spans(cu, 0, 0), chunk_slots.tolist())) if row0 else []) + (
            list(zip(_spans(None, T - row0, row0), row_slots.tolist())) if row0 < T else [])
        for (b, e), s in spans:
            p0 = int(positions[b])
            past = [ring[s, p % taps].float() if p >= 0 else torch.zeros(C) for p in range(p0 - taps + 1, p0)]
            xs = torch.cat([torch.stack(past) if past else torch.zeros(0, C), u[b:e]])
            x[b:e] = sum(xs[k:k + e - b] * a.conv[k] for k in range(taps))
            for t in range(max(b, e - taps), e):
                ring[s, (p0 + t - b) % taps] = u[t].to(dtype)
    x = x.view(T, heads, a.D)
    qk = x[:, :a.H + a.G]
    if a.whole:
        qk = torch.cat([_unit(t.flatten(1), t.shape[1] * a.dim, a.eps).view(t.shape) for t in (qk[:, :a.H], qk[:, a.H:])], 1)
    else:
        qk = _unit(qk, a.dim, a.eps)
    qk = qk * a.gain.view(a.H + a.G, a.D)
    if a.rot:
        ang = (positions.double()[:, None] * a.turns) * (2 * torch.pi)
        c, s = (ang.cos() * a.rot_mul).float()[:, None], (ang.sin() * a.rot_mul).float()[:, None]
        even, odd = qk[..., 0:a.rot:2].clone(), qk[..., 1:a.rot:2].clone()
        qk[..., 0:a.rot:2], qk[..., 1:a.rot:2] = even * c - odd * s, odd * c + even * s
    q = qk[:, :a.H]
    if a.t_coef:
        q = q * (1 + a.t_coef * torch.log((positions + 1).div(a.t_every, rounding_mode="floor").float() + 1))[:, None, None]
    v = x[:, a.H + a.G:]
    if mix is not None:
        first, lam = mix
        n = first.shape[-1]
        if lam is None:
            first.copy_(v[..., :n].to(dtype))
        else:
            v = v.clone()
            v[..., :n] = v[..., :n] + lam * (first.float() - v[..., :n])
    live = slots >= 0
    b, o = slots[live] // kc.shape[2], slots[live] % kc.shape[2]
    kc[b, :, o] = qk[live, a.H:].to(dtype)
    vc[b, :, o] = v[live].to(dtype)
    return q.to(dtype).contiguous()
