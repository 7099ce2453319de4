"""Plain-PyTorch references of ``ops.hybrid`` (recurrent mixers, chunked attention, experts): what CPU tensors run.

Projections may be finished rows [T, N] or split-K slabs [S, T, N]; ``cu`` lists the first row of every prompt
portion (None: one token per sequence).
"""
from __future__ import annotations

import torch
import torch.nn.functional as F


def total(y):
    return y.float().sum(0) if y.dim() == 3 else y.float()


def rms_residual(x, y, gain, n, eps, dtype, bias, pairs, ids, table, post=None, raw=False, fresh=False):
    add = torch.zeros_like(x)
    if y is not None:
        add += total(y)
    if bias is not None:
        add += bias
    if pairs is not None:
        add += pairs.float().view(x.shape[0], -1, x.shape[1]).sum(1)
    if post is not None:
        add = add * torch.rsqrt(add.pow(2).sum(-1, keepdim=True) / n + eps) * post
    if fresh:
        x.zero_()
    x += add
    if ids is not None:
        x += table[ids.long()].float()
    if gain is None:
        return x.to(dtype, copy=True) if raw else None
    r = torch.rsqrt(x.pow(2).sum(-1, keepdim=True) / n + eps)
    return (x * r * gain).to(dtype)


def qk_rope_write(y, col0, H, G, D, dim, rot, freq, eps, norm, positions, slots, kc, vc, dtype):
    T = positions.numel()
    x = total(y)[:, col0:col0 + (H + 2 * G) * D].to(dtype).float().view(T, H + 2 * G, D)
    qk = x[:, :H + G].clone()
    if rot:
        a = (positions.double()[:, None] * freq) * (2 * torch.pi)
        c, s = a.cos().float()[:, None], a.sin().float()[:, None]
        u, v = x[:, :H + G, 0:rot:2], x[:, :H + G, 1:rot:2]
        qk[..., 0:rot:2] = u * c - v * s
        qk[..., 1:rot:2] = v * c + u * s
    if norm:
        qk = qk * torch.rsqrt(qk.pow(2).sum(-1, keepdim=True) / dim + eps)
    live = slots >= 0
    bs = kc.shape[2]
    b, o = slots[live] // bs, slots[live] % bs
    kc[b, :, o] = qk[live, H:].to(dtype)
    vc[b, :, o] = x[live, H + G:].to(dtype)
    return qk[:, :H].to(dtype).contiguous()


def chunk_attention(q, kc, vc, bt, cu, ctx, scale, chunk, sink, out_scale, slopes=None):
    T, H, D = q.shape
    G, bs = kc.shape[1], kc.shape[2]
    out = torch.empty(T, H, D)
    rows = list(range(T + 1)) if cu is None else cu.tolist()
    for b in range(len(rows) - 1):
        n, m = rows[b + 1] - rows[b], int(ctx[b])
        pos = torch.arange(m)
        blk = bt[b].long()[pos // bs]
        k, v = (c[blk, :, pos % bs].float().repeat_interleave(H // G, 1) for c in (kc, vc))
        s = torch.einsum("qhd,khd->hqk", q[rows[b]:rows[b + 1]].float(), k) * scale
        i = torch.arange(m - n, m)[:, None]
        if slopes is not None:
            s = s - slopes.float().view(-1, 1, 1) * (i - pos[None])
        bad = pos[None] > i
        if chunk:
            bad = bad | (pos[None] // chunk != i // chunk)
        s = s.masked_fill(bad[None], float("-inf"))
        if sink is not None:
            s = torch.cat([s, sink.float().view(-1, 1, 1).expand(-1, n, 1)], -1)
        out[rows[b]:rows[b + 1]] = torch.einsum("hqk,khd->qhd", torch.softmax(s, -1)[..., :m], v) * out_scale
    return out


def _spans(cu, T, row0):
    return [(row0 + b, row0 + b + 1) for b in range(T)] if cu is None else list(zip(cu.tolist()[:-1], cu.tolist()[1:]))


def short_conv(y, col0, C, w, bias, ring, slot, pos, cu, dtype):
    """Convolves every portion (``cu``) or one token per sequence and updates the rings; -> [T, C]."""
    x = total(y)[:, col0:col0 + C].to(dtype)
    taps = w.shape[0]
    out = torch.zeros(x.shape[0], C)
    for b, (a, e) in enumerate(cu):
        p0, s = int(pos[a]), int(slot[b])
        past = [ring[s, p % taps].float() if p >= 0 else torch.zeros(C) for p in range(p0 - taps + 1, p0)]
        xs = torch.cat([torch.stack(past) if past else torch.zeros(0, C), x[a:e].float()])
        o = sum(xs[k:k + e - a] * w[k] for k in range(taps))
        out[a:e] = F.silu(o if bias is None else o + bias)
        for t in range(max(0, e - a - taps), e - a):
            ring[s, (p0 + t) % taps] = x[a + t]
    return out.to(dtype)


def gates(z, d, A, dt_bias):
    z = total(z)
    dt = F.softplus(z[:, d.a_col:d.a_col + d.H] + dt_bias)
    return torch.exp(-A * dt), torch.sigmoid(z[:, d.b_col:d.b_col + d.H]) if d.delta else dt


def state_scan(conv, d, z, A, dt_bias, skip, state, slot, pos, spans):
    """-> [T, H * V] (rows outside ``spans`` are zero)."""
    g, beta = gates(z, d, A, dt_bias)
    of = torch.arange(d.H) // (d.H // d.G)
    c = conv.float()
    q = c[:, d.q_col:d.q_col + d.G * d.D].view(-1, d.G, d.D)
    k = c[:, d.k_col:d.k_col + d.G * d.D].view(-1, d.G, d.D)
    v = c[:, d.v_col:d.v_col + d.H * d.V].view(-1, d.H, d.V)
    if d.delta:
        q = q * torch.rsqrt(q.pow(2).sum(-1, keepdim=True) + 1e-6) * d.D ** -0.5
        k = k * torch.rsqrt(k.pow(2).sum(-1, keepdim=True) + 1e-6)
    q, k = q[:, of], k[:, of]
    out = torch.zeros(conv.shape[0], d.H, d.V)
    for b, (a, e) in enumerate(spans):
        s = int(slot[b])
        S = state[s, :, :, :d.D] if int(pos[a]) else torch.zeros(d.H, d.V, d.D)  # [H, V, D]
        for t in range(a, e):
            S = S * g[t][:, None, None]
            u = v[t] - (S * k[t][:, None]).sum(-1) if d.delta else v[t]
            S = S + (beta[t][:, None] * u)[:, :, None] * k[t][:, None]
            out[t] = (S * q[t][:, None]).sum(-1)
        state[s, :, :, :d.D] = S
        state[s, :, :, d.D:] = 0
    if skip is not None:
        out = out + skip[:, None] * v
    return out.reshape(conv.shape[0], -1)


def gated_norm(y, gate, g_col, part, gate_first, per_head, w, eps, scale):
    n = y.shape[1]
    g = F.silu(total(gate)[:, g_col:g_col + n])
    v = (y.float() * g if gate_first else y.float()).view(-1, n // part, part)
    v = v * torch.rsqrt(v.pow(2).mean(-1, keepdim=True) + eps) * scale
    v = (v * w if per_head else v * w.view(-1, part)).reshape(-1, n)
    return v if gate_first else v * g


def moe_route(z, col0, E, top, scale, scores="softmax", correction=None):
    z = total(z)[:, col0:col0 + E]
    s = torch.sigmoid(z) if scores == "sigmoid" else torch.softmax(z, -1)
    idx = torch.topk(s if correction is None else s + correction, top, -1).indices
    v = s.gather(-1, idx)
    if scores != "softmax":
        return idx, v * scale
    return idx, v / (v.sum(-1, keepdim=True) + 1e-20) * scale


def moe_experts(h, idx, wt, gate_up, down, E, group, weigh="output"):
    """-> [T * top, W]: each choice's weighted expert output."""
    T, top = idx.shape
    F2, W = gate_up.shape[0] // E, down.shape[0] // E
    out = torch.zeros(T, top, W)
    for e in range(E):
        t, k = (idx == e).nonzero(as_tuple=True)
        if not t.numel():
            continue
        f = wt[t, k][:, None]
        y = h[t].float() @ gate_up[e * F2:(e + 1) * F2].float().T
        y, f = (y * f, 1.0) if weigh == "input" else (y, f)
        if group:
            y = y.view(-1, F2 // (2 * group), 2, group)
            act = (F.silu(y[:, :, 0]) * y[:, :, 1]).reshape(-1, F2 // 2)
        else:
            act = F.silu(y[:, :F2 // 2]) * y[:, F2 // 2:]
        out[t, k] = (act * f).to(h.dtype).float() @ down[e * W:(e + 1) * W].float().T
    return out.view(T * top, W).to(h.dtype)


def shared_glu(y, col0, n, z, sg_col):
    y, z = total(y), total(z)
    return F.silu(y[:, col0:col0 + n]) * y[:, col0 + n:col0 + 2 * n] * torch.sigmoid(z[:, sg_col:sg_col + 1])


def selective_scan(u, d, dt, low, y, A, dt_bias, skip, state, slot, pos, spans, dtype):
    """-> [T, C] (rows outside ``spans`` are zero); ``dt`` [T, C]: the step's projection."""
    dt = F.softplus(total(dt) + dt_bias)
    low, z, x = total(low), total(y)[:, d.z_col:d.z_col + d.C], u.float()
    B, Cn = low[:, d.b_col:d.b_col + d.Np], low[:, d.c_col:d.c_col + d.Np]
    out = torch.zeros(x.shape[0], d.C)
    for b, (a, e) in enumerate(spans):
        s = int(slot[b])
        S = state[s].clone() if int(pos[a]) else torch.zeros(d.C, d.Np)
        for t in range(a, e):
            S = torch.exp2(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t]
            out[t] = ((S @ Cn[t]) + skip * x[t]) * F.silu(z[t])
        state[s] = S
    return out.to(dtype)
