"""Plain fp64 implementation of the Vunelix decoder, one function per mechanism: the numerics oracle of the
framework's tests.  It keeps no cache, batches nothing, runs the recurrence token by token and shares no code
with the package.

A model is (config dict as read from config.json, tensors: name -> float64 torch tensor).
"""
from __future__ import annotations

import math

import torch


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


# ---------------------------------------------------------------- selective scan


def short_conv(x, taps, bias):
    """Causal convolution per channel and silu: x [n, C], taps [C, K], the last tap meets the token itself."""
    n, K = x.shape[0], taps.shape[1]
    pad = torch.cat([x.new_zeros(K - 1, x.shape[1]), x])
    return silu(sum(pad[t:t + n] * taps[:, t] for t in range(K)) + bias)


def selective_scan(x, dt, A, B, C, S=None):
    """x, dt [n, c], A [c, s] (< 0), B, C [n, s] -> (read-outs [n, c], state [c, s])."""
    S = torch.zeros_like(A) if S is None else S
    out = []
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None]
        out.append(S @ C[t])
    return torch.stack(out), S


def mamba1(h, m, w, p, planted=()):
    inner, N = m["inner"], m["state"]
    x, z = torch.split(h @ w[p + "in"].T, [inner, inner], 1)
    x = short_conv(x, w[p + "conv"], w[p + "conv.b"])
    dt, B, C = torch.split(x @ w[p + "x"].T, [m["dt_rank"], N, N], 1)
    dt = softplus(dt @ w[p + "dt"].T + w[p + "dt.b"])
    A = -torch.exp(w[p + "A_log"])
    if "decay_mean" in planted:
        A = A.mean(-1, keepdim=True).expand_as(A)
    y, _ = selective_scan(x, dt, A, B, C)
    if "skip" not in planted:
        y = y + w[p + "D"] * x
    return (y * silu(z)) @ w[p + "o"].T


# ---------------------------------------------------------------- latent attention


def frequencies(rot, planted=()):
    """Radians per position of every pair, and the factor on cosine and sine."""
    d, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / d) for i in range(d // 2)]
    if not sc or "yarn" in planted:
        return f, 1.0
    at = lambda t: d * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))  # noqa: E731
    lo, hi = max(math.floor(at(sc["fast"])), 0), min(math.ceil(at(sc["slow"])), d - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / sc["factor"] * r + x * (1.0 - r))
    return out, 1.0 if "yarn_gain" in planted else 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, rot, planted=()):
    """x [n, heads, dims], token t at position t; neighbours (2i, 2i + 1) are a pair."""
    f, g = frequencies(rot, planted)
    out = x.clone()
    for i, fi in enumerate(f):
        a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * fi
        c, s = torch.cos(a) * g, torch.sin(a) * g
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def latent_attention(h, m, w, p, eps, planted=()):
    n, H, D, P, V, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w[p + "q"].T).view(n, H, D + P)
    dkv = h @ w[p + "dkv"].T
    c = norm(dkv[:, :R], w[p + "dkv.norm"], eps)
    qr, kr = rotate(q[..., D:], m["rot"], planted), rotate(dkv[:, None, R:], m["rot"], planted)[:, 0]
    k = (c @ w[p + "uk"].T).view(n, H, D)
    v = (c @ w[p + "uv"].T).view(n, H, V)
    seen = torch.ones(n, n, dtype=torch.bool).tril()
    heads = []
    for x in range(H):
        s = (q[:, x, :D] @ k[:, x].T + qr[:, x] @ kr.T) * m["scale"]
        s = s.masked_fill(~seen, float("-inf"))
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        heads.append(e / e.sum(-1, keepdim=True) @ v[:, x])
    o = torch.stack(heads, 1).reshape(n, -1)
    if "out_gate" not in planted:
        o = o * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


# ---------------------------------------------------------------- feed-forward


def dense(h, w, p):
    return (torch.relu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, top):
    """Router logits [n, E] -> weights [n, E], zero outside each token's ``top`` experts."""
    s = torch.sigmoid(z)
    idx = torch.topk(s, top, -1).indices
    return torch.zeros_like(s).scatter(-1, idx, s.gather(-1, idx))


def moe(h, f, w, p, planted=()):
    r = f["router"]
    wt = route(h @ w[p + "router"].T, r["top"])
    if "renormalise" in planted:
        wt = wt / wt.sum(-1, keepdim=True)
    y = torch.zeros_like(h)
    for e in range(r["experts"]):
        k = wt[:, e:e + 1]
        y = y + (k * expert(h, w, f"{p}e{e}.") if "weigh_output" in planted else expert(k * h, w, f"{p}e{e}."))
    return y + expert(h, w, p + "shared.") if f.get("shared") else y


# ---------------------------------------------------------------- the model


def schedule(cfg):
    """(layer, pass that starts right before it or None) of every layer run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b, t = loop["start"], loop["stop"], loop["times"]
    return ([(i, None) for i in range(a)] + [(i, k if i == a else None) for k in range(t) for i in range(a, b)]
            + [(i, None) for i in range(b, n)])


def forward(cfg, w, tokens, trace=None, planted=()):
    """tokens (list of int) -> logits [n, vocab]; ``trace`` (list) collects the residual stream after every layer
    run.  ``planted``: mistakes to make on purpose, so a test can show that it would notice them."""
    eps = cfg["norm"]["eps"]
    x = emb = w["embed"][torch.as_tensor(tokens)]
    for i, start in schedule(cfg):
        p, L, m = f"l{i}.", cfg["layers"][i], cfg["layers"][i]["mixer"]
        if start is not None:
            x = torch.cat([x, emb], 1) @ w["loop.in"].T
            if "loop_step" not in planted:
                x = x + w["loop.step"][start]
        h = norm(x, w[p + "norm1"], eps)
        y = mamba1(h, m, w, p + "mix.", planted) if L["type"] == "mamba1" else \
            latent_attention(h, m, w, p + "mix.", eps, planted)
        x = x + norm(y, w[p + "norm1b"], eps)
        f = L.get("mlp")
        if f:
            h = norm(x, w[p + "norm2"], eps)
            y = dense(h, w, p + "mlp.") if f["kind"] == "dense" else moe(h, f, w, p + "mlp.", planted)
            x = x + (y if "post_norm" in planted else norm(y, w[p + "norm2b"], eps))
        if trace is not None:
            trace.append(x)
    z = norm(x, w["final.norm"], eps) @ w["embed"].T
    cap = cfg.get("logit_softcap")
    return z if not cap or "softcap" in planted else cap * torch.tanh(z / cap)
