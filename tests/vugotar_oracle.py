"""Plain fp64 implementation of the Vugotar decoder, one function per mechanism: the numerics oracle of
the framework's tests.  It keeps no cache, batches nothing, runs every recurrence token by token and shares
no code with the package.

A model is (config dict as read from config.json, tensors: name -> float64 torch tensor).
"""
from __future__ import annotations

import torch


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def rms(x, eps):
    """x over its root mean square (last dimension)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1.0 + w)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def rotate(x, dims, base):
    """Interleaved rotary positions: x [n, heads, dim], token t at position t, pairs (2i, 2i+1) of the first ``dims``."""
    out = x.clone()
    for i in range(dims // 2):
        a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * base ** (-2.0 * i / dims)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def chunk_softmax1(s, size, sink=1.0):
    """Rows of scores [n, n]: key j is seen by query i when j <= i and both lie in one chunk of ``size``; ``sink`` joins
    the denominator."""
    n = s.shape[0]
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = j <= i
    if size:
        seen = seen & (torch.div(i, size, rounding_mode="floor") == torch.div(j, size, rounding_mode="floor"))
    s = s.masked_fill(~seen, float("-inf"))
    top = s.max(-1, keepdim=True).values.clamp(min=0.0)
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + sink * torch.exp(-top))


def chunked_attention(h, m, w, p, eps, planted=()):
    n, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w[p + "q"].T).view(n, H, D)
    k = (h @ w[p + "k"].T).view(n, G, D)
    v = (h @ w[p + "v"].T).view(n, G, m["vdim"])
    if m.get("rot"):
        q, k = (rotate(x, m["rot"]["dims"], m["rot"]["base"]) for x in (q, k))
    if "qk_norm" not in planted:
        q, k = rms(q, eps), rms(k, eps)
    size = (m.get("mask") or {}).get("size", 0)
    if "chunk" in planted:
        size += 1
    heads = []
    for x in range(H):
        g = x // (H // G)
        pr = chunk_softmax1(q[:, x] @ k[:, g].T * m["scale"], size, 0.0 if "sink" in planted else 1.0)
        heads.append(pr @ v[:, g])
    return torch.stack(heads, 1).reshape(n, -1) @ w[p + "o"].T


def short_conv(x, taps, bias=None):
    """Causal convolution per channel and silu: x [n, C], taps [C, K], the last tap meets the token itself."""
    n, K = x.shape[0], taps.shape[1]
    pad = torch.cat([x.new_zeros(K - 1, x.shape[1]), x])
    y = sum(pad[t:t + n] * taps[:, t] for t in range(K))
    return silu(y if bias is None else y + bias)


def delta_rule(q, k, v, g, beta, S0=None):
    """Gated delta rule, token by token: q, k [n, H, D], v [n, H, V], g, beta [n, H] -> ([n, H, V], S [H, D, V])."""
    n, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if S0 is None else S0.clone()
    out = []
    for t in range(n):
        S = S * g[t][:, None, None]
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


def delta_mixer(h, m, w, p, eps, planted=()):
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ w[p + x].T, w[p + x + ".conv"]) for x in "qkv")
    q, k, v = q.view(n, G, D), k.view(n, G, D), v.view(n, H, V)
    q, k = unit(q) * D ** -0.5, unit(k)
    of = torch.arange(H) // (H // G)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    if "decay" in planted:
        g = torch.ones_like(g)
    o, _ = delta_rule(q[:, of], k[:, of], v, g, beta)
    o = rms(o, eps) * w[p + "norm"] * silu(h @ w[p + "g"].T).view(n, H, V)
    return o.reshape(n, -1) @ w[p + "o"].T


def ssd_scan(x, B, C, dt, A, S0=None):
    """State-space recurrence, token by token: x [n, H, V], B, C [n, H, N], dt [n, H], A [H] (> 0) -> ([n, H, V], S [H, N, V])."""
    n, H, V = x.shape
    S = torch.zeros(H, B.shape[-1], V, dtype=x.dtype) if S0 is None else S0.clone()
    out = []
    for t in range(n):
        S = torch.exp(-A * dt[t])[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        out.append(torch.einsum("hnv,hn->hv", S, C[t]))
    return torch.stack(out), S


def mamba2_mixer(h, m, w, p, eps, planted=()):
    n, H, V, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    z, xbc, dt = torch.split(h @ w[p + "in"].T, [inner, inner + 2 * G * N, H], 1)
    xbc = short_conv(xbc, w[p + "conv"], w[p + "conv.b"])
    x, B, C = torch.split(xbc, [inner, G * N, G * N], 1)
    x, B, C = x.view(n, H, V), B.view(n, G, N), C.view(n, G, N)
    of = torch.arange(H) // (H // G)
    y, _ = ssd_scan(x, B[:, of], C[:, of], softplus(dt + w[p + "dt_bias"]), torch.exp(w[p + "A_log"]))
    y = y + (0.0 if "skip" in planted else 1.0) * w[p + "D"][:, None] * x
    y = y.reshape(n, inner) * silu(z)
    y = rms(y.view(n, m["norm_groups"], -1), eps).reshape(n, inner) * w[p + "norm"]
    return y @ w[p + "o"].T


def glu(h, w, p, bias=False):
    b = (lambda name: w[p + name + ".b"]) if bias else (lambda name: 0.0)
    return (silu(h @ w[p + "gate"].T + b("gate")) * (h @ w[p + "up"].T + b("up"))) @ w[p + "down"].T + b("down")


def route(z, top, scale):
    """Router logits [n, E] -> weights [n, E], zero outside each token's ``top`` experts."""
    s = torch.softmax(z, -1)
    v, idx = torch.topk(s, top, -1)
    return torch.zeros_like(s).scatter(-1, idx, v / (v.sum(-1, keepdim=True) + 1e-20) * scale)


def moe(h, f, w, p, planted=()):
    r = f["router"]
    weights = route(h @ w[p + "router"].T, r["top"], 1.0 if "router_scale" in planted else r["scale"])
    y = sum(weights[:, e:e + 1] * glu(h, w, f"{p}e{e}.") for e in range(r["experts"]))
    if f.get("shared"):
        y = y + glu(h, w, p + "shared.") * torch.sigmoid(h @ w[p + "shared.sg"].T)
    return y


def schedule(cfg):
    """Layer of every layer run, and the runs before which the embedding output is added again."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n)), set()
    a, b, t = loop["start"], loop["stop"], loop["times"]
    return (list(range(a)) + list(range(a, b)) * t + list(range(b, n)), {a + i * (b - a) for i in range(1, t)} if b > a else set())


def forward(cfg, w, tokens, trace=None, planted=()):
    """tokens (list of int) -> logits [n, vocab]; ``trace`` (list) collects the residual stream after every layer
    run.  ``planted``: mistakes to make on purpose, so a test can show that it would notice them."""
    eps = cfg["norm"]["eps"]
    x = emb = w["embed"][torch.as_tensor(tokens)]
    runs, again = schedule(cfg)
    for r, i in enumerate(runs):
        p, L, m = f"l{i}.", cfg["layers"][i], cfg["layers"][i]["mixer"]
        if r in again and "loop_add" not in planted:
            x = x + emb
        h = norm(x, w[p + "norm1"], eps)
        if L["type"] == "mamba2":
            y = mamba2_mixer(h, m, w, p + "mix.", eps, planted)
        else:
            y = (m["left_scale"] * chunked_attention(h, m["left"], w, p + "mix.left.", eps, planted)
                 + m["right_scale"] * delta_mixer(h, m["right"], w, p + "mix.right.", eps, planted))
        f = L.get("mlp")
        if f:
            y = y + (glu(h, w, p + "mlp.", True) if f["kind"] == "dense" else moe(h, f, w, p + "mlp.", planted))
        x = x + y
        if trace is not None:
            trace.append(x)
    return norm(x, w["final.norm"], eps) @ w["head"].T
