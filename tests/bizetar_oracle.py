"""Plain fp64 implementation of the Bizetar decoder, one function per mechanism: the numerics oracle of the
framework's tests.  It keeps no cache, batches nothing and shares no code with the package.

A model is (config dict as read from config.json, tensors: name -> float64 torch tensor).
"""
from __future__ import annotations

import math

import torch


def silu(z):
    return z / (1.0 + torch.exp(-z))


def norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


# ---------------------------------------------------------------- attention


def short_conv(u, taps):
    """Causal convolution per channel: u [n, C], taps [C, K], the last tap meets the token itself."""
    n, K = u.shape[0], taps.shape[1]
    pad = torch.cat([u.new_zeros(K - 1, u.shape[1]), u])
    return sum(pad[t:t + n] * taps[:, t] for t in range(K))


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
    """x [n, heads, dim], token t at position t; neighbours (2i, 2i + 1) of the first rot.dims are a pair."""
    f, g = frequencies(rot, planted)
    out = x.clone()
    for i, fi in enumerate(f):
        a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * fi
        c, s = torch.cos(a) * g, torch.sin(a) * g
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def slopes(H):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=torch.float64)


def temperature(n, t):
    p = torch.arange(n, dtype=torch.float64)
    return 1.0 + t["coef"] * torch.log(torch.floor((p + 1) / t["every"]) + 1.0)


def mix_values(v, lam, first):
    return (1.0 - lam) * v + lam * first


def attend(q, k, v, scale, sink, slope=None):
    """q [n, H, D], k [n, G, D], v [n, G, V] -> [n, H, V]; every head's denominator also has exp(sink)."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    d = torch.arange(n)[:, None] - torch.arange(n)[None]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = q[:, h] @ k[:, g].T * scale
        if slope is not None:
            s = s - slope[h] * d
        s = s.masked_fill(d < 0, float("-inf"))
        m = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        e = torch.exp(s - m)
        out.append(e @ v[:, g] / (e.sum(-1, keepdim=True) + torch.exp(sink[h] - m)))
    return torch.stack(out, 1)


def attention(h, kind, m, w, p, eps, first, planted=()):
    """-> (the mixer's output, the values that later layers mix in)."""
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    x = {}
    for c in "qkv":
        x[c] = h @ w[p + c].T
        if kind == "attention_2":
            x[c] = x[c] + w[p + c + ".b"]
            if "conv" not in planted:
                x[c] = short_conv(x[c], w[p + c + ".conv"])
    q, k, v = x["q"], x["k"], x["v"].view(n, G, V)
    if kind == "attention":
        if "head_norm" in planted:
            q = norm(q.view(n, H, D), w[p + "q.norm"].view(H, D), eps)
            k = norm(k.view(n, G, D), w[p + "k.norm"].view(G, D), eps)
        else:
            q, k = norm(q, w[p + "q.norm"], eps).view(n, H, D), norm(k, w[p + "k.norm"], eps).view(n, G, D)
        if "q_temp" not in planted:
            q = q * temperature(n, m["q_temp"])[:, None, None]
    else:
        q, k = norm(q.view(n, H, D), w[p + "q.norm"], eps), norm(k.view(n, G, D), w[p + "k.norm"], eps)
        q, k = rotate(q, m["rot"], planted), rotate(k, m["rot"], planted)
    if m.get("v_mix"):
        if first is None:
            first = v
        elif "v_mix" not in planted:
            v = mix_values(v, w[p + "vmix"], first)
    sink = torch.full_like(w[p + "sink"], -1e30) if "sink" in planted else w[p + "sink"]
    o = attend(q, k, v, m["scale"], sink, slopes(H) if kind == "attention" and "slope" not in planted else None)
    g = torch.sigmoid(h @ w[p + "g"].T)
    if "out_gate" not in planted:
        o = o * g[:, :, None] if kind == "attention" else o * g.view(n, H, V)
    return o.reshape(n, -1) @ w[p + "o"].T, first


# ---------------------------------------------------------------- feed-forward


def poly_norm(z, act, eps):
    unit = lambda y: y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)  # noqa: E731
    return act[0] * unit(z) + act[1] * unit(z ** 2) + act[2] * unit(z ** 3) + act[3]


def dense(h, w, p, eps):
    return poly_norm(h @ w[p + "up"].T, w[p + "act"], eps) @ w[p + "down"].T


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, correction, top, planted=()):
    """Router logits [n, E] -> weights [n, E], zero outside each token's ``top`` experts."""
    s = torch.softmax(z, -1)
    idx = torch.topk(s if "correction" in planted else s + correction, top, -1).indices
    wt = torch.zeros_like(s).scatter(-1, idx, s.gather(-1, idx))
    return wt / wt.sum(-1, keepdim=True) if "renormalise" in planted else wt


def moe(h, f, w, p, planted=()):
    r = f["router"]
    wt = route(h @ w[p + "router"].T, w[p + "correction"], r["top"], planted)
    y = torch.zeros_like(h)
    for e in range(r["experts"]):
        y = y + wt[:, e:e + 1] * expert(h, w, f"{p}e{e}.")
    return y if "identity" in planted else y + wt[:, r["experts"]:].sum(-1, keepdim=True) * h


# ---------------------------------------------------------------- the model


def sublayer(x, y, w, p, k, eps, planted=()):
    """The stream after a sublayer: gate of the stream it read, norm of the result, sum."""
    if "res_gate" not in planted:
        y = y * torch.sigmoid(x @ w[f"{p}rg{k}"].T + w[f"{p}rg{k}.b"])
    return x + norm(y, w[f"{p}norm{k}"], eps)


def forward(cfg, w, tokens, trace=None, planted=()):
    """tokens (list of int) -> logits [n, vocab]; ``trace`` (list) collects the residual stream after every layer.
    ``planted``: mistakes to make on purpose, so a test can show that it would notice them."""
    eps = cfg["norm"]["eps"]
    x = norm(w["embed"][torch.as_tensor(tokens)], w["embed.norm"], eps)
    past, first = [x], None
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y, first = attention(x, L["type"], L["mixer"], w, p + "mix.", eps, first, planted)
        x = sublayer(x, y, w, p, 1, eps, planted)
        f = L.get("mlp")
        if f:
            y = dense(x, w, p + "mlp.", eps) if f["kind"] == "dense" else moe(x, f, w, p + "mlp.", planted)
            x = sublayer(x, y, w, p, 2, eps, planted)
        past.append(x)
        if "depth" not in planted:
            x = sum(w[p + "dwa"][j] * past[j] for j in range(i + 2))
        if trace is not None:
            trace.append(x)
    return norm(x, w["final.norm"], eps) @ w["head"].T
