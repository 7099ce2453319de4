"""Bizetar through the framework (checkpoint loading, engine, paged cache beside convolution rings, scheduler, sampling)
against the plain fp64 oracle of tests/bizetar_oracle.py.  Every engine test runs on the CPU reference ops in 32-bit and,
marked gpu, on the native kernels in 32-bit and bf16."""
import io
import json
import os
import random

import bizetar_oracle as oracle
import numpy as np
import pytest
import torch
from decoder_helpers import (
    GREEDY,
    MODES,
    VOCAB,
    assert_greedy,
    engine,
    error,
    feed_portions,
    greedy_oracle,
    prompt,
    write_checkpoint,
)

from django_assistant_bot_amd.engine.llm_engine import LLMEngine, SamplingParams
from django_assistant_bot_amd.models import decoder_config, is_decoder

TOL = {torch.float32: 3e-5, torch.bfloat16: 4e-2}


def sloped(heads, kv_heads, dim, vdim, scale, mlp, v_mix=False, temp=(0.4, 37)):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": v_mix,
         "q_temp": {"coef": temp[0], "every": temp[1]}}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def convolved(heads, kv_heads, dim, vdim, scale, conv, rot, mlp, v_mix=False, base=2000.0, yarn=(3.0, 90, 20.0, 1.5)):
    r = {"base": base, "dims": rot}
    if yarn:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": v_mix, "conv": conv, "rot": r}
    return {"type": "attention_2", "mixer": m, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, identity, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top}}


def config(width, layers, eps=1e-5):
    return {"architecture": "Bizetar", "vocab": VOCAB, "width": width, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # unequal everything: value heads unlike key heads, partial rotation, layers with and without mixed values and MLPs
    "uneven": config(200, [
        convolved(6, 2, 48, 24, 0.2, 3, 32, dense(168)),
        sloped(4, 2, 40, 56, 0.15, moe(7, 3, 3, 40), v_mix=True),
        convolved(4, 2, 72, 56, 0.12, 5, 72, None, v_mix=True, yarn=None),
        sloped(6, 2, 24, 56, 0.3, dense(72), v_mix=True, temp=(1.5, 11)),
        convolved(3, 3, 40, 16, 0.2, 4, 6, moe(9, 2, 4, 24), base=50.0, yarn=(2.0, 33, 4.0, 0.5))]),
    # ones and odd numbers: single heads, heads of one, one tap and many, one expert, identity experts only beside it
    "edge": config(65, [
        sloped(1, 1, 1, 1, 1.0, moe(1, 0, 1, 3), temp=(0.3, 1)),
        convolved(1, 1, 2, 3, 1.0, 1, 2, dense(1), base=10.0, yarn=(1.0, 5, 1.0, 1.0)),
        convolved(3, 1, 9, 13, 0.8, 16, 6, moe(1, 4, 3, 17), v_mix=True),
        sloped(5, 1, 7, 13, 0.5, dense(9), v_mix=True)], eps=1e-2),
    # heads outside the MFMA kernels' tiles, more experts than a wave has lanes
    "wide": config(136, [
        convolved(2, 1, 200, 40, 0.07, 2, 64, dense(72), v_mix=True),
        sloped(2, 1, 270, 40, 0.06, moe(70, 9, 5, 16), v_mix=True),
        convolved(2, 2, 300, 330, 0.05, 7, 300, None),
        sloped(2, 2, 520, 30, 0.05, None)]),
    # heads of 128, more than 16 heads on one key head
    "tiles": config(192, [
        sloped(18, 1, 100, 128, 0.1, dense(64), v_mix=True),
        convolved(18, 1, 128, 128, 0.08, 4, 128, moe(6, 6, 6, 32), v_mix=True),
        sloped(4, 2, 128, 96, 0.09, None)]),
    # no convolution anywhere: everything is paged, so prefixes are shared
    "paged": config(96, [sloped(4, 2, 64, 48, 0.14, dense(64)), sloped(2, 1, 32, 32, 0.2, moe(5, 1, 2, 24))]),
    # enough layers for several blocks of sums over depth
    "deep": config(64, [(sloped(2, 1, 32, 32, 0.2, None, v_mix=True), convolved(2, 1, 32, 32, 0.15, 3, 16, dense(48), v_mix=i % 4 == 1),
                         sloped(2, 2, 16, 24, 0.25, dense(40)))[i % 3] for i in range(19)]),
    # projection sizes that take the streaming decode GEMM (K % 128) and a split-K of several slabs
    "stream": config(512, [
        convolved(8, 2, 128, 128, 0.09, 4, 128, dense(1024), v_mix=True, base=10000.0, yarn=(4.0, 200, 32.0, 1.0)),
        sloped(8, 2, 96, 128, 0.1, moe(14, 3, 5, 256), v_mix=True, temp=(0.2, 64)),
        convolved(8, 4, 64, 64, 0.12, 4, 48, dense(512))]),
}


def tensors(cfg, seed=0):
    """Random bf16 tensors of ``cfg`` under the checkpoint's names.  Routing is decided by channels of the embedding that
    nothing else writes, with well-separated values, so that rounding never changes a token's experts; the corrections take
    one expert always and one never."""
    g = torch.Generator().manual_seed(seed)
    R = lambda *s, std=1.0: torch.randn(s, generator=g) * std  # noqa: E731
    W, w = cfg["width"], {}
    M = lambda o, i, std=1.0: R(o, i, std=std * i ** -0.5)  # noqa: E731
    outs = lambda f: f["router"]["experts"] + f["router"]["identity"]  # noqa: E731
    keep = max([outs(L["mlp"]) for L in cfg["layers"] if L["mlp"] and L["mlp"]["kind"] == "moe"] or [0])
    gain = lambda n, std=0.2: 1 + R(n, std=std)  # noqa: E731
    w["embed"], w["embed.norm"] = R(cfg["vocab"], W), gain(W)
    w["embed.norm"][W - keep:] = 1
    for t in range(cfg["vocab"]):
        w["embed"][t, W - keep:] = torch.linspace(-2.0, 2.0, max(keep, 2))[torch.randperm(max(keep, 2), generator=g)][:keep]
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        for k in "12" if f else "1":
            w[p + "norm" + k] = gain(W) * 0.4  # small steps: rounding does not grow from layer to layer
            w[p + "norm" + k][W - keep:] = 0
            w[p + "rg" + k], w[p + f"rg{k}.b"] = M(W, W), R(W, std=0.5)
        w[p + "dwa"] = R(i + 2, std=0.2).abs()
        w[p + "dwa"][-1] = 0.9
        q, H, G, D, V = p + "mix.", m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        two = L["type"] == "attention_2"
        for n, r in (("q", H * D), ("k", G * D), ("v", G * V)):
            w[q + n] = M(r, W)
            if two:
                w[q + n + ".b"], w[q + n + ".conv"] = R(r, std=0.3), R(r, m["conv"], std=m["conv"] ** -0.5)
        for n, h in (("q", H), ("k", G)):
            w[q + n + ".norm"] = gain(D if two else h * D, 0.3)
        w[q + "sink"] = R(H, std=0.7) + 1
        if m["v_mix"]:
            w[q + "vmix"] = torch.tensor(0.2 + 0.1 * i)
        w[q + "g"] = M(H * V if two else H, W)
        w[q + "o"] = M(W, H * V)
        q = p + "mlp."
        if f and f["kind"] == "dense":
            w[q + "up"], w[q + "down"], w[q + "act"] = M(f["ff"], W), M(W, f["ff"]), torch.tensor([0.7, -0.4, 0.5, 0.3])
        elif f:
            E, n = f["router"]["experts"], outs(f)
            w[q + "router"] = torch.zeros(n, W)
            w[q + "router"][torch.arange(n), W - keep + torch.randperm(keep, generator=g)[:n]] = 1.0
            w[q + "correction"] = torch.zeros(n)
            if n > 2:
                w[q + "correction"][0], w[q + "correction"][1] = -2.0, 2.0
            for e in range(E):
                w[f"{q}e{e}.gate"], w[f"{q}e{e}.up"] = M(f["expert"]["ff"], W), M(f["expert"]["ff"], W)
                w[f"{q}e{e}.down"] = M(W, f["expert"]["ff"], 3.0)
    w["final.norm"], w["head"] = gain(W), M(cfg["vocab"], W)
    w["final.norm"][W - keep:] = 0
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_DIRS: dict = {}


@pytest.fixture(scope="session")
def models(tmp_path_factory):
    """name -> (checkpoint directory, config, fp64 tensors)"""
    def get(name):
        if name not in _DIRS:
            d, cfg = str(tmp_path_factory.mktemp(f"bizetar-{name}")), CONFIGS[name]
            w = tensors(cfg, seed=len(name))
            write_checkpoint(d, cfg, w)
            _DIRS[name] = (d, cfg, {k: v.double() for k, v in w.items()})
        return _DIRS[name]
    return get


_WANT: dict = {}


def wanted(name, cfg, w, toks):
    """The oracle's logits, computed once per (model, prompt)."""
    key = (name, tuple(toks))
    if key not in _WANT:
        _WANT[key] = oracle.forward(cfg, w, toks)
    return _WANT[key]


def assert_rows(err, name, mode, *what):
    """Every row within tolerance; the bf16 "edge" model, whose one-element norms are signs that rounding may flip, at the
    median."""
    e = err.median() if name == "edge" and mode[1] == torch.bfloat16 else err.max()
    assert float(e) < TOL[mode[1]], (*what, int(err.argmax()), float(e))


def near(a, b, tol=1e-5):
    torch.testing.assert_close(a.double(), b.double(), atol=tol, rtol=tol)


# ------------------------------------------------------------------------------------------------ mechanisms


def heads_of(x, n, d, D):
    """[T, n d] -> [T, n D], each head in the low part of D columns."""
    out = x.new_zeros(x.shape[0], n, D)
    out[..., :d] = x.view(-1, n, d)
    return out.reshape(x.shape[0], n * D)


@pytest.mark.parametrize("whole", [False, True])
@pytest.mark.parametrize("taps", [0, 1, 3, 6])
def test_attention_input_mechanisms(whole, taps):
    """The reference op (the kernel is compared with it) against bias, convolution, both norms, rotation, temperature and value
    mix of the oracle, over a portion, a second one and decoded tokens."""
    from types import SimpleNamespace

    from django_assistant_bot_amd import ops

    g = torch.Generator().manual_seed(taps)
    R = lambda *s: torch.randn(s, generator=g).double()  # noqa: E731
    H, G, D, dim, vdim, T, eps, bs, lam = 4, 2, 16, 12, 9, 13, 1e-3, 4, 0.3
    parts = (("q", H, dim), ("k", G, dim), ("v", G, vdim))
    x = {n: R(T, h * d) for n, h, d in parts}
    b = {n: R(h * d) for n, h, d in parts}
    cw = {n: R(h * d, max(taps, 1)) for n, h, d in parts}
    rot = {"dims": 6, "base": 40.0, "scaling": {"factor": 2.0, "original": 30, "fast": 6.0, "slow": 1.0}}
    temp = {"coef": 0.7, "every": 5}
    gain = {"q": R(H * dim if whole else dim), "k": R(G * dim if whole else dim)}
    first, want = R(T, G, vdim), {}
    for n, h, d in parts:
        u = x[n] + b[n]
        u = oracle.short_conv(u, cw[n]) if taps else u
        if n == "v":
            want[n] = oracle.mix_values(u.view(T, h, d), lam, first)
            continue
        u = oracle.norm(u, gain[n], eps).view(T, h, d) if whole else oracle.norm(u.view(T, h, d), gain[n], eps)
        u = oracle.rotate(u, rot)
        want[n] = u * oracle.temperature(T, temp)[:, None, None] if n == "q" else u
    wide = lambda t, f: torch.cat([heads_of(f(t[n]), h, d, D) for n, h, d in parts], 1).float()  # noqa: E731
    gains = [heads_of((gain[n] if whole else gain[n].repeat(h))[None], h, dim, D)[0] for n, h in (("q", H), ("k", G))]
    a = ops.AttnInputs(H, G, D, dim, vdim, eps, whole, torch.cat(gains).float(), wide(b, lambda t: t[None])[0],
                       wide(cw, lambda t: t.t()).contiguous() if taps else None,
                       ops.rope_turns(6, 40.0, "cpu", SimpleNamespace(**rot["scaling"])), oracle.frequencies(rot)[1], 0.7, 5)
    y = torch.stack([wide(x, lambda t: t), torch.zeros(T, (H + 2 * G) * D)])
    y = torch.cat([torch.ones(2, T, 8), y], 2)  # (two slabs, eight columns of something else)
    kc, vc = torch.zeros(5, G, bs, D), torch.zeros(5, G, bs, D)
    slots = torch.arange(T) + 3
    ring = torch.full((3, taps, (H + 2 * G) * D), 9.0) if taps else None
    fw = torch.zeros(T, G, a.first_width)
    fw[..., :vdim] = first.float()
    got = torch.zeros(T, H, D)
    pos = torch.arange(T, dtype=torch.int32)
    for lo, hi in ((0, 7), (7, 9), (9, 10), (10, 11), (11, 12), (12, 13)):
        one = hi - lo == 1
        got[lo:hi] = ops.attn_inputs(y[:, lo:hi], 8, a, pos[lo:hi], slots[lo:hi], kc, vc, ring, None if one else torch.tensor([0, hi - lo]),
                                     hi - lo, torch.tensor([1]), torch.tensor([1]), 0 if one else hi - lo, (fw[lo:hi], lam))
    near(got[..., :dim], want["q"], 1e-4)
    k, v = (c.transpose(1, 2).reshape(-1, G, D)[3:3 + T] for c in (kc, vc))
    near(k[..., :dim], want["k"], 1e-4)
    near(v[..., :vdim], want["v"], 1e-4)
    assert float(got[..., dim:].abs().sum() + k[..., dim:].abs().sum() + v[..., vdim:].abs().sum()) == 0
    if taps:
        assert float(ring[[0, 2]].sub(9).abs().sum()) == 0  # other slots
    out = torch.zeros_like(fw)
    ops.attn_inputs(y, 8, a, pos, torch.full((T,), -1), kc * 0, vc * 0, ring, torch.tensor([0, T]), T, torch.tensor([0]), None, T, (out, None))
    near(oracle.mix_values(out[..., :vdim].double(), lam, first), want["v"], 1e-4)


def test_sublayer_and_feed_forward_mechanisms():
    from django_assistant_bot_amd import ops

    g = torch.Generator().manual_seed(2)
    R = lambda *s: torch.randn(s, generator=g).double()  # noqa: E731
    T, n, C, eps = 5, 20, 24, 1e-3

    def pad(t):
        return torch.cat([t, t.new_zeros(*t.shape[:-1], C - n)], -1).float().contiguous()

    x, y, gz, b, post, nxt = R(T, n), R(T, n), R(T, n), R(n), R(n), R(n)
    f = y * torch.sigmoid(gz + b)
    want = x + oracle.norm(f, post, eps)
    yy, gg = torch.stack([pad(y) / 4, pad(y) * 0.75]), torch.cat([torch.ones(T, 8), pad(gz)], 1)
    xs = torch.zeros(T, C)
    h = ops.gated_residual(pad(x), xs, yy, (gg, 8, pad(b)), pad(post), n, eps, torch.float32)
    near(xs, pad(want))
    near(h, xs)
    # the sum over depth, kept and not kept, with and without a norm behind it
    for k, gain in ((1, None), (3, nxt)):
        over, w = R(3, T, n), R(k + 1)
        res = want if k == 3 else want * 1.0
        total = sum(w[j] * over[j] for j in range(k)) + w[k] * res
        o = pad(over)
        h = ops.gated_residual(pad(x), xs, yy, (gg, 8, pad(b)), pad(post), n, eps, torch.float32, depth=(o, w.float(), k, None, 0),
                               gain=None if gain is None else pad(gain))
        near(xs, pad(total))
        near(h, pad(total if gain is None else oracle.norm(total, gain, eps)))
        if k < 3:
            near(o[k], pad(want))
        sums = ops.depth_ahead(o, torch.stack([w[:1], 2 * w[:1]]).float(), torch.zeros(8, T, C))
        near(sums[1], 2 * w[0] * o[0])
        h = ops.gated_residual(pad(x), xs, yy, (gg, 8, pad(b)), pad(post), n, eps, torch.float32, depth=(o, w.float(), k, sums[0], 1))
        near(xs, pad(total))
    # the embedding
    table, ids = R(7, n), torch.tensor([3, 0, 6, 6, 1], dtype=torch.int32)
    h = ops.norm_embed(ids, pad(table), pad(post), n, eps, xs)
    near(xs, pad(oracle.norm(table[ids.long()], post, eps)))
    near(h, xs)
    # PolyNorm, with padding behind it
    z, act = R(T, 11), [0.3, -0.7, 1.1, 0.4]
    got = ops.poly_norm(torch.cat([z, R(T, 13)], 1).float(), T, 11, 16, act, eps, torch.float32)
    near(got[:, :11], oracle.poly_norm(z, act, eps))
    assert float(got[:, 11:].abs().sum()) == 0
    # gates of whole heads
    o = R(T, 16).float()
    near(ops.sigmoid_gate(gz.float(), 3, o.clone(), 8), o * torch.sigmoid(gz[:, 3:5]).repeat_interleave(8, 1))
    # experts with corrections and identity experts
    for top in (1, 3, 7):
        f = {"router": {"experts": 5, "identity": 2, "top": top}, "expert": {"ff": 8}}
        wm = {"router": R(7, n), "correction": R(7) * 0.3}
        for e in range(5):
            wm.update({f"e{e}.gate": R(8, n), f"e{e}.up": R(8, n), f"e{e}.down": R(n, 8)})
        idx, wt = ops.moe_route((x @ wm["router"].T).float(), 0, 7, top, 1.0, T, "softmax_raw", wm["correction"].float())
        gu = torch.cat([torch.cat([wm[f"e{e}.gate"], wm[f"e{e}.up"]]) for e in range(5)]).float()
        rows = ops.moe_experts(x.float(), idx, wt, gu, torch.cat([wm[f"e{e}.down"] for e in range(5)]).float(), 5, 0)
        each = torch.where((idx < 5)[..., None], rows.view(T, top, n), wt[..., None] * x.float()[:, None])
        near(each.sum(1), oracle.moe(x, f, wm, ""), 1e-4)
        own = ops.RoutedRows(pad(rows), idx, wt, 5)
        ops.gated_residual(pad(x), xs, None, (gg, 8, pad(b)), pad(post), n, eps, torch.float32, own)
        f = oracle.moe(x, f, wm, "") * torch.sigmoid(gz + b)
        near(xs, pad(x + oracle.norm(f, post, eps)), 1e-4)


def test_sloped_attention_reference():
    from django_assistant_bot_amd import ops

    g = torch.Generator().manual_seed(3)
    H, G, D, n, bs = 6, 2, 8, 21, 4
    q, k, v = (torch.randn(n, h, D, generator=g) for h in (H, G, G))
    sink, slopes = torch.randn(H, generator=g), oracle.slopes(H).float()
    kc, vc = (torch.zeros(6, G, bs, D) for _ in "kv")
    for c, t in ((kc, k), (vc, v)):
        c.transpose(1, 2).reshape(-1, G, D)
        for i in range(n):
            c[i // bs, :, i % bs] = t[i]
    bt = torch.arange(6, dtype=torch.int32)[None]
    want = oracle.attend(q.double(), k.double(), v.double(), 0.3, sink.double(), oracle.slopes(H)).reshape(n, -1)
    out = torch.zeros(n, H * D)
    ops.chunk_prefill(q, kc, vc, bt, torch.tensor([0, n], dtype=torch.int32), torch.tensor([n], dtype=torch.int32), n, 0.3, 0, sink, out,
                      slopes=slopes)
    near(out, want)
    ops.chunk_decode(q[-1:], kc, vc, bt, torch.tensor([n], dtype=torch.int32), 0.3, 0, sink, out, slopes=slopes)
    near(out[:1], want[-1:])


MISTAKES = ("conv", "yarn", "yarn_gain", "head_norm", "q_temp", "v_mix", "sink", "slope", "out_gate", "correction", "identity",
            "res_gate", "depth")  # (the norm behind a sublayer hides the scale of its experts' weights)


def test_the_comparison_sees_every_planted_mistake(models):
    """The oracle with one mistake in it is far outside the tolerance the engine tests use."""
    _, cfg, w = models("uneven")
    toks = prompt(150)
    want = wanted("uneven", cfg, w, toks)
    for mistake in MISTAKES:
        assert error(oracle.forward(cfg, w, toks, planted=(mistake,)), want).max() > 100 * TOL[torch.float32], mistake


# ------------------------------------------------------------------------------------------------ prompts, portions, decoding


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_portions_and_decoding(models, name, mode):
    path, cfg, w = models(name)
    toks = prompt(150 if name == "edge" else 210, 3)
    want = wanted(name, cfg, w, toks)
    eng = engine(path, mode)
    for sizes in ([210], [130, 1], [2], [64], [3, 2, 61, 7, 1, 1, 90]):
        got = feed_portions(eng, 7, toks, sizes)
        assert_rows(error(got, want), name, mode, sizes)
        eng.release(7)
    assert eng.blocks.num_free_blocks() == eng.blocks.num_blocks()
    assert eng.blocks.num_free_state_slots() == (0 if name == "paged" else eng.max_batch)


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("name", ["uneven", "edge", "wide"])
def test_first_tokens_one_by_one(models, name, mode):
    path, cfg, w = models(name)
    toks = prompt(70, 5)
    want = wanted(name, cfg, w, toks)
    assert_rows(error(feed_portions(engine(path, mode), 0, toks, [1]), want), name, mode)


@pytest.mark.parametrize("mode", MODES)
def test_layer_results_match_the_oracle(models, mode):
    path, cfg, w = models("uneven")
    toks, taps, want = prompt(90, 1), [], []
    oracle.forward(cfg, w, toks, trace=want)
    eng = engine(path, mode)
    eng.model.layer_tap = lambda i, x: taps.append(x[:, :cfg["width"]].double().cpu())
    eng.feed([(0, toks, [0])])
    assert len(taps) == len(want) == 5
    for a, b in zip(taps, want):
        assert ((a - b).pow(2).mean() / b.pow(2).mean()).sqrt() < TOL[mode[1]]


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("name", ["uneven", "tiles"])
def test_mixed_batches_reused_pages_and_slots(models, mode, name):
    """Unequal requests side by side -- portions beside single tokens, requests that pause, a pool just large enough,
    pages and state slots freed and used again by later requests -- against each request alone."""
    path, cfg, w = models(name)
    rng = random.Random(11)
    reqs = {i: prompt(rng.choice([1, 2, 63, 64, 65, 129, 180]), 100 + i) for i in range(10)}
    want = {i: wanted(name, cfg, w, t) for i, t in reqs.items()}
    eng = engine(path, mode, tokens=4 * 192)
    at, todo, live, used = {}, list(reqs), [], set()
    while todo or live:
        while todo and len(live) < 4:
            live.append(todo.pop(0))
        entries = []
        for i in live:
            if at.get(i, 0) and rng.random() < 0.2:
                continue  # left out of this step
            left = len(reqs[i]) - at.get(i, 0)
            n = min(left, rng.choice([1, 1, 2, 3, 50, 64, 100]))
            entries.append((i, reqs[i][at.get(i, 0):at.get(i, 0) + n], range(n)))
        if not entries:
            continue
        rng.shuffle(entries)
        got, o = eng.feed(entries), 0
        for i, toks, _ in entries:
            lo = at.get(i, 0)
            e = error(got[o:o + len(toks)], want[i][lo:lo + len(toks)]).max()
            assert e < TOL[mode[1]] * 1.5, (i, lo, len(toks), float(e))
            o += len(toks)
            at[i] = lo + len(toks)
            used.update(eng.blocks.blocks(i))
            if at[i] == len(reqs[i]):
                live.remove(i)
                eng.release(i)
    assert eng.blocks.num_free_blocks() == eng.blocks.num_blocks()
    assert eng.blocks.num_free_state_slots() == 4
    assert sum(-(-len(t) // 64) for t in reqs.values()) > len(used)  # pages were used again


@pytest.mark.parametrize("mode", MODES)
def test_long_decoding_passes_pages(models, mode):
    path, cfg, w = models("stream")
    toks = prompt(330, 9)
    want = wanted("stream", cfg, w, toks)
    eng = engine(path, mode)
    got = [eng.feed([(0, toks[:20], range(20))])]
    got += [eng.feed([(0, toks[t:t + 1], [0])]) for t in range(20, 330)]
    err = error(torch.cat(got), want)
    assert err.max() < TOL[mode[1]], int(err.argmax())
    if mode[0] == "cuda":
        assert eng.stats["graph_replays"] == 310  # decode rows ran from captured graphs


def standing_out(special, kind):
    """A one-layer model in which one token's key stands out for every query, so that whether a query sees it (and how far away
    it is taken to be) decides the logits."""
    W, D = 64, 16
    mixer = sloped(1, 1, D, 32, 0.7, None, temp=(0.2, 50)) if kind == "sloped" else \
        convolved(1, 1, D, 32, 0.7, 3, 4, None, base=1e7, yarn=None)
    cfg = config(W, [mixer])
    w = tensors(cfg, 3)
    g = torch.Generator().manual_seed(2)
    w["embed"] = (torch.randn(VOCAB, W, generator=g) * 0.5).to(torch.bfloat16)
    w["embed"][:, :2] = 0
    w["embed"][:, 0] = 3.0
    w["embed"][special, 0], w["embed"][special, 1] = 0.0, 6.0
    w["embed.norm"] = w["embed.norm"] * 0 + 1
    q, k = w["l0.mix.q"].float() * 0.2, w["l0.mix.k"].float()
    at = 0 if kind == "sloped" else 2  # (a pair that hardly turns over the prompt)
    q[at] = 0
    k[at] = 0
    q[at, 0], k[at, 1] = 4.0, 8.0
    w["l0.mix.q"], w["l0.mix.k"] = q.to(torch.bfloat16), k.to(torch.bfloat16)
    for n in ("l0.mix.q.norm", "l0.mix.k.norm"):
        w[n] = w[n] * 0 + 1
    w["l0.dwa"] = torch.tensor([0.1, 1.0]).to(torch.bfloat16)
    if kind == "convolved":
        for n in "qkv":
            c = w[f"l0.mix.{n}.conv"] * 0
            c[:, -1] = 1  # a key belongs to its own token alone
            w[f"l0.mix.{n}.conv"], w[f"l0.mix.{n}.b"] = c, w[f"l0.mix.{n}.b"] * 0
    return cfg, w


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("kind", ["sloped", "convolved"])
def test_one_far_key_decides(tmp_path, mode, kind):
    """Hundreds of keys back, at the first token, at page borders and inside pages, asked for by a prompt, by a portion and by
    decoded tokens."""
    special, n = VOCAB - 1, 300
    cfg, w = standing_out(special, kind)
    write_checkpoint(str(tmp_path), cfg, w)
    wd = {k: v.double() for k, v in w.items()}
    eng = engine(str(tmp_path), mode)
    for pos in (0, 1, 63, 64, 130, 255):
        toks = [t % (VOCAB - 1) for t in prompt(n, 20)]
        other = oracle.forward(cfg, wd, toks)
        toks[pos] = special
        want = oracle.forward(cfg, wd, toks)
        assert error(other[pos + 1:], want[pos + 1:]).min() > 2 * TOL[torch.bfloat16]  # every later token sees it
        assert error(other[:pos + 1][:-1], want[:pos + 1][:-1]).sum() == 0
        for sizes in ([n], [n - 3, 1], [pos + 1, 1, 2, 1], [100]):
            err = error(feed_portions(eng, pos, toks, sizes), want)
            assert err.max() < TOL[mode[1]], (pos, sizes, int(err.argmax()), float(err.max()))
            eng.release(pos)


@pytest.mark.parametrize("mode", MODES)
def test_slopes_over_long_distances(tmp_path, mode):
    """Distances that turn steep heads away from all but their neighbours while flat ones see everything, across cuts."""
    cfg = config(96, [sloped(16, 2, 32, 32, 0.25, None, temp=(0.5, 200))])
    w = tensors(cfg, 4)
    write_checkpoint(str(tmp_path), cfg, w)
    toks = prompt(900, 8)
    want = oracle.forward(cfg, {k: v.double() for k, v in w.items()}, toks)
    eng = engine(str(tmp_path), mode)
    for sizes in ([900], [700, 1, 2, 1, 1], [128]):
        assert_rows(error(feed_portions(eng, 0, toks, sizes), want), "", mode, sizes)
        eng.release(0)


@pytest.mark.parametrize("mode", MODES)
def test_convolution_reaches_over_every_cut(tmp_path, mode):
    """Taps of equal weight: the inputs before a portion, a page or a decoded token count as much as its own."""
    for taps in (2, 4, 9):
        cfg = config(96, [convolved(2, 1, 32, 32, 0.2, taps, 16, dense(40))])
        w = tensors(cfg, 5)
        for n in "qkv":
            w[f"l0.mix.{n}.conv"] = w[f"l0.mix.{n}.conv"] * 0 + 0.5
        write_checkpoint(str(tmp_path), cfg, w)
        toks = prompt(140, taps)
        want = oracle.forward(cfg, {k: v.double() for k, v in w.items()}, toks)
        eng = engine(str(tmp_path), mode)
        for sizes in ([140], [2], [1, 1, 2, 3, 5, 64, 1], [64]):
            assert_rows(error(feed_portions(eng, 0, toks, sizes), want), "", mode, taps, sizes)
            eng.release(0)


@pytest.mark.gpu
def test_one_page_size_more(models):
    path, cfg, w = models("uneven")
    toks = prompt(300, 4)
    want = wanted("uneven", cfg, w, toks)
    eng = engine(path, ("cuda", torch.bfloat16), block_size=128)
    assert_rows(error(feed_portions(eng, 0, toks, [100, 150, 1]), want), "", (0, torch.bfloat16))


def test_small_pages_on_the_cpu(models):
    path, cfg, w = models("uneven")
    toks = prompt(120, 4)
    want = wanted("uneven", cfg, w, toks)
    for bs in (16, 8):
        eng = engine(path, ("cpu", torch.float32), tokens=256, block_size=bs)
        assert error(feed_portions(eng, 0, toks, [50, 1, 2, 17]), want).max() < TOL[torch.float32]


def test_bf16_engine_on_the_cpu(models):
    """The bf16 form of the layout (interleaved gate / up rows) on the reference ops."""
    for name in ("uneven", "tiles"):
        path, cfg, w = models(name)
        toks = prompt(100, 2)
        eng = engine(path, ("cpu", torch.bfloat16))
        assert_rows(error(feed_portions(eng, 0, toks, [60, 1, 30]), wanted(name, cfg, w, toks)) / 2, name, (0, torch.bfloat16))


# ------------------------------------------------------------------------------------------------ generation


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("mixed", [0, 48])
def test_greedy_generation_through_the_scheduler(models, mode, mixed):
    path, cfg, w = models("uneven")
    prompts = [prompt(n, 30 + n) for n in (1, 5, 64, 150)] + [[]]
    eng = engine(path, mode, max_prefill_tokens=100, mixed_prefill_tokens=mixed, max_batch=3, prefix_cache=True)
    n_new = [5, 9, 12, 7, 12]
    outs = eng.generate(prompts, [SamplingParams(max_new_tokens=n, **GREEDY) for n in n_new])
    for p, o, n in zip(prompts, outs, n_new):
        assert len(o.token_ids) == n and o.finish_reason == "length"
        if mode[1] == torch.float32 and len(p) < 100:
            assert o.token_ids == greedy_oracle(oracle, cfg, w, p or [0], n)
        assert_greedy(oracle, cfg, w, p or [0], o.token_ids, 2 * TOL[mode[1]])
    assert eng.blocks.num_free_blocks() == eng.blocks.num_blocks()
    assert eng.blocks.num_free_state_slots() == 3
    if mixed:
        assert eng.stats["mixed_steps"] > 0


@pytest.mark.parametrize("mode", MODES)
def test_preemption_recomputes_the_state(models, mode):
    """A pool too small for the batch: a preempted sequence gives its slot and pages back and starts over."""
    path, cfg, w = models("uneven")
    system = prompt(130, 77)
    prompts = [system + prompt(10 + i, i) for i in range(4)]
    sp = SamplingParams(max_new_tokens=60, **GREEDY)
    eng = engine(path, mode, tokens=9 * 64, max_model_len=256, prefix_cache=True)
    for p, o in zip(prompts, eng.generate(prompts, sp)):
        assert len(o.token_ids) == 60
        assert_greedy(oracle, cfg, w, p, o.token_ids, 2 * TOL[mode[1]])
    assert eng.stats["preemptions"] > 0 and eng.blocks.prefix_hits() == 0


@pytest.mark.parametrize("mode", MODES)
def test_prefixes_are_shared_without_convolutions(models, mode):
    """A model that keeps nothing but pages reuses those of a common prompt; values to mix are the step's own."""
    path, cfg, w = models("paged")
    system = prompt(140, 78)
    prompts = [system + prompt(5 + i, i) for i in range(3)]
    eng = engine(path, mode, prefix_cache=True)
    assert not eng.recurrent
    for _ in range(2):
        for p, o in zip(prompts, eng.generate(prompts, SamplingParams(max_new_tokens=6, **GREEDY))):
            assert_greedy(oracle, cfg, w, p, o.token_ids, 2 * TOL[mode[1]])
    assert eng.blocks.prefix_hits() > 0


@pytest.mark.gpu
def test_graph_replays_match_eager_steps(models):
    """The captured decode step, replayed with the program's own eager work and synchronisations between the replays,
    writes the logits of the eager step; capturing does not advance a convolution."""
    path, cfg, w = models("stream")
    toks = [prompt(100, s) for s in (1, 2, 3)]
    g = engine(path, ("cuda", torch.bfloat16))
    e = engine(path, ("cuda", torch.bfloat16), use_graphs=False)
    for eng in (g, e):
        eng.feed([(i, t[:60], []) for i, t in enumerate(toks)])
    for t in range(60, 90):
        step = [(i, toks[i][t:t + 1], [0]) for i in range(3 if t % 3 else 2)]
        if t % 3 == 0:
            step.append((2, toks[2][t:t + 1], [0]))
        a, b = g.feed(step), e.feed(step)
        assert torch.equal(a, b), t
        if t % 5 == 0:
            torch.randn(1 << 20, device="cuda").sum().item()
            torch.cuda.synchronize()
    assert g.stats["graph_replays"] == 30 and e.stats["graph_replays"] == 0


@pytest.mark.gpu
def test_large_decode_batches(models):
    """Unequal sequences, more than the split-K steps of small batches take, against each alone."""
    path, cfg, w = models("stream")
    for B in (37, 140):
        lens = [1 + (7 * i) % 40 for i in range(B)]
        toks = [prompt(n + 2, 200 + i) for i, n in enumerate(lens)]
        eng = engine(path, ("cuda", torch.bfloat16), tokens=64 * (B + 3), max_batch=B, max_model_len=64)
        eng.feed([(i, t[:-2], []) for i, t in enumerate(toks)])
        for k in (2, 1):
            got = eng.feed([(i, t[len(t) - k:len(t) - k + 1], [0]) for i, t in enumerate(toks)])
            for i, t in enumerate(toks):
                if i % 9 == 0 or i > B - 3:
                    want = oracle.forward(cfg, w, t[:len(t) - k + 1])[-1:]
                    assert error(got[i:i + 1], want).max() < 1.5 * TOL[torch.bfloat16], (k, i)


def test_sampling_and_string_prompts(models):
    path, _, _ = models("uneven")
    eng = engine(path, ("cpu", torch.float32))
    outs = eng.generate(["hello world", "again"], SamplingParams(max_new_tokens=5, top_k=5, seed=3))
    assert all(len(o.token_ids) == 5 and all(0 <= t < VOCAB for t in o.token_ids) for o in outs)


def test_served_by_the_dialog_provider(models, monkeypatch):
    """The application's in-process provider serves a Bizetar checkpoint directory, JSON mode included."""
    import asyncio

    from assistant.ai.providers.transformers import TransformersProvider
    from django_assistant_bot_amd.engine import serving

    path, _, _ = models("edge")
    monkeypatch.setattr(serving, "_llm", {})
    p = TransformersProvider(path, device="cpu", dtype=torch.float32)
    try:
        msg = [{"role": "user", "content": "hello there"}]
        r = asyncio.run(p.get_response(msg, max_tokens=6))
        assert r.length_limited and r.usage["completion_tokens"] == 6
        assert isinstance(asyncio.run(p.get_response(msg, max_tokens=40, json_format=True)).result, dict)
    finally:
        p._worker.stop()


@pytest.mark.gpu
def test_decoder_bench_option():
    from benchmarks import decoder_bench

    out = decoder_bench.run(["tiny-bizetar", "tiny-llama"], prefill=((2, 64),), decode=((2, 100),), iters=2, repeat=1)
    assert [(r["model"], r["metric"].split()[0]) for r in out] == [
        (m, k) for k in ("prefill", "decode") for m in ("tiny-bizetar", "tiny-llama")]
    assert all(r["value"] > 0 for r in out)


# ------------------------------------------------------------------------------------------------ configuration, loading, tools


def test_registry_and_presets():
    from django_assistant_bot_amd.models import BizetarModel, decoder_family, random_bizetar_weights

    cfg = decoder_config("tiny-bizetar")
    assert is_decoder("tiny-bizetar") and decoder_family(cfg).model is BizetarModel
    n = sum(v.numel() for v in random_bizetar_weights(cfg).values() if torch.is_tensor(v))
    assert n >= cfg.params()  # padding only adds
    assert 6.5e9 < decoder_config("bizetar-8b").params() < 8.5e9
    eng = LLMEngine("tiny-bizetar", "cpu", max_batch=2, max_model_len=128, num_blocks=8)
    assert len(eng.generate([[1, 2, 3]], SamplingParams(max_new_tokens=4, ignore_eos=True))[0].token_ids) == 4


def test_parameter_count_is_exact(models):
    for name in CONFIGS:
        path, _, w = models(name)
        assert decoder_config(path).params() == sum(v.numel() for v in w.values()), name


def test_checkpoint_directory(models):
    path, cfg, w = models("uneven")
    c = decoder_config(path)
    assert is_decoder(path) and c.vocab_size == VOCAB and c.layers == 5 and c.first_mix == 1
    assert c.blocks[0].mixer.rot.scaling.original == 90 and c.blocks[2].mixer.rot.scaling is None
    assert c.blocks[0].mixer.temp is None and c.blocks[3].mixer.temp.every == 11 and c.blocks[3].mixer.slopes
    assert c.blocks[2].mlp is None and c.blocks[1].mlp.identity == 3 and c.blocks[1].mlp.outputs == 10
    assert decoder_config(models("paged")[0]).first_mix is None


def test_bad_checkpoints_are_refused(models, tmp_path):
    path, cfg, _ = models("uneven")
    w = tensors(cfg)
    for change, what in ((lambda c: c["layers"][0].update(type="other"), "mixer type"),
                         (lambda c: c["layers"][0]["mlp"].update(kind="routed"), "mlp kind"),
                         (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=11), "pairs"),
                         (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=50), "pairs"),
                         (lambda c: c["layers"][0]["mixer"].update(conv=17), "taps"),
                         (lambda c: c["layers"][0]["mixer"].update(heads=5), "groups"),
                         (lambda c: c["layers"][0]["mixer"].update(vdim=1100), "wide"),
                         (lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0), "period"),
                         (lambda c: c["layers"][1]["mixer"].update(vdim=48), "equal value heads"),
                         (lambda c: c["layers"][1]["mlp"]["router"].update(top=11), "experts"),
                         (lambda c: c["layers"][0]["mlp"].update(ff=70000), "MLP"),
                         (lambda c: c.update(width=17000), "width"),
                         (lambda c: c["layers"][0]["mixer"].update(dim=52), "config.json says")):
        c = json.loads(json.dumps(cfg))
        change(c)
        write_checkpoint(str(tmp_path), c, w)
        with pytest.raises(ValueError, match=what):
            LLMEngine(str(tmp_path), "cpu", dtype=torch.float32, max_batch=1, max_model_len=64, num_blocks=4)
    with pytest.raises(ValueError, match="tp_size"):
        LLMEngine("tiny-bizetar", "cpu", tp_size=2)


def test_memory_of_the_layers(models):
    path, cfg, _ = models("uneven")
    eng = engine(path, ("cpu", torch.float32))
    kv = eng.kv
    assert [r is not None for r in kv.ring] == [True, False, True, False, True] and not any(s is not None for s in kv.state)
    assert eng.model.state_bytes(5) == sum(t.numel() * t.element_size() for t in kv.ring if t is not None)
    assert eng.model.cache_bytes_per_block(64) * eng.blocks.num_blocks() == sum(t.numel() * t.element_size() for t in kv.k + kv.v)
    assert eng.model.step_bytes(10) == 10 * 5 * 256 * 4 and not eng.model.ahead
    deep = engine(models("deep")[0], ("cpu", torch.float32)).model
    assert {b: tuple(t.shape) for b, t in deep.ahead.items()} == {8: (8, 9), 16: (3, 17)}


def test_feed_guards(models):
    path, _, _ = models("edge")
    eng = engine(path, ("cpu", torch.float32), tokens=128, max_batch=2)
    eng.feed([(0, [1, 2], []), (1, [3], [])])
    with pytest.raises(RuntimeError, match="live"):
        eng.feed([(2, [1], [0])])
    with pytest.raises(RuntimeError, match="cache exhausted"):
        eng.feed([(0, [1] * 70, [])])
    eng.release(1)
    assert eng.feed([(3, [4], [0])]).shape == (1, VOCAB)


@pytest.mark.parametrize("mode", MODES)
def test_trace_replay(models, tmp_path, mode, monkeypatch, capsys):
    """The command-line runner: files, order of rows, request names that come back, several requests in a step."""
    from django_assistant_bot_amd.engine import trace_replay

    path, cfg, w = models("uneven")
    a, b = prompt(80, 1), prompt(9, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:70], "want": [69, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b, "want": []}, {"id": "a", "tokens": a[70:71], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[71:72], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "b", "tokens": b[:1], "want": [0]}, {"id": "a", "tokens": a[72:], "want": [7, 0]}], "end": ["a", "b"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    rc = trace_replay.main(["--model", path, "--dtype", "float32" if mode[1] == torch.float32 else "bfloat16", "--out",
                            str(tmp_path), "--max-tokens", "192", "--device", mode[0]])
    assert rc == 0
    assert [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(4)]
    wa, wb = oracle.forward(cfg, w, a), oracle.forward(cfg, w, b)
    want = {0: wa[[69, 3]], 1: wa[[70]], 3: torch.stack([wb[0], wa[79], wa[72]])}
    assert sorted(os.listdir(tmp_path)) == ["0.f32", "1.f32", "3.f32"]
    for s, rows in want.items():
        got = torch.from_numpy(np.fromfile(tmp_path / f"{s}.f32", "<f4").reshape(len(rows), VOCAB))
        assert error(got, rows).max() < TOL[mode[1]]
