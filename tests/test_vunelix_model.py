"""Vunelix through the framework (checkpoint loading, engine, paged latents beside state slots, scheduler, sampling) against
the plain fp64 oracle of tests/vunelix_oracle.py.  Every engine test runs on the CPU reference ops in 32-bit and, marked
gpu, on the native kernels in 32-bit and bf16."""
import io
import json
import os
import random

import numpy as np
import pytest
import torch
import vunelix_oracle as oracle
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


def mamba(inner, state, dt_rank, conv, mlp):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}, "mlp": mlp}


def latent(heads, dim, rot_dim, vdim, rank, scale, mlp, base=2000.0, yarn=(3.0, 90, 20.0, 1.5)):
    rot = {"base": base, "dims": rot_dim}
    if yarn:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale, "rot": rot}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def config(width, layers, loop=None, eps=1e-5, cap=9.0):
    c = {"architecture": "Vunelix", "vocab": VOCAB, "width": width, "norm": {"eps": eps}, "layers": layers}
    if cap:
        c["logit_softcap"] = cap
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CONFIGS = {
    # unequal everything: value heads unlike key heads, experts with and without a shared one, layers without MLP, a loop
    # over both kinds of mixers that starts and ends inside
    "uneven": config(200, [
        latent(3, 40, 12, 24, 80, 0.3, dense(168)),
        mamba(152, 20, 9, 3, moe(12, 3, 40, 72)),
        latent(5, 16, 32, 56, 48, 0.2, moe(5, 1, 24), yarn=None),
        mamba(96, 33, 20, 5, None),
        latent(2, 64, 8, 64, 100, 0.25, None, base=50.0, yarn=(2.0, 33, 4.0, 0.5))], loop=(1, 3, 3)),
    # ones and odd numbers: single heads, one tap, one state entry, one step dimension, one expert, odd widths
    "edge": config(65, [
        mamba(7, 1, 1, 1, moe(1, 1, 3, 5)),
        latent(1, 1, 2, 1, 1, 1.0, dense(9)),
        latent(2, 9, 6, 13, 5, 0.8, moe(3, 3, 17), yarn=(1.0, 5, 1.0, 1.0)),
        mamba(33, 5, 3, 16, moe(4, 2, 8))], loop=(0, 4, 2), eps=1e-2, cap=2.0),
    # latents and heads outside the MFMA kernels' tiles, many state entries, long step projections
    "wide": config(136, [
        mamba(72, 100, 70, 2, dense(72)),
        latent(2, 200, 64, 270, 40, 0.1, None),
        latent(3, 32, 32, 40, 560, 0.2, moe(70, 5, 16, 24)),
        mamba(40, 200, 5, 4, None)], cap=None),
    # rows that end with a rotated key (256 + 64, 512 + 64), heads of 128, more than 16 heads
    "tiles": config(192, [
        latent(4, 72, 48, 128, 256, 0.12, dense(64)),
        latent(18, 40, 24, 48, 510, 0.15, None, base=300.0),
        mamba(256, 64, 16, 4, None)], loop=(0, 1, 1)),
    # no attention anywhere: nothing is paged
    "recurrent": config(96, [mamba(64, 16, 8, 4, dense(64)), mamba(48, 24, 6, 2, moe(6, 2, 24))], loop=(0, 2, 2)),
    # projection sizes that take the streaming decode GEMM (K % 128) and a split-K of several slabs
    "stream": config(512, [
        mamba(1024, 16, 64, 4, dense(1024)),
        latent(8, 96, 32, 128, 128, 0.09, moe(14, 5, 256, 512), base=10000.0, yarn=(4.0, 200, 32.0, 1.0)),
        latent(8, 32, 32, 64, 96, 0.12, dense(512))], loop=(0, 2, 2)),
}


def tensors(cfg, seed=0):
    """Random bf16 tensors of ``cfg`` under the checkpoint's names.  Routing is decided by channels of the embedding that
    nothing else writes, with well-separated values, so that rounding never changes a token's experts."""
    g = torch.Generator().manual_seed(seed)
    R = lambda *s, std=1.0: torch.randn(s, generator=g) * std  # noqa: E731
    W, w = cfg["width"], {}
    M = lambda o, i, std=1.0: R(o, i, std=std * i ** -0.5)  # noqa: E731
    keep = max([L["mlp"]["router"]["experts"] for L in cfg["layers"] if L["mlp"] and L["mlp"]["kind"] == "moe"] or [0])

    def down(o, i, std=1.0):
        t = M(o, i, std)
        t[W - keep:] = 0
        return t

    def gain(n, std=0.2):
        t = 1 + R(n, std=std)
        if n == W:
            t[W - keep:] = 1
        return t

    w["embed"] = R(cfg["vocab"], W)
    for t in range(cfg["vocab"]):
        w["embed"][t, W - keep:] = torch.linspace(-2.0, 2.0, max(keep, 2))[torch.randperm(max(keep, 2), generator=g)][:keep]
    if cfg.get("loop"):
        w["loop.in"], w["loop.step"] = down(W, 2 * W), R(cfg["loop"]["times"], W, std=0.5)
        w["loop.in"][torch.arange(W - keep, W), torch.arange(W - keep, W)] = 1
        w["loop.step"][:, W - keep:] = 0
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            w[p + n] = gain(W) * (0.3 if n.endswith("b") else 1.0)  # small steps: rounding does not grow from layer to layer
        q = p + "mix."
        if L["type"] == "mamba1":
            C, N, K = m["inner"], m["state"], m["dt_rank"]
            w[q + "in"] = M(2 * C, W)
            w[q + "conv"], w[q + "conv.b"] = R(C, m["conv"], std=m["conv"] ** -0.5), R(C, std=0.2)
            w[q + "x"], w[q + "dt"], w[q + "dt.b"] = M(K + 2 * N, C), M(C, K, 0.7), R(C, std=0.5) - 2
            w[q + "A_log"], w[q + "D"] = R(C, N, std=0.7), gain(C, 0.3)
            w[q + "o"] = down(W, C)
        else:
            H, D, P, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            w[q + "q"], w[q + "dkv"], w[q + "dkv.norm"] = M(H * (D + P), W), M(K + P, W), gain(K)
            w[q + "uk"], w[q + "uv"], w[q + "g"] = M(H * D, K), M(H * V, K), M(H * V, W)
            w[q + "o"] = down(W, H * V)
        q = p + "mlp."

        def glu(q, ff):
            w[q + "gate"], w[q + "up"], w[q + "down"] = M(ff, W), M(ff, W), down(W, ff)

        if f and f["kind"] == "dense":
            glu(q, f["ff"])
        elif f:
            E = f["router"]["experts"]
            w[q + "router"] = torch.zeros(E, W)
            w[q + "router"][torch.arange(E), W - keep + torch.randperm(keep, generator=g)[:E]] = 1.0
            for e in range(E):
                glu(f"{q}e{e}.", f["expert"]["ff"])
            if f.get("shared"):
                glu(q + "shared.", f["shared"]["ff"])
    w["final.norm"] = gain(W)
    w["final.norm"][W - keep:] = 0
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_DIRS: dict = {}


@pytest.fixture(scope="session")
def models(tmp_path_factory):
    """name -> (checkpoint directory, config, fp64 tensors)"""
    def get(name):
        if name not in _DIRS:
            d, cfg = str(tmp_path_factory.mktemp(f"vunelix-{name}")), CONFIGS[name]
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


# ------------------------------------------------------------------------------------------------ mechanisms


def assert_rows(err, name, mode, *what):
    """Every row within tolerance; the bf16 "edge" model, whose latents of one element are signs that rounding may flip, at
    the median."""
    e = err.median() if name == "edge" and mode[1] == torch.bfloat16 else err.max()
    assert float(e) < TOL[mode[1]], (*what, int(err.argmax()), float(e))


def near(a, b, tol=1e-5):
    torch.testing.assert_close(a.double(), b.double(), atol=tol, rtol=tol)


def test_selective_scan_mechanisms():
    """The reference ops of the scan alone (the kernels are compared with these): convolution step, portions, decoded tokens,
    steps from the low-rank projection."""
    from django_assistant_bot_amd import ops

    g = torch.Generator().manual_seed(1)
    R = lambda *s: torch.randn(s, generator=g).double()  # noqa: E731
    T, C, N, K, taps = 11, 8, 5, 32, 4
    x, cw, cb = R(T, C), R(C, taps), R(C)
    ring, u = torch.zeros(2, taps, C), torch.zeros(T, C)
    pos = torch.arange(T, dtype=torch.int32)
    u[:4] = ops.short_conv(x[:4].float(), 0, cw.t().contiguous().float(), cb.float(), ring, torch.tensor([1]), pos[:4],
                           torch.tensor([0, 4]), 4)
    for t in range(4, T):
        z = torch.zeros(T, C)
        both = torch.cat([x, 2 * x], 1).float()
        ops.short_conv_step(both, 0, cw.t().contiguous().float(), cb.float(), ring, torch.tensor([1]), pos, t, u, C, z)
        near(z[t], 2 * x[t])
        assert float(z.abs().sum(1).gt(0).sum()) == 1
    near(u, oracle.short_conv(x, cw, cb))
    Np = 16
    d = ops.SelectiveShape(C, Np, K, K, K + Np, C)
    low, y, dtw, dtb, skip = R(T, K + 2 * Np), R(T, 2 * C), R(C, K) * 0.2, R(C), R(C)
    low[:, K + N:K + Np] = 0
    low[:, K + Np + N:] = 0
    A = -R(C, N).exp()
    Af = torch.zeros(C, Np)
    Af[:, :N] = (A / np.log(2)).float()
    st = torch.full((3, C, Np), 7.0)
    out, dt = torch.zeros(T, C), low[:, :K] @ dtw.T
    a = (Af, dtb.float(), skip.float(), st, torch.tensor([2], dtype=torch.int32), pos)
    ux = R(T, C)
    for lo, hi in ((0, 3), (3, 5)):
        o = torch.zeros(hi - lo, C)
        ops.selective_scan(ux[lo:hi].float(), d, dt[lo:hi].float(), low[lo:hi].float(), y[lo:hi].float(), *a[:5], pos[lo:hi],
                           torch.tensor([0, hi - lo]), hi - lo, o)
        out[lo:hi] = o
    step = low[:, :K].float()
    out[5:] = y[5:, C:].float()
    for t in range(5, T):
        ops.selective_step(ux.float(), d, dtw.float(), step, low.float(), *a, t, out)
    S, want = oracle.selective_scan(ux, oracle.softplus(dt + dtb), A, low[:, K:K + N], low[:, K + Np:K + Np + N])[::-1]
    near(out, (want + skip * ux) * oracle.silu(y[:, C:]))
    near(st[2, :, :N], S)
    assert float(st[:2].sub(7).abs().sum()) == 0


def test_latent_and_feed_forward_mechanisms():
    from types import SimpleNamespace

    from django_assistant_bot_amd import ops
    from django_assistant_bot_amd.models.configs import Rotary, Yarn
    from django_assistant_bot_amd.ops import reference as ref

    g = torch.Generator().manual_seed(2)
    R = lambda *s: torch.randn(s, generator=g).double()  # noqa: E731
    # frequencies, with every branch of the ramp
    for dims, base, y in ((16, 1e4, (4.0, 100, 32.0, 1.0)), (8, 50.0, (2.0, 20, 2.0, 2.0)), (64, 5e5, (1.5, 4096, 32.0, 1.0)),
                          (2, 10.0, (3.0, 1000, 400.0, 0.01)), (6, 1e3, None)):
        rot = {"dims": dims, "base": base}
        if y:
            rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), y))
        f, gain = oracle.frequencies(rot)
        r = Rotary(dims, base, Yarn(*y) if y else None)
        near(ops.rope_turns(dims, base, "cpu", r.scaling) * 2 * torch.pi, torch.tensor(f, dtype=torch.float64), 1e-12)
        assert abs(r.gain - gain) < 1e-12
    # latent norm, both rotations, cache write
    H, D, dim, P, rank, T, bs = 3, 24, 9, 6, 11, 5, 4
    rot = {"dims": P, "base": 30.0, "scaling": {"factor": 2.0, "original": 40, "fast": 9.0, "slow": 1.0}}
    q, row, gain = R(T, H, dim + P), R(T, rank + P), R(rank)
    y = torch.zeros(2, T, H * D + 24 + 8).double()
    y[:, :, :H * D].view(2, T, H, D)[1][..., :dim], y[:, :, :H * D].view(2, T, H, D)[0][..., 16:16 + P] = q[..., :dim], q[..., dim:]
    y[1, :, H * D:H * D + rank], y[0, :, H * D + 16:H * D + 16 + P] = row[:, :rank], row[:, rank:]
    cache, slots = torch.zeros(3, bs, 24), torch.tensor([4, 5, -1, 8, 9])
    rope = ops.LatentRope(ops.rope_turns(P, 30.0, "cpu", SimpleNamespace(**rot["scaling"])), oracle.frequencies(rot)[1], P, D, 16, 16,
                          torch.arange(T, dtype=torch.int32))
    gp = torch.zeros(24)
    gp[:rank] = gain.float()
    got = ops.latent_write(y.float(), H * D, gp, cache, slots, rank, 1e-3, rope).view(T, H, D)
    near(got[..., :dim], q[..., :dim])
    near(got[..., 16:16 + P], oracle.rotate(q[..., dim:], rot))
    near(cache[2, 1, :rank], oracle.norm(row[4, :rank], gain, 1e-3))
    near(cache[1, 1, 16:16 + P], oracle.rotate(row[:, None, rank:], rot)[1, 0])
    assert float(cache[1, 2:].abs().sum()) == 0
    k = torch.zeros(4, 2, 24)
    assert float(ops.latent_key_fill(k, torch.ones(4, 24), 8, 16, 6).sum()) == 48 and float(k[:, :, 8:14].sum()) == 48
    # what is added passes a norm of its own; the stream itself as the result; an fp32 table
    x, yy, post, nxt, pairs, table = R(4, 24), R(3, 4, 24), R(20), R(20), R(8, 24), R(7, 24)
    for t in (x, yy, pairs, table):
        t[..., 20:] = 0
    pad = lambda t: torch.cat([t, torch.zeros(4).double()]).float()  # noqa: E731
    xs = x.float().clone()
    h = ops.rms_residual(xs, yy.float(), pad(nxt), 20, 1e-3, torch.float32, None, pairs.float(), post=pad(post))
    want = x[:, :20] + oracle.norm((yy.sum(0) + pairs.view(4, 2, 24).sum(1))[:, :20], post, 1e-3)
    near(xs[:, :20], want)
    near(h[:, :20], oracle.norm(want, nxt, 1e-3))
    ids = torch.tensor([3, 0, 6, 6], dtype=torch.int32)
    h = ops.rms_residual(xs, yy.float(), None, 20, 1e-3, torch.float32, again=(ids, table.float()), fresh=True, raw=True)
    near(xs, yy.sum(0) + table[ids.long()])
    near(h, xs)
    # gates, cap, activations
    o = R(4, 16).float()
    near(ops.sigmoid_gate(yy.float(), 8, o.clone()), o * torch.sigmoid(yy.sum(0)[:, 8:24]))
    near(ops.softcap(yy.float(), 3.0), 3 * torch.tanh(yy.sum(0) / 3))
    gu = torch.stack([R(8, 16).view(1, 8, 16), R(8, 16).view(1, 8, 16)], 1).reshape(16, 16)
    hh = R(5, 16)
    near(ref.gemm_bt(hh.float(), gu.float(), epilogue=ops.EPI_REGLU8, out_f32=True), torch.relu(hh @ gu[:8].T) * (hh @ gu[8:].T))
    near(ops.glu_f32((hh @ gu.T).float(), "relu"), torch.relu(hh @ gu[:8].T) * (hh @ gu[8:].T))
    # experts of the weighted input, sigmoid scores as they are
    for top in (1, 2, 5):
        f = {"router": {"experts": 5, "top": top}, "expert": {"ff": 8}}
        wm = {"router": R(5, 16)}
        for e in range(5):
            wm.update({f"e{e}.gate": R(8, 16), f"e{e}.up": R(8, 16), f"e{e}.down": R(16, 8)})
        idx, wt = ops.moe_route((hh @ wm["router"].T).float(), 0, 5, top, 1.0, 5, "sigmoid")
        gu = torch.cat([torch.cat([wm[f"e{e}.gate"], wm[f"e{e}.up"]]) for e in range(5)]).float()
        rows = ops.moe_experts(hh.float(), idx, wt, gu, torch.cat([wm[f"e{e}.down"] for e in range(5)]).float(), 5, 0, "input")
        near(rows.view(5, top, 16).sum(1), oracle.moe(hh, f, wm, ""), 1e-4)


MISTAKES = ("decay_mean", "skip", "yarn", "yarn_gain", "out_gate", "renormalise", "weigh_output", "loop_step", "post_norm", "softcap")


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
    assert eng.blocks.num_free_state_slots() == eng.max_batch


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("name", ["uneven", "edge"])
def test_first_tokens_one_by_one(models, name, mode):
    path, cfg, w = models(name)
    toks = prompt(70, 5)
    want = wanted(name, cfg, w, toks)
    assert_rows(error(feed_portions(engine(path, mode), 0, toks, [1]), want), name, mode)


@pytest.mark.parametrize("mode", MODES)
def test_layer_runs_match_the_oracle(models, mode):
    path, cfg, w = models("uneven")
    toks, taps, want = prompt(90, 1), [], []
    oracle.forward(cfg, w, toks, trace=want)
    eng = engine(path, mode)
    eng.model.layer_tap = lambda i, x: taps.append(x[:, :cfg["width"]].double().cpu())
    eng.feed([(0, toks, [0])])
    assert len(taps) == len(want) == 9
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


def standing_out(special, rotated: bool):
    """A one-layer model in which one token's key stands out for every query -- in the latent part, or in the rotated part,
    where the score also depends on the distance --, so that whether a query sees it decides the logits."""
    W, H, D, P, V, K = 64, 1, 16, 4, 32, 32
    cfg = config(W, [latent(H, D, P, V, K, 0.5, None, base=1e6, yarn=None)])
    w = tensors(cfg, 3)
    g = torch.Generator().manual_seed(2)
    w["embed"] = (torch.randn(VOCAB, W, generator=g) * 0.5).to(torch.bfloat16)
    w["embed"][:, :2] = 0
    w["embed"][:, 0] = 2.0
    w["embed"][special, 0], w["embed"][special, 1] = 0.0, 6.0
    q, dkv, uk = w["l0.mix.q"].float() * 0.2, w["l0.mix.dkv"].float(), w["l0.mix.uk"].float() * 0.2
    dkv[K:] *= 0.2
    dkv[0] = 0
    uk[0] = 0
    if rotated:  # the pair that turns slowest: its score hardly changes over the prompt
        q[D + P - 2:] = 0
        dkv[K + P - 2:] = 0
        q[D + P - 2, 0], dkv[K + P - 2, 1] = 8.0, 8.0
    else:  # latent axis 0 is the special token's
        q[0] = 0
        dkv[0, 1], uk[0, 0], q[0, 0] = 8.0, 8.0, 8.0
    w["l0.mix.q"], w["l0.mix.dkv"], w["l0.mix.uk"] = (t.to(torch.bfloat16) for t in (q, dkv, uk))
    return cfg, w


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("rotated", [False, True])
def test_one_far_key_decides(tmp_path, mode, rotated):
    """Hundreds of keys back, at the first token, at page borders and inside pages, asked for by a prompt, by a portion and by
    decoded tokens."""
    special, n = VOCAB - 1, 300
    cfg, w = standing_out(special, rotated)
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
def test_a_write_to_the_state_is_read_far_away(models, tmp_path, mode):
    """Decays near one and no attention: a token's write is still in every state hundreds of tokens later, across portions."""
    _, cfg, _ = models("recurrent")
    w = tensors(cfg, 6)
    for k in w:
        if k.endswith("dt.b"):
            w[k] = w[k] * 0 - 5
        if k.endswith("A_log"):
            w[k] = w[k] - 4
    write_checkpoint(str(tmp_path), cfg, w)
    wd = {k: v.double() for k, v in w.items()}
    toks = prompt(300, 8)
    other = list(toks)
    other[3] = (toks[3] + 1) % VOCAB
    want, moved = oracle.forward(cfg, wd, toks), oracle.forward(cfg, wd, other)
    assert error(moved[-40:], want[-40:]).min() > 10 * TOL[torch.float32]  # token 3 matters at the end
    eng = engine(str(tmp_path), mode)
    for sizes in ([300], [150, 2, 1, 1, 120], [64, 1]):
        assert_rows(error(feed_portions(eng, 0, toks, sizes), want), "", mode, sizes)
        eng.release(0)


@pytest.mark.parametrize("mode", MODES)
def test_fast_decays_forget(models, tmp_path, mode):
    """Steps so long that the state is forgotten within a token, beside entries that hardly decay."""
    _, cfg, _ = models("recurrent")
    w = tensors(cfg, 7)
    for k in w:
        if k.endswith("A_log"):
            w[k] = torch.linspace(-12, 5, w[k].shape[1]).expand_as(w[k]).to(torch.bfloat16).contiguous()
        if k.endswith("dt.b"):
            w[k] = w[k] + 3
    write_checkpoint(str(tmp_path), cfg, w)
    toks = prompt(140, 8)
    want = oracle.forward(cfg, {k: v.double() for k, v in w.items()}, toks)
    eng = engine(str(tmp_path), mode)
    for sizes in ([140], [70, 1, 1, 2]):
        assert_rows(error(feed_portions(eng, 0, toks, sizes), want), "", mode, sizes)
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
    """The bf16 form of the layout (interleaved gate / up rows, expanded keys) on the reference ops."""
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


@pytest.mark.gpu
def test_graph_replays_match_eager_steps(models):
    """The captured decode step, replayed with the program's own eager work and synchronisations between the replays,
    writes the logits of the eager step; capturing does not advance a recurrence."""
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
    """More sequences than a workgroup of the state step takes, of unequal lengths, against each alone."""
    path, cfg, w = models("stream")
    lens = [1 + (7 * i) % 40 for i in range(37)]
    toks = [prompt(n + 2, 200 + i) for i, n in enumerate(lens)]
    eng = engine(path, ("cuda", torch.bfloat16), tokens=64 * 40, max_batch=37, max_model_len=64)
    eng.feed([(i, t[:-2], []) for i, t in enumerate(toks)])
    for k in (2, 1):
        got = eng.feed([(i, t[len(t) - k:len(t) - k + 1], [0]) for i, t in enumerate(toks)])
        for i, t in enumerate(toks):
            if i % 4 == 0 or i > 33:
                want = oracle.forward(cfg, w, t[:len(t) - k + 1])[-1:]
                assert error(got[i:i + 1], want).max() < 1.5 * TOL[torch.bfloat16], (k, i)


def test_sampling_and_string_prompts(models):
    path, _, _ = models("uneven")
    eng = engine(path, ("cpu", torch.float32))
    outs = eng.generate(["hello world", "again"], SamplingParams(max_new_tokens=5, top_k=5, seed=3))
    assert all(len(o.token_ids) == 5 and all(0 <= t < VOCAB for t in o.token_ids) for o in outs)


def test_served_by_the_dialog_provider(models, monkeypatch):
    """The application's in-process provider serves a Vunelix checkpoint directory, JSON mode included."""
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

    out = decoder_bench.run(["tiny-vunelix", "tiny-llama"], prefill=((2, 64),), decode=((2, 100),), iters=2, repeat=1)
    assert [(r["model"], r["metric"].split()[0]) for r in out] == [
        (m, k) for k in ("prefill", "decode") for m in ("tiny-vunelix", "tiny-llama")]
    assert all(r["value"] > 0 for r in out)


# ------------------------------------------------------------------------------------------------ configuration, loading, tools


def test_registry_and_presets():
    from django_assistant_bot_amd.models import VunelixModel, decoder_family, random_vunelix_weights

    cfg = decoder_config("tiny-vunelix")
    assert is_decoder("tiny-vunelix") and decoder_family(cfg).model is VunelixModel
    n = sum(v.numel() for v in random_vunelix_weights(cfg).values())
    assert n >= cfg.params()  # padding only adds
    assert 6.5e9 < decoder_config("vunelix-8b").params() < 8.5e9
    eng = LLMEngine("tiny-vunelix", "cpu", max_batch=2, max_model_len=128, num_blocks=8)
    assert len(eng.generate([[1, 2, 3]], SamplingParams(max_new_tokens=4, ignore_eos=True))[0].token_ids) == 4


def test_parameter_count_is_exact(models):
    for name in CONFIGS:
        path, _, w = models(name)
        assert decoder_config(path).params() == sum(v.numel() for v in w.values()), name


def test_checkpoint_directory(models):
    path, cfg, w = models("uneven")
    c = decoder_config(path)
    assert is_decoder(path) and c.vocab_size == VOCAB and c.layers == 5 and c.loop == (1, 3, 3) and c.softcap == 9.0
    assert c.runs() == oracle.schedule(cfg) and c.passes == 3
    assert c.blocks[0].mixer.rot.scaling.original == 90 and c.blocks[2].mixer.rot.scaling is None
    assert c.blocks[3].mlp is None and c.blocks[2].mlp.shared is None and c.blocks[1].mlp.weigh == "input"
    assert decoder_config(models("wide")[0]).softcap is None and decoder_config(models("wide")[0]).passes == 0


def test_empty_loops_are_no_loops(models, tmp_path):
    """A loop over no layers has no first layer of a pass to mix before."""
    _, cfg, _ = models("wide")
    cfg = dict(cfg, loop={"start": 1, "stop": 1, "times": 2})
    w = tensors(cfg)
    write_checkpoint(str(tmp_path), cfg, w)
    toks = prompt(20)
    want = oracle.forward({k: v for k, v in cfg.items() if k != "loop"}, {k: v.double() for k, v in w.items()}, toks)
    eng = engine(str(tmp_path), ("cpu", torch.float32))
    assert error(eng.feed([(0, toks, range(20))]), want).max() < TOL[torch.float32]


def test_bad_checkpoints_are_refused(models, tmp_path):
    path, cfg, _ = models("uneven")
    w = tensors(cfg)
    for change, what in ((lambda c: c["layers"][0].update(type="other"), "mixer type"),
                         (lambda c: c["layers"][0]["mlp"].update(kind="routed"), "mlp kind"),
                         (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10), "rot.dims"),
                         (lambda c: (c["layers"][0]["mixer"].update(rot_dim=5), c["layers"][0]["mixer"]["rot"].update(dims=5)), "pairs"),
                         (lambda c: c["layers"][0]["mixer"].update(kv_rank=2100), "latent"),
                         (lambda c: c["layers"][1]["mixer"].update(state=300), "state"),
                         (lambda c: c["layers"][1]["mixer"].update(conv=17), "taps"),
                         (lambda c: c["layers"][1]["mlp"]["router"].update(top=13), "experts"),
                         (lambda c: c["loop"].update(stop=9), "loop"),
                         (lambda c: c["layers"][1]["mixer"].update(inner=160), "config.json says")):
        c = json.loads(json.dumps(cfg))
        change(c)
        write_checkpoint(str(tmp_path), c, w)
        with pytest.raises(ValueError, match=what):
            LLMEngine(str(tmp_path), "cpu", dtype=torch.float32, max_batch=1, max_model_len=64, num_blocks=4)
    with pytest.raises(ValueError, match="tp_size"):
        LLMEngine("tiny-vunelix", "cpu", tp_size=2)


def test_every_pass_has_its_own_memory(models):
    path, cfg, _ = models("uneven")
    eng = engine(path, ("cpu", torch.float32))
    kv = eng.kv
    scan = [False, True, False, True, False, True, False, True, False]
    assert [s is not None for s in kv.state] == [r is not None for r in kv.ring] == scan
    assert [c is None for c in kv.c] == scan
    mem = [t for t in kv.c + kv.state + kv.ring if t is not None]
    assert len({t.data_ptr() for t in mem}) == len(mem)
    assert eng.model.state_bytes(5) == sum(t.numel() * t.element_size() for t in kv.state + kv.ring if t is not None)
    assert eng.model.cache_bytes_per_block(64) * eng.blocks.num_blocks() == sum(
        t.numel() * t.element_size() for t in kv.c if t is not None)


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
