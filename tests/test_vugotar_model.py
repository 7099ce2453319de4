"""Vugotar through the framework (checkpoint loading, engine, paged K / V beside state slots, scheduler, sampling) against
the plain fp64 oracle of tests/vugotar_oracle.py.  Every engine test runs on the CPU reference ops in 32-bit and, marked
gpu, on the native kernels in 32-bit and bf16."""
import json
import os
import random

import numpy as np
import pytest
import torch
import vugotar_oracle as oracle
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

TOL = {torch.float32: 3e-5, torch.bfloat16: 2.5e-2}


def parallel(left, right, mlp, scales=(0.7, 0.4)):
    """left = (heads, kv_heads, dim, vdim, scale, chunk, rotated dims), right = (heads, kv_heads, dim, vdim, taps)"""
    H, G, D, V, sc, chunk, rot = left
    a = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": sc, "rot": {"base": 3000.0, "dims": rot}, "mask": {"size": chunk}}
    d = dict(zip(("heads", "kv_heads", "dim", "vdim", "conv"), right))
    return {"type": "parallel", "mixer": {"left": a, "right": d, "left_scale": scales[0], "right_scale": scales[1]}, "mlp": mlp}


def mamba(heads, vdim, state, groups, conv, norm_groups, mlp):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": norm_groups}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, scale, ff, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def config(width, layers, loop=None, eps=1e-5):
    c = {"architecture": "Vugotar", "vocab": VOCAB, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CONFIGS = {
    # unequal everything: grouped heads, value heads narrower than keys, partial rotation, norm groups that cut heads, a
    # loop over both kinds of layers, experts with and without a shared one, a layer without MLP
    "uneven": config(200, [
        mamba(6, 24, 40, 3, 3, 4, dense(168)),
        parallel((6, 2, 48, 40, 0.4, 37, 32), (6, 2, 40, 24, 4), moe(12, 3, 1.7, 40, 72)),
        mamba(4, 32, 16, 2, 4, 2, None),
        parallel((3, 3, 64, 64, 0.3, 100, 64), (2, 2, 64, 64, 2), moe(5, 2, 0.8, 24)),
        parallel((4, 1, 24, 56, 0.6, 64, 8), (3, 1, 32, 48, 4), dense(96), (1.0, 1.0))], loop=(1, 3, 3)),
    # ones and odd numbers: single heads and groups, one tap, one expert, chunks of one token, odd value widths
    "edge": config(65, [
        mamba(1, 7, 5, 1, 1, 1, dense(9)),
        parallel((1, 1, 2, 1, 1.0, 1, 2), (1, 1, 3, 5, 1), moe(1, 1, 1.0, 3, 5)),
        parallel((2, 1, 10, 6, 0.8, 3, 0), (3, 3, 12, 7, 5), moe(3, 3, 2.0, 17), (0.3, 1.6)),
        mamba(3, 9, 33, 3, 6, 1, moe(4, 1, 0.5, 8))], loop=(0, 4, 2), eps=1e-2),
    # heads wider than the MFMA kernels tile, groups of more than 16 queries, state rows past 128
    "wide": config(136, [
        parallel((2, 1, 264, 100, 0.15, 50, 100), (2, 1, 160, 100, 4), dense(64)),
        parallel((20, 1, 16, 16, 0.7, 90, 16), (4, 4, 96, 40, 9), None),
        mamba(2, 70, 136, 1, 4, 2, moe(70, 5, 1.5, 16, 24)),
        parallel((2, 2, 160, 136, 0.2, 70, 160), (1, 1, 200, 33, 4), dense(72))]),
    # no attention anywhere: nothing is paged
    "recurrent": config(96, [mamba(4, 16, 24, 2, 4, 4, dense(64)), mamba(2, 48, 8, 1, 2, 1, moe(6, 2, 1.1, 24))], loop=(0, 2, 1)),
    # projection sizes that take the streaming decode GEMM (K % 128) and a split-K of several slabs
    "stream": config(512, [
        mamba(8, 64, 128, 2, 4, 1, dense(1024)),
        parallel((8, 2, 64, 64, 0.3, 96, 64), (4, 2, 128, 128, 4), moe(14, 5, 1.3, 256, 512)),
        parallel((8, 8, 64, 64, 0.3, 200, 32), (8, 4, 64, 64, 4), dense(1024))], loop=(1, 2, 2)),
}


def tensors(cfg, seed=0):
    """Random bf16 tensors of ``cfg`` under the checkpoint's names.  Routing is decided by channels of the embedding that
    nothing else writes, with well-separated values, so that rounding never changes a token's experts."""
    g = torch.Generator().manual_seed(seed)
    R = lambda *s, std=1.0: torch.randn(s, generator=g) * std  # noqa: E731
    W, w = cfg["width"], {}
    M = lambda o, i, std=1.0: R(o, i, std=std * i ** -0.5)  # noqa: E731
    reserved = max([L["mlp"]["router"]["experts"] for L in cfg["layers"] if L["mlp"] and L["mlp"]["kind"] == "moe"] or [0])

    def down(o, i, std=1.0):
        t = M(o, i, std)
        t[W - reserved:] = 0
        return t

    w["embed"], w["head"] = R(cfg["vocab"], W), M(cfg["vocab"], W)
    for t in range(cfg["vocab"]):
        w["embed"][t, W - reserved:] = torch.linspace(-2.0, 2.0, max(reserved, 2))[torch.randperm(max(reserved, 2), generator=g)][:reserved]
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        w[p + "norm1"] = R(W, std=0.2)
        w[p + "norm1"][W - reserved:] = 0
        q = p + "mix."
        if L["type"] == "mamba2":
            inner, c = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            w[q + "in"] = M(inner + c + m["heads"], W)
            w[q + "conv"], w[q + "conv.b"] = R(c, m["conv"], std=m["conv"] ** -0.5), R(c, std=0.2)
            w[q + "dt_bias"], w[q + "A_log"] = R(m["heads"], std=0.5) - 2, R(m["heads"], std=0.5)
            w[q + "D"], w[q + "norm"] = 1 + R(m["heads"], std=0.3), 1 + R(inner, std=0.2)
            w[q + "o"] = down(W, inner, 0.7)
        else:
            a, d = m["left"], m["right"]
            w[q + "left.q"], w[q + "left.k"] = M(a["heads"] * a["dim"], W), M(a["kv_heads"] * a["dim"], W)
            w[q + "left.v"], w[q + "left.o"] = M(a["kv_heads"] * a["vdim"], W), down(W, a["heads"] * a["vdim"], 2.0)
            q += "right."
            for x, n in (("q", d["kv_heads"] * d["dim"]), ("k", d["kv_heads"] * d["dim"]), ("v", d["heads"] * d["vdim"])):
                w[q + x], w[q + x + ".conv"] = M(n, W), R(n, d["conv"], std=d["conv"] ** -0.5)
            w[q + "a"], w[q + "b"] = M(d["heads"], W), M(d["heads"], W)
            w[q + "dt_bias"], w[q + "A_log"] = R(d["heads"], std=0.5) - 3, R(d["heads"], std=0.5)
            w[q + "g"], w[q + "norm"] = M(d["heads"] * d["vdim"], W), 1 + R(d["vdim"], std=0.2)
            w[q + "o"] = down(W, d["heads"] * d["vdim"], 0.7)
        q = p + "mlp."

        def glu(q, ff, bias):
            w[q + "gate"], w[q + "up"], w[q + "down"] = M(ff, W), M(ff, W), down(W, ff)
            if bias:
                w[q + "gate.b"], w[q + "up.b"], w[q + "down.b"] = R(ff, std=0.3), R(ff, std=0.3), R(W, std=0.3)
                w[q + "down.b"][W - reserved:] = 0

        if f and f["kind"] == "dense":
            glu(q, f["ff"], True)
        elif f:
            E = f["router"]["experts"]
            w[q + "router"] = torch.zeros(E, W)
            w[q + "router"][torch.arange(E), W - reserved + torch.randperm(reserved, generator=g)[:E]] = 1.0
            for e in range(E):
                glu(f"{q}e{e}.", f["expert"]["ff"], False)
            if f.get("shared"):
                glu(q + "shared.", f["shared"]["ff"], False)
                w[q + "shared.sg"] = M(1, W)
    w["final.norm"] = R(W, std=0.2)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_DIRS: dict = {}


@pytest.fixture(scope="session")
def models(tmp_path_factory):
    """name -> (checkpoint directory, config, fp64 tensors)"""
    def get(name):
        if name not in _DIRS:
            d, cfg = str(tmp_path_factory.mktemp(f"vugotar-{name}")), CONFIGS[name]
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


def test_mechanisms_against_the_oracle():
    """Each reference op of the product path alone (the kernels are compared with these)."""
    from django_assistant_bot_amd import ops
    from django_assistant_bot_amd.ops import reference_hybrid as ref

    g = torch.Generator().manual_seed(1)
    R = lambda *s: torch.randn(s, generator=g).double()  # noqa: E731
    near = lambda a, b, tol=1e-5: torch.testing.assert_close(a.double(), b.double(), atol=tol, rtol=tol)  # noqa: E731
    # residual sum, bias, expert rows, embedding and the norm over the true width
    x, y, w, bias, table = R(5, 24), R(3, 5, 24), R(20), R(24), R(7, 24)
    pairs, ids = R(10, 24), torch.tensor([1, 0, 6, 2, 2], dtype=torch.int32)
    for t in (x, y, bias, table, pairs):
        t[..., 20:] = 0
    xs, gain = x.float().clone(), torch.cat([1 + w, torch.zeros(4).double()]).float()
    h = ref.rms_residual(xs, y.float(), gain, 20, 1e-3, torch.float32, bias.float(), pairs.float(), ids, table.float())
    want = x + y.sum(0) + bias + pairs.view(5, 2, 24).sum(1) + table[ids.long()]
    near(xs, want)
    near(h[:, :20], oracle.norm(want[:, :20], w, 1e-3))
    # rotary positions, q / k norm, cache write
    H, G, D, dim, rot = 4, 2, 8, 6, 4
    T, bs = 5, 4
    proj = R(T, (H + 2 * G) * D).view(T, H + 2 * G, D)
    proj[:, :H + G, dim:] = 0
    kc, vc = torch.zeros(3, G, bs, D), torch.zeros(3, G, bs, D)
    slots = torch.tensor([4, 5, -1, 8, 9])
    q = ops.qk_rope_write(proj.reshape(T, -1).float(), 0, H, G, D, dim, rot, ops.rope_turns(rot, 50.0, "cpu"), 1e-5, True,
                          torch.arange(T, dtype=torch.int32), slots, kc, vc)
    want = oracle.rms(oracle.rotate(proj[:, :H + G, :dim], rot, 50.0), 1e-5)
    near(q[..., :dim], want[:, :H])
    near(kc[2, :, 1, :dim], want[4, H:])
    near(vc[1, :, 0], proj[0, H + G:])
    assert float(kc[1, :, 2:].abs().sum()) == 0
    # chunked attention with a sink of 1
    n = 11
    k, v, q = R(n, G, D), R(n, G, D), R(n, H, D)
    kc, vc = (c.view(3, bs, G, D).transpose(1, 2).float() for c in (torch.cat([t, torch.zeros(1, G, D)]) for t in (k, v)))
    for chunk in (0, 1, 4, 5, 20):
        out = torch.zeros(n, H * D)
        ops.chunk_prefill(q.float(), kc, vc, torch.tensor([[0, 1, 2]], dtype=torch.int32), torch.tensor([0, n]), torch.tensor([n]),
                          n, 0.7, chunk, torch.zeros(H), out, 0.3)
        for hd in range(H):
            p = oracle.chunk_softmax1(q[:, hd] @ k[:, hd // 2].T * 0.7, chunk)
            near(out.view(n, H, D)[:, hd], 0.3 * p @ v[:, hd // 2])
    # convolution and its ring, in portions
    C, taps = 6, 4
    xin, taps_w, b = R(9, C), R(C, taps), R(C)
    ring, out = torch.zeros(2, taps, C), []
    for a, e in ((0, 2), (2, 3), (3, 9)):
        out.append(ops.short_conv(xin[a:e].float(), 0, taps_w.t().float(), b.float(), ring, torch.tensor([1]),
                                  torch.arange(a, e, dtype=torch.int32), torch.tensor([0, e - a]), e - a))
    near(torch.cat(out), oracle.short_conv(xin, taps_w, b))
    # both recurrences, a portion and then decoded tokens
    H, G, D, V, T = 4, 2, 5, 3, 8
    of = torch.arange(H) // 2
    z, A, dtb, skip = R(T, 2 * H), R(H).exp(), R(H), R(H)
    dt = oracle.softplus(z[:, :H] + dtb)
    c = R(T, 2 * G * D + H * V)
    q, k, v = c[:, :G * D].view(T, G, D), c[:, G * D:2 * G * D].view(T, G, D), c[:, 2 * G * D:].view(T, H, V)
    pos = torch.arange(T, dtype=torch.int32)
    for delta in (True, False):
        d = ops.RecurrentShape(delta, H, G, D, V, c.shape[1], 0, G * D, 2 * G * D, 0, H)
        st = torch.full((3, H, V, d.Dp), 7.0)
        got = [ops.state_scan(c[a:e].float(), d, z[a:e].float(), A.float(), dtb.float(), None if delta else skip.float(), st,
                              torch.tensor([2]), pos[a:e], torch.tensor([0, e - a]), e - a) for a, e in ((0, 5), (5, 6), (6, 8))]
        if delta:
            want, S = oracle.delta_rule(oracle.unit(q)[:, of] * D ** -0.5, oracle.unit(k)[:, of], v, torch.exp(-A * dt),
                                        torch.sigmoid(z[:, H:]))
        else:
            want, S = oracle.ssd_scan(v, k[:, of], q[:, of], dt, A)
            want = want + skip[:, None] * v
        near(torch.cat(got).view(T, H, V), want)
        near(st[2, :, :, :D].transpose(1, 2), S)
        assert float(st[:2].sub(7).abs().sum()) == 0
    # gated norms
    y, gate, wn = R(4, 12), R(4, 12), R(12)
    near(ref.gated_norm(y, gate, 0, 4, True, False, wn, 1e-3, 1.0),
         oracle.rms((y * oracle.silu(gate)).view(4, 3, 4), 1e-3).reshape(4, 12) * wn)
    near(ref.gated_norm(y, gate, 0, 4, False, True, wn[:4], 1e-3, 0.5),
         0.5 * (oracle.rms(y.view(4, 3, 4), 1e-3) * wn[:4]).reshape(4, 12) * oracle.silu(gate))
    # experts
    f = {"router": {"experts": 5, "top": 2, "scale": 1.3}, "expert": {"ff": 8}}
    wm = {"router": R(5, 16)}
    for e in range(5):
        wm.update({f"e{e}.gate": R(8, 16), f"e{e}.up": R(8, 16), f"e{e}.down": R(16, 8)})
    h = R(6, 16)
    idx, wt = ops.moe_route((h @ wm["router"].T).float(), 0, 5, 2, 1.3, 6)
    gu = torch.cat([torch.cat([wm[f"e{e}.gate"], wm[f"e{e}.up"]]) for e in range(5)]).float()
    rows = ops.moe_experts(h.float(), idx, wt, gu, torch.cat([wm[f"e{e}.down"] for e in range(5)]).float(), 5, 0)
    near(rows.view(6, 2, 16).sum(1), oracle.moe(h, f, wm, ""), 1e-4)


def test_the_comparison_sees_every_planted_mistake(models):
    """The oracle with one mistake in it is far outside the tolerance the engine tests use."""
    _, cfg, w = models("uneven")
    toks = prompt(150)
    want = wanted("uneven", cfg, w, toks)
    for mistake in ("chunk", "sink", "qk_norm", "decay", "skip", "router_scale", "loop_add"):
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
        err = error(got, want)
        assert err.max() < TOL[mode[1]], (sizes, int(err.argmax()), float(err.max()))
        eng.release(7)
    assert eng.blocks.num_free_blocks() == eng.blocks.num_blocks()
    assert eng.blocks.num_free_state_slots() == eng.max_batch


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("name", ["uneven", "edge"])
def test_first_tokens_one_by_one(models, name, mode):
    path, cfg, w = models(name)
    toks = prompt(70, 5)
    want = wanted(name, cfg, w, toks)
    eng = engine(path, mode)
    err = error(feed_portions(eng, 0, toks, [1]), want)
    assert err.max() < TOL[mode[1]], int(err.argmax())


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
def test_mixed_batches_reused_pages_and_slots(models, mode):
    """Unequal requests side by side -- portions beside single tokens, requests that pause, a pool just large enough,
    pages and state slots freed and used again by later requests -- against each request alone."""
    path, cfg, w = models("uneven")
    rng = random.Random(11)
    reqs = {i: prompt(rng.choice([1, 2, 63, 64, 65, 129, 180]), 100 + i) for i in range(12)}
    want = {i: wanted("uneven", cfg, w, t) for i, t in reqs.items()}
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
def test_long_decoding_passes_chunks_and_pages(models, mode):
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


def standing_out(chunk, special):
    """A one-layer model in which one token's key stands out for every query, so that whether a query still sees it
    decides the logits."""
    W = 64
    cfg = config(W, [parallel((1, 1, 32, 32, 0.4, chunk, 0), (1, 1, 16, 16, 4), None, (1.0, 0.02))])
    w = tensors(cfg, 3)
    w["embed"] = (torch.randn(VOCAB, W, generator=torch.Generator().manual_seed(2)) * 0.5).to(torch.bfloat16)
    w["embed"][:, :2] = 0
    w["embed"][:, 0] = 2.0
    w["embed"][special, 0], w["embed"][special, 1] = 0.0, 6.0
    for n in ("q", "k"):
        w[f"l0.mix.left.{n}"].mul_(0.2)
    w["l0.mix.left.q"][0].zero_()
    w["l0.mix.left.k"][0].zero_()
    w["l0.mix.left.q"][0, 0] = 8.0  # every query asks for axis 0, which only the special token's key has
    w["l0.mix.left.k"][0, 1] = 8.0
    return cfg, w


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("chunk", [70, 64, 128])
def test_one_key_at_the_chunk_edge(tmp_path, mode, chunk):
    """A query in the special key's chunk copies its value, the first one of the next chunk does not, whether it is in
    a prompt, a portion or decoded, at page borders and inside pages."""
    special = VOCAB - 1
    cfg, w = standing_out(chunk, special)
    write_checkpoint(str(tmp_path), cfg, w)
    wd = {k: v.double() for k, v in w.items()}
    eng = engine(str(tmp_path), mode)
    for k, pos in enumerate((0, chunk - 1, chunk, 2 * chunk - 6)):
        edge = (pos // chunk + 1) * chunk  # the first token of the next chunk
        toks = [t % (VOCAB - 1) for t in prompt(edge + 9, pos)]
        toks[pos] = special
        want = oracle.forward(cfg, wd, toks)
        wrong = oracle.forward(cfg, wd, toks, planted=("chunk",))
        if pos < chunk:
            assert error(wrong[edge:edge + 1], want[edge:edge + 1]) > 3 * TOL[torch.bfloat16]  # the edge decides
        for sizes in ([len(toks)], [edge, 1], [edge - 1, 2, 1], [max(pos, 1), 1] if k else [2, 1]):
            got = feed_portions(eng, pos, toks, sizes)
            e = error(got[edge - 2:edge + 3], want[edge - 2:edge + 3])
            assert e.max() < TOL[mode[1]], (pos, sizes, e)
            eng.release(pos)


@pytest.mark.parametrize("mode", MODES)
def test_a_write_to_the_state_is_read_far_away(models, tmp_path, mode):
    """Decays near one: a token's write is still in every state hundreds of tokens later, across portions."""
    _, cfg, _ = models("uneven")
    w = tensors(cfg, 6)
    for k in w:
        if k.endswith("dt_bias"):
            w[k] = w[k] * 0 - 9
    write_checkpoint(str(tmp_path), cfg, w)
    wd = {k: v.double() for k, v in w.items()}
    toks = prompt(300, 8)
    other = list(toks)
    other[3] = (toks[3] + 1) % VOCAB
    want, moved = oracle.forward(cfg, wd, toks), oracle.forward(cfg, wd, other)
    assert error(moved[-40:], want[-40:]).min() > 10 * TOL[torch.float32]  # token 3 matters at the end
    eng = engine(str(tmp_path), mode)
    for sizes in ([300], [150, 2, 1, 1, 120], [64, 1]):
        assert error(feed_portions(eng, 0, toks, sizes), want).max() < TOL[mode[1]], sizes
        eng.release(0)


@pytest.mark.gpu
def test_one_page_size_more(models):
    path, cfg, w = models("uneven")
    toks = prompt(300, 4)
    want = wanted("uneven", cfg, w, toks)
    eng = engine(path, ("cuda", torch.bfloat16), block_size=128)
    assert error(feed_portions(eng, 0, toks, [100, 150, 1]), want).max() < TOL[torch.bfloat16]


def test_small_pages_on_the_cpu(models):
    path, cfg, w = models("uneven")
    toks = prompt(120, 4)
    want = wanted("uneven", cfg, w, toks)
    for bs in (16, 8):
        eng = engine(path, ("cpu", torch.float32), tokens=256, block_size=bs)
        assert error(feed_portions(eng, 0, toks, [50, 1, 2, 17]), want).max() < TOL[torch.float32]


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
    """A pool too small for the batch: a preempted sequence gives its slot and pages back and starts over.  Prefix reuse,
    asked for, stays off (a slot holds the state of a whole prefix)."""
    path, cfg, w = models("uneven")
    system = prompt(130, 77)
    prompts = [system + prompt(10 + i, i) for i in range(4)]
    sp = SamplingParams(max_new_tokens=60, **GREEDY)
    eng = engine(path, mode, tokens=9 * 64, max_model_len=256, prefix_cache=True)
    for p, o in zip(prompts, eng.generate(prompts, sp)):
        assert len(o.token_ids) == 60
        assert_greedy(oracle, cfg, w, p, o.token_ids, 2 * TOL[mode[1]])
    assert eng.stats["preemptions"] > 0 and eng.blocks.prefix_hits() == 0


def test_abort_and_failure_give_slots_back(models):
    path, _, _ = models("edge")
    eng = engine(path, ("cpu", torch.float32), max_batch=2)
    ids = [eng.add_request(prompt(5, i), SamplingParams(max_new_tokens=50, ignore_eos=True)) for i in range(3)]
    for _ in range(4):
        eng.step()
    assert eng.blocks.num_free_state_slots() == 0
    eng.abort(ids[0])
    assert eng.blocks.num_free_state_slots() == 1
    eng.fail_all()
    assert eng.blocks.num_free_state_slots() == 2


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


def test_sampling_and_string_prompts(models):
    path, _, _ = models("uneven")
    eng = engine(path, ("cpu", torch.float32))
    outs = eng.generate(["hello world", "again"], SamplingParams(max_new_tokens=5, top_k=5, seed=3))
    assert all(len(o.token_ids) == 5 and all(0 <= t < VOCAB for t in o.token_ids) for o in outs)


def test_served_by_the_dialog_provider(models, monkeypatch):
    """The application's in-process provider serves a Vugotar checkpoint directory, JSON mode included."""
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

    out = decoder_bench.run(["tiny-vugotar", "tiny-llama"], prefill=((2, 64),), decode=((2, 100),), iters=2, repeat=1)
    assert [(r["model"], r["metric"].split()[0]) for r in out] == [
        (m, k) for k in ("prefill", "decode") for m in ("tiny-vugotar", "tiny-llama")]
    assert all(r["value"] > 0 for r in out)


# ------------------------------------------------------------------------------------------------ configuration, loading, tools


def test_registry_and_presets():
    from django_assistant_bot_amd.models import VugotarModel, decoder_family, random_vugotar_weights

    cfg = decoder_config("tiny-vugotar")
    assert is_decoder("tiny-vugotar") and decoder_family(cfg).model is VugotarModel
    n = sum(v.numel() for v in random_vugotar_weights(cfg).values())
    assert n >= cfg.params()  # padding only adds
    assert 7.5e9 < decoder_config("vugotar-8b").params() < 8.5e9
    eng = LLMEngine("tiny-vugotar", "cpu", max_batch=2, max_model_len=128, num_blocks=8)
    assert len(eng.generate([[1, 2, 3]], SamplingParams(max_new_tokens=4, ignore_eos=True))[0].token_ids) == 4


def test_parameter_count_is_exact(models):
    for name in CONFIGS:
        path, _, w = models(name)
        assert decoder_config(path).params() == sum(v.numel() for v in w.values()), name


def test_checkpoint_directory(models):
    path, cfg, w = models("uneven")
    c = decoder_config(path)
    assert is_decoder(path) and c.vocab_size == VOCAB and c.layers == 5 and c.loop == (1, 3, 3)
    assert [i for i, _ in c.runs()] == oracle.schedule(cfg)[0]
    assert {r for r, (_, again) in enumerate(c.runs()) if again} == oracle.schedule(cfg)[1]
    assert c.blocks[1].mixer.left.chunk == 37 and c.blocks[2].mlp is None and c.blocks[3].mlp.shared is None


def test_bad_checkpoints_are_refused(models, tmp_path):
    path, cfg, _ = models("uneven")
    w = tensors(cfg)
    for change, what in ((lambda c: c["layers"][0].update(type="other"), "mixer type"),
                         (lambda c: c["layers"][0]["mlp"].update(kind="routed"), "mlp kind"),
                         (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4), "kv_heads"),
                         (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=50), "rotated"),
                         (lambda c: c["layers"][0]["mixer"].update(norm_groups=5), "norm groups"),
                         (lambda c: c["layers"][0]["mixer"].update(state=300), "state rows"),
                         (lambda c: c["layers"][1]["mlp"]["router"].update(top=13), "experts"),
                         (lambda c: c["loop"].update(stop=9), "loop"),
                         (lambda c: c["layers"][0]["mixer"].update(heads=12, vdim=12), "config.json says")):
        c = json.loads(json.dumps(cfg))
        change(c)
        write_checkpoint(str(tmp_path), c, w)
        with pytest.raises(ValueError, match=what):
            LLMEngine(str(tmp_path), "cpu", dtype=torch.float32, max_batch=1, max_model_len=64, num_blocks=4)
    with pytest.raises(ValueError, match="tp_size"):
        LLMEngine("tiny-vugotar", "cpu", tp_size=2)


def test_every_pass_has_its_own_memory(models):
    path, cfg, _ = models("uneven")
    eng = engine(path, ("cpu", torch.float32))
    kv = eng.kv
    assert len(kv.k) == 9 and len({t.data_ptr() for t in kv.state}) == 9
    assert [k is not None for k in kv.k] == [False, True, False, True, False, True, False, True, True]
    assert kv.state[1].shape == (5, 6, 24, 64) and kv.ring[1].shape == (5, 4, 2 * 2 * 40 + 6 * 24)
    assert eng.model.state_bytes(5) == sum(t.numel() * t.element_size() for t in kv.state + kv.ring)
    assert eng.model.cache_bytes_per_block(64) * eng.blocks.num_blocks() == sum(
        t.numel() * t.element_size() for t in kv.k + kv.v if t is not None)


def test_feed_guards(models):
    path, _, _ = models("edge")
    eng = engine(path, ("cpu", torch.float32), tokens=128, max_batch=2)
    eng.feed([(0, [1, 2], []), (1, [3], [])])
    with pytest.raises(RuntimeError, match="live"):
        eng.feed([(2, [1], [0])])
    with pytest.raises(ValueError, match="vocabulary"):
        eng.feed([(0, [VOCAB], [0])])
    with pytest.raises(RuntimeError, match="cache exhausted"):
        eng.feed([(0, [1] * 70, [])])
    eng.release(1)
    assert eng.feed([(3, [4], [0])]).shape == (1, VOCAB)


@pytest.mark.parametrize("mode", MODES)
def test_trace_replay(models, tmp_path, mode, monkeypatch, capsys):
    """The command-line runner: files, order of rows, request names that come back, several requests in a step."""
    import io

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
