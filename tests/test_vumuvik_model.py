"""Vumuvik through the framework (checkpoint loading, engine, paged latents, scheduler, sampling) against the plain
fp64 oracle of tests/vumuvik_oracle.py.  Every engine test runs on the CPU reference ops in 32-bit and, marked gpu,
on the native kernels in 32-bit and bf16."""
import json
import os
import random

import numpy as np
import pytest
import torch
import vumuvik_oracle as oracle
from decoder_helpers import (
    GREEDY,
    MODES,
    TOL,
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


def layer(heads, dim, vdim, rank, window, ff, kv_from=None, scale=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale or dim ** -0.5}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, layers, eps=1e-5, scale=9.0, vocab=VOCAB):
    return {"architecture": "Vumuvik", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "layers": layers}


CONFIGS = {
    # unequal heads / widths / ranks / windows, shared latents read by two layers, a layer without MLP
    "uneven": config(200, [layer(4, 48, 40, 80, 70, 344), layer(3, 64, 64, 80, 33, 200, kv_from=0),
                           layer(2, 16, 24, 80, 128, None, kv_from=0), layer(5, 32, 56, 48, 0, 152)]),
    # window 1 (a token sees itself only), one head, sizes of one tile
    "edge": config(64, [layer(1, 8, 8, 16, 1, 24, scale=1.0), layer(1, 64, 64, 64, 64, 64), layer(2, 64, 32, 64, 65, 64, kv_from=1)],
                   eps=1e-2, scale=1.0),
    # heads and latents wider than the flash / MFMA decode tiles, more heads than one workgroup's 64
    "wide": config(136, [layer(2, 264, 100, 520, 50, 64), layer(70, 16, 16, 24, 90, 72), layer(3, 160, 136, 320, 40, None)]),
    # projection sizes that take the streaming decode GEMM (K % 128) and a split-K of several slabs
    "stream": config(512, [layer(8, 64, 64, 128, 96, 1024), layer(8, 64, 64, 128, 200, 1024, kv_from=0)]),
}


def tensors(cfg, seed=0, share=1.0):
    """Random bf16 tensors of ``cfg`` under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    R = lambda *s, std=1.0: torch.randn(s, generator=g) * std  # noqa: E731
    W, w = cfg["width"], {}

    def norm(name):
        w[name], w[name + ".b"], w[name + ".alpha"] = 1 + R(W, std=0.2), R(W, std=0.2), torch.tensor(0.4) + R(std=0.1)

    w["embed"], w["head"] = R(cfg["vocab"], W, std=0.1), R(cfg["vocab"], W, std=W ** -0.5)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H = m["heads"]
        # queries and keys large enough for peaked attention: a wrong key or a lost sink then shows
        w[p + "mix.q"] = R(H * m["dim"], W, std=2.0 * W ** -0.5)
        if "kv_from" not in m:
            w[p + "mix.dkv"], w[p + "mix.dkv.norm"] = R(m["kv_rank"], W, std=W ** -0.5), 1 + R(m["kv_rank"], std=0.2)
        w[p + "mix.uk"] = R(H * m["dim"], m["kv_rank"], std=1.5 * m["kv_rank"] ** -0.5)
        w[p + "mix.uv"] = R(H * m["vdim"], m["kv_rank"], std=m["kv_rank"] ** -0.5)
        w[p + "mix.sink"] = 2 + R(H, std=0.5)
        w[p + "mix.o"] = R(W, H * m["vdim"], std=2.0 * (H * m["vdim"]) ** -0.5)
        norm(p + "norm1"), norm(p + "norm1b")
        w[p + "ls1"] = 0.8 + R(W, std=0.2)
        if L["mlp"]:
            F = L["mlp"]["ff"]
            w[p + "mlp.gate"], w[p + "mlp.up"] = R(F, W, std=W ** -0.5), R(F, W, std=W ** -0.5)
            w[p + "mlp.down"] = R(W, F, std=2.0 * F ** -0.5)
            norm(p + "norm2"), norm(p + "norm2b")
            w[p + "ls2"] = 0.8 + R(W, std=0.2)
    norm("final.norm")
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_DIRS: dict = {}


@pytest.fixture(scope="session")
def models(tmp_path_factory):
    """name -> (checkpoint directory, config, fp64 tensors)"""
    def get(name):
        if name not in _DIRS:
            d, cfg = str(tmp_path_factory.mktemp(f"vumuvik-{name}")), CONFIGS[name]
            w = tensors(cfg, seed=len(name))
            write_checkpoint(d, cfg, w)
            _DIRS[name] = (d, cfg, {k: v.double() for k, v in w.items()})
        return _DIRS[name]
    return get


# ------------------------------------------------------------------------------------------------ mechanisms


def test_mechanisms_against_the_oracle():
    """Each reference op of the product path alone."""
    from django_assistant_bot_amd.ops import reference as ref

    g = torch.Generator().manual_seed(1)
    R = lambda *s: torch.randn(s, generator=g).double()  # noqa: E731
    x, w, b = R(5, 24), R(24), R(24)
    assert torch.allclose(ref.dyt(x, (0.7, w, b)), oracle.dyt(x, 0.7, w, b))
    # norm, scale, residual, next norm in one op
    y, ls = R(5, 24).float(), R(24).float()
    xs = x.float().clone()
    h = ref.dyt_residual(xs, y, (0.7, w.float(), b.float()), ls, (0.3, b.float(), w.float()), torch.float32)
    want = x + oracle.dyt(y.double(), 0.7, w, b) * ls.double()
    assert torch.allclose(xs.double(), want, atol=1e-5)
    assert torch.allclose(h.double(), oracle.dyt(want, 0.3, b, w), atol=1e-5)
    # latent norm over the true rank although the row is padded
    q_cols, rank = 8, 10
    proj = torch.cat([R(3, q_cols), R(3, rank), torch.zeros(3, 6).double()], 1).float()
    gain, cache = torch.cat([w[:rank], torch.zeros(6).double()]).float(), torch.zeros(2, 4, 16)
    ref.latent_write(proj, q_cols, gain, cache, torch.tensor([5, -1, 0]), rank, 1e-3)
    c = oracle.rms(proj[:, q_cols:q_cols + rank].double(), w[:rank], 1e-3)
    assert torch.allclose(cache[1, 1, :rank].double(), c[0], atol=1e-5) and torch.equal(cache[1, 1, rank:], torch.zeros(6))
    assert torch.allclose(cache[0, 0, :rank].double(), c[2], atol=1e-5) and float(cache[1, 2].abs().sum()) == 0
    # window + sink softmax
    q, k, v, sink = R(6, 2, 4), R(9, 2, 4), R(9, 2, 4), R(2)
    for window in (0, 1, 3, 9):
        got = ref._attend_window(q, k, v, 0.5, window, sink, 3)
        for hd in range(2):
            p = oracle.window_sink_softmax(q[:, hd] @ k[:, hd].T * 0.5, sink[hd], window or 99, 3)
            assert torch.allclose(got[:, hd].double(), p @ v[:, hd], atol=1e-6)
    # gated MLP
    xg, wg, wu, wd = R(4, 16), R(32, 16), R(32, 16), R(16, 32)
    from django_assistant_bot_amd import ops

    gu = ops.interleave_gate_up(wg, wu, 8).float()
    act = ref.gemm_bt(xg.float(), gu, epilogue=ops.EPI_GEGLU8)
    assert torch.allclose((act.double() @ wd.T), oracle.glu(xg, wg, wu, wd), atol=1e-3)


def test_the_comparison_sees_every_planted_mistake(models):
    """The oracle with one mistake in it is far outside the tolerance the engine tests use."""
    _, cfg, w = models("uneven")
    toks = prompt(150)
    want = oracle.forward(cfg, w, toks)
    for mistake in ("window", "sink", "ls", "post_norm"):
        assert error(oracle.forward(cfg, w, toks, planted=(mistake,)), want).max() > 50 * TOL[torch.float32], mistake
    assert error(oracle.forward(cfg, w, toks, planted=("own_latent",)), want).max() > 50 * TOL[torch.float32]


# ------------------------------------------------------------------------------------------------ prompts, portions, decoding


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_portions_and_decoding(models, name, mode):
    path, cfg, w = models(name)
    toks = prompt(210, 3)
    want = oracle.forward(cfg, w, toks)
    eng = engine(path, mode)
    for sizes in ([210], [130, 1], [2], [64], [3, 2, 61, 7, 1, 1, 90]):
        got = feed_portions(eng, 7, toks, sizes)
        err = error(got, want)
        assert err.max() < TOL[mode[1]], (sizes, int(err.argmax()), float(err.max()))
        eng.release(7)
    assert eng.blocks.num_free_blocks() == eng.blocks.num_blocks()


@pytest.mark.parametrize("mode", MODES)
def test_first_tokens_one_by_one(models, mode):
    path, cfg, w = models("edge")
    toks = prompt(70, 5)
    want = oracle.forward(cfg, w, toks)
    eng = engine(path, mode)
    err = error(feed_portions(eng, 0, toks, [1]), want)
    assert err.max() < TOL[mode[1]], int(err.argmax())


@pytest.mark.parametrize("mode", MODES)
def test_layers_match_the_oracle(models, mode):
    path, cfg, w = models("uneven")
    toks, taps, want = prompt(90, 1), [], []
    oracle.forward(cfg, w, toks, trace=want)
    eng = engine(path, mode)
    eng.model.layer_tap = lambda i, x: taps.append(x[:, :cfg["width"]].double().cpu())
    eng.feed([(0, toks, [0])])
    assert len(taps) == len(want)
    for a, b in zip(taps, want):
        assert ((a - b).pow(2).mean() / b.pow(2).mean()).sqrt() < TOL[mode[1]]


@pytest.mark.parametrize("mode", MODES)
def test_mixed_batches_and_reused_pages(models, mode):
    """Unequal requests side by side -- portions beside single tokens, requests that pause, a pool just large
    enough, pages freed and used again by later requests -- against each request alone."""
    path, cfg, w = models("uneven")
    rng = random.Random(11)
    reqs = {i: prompt(rng.choice([1, 2, 63, 64, 65, 129, 180]), 100 + i) for i in range(12)}
    want = {i: oracle.forward(cfg, w, t) for i, t in reqs.items()}
    eng = engine(path, mode, tokens=4 * 192)
    at, todo, live, worst, used = {}, list(reqs), [], 0.0, set()
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
        for i, toks, rows in entries:
            lo = at.get(i, 0)
            e = error(got[o:o + len(toks)], want[i][lo:lo + len(toks)]).max()
            assert e < TOL[mode[1]] * 1.5, (i, lo, len(toks), float(e))
            worst, o = max(worst, float(e)), o + len(toks)
            at[i] = lo + len(toks)
            used.update(eng.blocks.blocks(i))
            if at[i] == len(reqs[i]):
                live.remove(i)
                eng.release(i)
    assert eng.blocks.num_free_blocks() == eng.blocks.num_blocks()
    assert sum(-(-len(t) // 64) for t in reqs.values()) > len(used)  # pages were used again


@pytest.mark.parametrize("mode", MODES)
def test_long_decoding_passes_windows_and_pages(models, mode):
    path, cfg, w = models("stream")
    toks = prompt(330, 9)
    want = oracle.forward(cfg, w, toks)
    eng = engine(path, mode)
    got = [eng.feed([(0, toks[:20], range(20))])]
    got += [eng.feed([(0, toks[t:t + 1], [0])]) for t in range(20, 330)]
    err = error(torch.cat(got), want)
    assert err.max() < TOL[mode[1]], int(err.argmax())
    if mode[0] == "cuda":
        assert eng.stats["graph_replays"] == 310  # decode rows ran from captured graphs


@pytest.mark.parametrize("mode", MODES)
@pytest.mark.parametrize("back", [0, 1])
def test_one_key_at_the_window_edge(tmp_path, mode, back):
    """One token's key stands out for every query.  A query `window` - 1 later still copies its value, one a token later
    does not, whether the query is in a prompt, a portion or decoded -- on a page's border."""
    window, W = 70, 64
    cfg = config(W, [layer(1, 32, 32, 32, window, None)], scale=1.0)
    w = tensors(cfg, 3)
    w["embed"] = (torch.randn(VOCAB, W, generator=torch.Generator().manual_seed(2)) * 0.5).to(torch.bfloat16)
    # the special token's latent points along one axis; every query asks for that axis
    special = VOCAB - 1
    w["embed"][:, :2] = 0
    w["embed"][:, 0] = 2.0
    w["embed"][special, 1] = 2.0
    w["l0.norm1.b"].zero_()
    w["l0.mix.q"].zero_()
    w["l0.mix.q"][0, 0] = 8.0
    w["l0.mix.dkv"][0] = 0
    w["l0.mix.dkv"][0, 1] = 8.0
    w["l0.mix.uk"].zero_()
    w["l0.mix.uk"][0, 0] = 4.0
    w["l0.mix.sink"].zero_()
    write_checkpoint(str(tmp_path), cfg, w)
    wd = {k: v.double() for k, v in w.items()}
    eng = engine(str(tmp_path), mode)
    for pos in (57, 63, 64, 65 - back):
        toks = [t % (VOCAB - 1) for t in prompt(pos + window + 8, pos)]
        toks[pos] = special
        want = oracle.forward(cfg, wd, toks)
        wrong = oracle.forward(cfg, wd, toks, planted=("window",))
        edge = pos + window
        assert error(wrong[edge:edge + 1], want[edge:edge + 1]) > 3 * TOL[torch.bfloat16]  # the edge decides
        for sizes in ([len(toks)], [edge, 1], [edge - 1, 2, 1], [1] if pos == 63 else [edge - back, 1]):
            got = feed_portions(eng, pos, toks, sizes)
            e = error(got[edge - 2:edge + 3], want[edge - 2:edge + 3])
            assert e.max() < TOL[mode[1]], (pos, sizes, e)
            eng.release(pos)


@pytest.mark.gpu
def test_one_page_size_more(models):
    path, cfg, w = models("uneven")
    toks = prompt(300, 4)
    want = oracle.forward(cfg, w, toks)
    eng = engine(path, ("cuda", torch.bfloat16), block_size=128)
    assert error(feed_portions(eng, 0, toks, [100, 150, 1]), want).max() < TOL[torch.bfloat16]


def test_small_pages_on_the_cpu(models):
    path, cfg, w = models("uneven")
    toks = prompt(120, 4)
    want = oracle.forward(cfg, w, toks)
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
        if mode[1] == torch.float32:
            assert o.token_ids == greedy_oracle(oracle, cfg, w, p or [0], n)
        assert_greedy(oracle, cfg, w, p or [0], o.token_ids, 2 * TOL[mode[1]])
    assert eng.blocks.num_free_blocks() == eng.blocks.num_blocks()
    if mixed:
        assert eng.stats["mixed_steps"] > 0


@pytest.mark.parametrize("mode", MODES)
def test_preemption_and_prefix_reuse(models, mode):
    path, cfg, w = models("uneven")
    system = prompt(130, 77)
    prompts = [system + prompt(10 + i, i) for i in range(4)]
    eng = engine(path, mode, tokens=10 * 64, prefix_cache=True, max_model_len=256)
    sp = SamplingParams(max_new_tokens=60, **GREEDY)
    outs = eng.generate(prompts, sp) + eng.generate(prompts[:1], sp)
    assert eng.blocks.prefix_hits() > 0
    for p, o in zip(prompts + prompts[:1], outs):
        assert len(o.token_ids) == 60
        assert_greedy(oracle, cfg, w, p, o.token_ids, 2 * TOL[mode[1]])
    tight = engine(path, mode, tokens=9 * 64, max_model_len=256)
    for p, o in zip(prompts, tight.generate(prompts, sp)):
        assert_greedy(oracle, cfg, w, p, o.token_ids, 2 * TOL[mode[1]])
    assert tight.stats["preemptions"] > 0


@pytest.mark.gpu
def test_graph_replays_match_eager_steps(models):
    """The captured decode step, replayed with the program's own eager work and synchronisations between the
    replays, writes the logits of the eager step."""
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
    """The application's in-process provider serves a Vumuvik checkpoint directory, JSON mode included."""
    import asyncio

    from assistant.ai.providers.transformers import TransformersProvider
    from django_assistant_bot_amd.engine import serving

    path, _, _ = models("uneven")
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

    out = decoder_bench.run(["tiny-vumuvik", "tiny-llama"], prefill=((2, 64),), decode=((2, 100),), iters=2, repeat=1)
    assert [(r["model"], r["metric"].split()[0]) for r in out] == [
        (m, k) for k in ("prefill", "decode") for m in ("tiny-vumuvik", "tiny-llama")]
    assert all(r["value"] > 0 for r in out)


# ------------------------------------------------------------------------------------------------ configuration, loading, tools


def test_registry_and_presets():
    from django_assistant_bot_amd.models import VumuvikModel, decoder_family, random_vumuvik_weights

    cfg = decoder_config("tiny-vumuvik")
    assert is_decoder("tiny-vumuvik") and decoder_family(cfg).model is VumuvikModel
    n = sum(v.numel() for k, v in random_vumuvik_weights(cfg).items() if torch.is_tensor(v))
    assert n >= cfg.params() - 6 * cfg.hidden * len(cfg.blocks)  # padding only adds
    eng = LLMEngine("tiny-vumuvik", "cpu", max_batch=2, max_model_len=128, num_blocks=8)
    assert len(eng.generate([[1, 2, 3]], SamplingParams(max_new_tokens=4, ignore_eos=True))[0].token_ids) == 4


def test_checkpoint_directory(models):
    path, cfg, w = models("uneven")
    c = decoder_config(path)
    assert is_decoder(path) and c.vocab_size == VOCAB and c.layers == 4
    assert [c.source(i) for i in range(4)] == [0, 0, 0, 3]
    assert c.blocks[2].ff is None and c.blocks[3].mixer.window == 0 and c.blocks[1].mixer.window == 33


def test_bad_checkpoints_are_refused(models, tmp_path):
    path, cfg, _ = models("uneven")
    w = tensors(cfg)
    for change, what in ((lambda c: c["layers"][0].update(type="other"), "mixer type"),
                         (lambda c: c["layers"][0]["mlp"].update(kind="routed"), "mlp kind"),
                         (lambda c: c["layers"][1]["mixer"].update(kv_rank=48), "rank"),
                         (lambda c: c["layers"][1]["mixer"].update(kv_from=2), "latent"),
                         (lambda c: c["layers"][0]["mixer"].update(heads=5), "config.json says")):
        c = json.loads(json.dumps(cfg))
        change(c)
        write_checkpoint(str(tmp_path), c, w)
        with pytest.raises(ValueError, match=what):
            LLMEngine(str(tmp_path), "cpu", dtype=torch.float32, max_batch=1, max_model_len=64, num_blocks=4)
    with pytest.raises(ValueError, match="tp_size"):
        LLMEngine("tiny-vumuvik", "cpu", tp_size=2)


def test_shared_latents_share_one_cache(models):
    path, cfg, _ = models("uneven")
    eng = engine(path, ("cpu", torch.float32))
    c = eng.kv.c
    assert c[1] is c[0] and c[2] is c[0] and c[3] is not c[0]
    assert c[0].shape[-1] == 128 and c[3].shape[-1] == 64
    assert eng.model.cache_bytes_per_block(64) == (128 + 64) * 64 * 4


def test_feed_guards(models):
    path, _, _ = models("uneven")
    eng = engine(path, ("cpu", torch.float32), tokens=128, max_batch=2)
    eng.feed([(0, [1, 2], []), (1, [3], [])])
    with pytest.raises(RuntimeError, match="live"):
        eng.feed([(2, [1], [0])])
    with pytest.raises(ValueError, match="vocabulary"):
        eng.feed([(0, [VOCAB], [0])])
    with pytest.raises(RuntimeError, match="cache exhausted"):
        eng.feed([(0, [1] * 70, [])])
    assert eng.feed([]).shape == (0, VOCAB)
    with pytest.raises(RuntimeError, match="prefix"):
        engine(path, ("cpu", torch.float32), prefix_cache=True).feed([(0, [1], [0])])


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


def test_trace_replay_refuses_32_bit_where_there_is_none():
    from django_assistant_bot_amd.engine import trace_replay

    assert trace_replay.main(["--model", "llama-3-8b", "--dtype", "float32", "--out", ".", "--max-tokens", "64",
                              "--device", "cuda:0"]) == 3
