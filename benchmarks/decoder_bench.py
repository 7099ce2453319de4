"""Prefill and decode throughput of decoder presets at the engine's own step functions (random weights).

    python bench.py --decoder-bench vugotar-8b,llama-3-8b [--decoder-shapes ...]

Per model: prefill steps of packed prompts (model forward + last-token logits, as ``LLMEngine._run_prefill``
enqueues them) and decode steps replayed from the engine's HIP graphs (forward + LM head + sampling) at a
fixed context.  Models are measured in turn, ``repeat`` times, and the best time of each is kept.  Prints
one JSON line per (model, shape).
"""
from __future__ import annotations

import json
import random

PREFILL = ((16, 1024), (4, 4096), (1, 8192))  # (prompts, tokens each)
DECODE = ((1, 2048), (16, 2048), (128, 2048), (128, 4096))  # (batch, context)


def _engine(name, max_batch, max_len):
    import torch

    from django_assistant_bot_amd.engine.llm_engine import LLMEngine

    eng = LLMEngine(name, "cuda", max_batch=max_batch, max_model_len=max_len, prefix_cache=False,
                    num_blocks=max_batch * 4224 // 64)
    torch.cuda.synchronize()
    return eng


def _time(fn, iters):
    import torch

    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    fn()
    torch.cuda.synchronize()
    a.record()
    for _ in range(iters):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / iters


def prefill_step(eng, n, length):
    """A closure that runs one packed prefill step of ``n`` fresh prompts."""
    rng = random.Random(0)
    V = eng.cfg.vocab_size
    toks = [[rng.randrange(V) for _ in range(length)] for _ in range(n)]
    for i, t in enumerate(toks):
        assert eng.blocks.add_sequence(i, t, 0) == 0
    ids, cu, meta = eng._prefill_inputs([(i, t, 0, length) for i, t in enumerate(toks)])
    import torch

    last = torch.as_tensor(cu[1:].astype("int64") - 1).cuda()

    def run():
        h = eng.model.forward(ids, meta, eng.kv)
        return eng.model.logits(h.index_select(0, last))
    return run


def decode_step(eng, batch, ctx):
    """A closure that replays the captured decode step of ``batch`` sequences of ``ctx`` tokens."""
    rng = random.Random(1)
    for i in range(batch):
        assert eng.blocks.add_sequence(i, [rng.randrange(eng.cfg.vocab_size) for _ in range(ctx - 1)], 0) == 0
    h = (eng._h_ids, eng._h_pos, eng._h_slots, eng._h_ctx, eng._h_bt)
    # tokens of their own, so that experts are loaded as unequal requests load them
    assert eng.blocks.prepare_decode_into(list(range(batch)), [rng.randrange(eng.cfg.vocab_size) for _ in range(batch)],
                                          eng.max_blocks_per_seq,
                                          *(t.data_ptr() for t in h)) < 0
    eng._decode_logits(batch)
    key = (next(b for b in eng._buckets if b >= batch), True, False)
    if eng.use_graphs:
        return eng._graphs[key].replay
    return lambda: eng._decode_body(batch)


def run(models, prefill=PREFILL, decode=DECODE, iters=20, repeat=3, emit=print):
    import torch

    engines = {m: _engine(m, 128, 8320) for m in models}
    shapes = [("prefill", n, s) for n, s in prefill] + [("decode", n, s) for n, s in decode]
    out = []
    for kind, n, s in shapes:
        best, steps = {}, {}
        for m, eng in engines.items():
            steps[m] = (prefill_step if kind == "prefill" else decode_step)(eng, n, s)
        for _ in range(repeat):
            for m in engines:
                t = _time(steps[m], max(1, iters // 4) if kind == "prefill" else iters)
                best[m] = min(best.get(m, t), t)
        for m, eng in engines.items():
            for i in range(n):
                eng.blocks.free_sequence(i)
            toks = n * s if kind == "prefill" else n
            rec = {"metric": f"{kind} tokens/s", "model": m, "batch": n, "context": s, "value": round(toks / best[m] * 1e3, 1),
                   "unit": "tokens/s", "ms_per_step": round(best[m], 3), "dtype": "bf16", "data": "synthetic (random weights)"}
            out.append(rec)
            emit(json.dumps(rec), flush=True)
        torch.cuda.synchronize()
    return out
