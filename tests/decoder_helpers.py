"""What the decoder-family tests share: small checkpoints, engines of every mode, feeding and comparing."""
import json
import os
import random
import struct

import pytest
import torch

from django_assistant_bot_amd.engine.llm_engine import LLMEngine

VOCAB = 211


def write_checkpoint(path, cfg, w):
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blob = {}, b""
    for k, v in w.items():
        raw = v.contiguous().view(torch.int16).numpy().tobytes()
        head[k] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [len(blob), len(blob) + len(raw)]}
        blob += raw
    h = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + blob)


MODES = [pytest.param(("cpu", torch.float32), id="cpu-f32"),
         pytest.param(("cuda", torch.float32), id="gpu-f32", marks=pytest.mark.gpu),
         pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=pytest.mark.gpu)]
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.5e-2}


def engine(path, mode, tokens=1024, **kw):
    dev, dtype = mode
    kw.setdefault("prefix_cache", False)
    kw.setdefault("max_batch", 4)
    kw.setdefault("max_model_len", tokens)
    bs = kw.setdefault("block_size", 64)
    return LLMEngine(path, dev, dtype=dtype, num_blocks=tokens // bs, **kw)


def error(got, want):
    """rms over the vocabulary of the mean-free difference, per row, over the rms of the wanted logits."""
    d = got.double() - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def prompt(n, seed=0):
    r = random.Random(seed)
    return [r.randrange(VOCAB) for _ in range(n)]


def feed_portions(eng, rid, toks, sizes):
    """Feeds ``toks`` in portions of the given sizes (repeated), every row wanted -> [n, vocab]."""
    out, at, k = [], 0, 0
    while at < len(toks):
        n = min(sizes[k % len(sizes)], len(toks) - at)
        out.append(eng.feed([(rid, toks[at:at + n], range(n))]))
        at, k = at + n, k + 1
    return torch.cat(out)


def greedy_oracle(oracle, cfg, w, toks, n):
    toks = list(toks)
    for _ in range(n):
        toks.append(int(oracle.forward(cfg, w, toks)[-1].argmax()))
    return toks[-n:]


def assert_greedy(oracle, cfg, w, toks, out, tol):
    """Every generated token is the oracle's best, up to ``tol`` of the logit spread (rounding ties)."""
    lg = oracle.forward(cfg, w, list(toks) + list(out))
    for i, t in enumerate(out):
        row = lg[len(toks) - 1 + i]
        assert row.max() - row[t] <= tol * row.std(), (i, float(row.max() - row[t]))


GREEDY = dict(do_sample=False, temperature=0.0, ignore_eos=True)
