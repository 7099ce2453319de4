"""Weight factories: seeded random init with the real shapes, or HF safetensors checkpoints.

Random init is what the benchmarks use (no network, BASELINE.json "random-init weights"); it is
generated directly on the target device, shard by shard for tensor parallelism, so a 70B TP=8 rank
never materialises more than its own ~17.6 GB.  Checkpoint loading maps HF tensor names to the
engine's fused layouts (QKV concatenated, gate/up stacked or interleaved for the fused SwiGLU GEMM)
and slices the tensor-parallel shard of each projection (Megatron column / row split).
"""
from __future__ import annotations

import glob
import math
import os
import re
from dataclasses import dataclass

import torch

from ..ops.selective import state_width

from .configs import (
    BizetarConfig,
    DecoderConfig,
    DenseMlp,
    EncoderConfig,
    MoeMlp,
    ParallelMixer,
    PolyMlp,
    SelectiveMixer,
    VugotarConfig,
    VumuvikConfig,
    VunelixConfig,
    _up,
)

STD = 0.02


def _randn(shape, gen, device, dtype, std=STD):
    t = torch.empty(shape, device=device, dtype=torch.float32)
    t.normal_(0.0, std, generator=gen)
    return t.to(dtype)


def _gen(device, seed):
    g = torch.Generator(device=device)
    g.manual_seed(int(seed))
    return g


def random_encoder_weights(cfg: EncoderConfig, device="cpu", dtype=torch.bfloat16, seed=0) -> dict:
    device = torch.device(device)
    g = _gen(device, seed)
    H, F = cfg.hidden, cfg.intermediate
    ones = lambda n: torch.ones(n, device=device, dtype=dtype)  # noqa: E731
    zeros = lambda n: torch.zeros(n, device=device, dtype=dtype)  # noqa: E731
    w = {
        "word_emb": _randn((cfg.vocab_size, H), g, device, dtype),
        "pos_emb": _randn((cfg.max_position, H), g, device, dtype),
        "type_emb": _randn((cfg.type_vocab, H), g, device, dtype),
        "emb_ln_g": ones(H),
        "emb_ln_b": zeros(H),
    }
    for i in range(cfg.layers):
        w[f"l{i}.qkv_w"] = _randn((3 * H, H), g, device, dtype)
        w[f"l{i}.qkv_b"] = _randn((3 * H,), g, device, dtype)
        w[f"l{i}.o_w"] = _randn((H, H), g, device, dtype)
        w[f"l{i}.o_b"] = _randn((H,), g, device, dtype)
        w[f"l{i}.ln1_g"] = ones(H)
        w[f"l{i}.ln1_b"] = zeros(H)
        w[f"l{i}.i_w"] = _randn((F, H), g, device, dtype)
        w[f"l{i}.i_b"] = _randn((F,), g, device, dtype)
        w[f"l{i}.d_w"] = _randn((H, F), g, device, dtype)
        w[f"l{i}.d_b"] = _randn((H,), g, device, dtype)
        w[f"l{i}.ln2_g"] = ones(H)
        w[f"l{i}.ln2_b"] = zeros(H)
    return w


MLP_GROUP = 8  # gate|up row groups of the fused SwiGLU GEMMs (EPI_SWIGLU8: any 16-row tile holds pairs)


def _mlp_group(interleave_mlp) -> int:
    """``interleave_mlp``: False / 0 = stacked [gate; up], True = the engine's 8-row groups, or an
    explicit group size (8 / 16)."""
    if interleave_mlp is True:
        return MLP_GROUP
    return int(interleave_mlp or 0)


def _gate_up(gate: torch.Tensor, up: torch.Tensor, interleave_mlp) -> torch.Tensor:
    grp = _mlp_group(interleave_mlp)
    if not grp:
        return torch.cat([gate, up], 0)
    Fd, H = gate.shape
    return torch.stack([gate.reshape(Fd // grp, grp, H), up.reshape(Fd // grp, grp, H)], dim=1).reshape(2 * Fd, H)


def random_decoder_weights(cfg: DecoderConfig, device="cpu", dtype=torch.bfloat16, seed=0, tp_rank=0, tp_size=1,
                           interleave_mlp=False) -> dict:
    """Shard `tp_rank` of a seeded random-init decoder.  With tp_size == 1 this is the full model."""
    device = torch.device(device)
    H, F, D = cfg.hidden, cfg.intermediate, cfg.head_dim
    assert cfg.heads % tp_size == 0 and cfg.kv_heads % tp_size == 0 and F % tp_size == 0
    hq, hkv, f = cfg.heads // tp_size, cfg.kv_heads // tp_size, F // tp_size
    # replicated tensors (embedding, LM head) are identical on every rank; the layer shards draw from
    # a per-rank stream (tp_size == 1 keeps the single stream)
    g = _gen(device, seed * 1000003)
    w = {
        "embed": _randn((cfg.vocab_size, H), g, device, dtype),
        "final_norm": torch.ones(H, device=device, dtype=dtype),
    }
    if not cfg.tie_embeddings:
        w["lm_head"] = _randn((cfg.vocab_size, H), g, device, dtype)
    if tp_size > 1:
        g = _gen(device, seed * 1000003 + 1 + tp_rank)
    for i in range(cfg.layers):
        w[f"l{i}.attn_norm"] = torch.ones(H, device=device, dtype=dtype)
        w[f"l{i}.qkv_w"] = _randn(((hq + 2 * hkv) * D, H), g, device, dtype)
        w[f"l{i}.o_w"] = _randn((H, hq * D), g, device, dtype)
        w[f"l{i}.mlp_norm"] = torch.ones(H, device=device, dtype=dtype)
        gate = _randn((f, H), g, device, dtype)
        up = _randn((f, H), g, device, dtype)
        w[f"l{i}.gate_up_w"] = _gate_up(gate, up, interleave_mlp)
        del gate, up
        w[f"l{i}.down_w"] = _randn((H, f), g, device, dtype)
    return w


def shard_decoder_weights(full: dict, cfg: DecoderConfig, tp_rank: int, tp_size: int, interleave_mlp=False) -> dict:
    """Megatron split of a full (stacked gate|up) decoder state: QKV / gate-up by output rows
    (column parallel), O / down by input columns (row parallel)."""
    H, F, D = cfg.hidden, cfg.intermediate, cfg.head_dim
    hq, hkv, f = cfg.heads // tp_size, cfg.kv_heads // tp_size, F // tp_size
    out = {k: v for k, v in full.items() if not re.match(r"l\d+\.", k)}  # embed, final_norm, lm_head
    for i in range(cfg.layers):
        qkv = full[f"l{i}.qkv_w"]
        q = qkv[: cfg.heads * D].view(cfg.heads, D, H)[tp_rank * hq:(tp_rank + 1) * hq].reshape(-1, H)
        k = qkv[cfg.heads * D:(cfg.heads + cfg.kv_heads) * D].view(cfg.kv_heads, D, H)
        v = qkv[(cfg.heads + cfg.kv_heads) * D:].view(cfg.kv_heads, D, H)
        k = k[tp_rank * hkv:(tp_rank + 1) * hkv].reshape(-1, H)
        v = v[tp_rank * hkv:(tp_rank + 1) * hkv].reshape(-1, H)
        out[f"l{i}.qkv_w"] = torch.cat([q, k, v], 0).contiguous()
        out[f"l{i}.o_w"] = full[f"l{i}.o_w"][:, tp_rank * hq * D:(tp_rank + 1) * hq * D].contiguous()
        gu = full[f"l{i}.gate_up_w"]
        gate = gu[:F][tp_rank * f:(tp_rank + 1) * f]
        up = gu[F:][tp_rank * f:(tp_rank + 1) * f]
        out[f"l{i}.gate_up_w"] = _gate_up(gate, up, interleave_mlp).contiguous()
        out[f"l{i}.down_w"] = full[f"l{i}.down_w"][:, tp_rank * f:(tp_rank + 1) * f].contiguous()
        out[f"l{i}.attn_norm"] = full[f"l{i}.attn_norm"]
        out[f"l{i}.mlp_norm"] = full[f"l{i}.mlp_norm"]
    return out


# ------------------------------------------------------------------------------------------------
# HF checkpoints (safetensors only: nothing executable is ever loaded)


class SafetensorsDir:
    """Lazy reader over the ``*.safetensors`` files of a checkpoint (``safe_open``: memory-mapped,
    nothing executable).  ``get`` materialises a whole tensor, ``rows`` / ``cols`` only a slice, so
    a tensor-parallel rank reads about 1/tp of every sharded projection.  ``bytes_read`` counts the
    bytes materialised (tests / logs)."""

    def __init__(self, path: str):
        from safetensors import safe_open

        files = sorted(glob.glob(os.path.join(path, "*.safetensors"))) if os.path.isdir(path) else [path]
        if not files:
            raise FileNotFoundError(f"no .safetensors files under {path}")
        self._handles = [safe_open(f, framework="pt") for f in files]
        self._where = {k: h for h in self._handles for k in h.keys()}
        self.bytes_read = 0

    def keys(self):
        return self._where.keys()

    def __contains__(self, name):
        return name in self._where

    def _count(self, t):
        self.bytes_read += t.numel() * t.element_size()
        return t

    def get(self, name):
        return self._count(self._where[name].get_tensor(name))

    def rows(self, name, a: int, b: int):
        return self._count(self._where[name].get_slice(name)[a:b])

    def cols(self, name, a: int, b: int):
        return self._count(self._where[name].get_slice(name)[:, a:b])


def _read_safetensors(path: str) -> dict:
    st = SafetensorsDir(path)
    return {k: st.get(k) for k in st.keys()}


def load_encoder_checkpoint(path: str, cfg: EncoderConfig, dtype=torch.bfloat16) -> dict:
    st = _read_safetensors(path)
    pre = "bert." if any(k.startswith("bert.") for k in st) else ""
    get = lambda k: st[pre + k].to(dtype)  # noqa: E731
    w = {
        "word_emb": get("embeddings.word_embeddings.weight"),
        "pos_emb": get("embeddings.position_embeddings.weight"),
        "type_emb": get("embeddings.token_type_embeddings.weight"),
        "emb_ln_g": get("embeddings.LayerNorm.weight"),
        "emb_ln_b": get("embeddings.LayerNorm.bias"),
    }
    for i in range(cfg.layers):
        p = f"encoder.layer.{i}."
        w[f"l{i}.qkv_w"] = torch.cat([get(p + f"attention.self.{n}.weight") for n in ("query", "key", "value")], 0)
        w[f"l{i}.qkv_b"] = torch.cat([get(p + f"attention.self.{n}.bias") for n in ("query", "key", "value")], 0)
        w[f"l{i}.o_w"] = get(p + "attention.output.dense.weight")
        w[f"l{i}.o_b"] = get(p + "attention.output.dense.bias")
        w[f"l{i}.ln1_g"] = get(p + "attention.output.LayerNorm.weight")
        w[f"l{i}.ln1_b"] = get(p + "attention.output.LayerNorm.bias")
        w[f"l{i}.i_w"] = get(p + "intermediate.dense.weight")
        w[f"l{i}.i_b"] = get(p + "intermediate.dense.bias")
        w[f"l{i}.d_w"] = get(p + "output.dense.weight")
        w[f"l{i}.d_b"] = get(p + "output.dense.bias")
        w[f"l{i}.ln2_g"] = get(p + "output.LayerNorm.weight")
        w[f"l{i}.ln2_b"] = get(p + "output.LayerNorm.bias")
    return {k: v.contiguous() for k, v in w.items()}


def load_decoder_checkpoint(path: str, cfg: DecoderConfig, dtype=torch.bfloat16, tp_rank=0, tp_size=1,
                            interleave_mlp=False, reader: SafetensorsDir | None = None) -> dict:
    """The rank's tensor-parallel shard of an HF Llama checkpoint, read slice by slice: q / k / v /
    gate / up by output rows (column parallel), o / down by input columns (row parallel), so a rank
    of a 70B TP-8 group materialises ~1/8 of every projection (~17.5 GB) instead of the whole
    140 GB state.  Replicated tensors (embedding, LM head, norms) are read whole.  Same result as
    ``shard_decoder_weights`` of the full state (tests/test_models_cpu.py)."""
    st = reader or SafetensorsDir(path)
    H, F, D = cfg.hidden, cfg.intermediate, cfg.head_dim
    hq, hkv, f = cfg.heads // tp_size, cfg.kv_heads // tp_size, F // tp_size
    cast = lambda t: t.to(dtype).contiguous()  # noqa: E731
    w = {"embed": cast(st.get("model.embed_tokens.weight")), "final_norm": cast(st.get("model.norm.weight"))}
    if not cfg.tie_embeddings:
        w["lm_head"] = cast(st.get("lm_head.weight"))
    r = tp_rank
    for i in range(cfg.layers):
        p = f"model.layers.{i}."
        w[f"l{i}.attn_norm"] = cast(st.get(p + "input_layernorm.weight"))
        w[f"l{i}.mlp_norm"] = cast(st.get(p + "post_attention_layernorm.weight"))
        q = st.rows(p + "self_attn.q_proj.weight", r * hq * D, (r + 1) * hq * D)
        k = st.rows(p + "self_attn.k_proj.weight", r * hkv * D, (r + 1) * hkv * D)
        v = st.rows(p + "self_attn.v_proj.weight", r * hkv * D, (r + 1) * hkv * D)
        w[f"l{i}.qkv_w"] = cast(torch.cat([q, k, v], 0))
        w[f"l{i}.o_w"] = cast(st.cols(p + "self_attn.o_proj.weight", r * hq * D, (r + 1) * hq * D))
        gate = st.rows(p + "mlp.gate_proj.weight", r * f, (r + 1) * f).to(dtype)
        up = st.rows(p + "mlp.up_proj.weight", r * f, (r + 1) * f).to(dtype)
        w[f"l{i}.gate_up_w"] = _gate_up(gate, up, interleave_mlp).contiguous()
        w[f"l{i}.down_w"] = cast(st.cols(p + "mlp.down_proj.weight", r * f, (r + 1) * f))
    return w


# ------------------------------------------------------------------------------------------------
# Vumuvik: the engine's layout from named checkpoint tensors (file or random init)


def _pad(t: torch.Tensor, *shape) -> torch.Tensor:
    """``t`` in the low corner of a zero tensor of ``shape``."""
    if tuple(t.shape) == shape:
        return t
    out = t.new_zeros(shape)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def _vumuvik_layout(cfg: VumuvikConfig, get, device, dtype, interleave_mlp) -> dict:
    """``get(name, shape)`` -> the engine's tensors: projections fused ([q | latent], [K; V] expansion, gate /
    up), every size padded with zeros (``VumuvikConfig.padded_*``), W_uk also per head transposed for the
    absorbed decode queries; gains, biases, scales and sinks in fp32."""
    W, Wp = cfg.hidden, cfg.padded_hidden

    def mat(name, *shape):
        return get(name, shape).to(device=device, dtype=dtype)

    def vec(name, n, pad):
        return _pad(get(name, (n,)).to(device=device, dtype=torch.float32), pad)

    def norm(name):
        return (float(get(name + ".alpha", ())), vec(name, W, Wp), vec(name + ".b", W, Wp))

    w = {"embed": _pad(mat("embed", cfg.vocab_size, W), cfg.vocab_size, Wp),
         "lm_head": _pad(mat("head", cfg.vocab_size, W), cfg.padded_vocab, Wp), "final_norm": norm("final.norm")}
    for i, blk in enumerate(cfg.blocks):
        p, m = f"l{i}.", blk.mixer
        H, D, R = m.heads, cfg.padded_head(i), cfg.padded_rank(i)
        qd = _pad(mat(p + "mix.q", H * m.dim, W).view(H, m.dim, W), H, D, Wp).reshape(H * D, Wp)
        if m.kv_from is None:
            qd = torch.cat([qd, _pad(mat(p + "mix.dkv", m.rank, W), R, Wp)])
            w[p + "latent_norm"] = vec(p + "mix.dkv.norm", m.rank, R)
        w[p + "qd_w"] = qd.contiguous()
        uk = _pad(mat(p + "mix.uk", H * m.dim, m.rank).view(H, m.dim, m.rank), H, D, R)
        uv = _pad(mat(p + "mix.uv", H * m.vdim, m.rank).view(H, m.vdim, m.rank), H, D, R)
        w[p + "kv_w"] = torch.cat([uk.reshape(H * D, R), uv.reshape(H * D, R)])
        w[p + "absorb_w"] = uk.transpose(1, 2).reshape(H * R, D).contiguous()
        w[p + "sink"] = get(p + "mix.sink", (H,)).to(device=device, dtype=torch.float32).contiguous()
        o = mat(p + "mix.o", W, H * m.vdim).view(W, H, m.vdim)
        w[p + "o_w"] = _pad(o, Wp, H, D).reshape(Wp, H * D)
        for n in ("norm1", "norm1b"):
            w[p + n] = norm(p + n)
        w[p + "ls1"] = vec(p + "ls1", W, Wp)
        if blk.ff is not None:
            F = cfg.padded_ff(i)
            w[p + "gate_up_w"] = _gate_up(_pad(mat(p + "mlp.gate", blk.ff, W), F, Wp),
                                          _pad(mat(p + "mlp.up", blk.ff, W), F, Wp), interleave_mlp).contiguous()
            w[p + "down_w"] = _pad(mat(p + "mlp.down", W, blk.ff), Wp, F)
            for n in ("norm2", "norm2b"):
                w[p + n] = norm(p + n)
            w[p + "ls2"] = vec(p + "ls2", W, Wp)
    return w


def _checked(path: str, reader: SafetensorsDir | None):
    """``get(name, shape)`` over a checkpoint directory."""
    st = reader or SafetensorsDir(path)

    def get(name, shape):
        t = st.get(name)
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"{path}: tensor {name} is {tuple(t.shape)}, config.json says {tuple(shape)}")
        return t

    return get


def load_vumuvik_checkpoint(path: str, cfg: VumuvikConfig, device="cpu", dtype=torch.bfloat16, interleave_mlp=False,
                            reader: SafetensorsDir | None = None) -> dict:
    return _vumuvik_layout(cfg, _checked(path, reader), torch.device(device), dtype, interleave_mlp)


def random_vumuvik_tensors(cfg: VumuvikConfig, device="cpu", dtype=torch.bfloat16, seed=0):
    """Seeded ``get(name, shape)`` of a random Vumuvik: fan-in scaled matrices, alphas, gains and scales near
    one half / one, small biases and sinks."""
    g = _gen(torch.device(device), seed * 1000003)

    def get(name, shape):
        if name.endswith(".alpha"):
            return torch.tensor(0.5)
        if len(shape) == 2:
            return _randn(shape, g, device, dtype, std=STD if name in ("embed", "head") else shape[1] ** -0.5)
        t = _randn(shape, g, device, torch.float32, std=0.1)
        return t if name.endswith((".b", ".sink")) else t + 1.0

    return get


def random_vumuvik_weights(cfg: VumuvikConfig, device="cpu", dtype=torch.bfloat16, seed=0, interleave_mlp=False) -> dict:
    device = torch.device(device)
    return _vumuvik_layout(cfg, random_vumuvik_tensors(cfg, device, dtype, seed), device, dtype, interleave_mlp)


# ------------------------------------------------------------------------------------------------
# Vugotar


class Columns:
    """Named blocks of output rows of one fused projection, each starting at a multiple of ``align``."""

    def __init__(self, align: int = 16):
        self.align, self.at, self.width = align, {}, 0

    def add(self, name: str, n: int) -> None:
        self.at[name] = self.width
        self.width = _up(self.width + n, self.align)

    def fill(self, parts: dict, cols: int, total: int, like: torch.Tensor) -> torch.Tensor:
        out = like.new_zeros((total, cols))
        for name, t in parts.items():
            out[self.at[name]:self.at[name] + t.shape[0], :t.shape[1]] = t
        return out


@dataclass(frozen=True)
class HybridLayout:
    """Where things are in a Vugotar layer's fused tensors."""

    inp: Columns  # input projection: mixer columns, the shared expert's [gate | up]
    aux: Columns  # fp32 projection: recurrence gates, router, shared gate
    ff: int  # padded MLP columns at the head of the output projection's input (0: none)
    mix: int  # its column of the recurrent mixer's output, the last block
    width: int  # its columns
    expert_ff: int  # padded expert width
    conv: int  # convolution channels, a multiple of 8


def hybrid_layout(cfg: VugotarConfig, i: int) -> HybridLayout:
    m, f = cfg.blocks[i].mixer, cfg.blocks[i].mlp
    inp, aux = Columns(), Columns(1)
    if isinstance(m, ParallelMixer):
        a, d = m.left, m.right
        inp.add("qkv", (a.heads + 2 * a.kv_heads) * cfg.padded_head(a))
        conv = _up(2 * d.kv_heads * d.dim + d.heads * d.vdim, 8)
        inp.add("conv", conv)
        inp.add("gate", d.heads * d.vdim)
        aux.add("a", d.heads)
        aux.add("b", d.heads)
        attn, rec = a.heads * cfg.padded_head(a), d.heads * d.vdim
    else:
        rec = m.heads * m.vdim
        conv = _up(rec + 2 * m.groups * m.state, 8)
        inp.add("gate", rec)
        inp.add("conv", conv)
        aux.add("a", m.heads)
        attn = 0
    ff = eff = 0
    if isinstance(f, DenseMlp):
        ff = _up(f.ff, 128)
    elif isinstance(f, MoeMlp):
        aux.add("router", f.experts)
        eff = _up(f.ff, 64)
        if f.shared:
            ff = _up(f.shared, 128)
            inp.add("shared", 2 * ff)
            aux.add("sg", 1)
    return HybridLayout(inp, aux, ff, ff + attn, _up(ff + attn + rec, 128), eff, conv)


def _vugotar_layout(cfg: VugotarConfig, get, device, dtype, interleave_mlp) -> dict:
    """``get(name, shape)`` -> the engine's tensors.  Both sublayers of a layer read one norm, so a layer has one input
    projection (``in_w``: attention q | k | v, convolution channels, gates, shared expert), one small fp32 projection
    (``aux_w``: recurrence gates, router logits) and one output projection over the concatenated activations
    [MLP | attention | recurrence] (``out_w``); a dense MLP's [gate | up] stays apart for the fused GLU epilogue.
    Sizes are padded with zeros; gains (1 + w), biases, taps and recurrence constants are fp32."""
    W, Wp = cfg.hidden, cfg.padded_hidden

    def mat(name, *shape):
        return get(name, shape).to(device=device, dtype=dtype)

    def vec(name, *shape):
        return get(name, shape).to(device=device, dtype=torch.float32).contiguous()

    def glu(p, ff, to):
        return _gate_up(_pad(mat(p + "gate", ff, W), to, Wp), _pad(mat(p + "up", ff, W), to, Wp), interleave_mlp)

    w = {"embed": _pad(mat("embed", cfg.vocab_size, W), cfg.vocab_size, Wp),
         "lm_head": _pad(mat("head", cfg.vocab_size, W), cfg.padded_vocab, Wp),
         "final_norm": _pad(1 + vec("final.norm", W), Wp)}
    for i, blk in enumerate(cfg.blocks):
        p, m, f, lay = f"l{i}.", blk.mixer, blk.mlp, hybrid_layout(cfg, i)
        w[p + "norm1"] = _pad(1 + vec(p + "norm1", W), Wp)
        inp, aux, q = {}, {}, p + "mix."
        out = w["embed"].new_zeros((Wp, lay.width))
        if isinstance(m, ParallelMixer):
            a, d, D = m.left, m.right, cfg.padded_head(m.left)
            inp["qkv"] = torch.cat([_pad(mat(q + "left." + n, h * c, W).view(h, c, W), h, D, W).reshape(h * D, W)
                                    for n, h, c in (("q", a.heads, a.dim), ("k", a.kv_heads, a.dim), ("v", a.kv_heads, a.vdim))])
            out[:W, lay.ff:lay.mix] = _pad(mat(q + "left.o", W, a.heads * a.vdim).view(W, a.heads, a.vdim),
                                           W, a.heads, D).reshape(W, a.heads * D)
            q += "right."
            rows = {"q": d.kv_heads * d.dim, "k": d.kv_heads * d.dim, "v": d.heads * d.vdim}
            inp["conv"] = torch.cat([mat(q + n, r, W) for n, r in rows.items()])
            w[p + "conv_w"] = _pad(torch.cat([vec(q + n + ".conv", r, d.conv) for n, r in rows.items()]).t(), d.conv, lay.conv)
            inp["gate"] = mat(q + "g", d.heads * d.vdim, W)
            aux["a"], aux["b"] = mat(q + "a", d.heads, W), mat(q + "b", d.heads, W)
            w[p + "rec_norm"] = vec(q + "norm", d.vdim)
            heads, rec = d.heads, d.heads * d.vdim
        else:
            heads, rec = m.heads, m.heads * m.vdim
            conv = rec + 2 * m.groups * m.state
            full = mat(q + "in", rec + conv + heads, W)
            inp["gate"], inp["conv"], aux["a"] = full[:rec], full[rec:rec + conv], full[rec + conv:]
            w[p + "conv_w"] = _pad(vec(q + "conv", conv, m.conv).t(), m.conv, lay.conv)
            w[p + "conv_b"] = _pad(vec(q + "conv.b", conv), lay.conv)
            w[p + "skip"], w[p + "rec_norm"] = vec(q + "D", heads), vec(q + "norm", rec)
        out[:W, lay.mix:lay.mix + rec] = mat(q + "o", W, rec)
        w[p + "A"] = torch.exp(vec(q + "A_log", heads).double()).float()
        w[p + "dt_bias"] = vec(q + "dt_bias", heads)
        q = p + "mlp."
        if isinstance(f, DenseMlp):
            w[p + "gate_up_w"] = glu(q, f.ff, lay.ff).contiguous()
            w[p + "gate_up_b"] = torch.cat([_pad(vec(q + n + ".b", f.ff), lay.ff) for n in ("gate", "up")])
            out[:W, :f.ff] = mat(q + "down", W, f.ff)
            w[p + "down_b"] = _pad(vec(q + "down.b", W), Wp)
        elif f is not None:
            aux["router"] = mat(q + "router", f.experts, W)
            ex, F = [f"{q}e{e}." for e in range(f.experts)], lay.expert_ff
            w[p + "expert_gate_up_w"] = torch.cat([glu(e, f.ff, F) for e in ex])
            w[p + "expert_down_w"] = torch.cat([_pad(mat(e + "down", W, f.ff), Wp, F) for e in ex])
            if f.shared:
                inp["shared"] = torch.cat([_pad(mat(q + "shared." + n, f.shared, W), lay.ff, W) for n in ("gate", "up")])
                aux["sg"] = mat(q + "shared.sg", 1, W)
                out[:W, :f.shared] = mat(q + "shared.down", W, f.shared)
        w[p + "in_w"] = lay.inp.fill(inp, Wp, _up(lay.inp.width, 128), out)
        w[p + "aux_w"] = lay.aux.fill(aux, Wp, _up(lay.aux.width, 128), out)
        w[p + "out_w"] = out
    return w


def load_vugotar_checkpoint(path: str, cfg: VugotarConfig, device="cpu", dtype=torch.bfloat16, interleave_mlp=False,
                            reader: SafetensorsDir | None = None) -> dict:
    return _vugotar_layout(cfg, _checked(path, reader), torch.device(device), dtype, interleave_mlp)


def random_vugotar_tensors(cfg: VugotarConfig, device="cpu", dtype=torch.bfloat16, seed=0):
    """Seeded ``get(name, shape)`` of a random Vugotar: fan-in scaled matrices, small norm weights around zero, plain
    norms and skips near one, decays between about 0.9 and 0.999 per step."""
    g = _gen(torch.device(device), seed * 1000003)

    def get(name, shape):
        if name.endswith(".conv"):
            return _randn(shape, g, device, torch.float32, std=shape[1] ** -0.5)
        if len(shape) == 2:
            return _randn(shape, g, device, dtype, std=STD if name in ("embed", "head") else shape[1] ** -0.5)
        t = _randn(shape, g, device, torch.float32, std=0.1)
        if name.endswith(".A_log"):
            return t
        if name.endswith(".dt_bias"):
            return t - 4.0
        return t + 1.0 if name.endswith((".D", "mix.norm", "right.norm")) else t

    return get


def random_vugotar_weights(cfg: VugotarConfig, device="cpu", dtype=torch.bfloat16, seed=0, interleave_mlp=False) -> dict:
    device = torch.device(device)
    return _vugotar_layout(cfg, random_vugotar_tensors(cfg, device, dtype, seed), device, dtype, interleave_mlp)


# ------------------------------------------------------------------------------------------------
# Vunelix


@dataclass(frozen=True)
class SelectiveLayout:
    """Padded sizes of a selective-scan layer: channels, state entries, step dimensions; columns of the narrow projection."""

    inner: int
    state: int
    rank: int
    b_col: int
    c_col: int
    narrow: int


def selective_layout(m: SelectiveMixer) -> SelectiveLayout:
    Np, R = state_width(m.state), _up(m.dt_rank, 64)
    return SelectiveLayout(_up(m.inner, 128), Np, R, R, R + Np, R + 2 * Np)


def _vunelix_layout(cfg: VunelixConfig, get, device, dtype, interleave_mlp) -> dict:
    """``get(name, shape)`` -> the engine's tensors.  Scan layers: ``in_w`` [x; z], ``x_w`` (step | input | read-out, the fp32
    projection), ``dt_w``, ``o_w``; attention layers: ``in_w`` [q; latent | rotated key; output gate], ``kv_w`` (K rows, with an
    identity block for a rotated key among their columns, then V rows), ``absorb_w`` (the K rows of every head transposed), ``o_w``.  Sizes
    are padded with zeros; gains, biases, taps and recurrence constants are fp32, decays as -exp(A_log) log2(e)."""
    W, Wp = cfg.hidden, cfg.padded_hidden

    def mat(name, *shape):
        return get(name, shape).to(device=device, dtype=dtype)

    def vec(name, *shape):
        return get(name, shape).to(device=device, dtype=torch.float32).contiguous()

    def glu(p, ff, to):
        return _gate_up(_pad(mat(p + "gate", ff, W), to, Wp), _pad(mat(p + "up", ff, W), to, Wp), interleave_mlp).contiguous()

    def heads(t, H, n, at, D, cols):
        """Rows of H heads of n -> H heads of D, from row ``at`` of each; columns padded to ``cols``."""
        out = t.new_zeros((H, D, cols))
        out[:, at:at + n, :t.shape[1]] = t.view(H, n, t.shape[1])
        return out

    embed = _pad(mat("embed", cfg.vocab_size, W), cfg.vocab_size, Wp)
    w = {"embed": embed, "lm_head": _pad(embed, cfg.padded_vocab, Wp), "final_norm": _pad(vec("final.norm", W), Wp)}
    if cfg.passes:
        mix = mat("loop.in", W, 2 * W)
        w["loop_w"] = torch.stack([_pad(mix[:, :W], Wp, Wp), _pad(mix[:, W:], Wp, Wp)])
        w["loop_step"] = _pad(vec("loop.step", cfg.loop[2], W), cfg.loop[2], Wp)
    for i, blk in enumerate(cfg.blocks):
        p, m, f = f"l{i}.", blk.mixer, blk.mlp
        q = p + "mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ()):
            w[p + n] = _pad(vec(p + n, W), Wp)
        if isinstance(m, SelectiveMixer):
            lay, N, R = selective_layout(m), m.state, m.dt_rank
            I = lay.inner
            w[p + "in_w"] = _pad(mat(q + "in", 2 * m.inner, W).view(2, m.inner, W), 2, I, Wp).reshape(2 * I, Wp)
            w[p + "conv_w"] = _pad(vec(q + "conv", m.inner, m.conv).t(), m.conv, I).contiguous()
            w[p + "conv_b"] = _pad(vec(q + "conv.b", m.inner), I)
            x, xw = mat(q + "x", R + 2 * N, m.inner), embed.new_zeros((_up(lay.narrow, 128), I))
            for at, a, b in ((0, 0, R), (lay.b_col, R, R + N), (lay.c_col, R + N, R + 2 * N)):
                xw[at:at + b - a, :m.inner] = x[a:b]
            w[p + "x_w"] = xw
            w[p + "dt_w"] = _pad(mat(q + "dt", m.inner, R), I, lay.rank)
            w[p + "dt_bias"] = _pad(vec(q + "dt.b", m.inner), I)
            decay = -torch.exp(vec(q + "A_log", m.inner, N).double()) * math.log2(math.e)
            w[p + "A"] = _pad(decay.float(), I, lay.state).contiguous()
            w[p + "skip"] = _pad(vec(q + "D", m.inner), I)
            w[p + "o_w"] = _pad(mat(q + "o", W, m.inner), Wp, I)
        else:
            H, D, R, P = m.heads, m.padded_head(), m.padded_row(), m.rot.dims if m.rot else 0
            V = m.padded_latent()
            full = mat(q + "q", H * (m.dim + P), W).view(H, m.dim + P, W)
            qw = embed.new_zeros((H, D, Wp))
            qw[:, :m.dim, :W] = full[:, :m.dim]
            qw[:, m.q_at:m.q_at + P, :W] = full[:, m.dim:]
            dkv = mat(q + "dkv", m.rank + P, W)
            row = embed.new_zeros((R, Wp))
            row[:m.rank, :W] = dkv[:m.rank]
            row[m.c_at:m.c_at + P, :W] = dkv[m.rank:]
            parts = [qw.reshape(H * D, Wp), row]
            if m.gate:
                parts.append(heads(mat(q + "g", H * m.vdim, W), H, m.vdim, 0, D, Wp).reshape(H * D, Wp))
            fused = torch.cat(parts)
            w[p + "in_w"] = _pad(fused, _up(fused.shape[0], 256 if fused.shape[0] > 2048 else 128), Wp)
            w[p + "latent_norm"] = _pad(vec(q + "dkv.norm", m.rank), R)
            uk = heads(mat(q + "uk", H * m.dim, m.rank), H, m.dim, 0, D, R)
            for k in range(P):  # the rotated key part passes through
                uk[:, m.q_at + k, m.c_at + k] = 1.0
            uv = heads(mat(q + "uv", H * m.vdim, m.rank), H, m.vdim, 0, D, V)
            w[p + "kv_w"] = torch.cat([uk[:, :, :V].reshape(H * D, V), uv.reshape(H * D, V)])
            w[p + "absorb_w"] = uk.transpose(1, 2).reshape(H * R, D).contiguous()
            w[p + "o_w"] = _pad(mat(q + "o", W, H * m.vdim).view(W, H, m.vdim), Wp, H, D).reshape(Wp, H * D)
        q = p + "mlp."
        if isinstance(f, DenseMlp):
            F = _up(f.ff, 128)
            w[p + "gate_up_w"], w[p + "down_w"] = glu(q, f.ff, F), _pad(mat(q + "down", W, f.ff), Wp, F)
        elif f is not None:
            w[p + "router_w"] = _pad(mat(q + "router", f.experts, W), _up(f.experts, 128), Wp)
            ex, F = [f"{q}e{e}." for e in range(f.experts)], _up(f.ff, 64)
            w[p + "expert_gate_up_w"] = torch.cat([glu(e, f.ff, F) for e in ex])
            w[p + "expert_down_w"] = torch.cat([_pad(mat(e + "down", W, f.ff), Wp, F) for e in ex])
            if f.shared:
                F = _up(f.shared, 128)
                w[p + "gate_up_w"] = glu(q + "shared.", f.shared, F)
                w[p + "down_w"] = _pad(mat(q + "shared.down", W, f.shared), Wp, F)
    return w


def load_vunelix_checkpoint(path: str, cfg: VunelixConfig, device="cpu", dtype=torch.bfloat16, interleave_mlp=False,
                            reader: SafetensorsDir | None = None) -> dict:
    return _vunelix_layout(cfg, _checked(path, reader), torch.device(device), dtype, interleave_mlp)


def random_vunelix_tensors(cfg: VunelixConfig, device="cpu", dtype=torch.bfloat16, seed=0):
    """Seeded ``get(name, shape)`` of a random Vunelix: fan-in scaled matrices, norms and skips near one, small biases, decays
    between about 0.9 and 0.999 per step."""
    g = _gen(torch.device(device), seed * 1000003)

    def get(name, shape):
        if name.endswith(".conv"):
            return _randn(shape, g, device, torch.float32, std=shape[1] ** -0.5)
        if name.endswith(".A_log"):
            return _randn(shape, g, device, torch.float32, std=0.1)
        if len(shape) == 2 and name != "loop.step":
            return _randn(shape, g, device, dtype, std=STD if name == "embed" else shape[1] ** -0.5)
        t = _randn(shape, g, device, torch.float32, std=0.1)
        if name.endswith(".dt.b"):
            return t - 4.0
        return t if name == "loop.step" or name.endswith(".conv.b") else t + 1.0

    return get


def random_vunelix_weights(cfg: VunelixConfig, device="cpu", dtype=torch.bfloat16, seed=0, interleave_mlp=False) -> dict:
    device = torch.device(device)
    return _vunelix_layout(cfg, random_vunelix_tensors(cfg, device, dtype, seed), device, dtype, interleave_mlp)


# ------------------------------------------------------------------------------------------------
# Bizetar


def bizetar_columns(cfg: BizetarConfig, i: int) -> Columns:
    """Output rows of a layer's input projection: queries, keys and values, output gate, gate of the mixer's result."""
    m, inp = cfg.blocks[i].mixer, Columns()
    inp.add("qkv", (m.heads + 2 * m.kv_heads) * m.padded_head())
    inp.add("g", m.heads * (m.padded_head() if m.gate == "element" else 1))
    inp.add("rg", cfg.padded_hidden)
    return inp


def _bizetar_layout(cfg: BizetarConfig, get, device, dtype, interleave_mlp) -> dict:
    """``get(name, shape)`` -> the engine's tensors.  Everything that reads a sublayer's input is one projection: ``in_w``
    (``bizetar_columns``) for the mixer, ``up_w`` [up; gate of the result] or, with experts, ``rg_w`` (the gate alone) beside
    the fp32 ``router_w``.  Sizes are padded with zeros; gains (``qk_norm``: of every query and key head), biases, taps,
    sinks and the weights over depth are fp32; single numbers are floats."""
    W, Wp = cfg.hidden, cfg.padded_hidden

    def mat(name, *shape):
        return get(name, shape).to(device=device, dtype=dtype)

    def vec(name, *shape):
        return get(name, shape).to(device=device, dtype=torch.float32).contiguous()

    def glu(p, ff, to):
        return _gate_up(_pad(mat(p + "gate", ff, W), to, Wp), _pad(mat(p + "up", ff, W), to, Wp), interleave_mlp).contiguous()

    embed = _pad(mat("embed", cfg.vocab_size, W), cfg.vocab_size, Wp)
    w = {"embed": embed, "embed_norm": _pad(vec("embed.norm", W), Wp),
         "lm_head": _pad(mat("head", cfg.vocab_size, W), cfg.padded_vocab, Wp), "final_norm": _pad(vec("final.norm", W), Wp)}
    for i, blk in enumerate(cfg.blocks):
        p, m, f = f"l{i}.", blk.mixer, blk.mlp
        q, H, G, D = p + "mix.", m.heads, m.kv_heads, m.padded_head()
        parts = (("q", H, m.dim), ("k", G, m.dim), ("v", G, m.vdim))

        def heads(of, cols):  # rows of every q, k and v head, each padded to D
            return torch.cat([_pad(of(n, h * d).view(h, d, cols), h, D, cols).reshape(h * D, cols) for n, h, d in parts])

        inp = bizetar_columns(cfg, i)
        rows = {"qkv": heads(lambda n, r: mat(q + n, r, W), W), "rg": mat(p + "rg1", W, W)}
        if m.gate == "element":
            rows["g"] = _pad(mat(q + "g", H * m.vdim, W).view(H, m.vdim, W), H, D, W).reshape(H * D, W)
        else:
            rows["g"] = mat(q + "g", H, W)
        w[p + "in_w"] = inp.fill(rows, Wp, _up(inp.width, 256 if inp.width > 2048 else 128), embed)
        if m.bias:
            w[p + "qkv_b"] = heads(lambda n, r: vec(q + n + ".b", r), 1).view(-1).contiguous()
        if m.conv:
            w[p + "conv_w"] = heads(lambda n, r: vec(q + n + ".conv", r, m.conv), m.conv).t().contiguous()
        if m.norm == "whole":
            gains = [_pad(vec(q + n + ".norm", h * m.dim).view(h, m.dim), h, D) for n, h in (("q", H), ("k", G))]
        else:
            gains = [_pad(vec(q + n + ".norm", m.dim), D).expand(h, D) for n, h in (("q", H), ("k", G))]
        w[p + "qk_norm"] = torch.cat(gains).reshape(-1).contiguous()
        w[p + "sink"] = vec(q + "sink", H)
        if m.slopes:
            w[p + "slopes"] = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=torch.float32, device=device)
        if m.v_mix:
            w[p + "vmix"] = float(get(q + "vmix", ()))
        w[p + "o_w"] = _pad(mat(q + "o", W, H * m.vdim).view(W, H, m.vdim), Wp, H, D).reshape(Wp, H * D)
        w[p + "norm1"], w[p + "rg1_b"] = _pad(vec(p + "norm1", W), Wp), _pad(vec(p + "rg1.b", W), Wp)
        w[p + "depth"] = vec(p + "dwa", i + 2)
        if f is None:
            continue
        w[p + "norm2"], w[p + "rg2_b"] = _pad(vec(p + "norm2", W), Wp), _pad(vec(p + "rg2.b", W), Wp)
        gate = _pad(mat(p + "rg2", W, W), Wp, Wp)
        q = p + "mlp."
        if isinstance(f, PolyMlp):
            F = _up(f.ff, 128)
            w[p + "up_w"] = torch.cat([_pad(mat(q + "up", f.ff, W), F, Wp), gate])
            w[p + "down_w"] = _pad(mat(q + "down", W, f.ff), Wp, F)
            w[p + "act"] = tuple(float(x) for x in get(q + "act", (4,)))
        else:
            w[p + "rg_w"] = gate
            w[p + "router_w"] = _pad(mat(q + "router", f.outputs, W), _up(f.outputs, 128), Wp)
            w[p + "correction"] = vec(q + "correction", f.outputs)
            ex, F = [f"{q}e{e}." for e in range(f.experts)], _up(f.ff, 64)
            w[p + "expert_gate_up_w"] = torch.cat([glu(e, f.ff, F) for e in ex])
            w[p + "expert_down_w"] = torch.cat([_pad(mat(e + "down", W, f.ff), Wp, F) for e in ex])
    return w


def load_bizetar_checkpoint(path: str, cfg: BizetarConfig, device="cpu", dtype=torch.bfloat16, interleave_mlp=False,
                            reader: SafetensorsDir | None = None) -> dict:
    return _bizetar_layout(cfg, _checked(path, reader), torch.device(device), dtype, interleave_mlp)


def random_bizetar_tensors(cfg: BizetarConfig, device="cpu", dtype=torch.bfloat16, seed=0):
    """Seeded ``get(name, shape)`` of a random Bizetar: fan-in scaled matrices, norms near one, small biases and sinks, weights
    over depth that keep most of the newest result."""
    g = _gen(torch.device(device), seed * 1000003)

    def get(name, shape):
        if name.endswith(".vmix"):
            return torch.tensor(0.3)
        if name.endswith(".act"):
            return torch.tensor([0.8, 0.4, 0.3, 0.1])
        if name.endswith(".dwa"):
            t = _randn(shape, g, device, torch.float32, std=0.2 / shape[0])
            t[-1] += 0.9
            return t
        if name.endswith(".conv"):
            return _randn(shape, g, device, torch.float32, std=shape[1] ** -0.5)
        if len(shape) == 2:
            return _randn(shape, g, device, dtype, std=STD if name in ("embed", "head") else shape[1] ** -0.5)
        t = _randn(shape, g, device, torch.float32, std=0.1)
        if name.endswith(".correction"):
            return t / shape[0]
        return t if name.endswith((".b", ".sink")) else t + 1.0

    return get


def random_bizetar_weights(cfg: BizetarConfig, device="cpu", dtype=torch.bfloat16, seed=0, interleave_mlp=False) -> dict:
    device = torch.device(device)
    return _bizetar_layout(cfg, random_bizetar_tensors(cfg, device, dtype, seed), device, dtype, interleave_mlp)
