"""Model shape presets (public architecture configs) for the encoder and decoder families.

The reference names models by HF hub id (gpu_service/models.py:1-9, settings EMBEDDING_AI_MODEL /
DIALOG_*_AI_MODEL); the engine resolves the same ids (and short aliases) to these presets, builds
random-init weights of the exact shapes (benchmarks) or loads safetensors checkpoints when a local
directory is given.
"""
from __future__ import annotations

import json
import math
import os
from dataclasses import asdict, dataclass, field, replace


@dataclass(frozen=True)
class EncoderConfig:
    name: str
    vocab_size: int = 30522
    hidden: int = 768
    layers: int = 12
    heads: int = 12
    intermediate: int = 3072
    max_position: int = 512
    type_vocab: int = 2
    eps: float = 1e-12
    normalize: bool = False  # reference mean-pools and does NOT L2-normalise (embedders/transformers.py:25)

    @property
    def head_dim(self) -> int:
        return self.hidden // self.heads

    def to_dict(self):
        return asdict(self)


@dataclass(frozen=True)
class DecoderConfig:
    name: str
    vocab_size: int = 128256
    hidden: int = 4096
    layers: int = 32
    heads: int = 32
    kv_heads: int = 8
    intermediate: int = 14336
    rope_theta: float = 500000.0
    rope_scaling: dict | None = field(default_factory=lambda: {
        "factor": 8.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0, "original_max_position_embeddings": 8192})
    eps: float = 1e-5
    max_position: int = 8192
    bos_id: int = 128000
    eos_ids: tuple = (128001, 128009)
    tie_embeddings: bool = False

    @property
    def head_dim(self) -> int:
        return self.hidden // self.heads

    def to_dict(self):
        return asdict(self)

    def params(self) -> int:
        H, F, V, L = self.hidden, self.intermediate, self.vocab_size, self.layers
        D = self.head_dim
        attn = H * (self.heads * D) + 2 * H * (self.kv_heads * D) + (self.heads * D) * H
        mlp = 3 * H * F
        emb = V * H * (1 if self.tie_embeddings else 2)
        return L * (attn + mlp + 2 * H) + emb + H


# ------------------------------------------------------------------ latent-attention decoders (Vumuvik)

# cached row widths of the MFMA decode kernel, and rows of (width, latent part) whose rest is a rotated key
LATENT_TILES = (64, 128, 192, 256, 384, 512)
ROTARY_TILES = ((320, 256), (576, 512))


def _up(n: int, m: int) -> int:
    return -(-n // m) * m


@dataclass(frozen=True)
class Yarn:
    """YaRN scaling of rotary frequencies: divided by ``factor`` where a pair turns fewer than ``slow`` times in ``original``
    positions, as they are where it turns more than ``fast`` times, a ramp over the pairs between."""

    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class Rotary:
    """Rotary positions on ``dims`` dimensions, neighbours (2i, 2i + 1) being a pair."""

    dims: int
    base: float = 10000.0
    scaling: Yarn | None = None

    @property
    def gain(self) -> float:
        """Factor on cosine and sine."""
        return 1.0 if self.scaling is None else 0.1 * math.log(self.scaling.factor) + 1.0


@dataclass(frozen=True)
class LatentMixer:
    """One latent-attention mixer: every head's keys and values are images of one ``rank``-wide latent.  With ``rot`` a
    head also has ``rot.dims`` rotated query dimensions, which meet one rotated key part that all heads share."""

    heads: int
    dim: int  # query / key width of a head
    vdim: int  # value width of a head
    rank: int
    scale: float
    window: int = 0  # keys a query sees, itself included (0: all before it)
    kv_from: int | None = None  # layer whose cached latent this mixer reads (None: its own)
    rot: Rotary | None = None
    gate: bool = False  # the heads' output is multiplied with the sigmoid of a projection of the layer's input

    # where the rotated parts start in a head and in a cached row (multiples of 8), and the widths up to their ends
    @property
    def q_at(self) -> int:
        return _up(self.dim, 8)

    @property
    def c_at(self) -> int:
        return _up(self.rank, 8)

    @property
    def head_width(self) -> int:
        return max(self.q_at + self.rot.dims if self.rot else self.dim, self.vdim)

    @property
    def row_width(self) -> int:
        return self.c_at + self.rot.dims if self.rot else self.rank

    def padded_head(self) -> int:
        """Common padded width of the query / key and value heads."""
        return next((p for p in (64, 128, 256) if self.head_width <= p), _up(self.head_width, 64))

    def padded_row(self) -> int:
        """Padded width of a cached row: a tile of the MFMA decode kernel where one fits."""
        tiles = LATENT_TILES if self.rot is None else sorted(LATENT_TILES + tuple(r for r, _ in ROTARY_TILES))
        values = dict(ROTARY_TILES)
        return next((p for p in tiles if self.row_width <= p and self.rank <= values.get(p, p)), _up(self.row_width, 64))

    def padded_latent(self) -> int:
        """Columns of a cached row that values come from (all of them where latent and rotated key share a tile)."""
        return dict(ROTARY_TILES).get(self.padded_row(), self.padded_row()) if self.rot else self.padded_row()


@dataclass(frozen=True)
class LatentLayer:
    mixer: LatentMixer
    ff: int | None  # hidden width of the gated MLP (None: the layer has no feed-forward)


@dataclass(frozen=True)
class VumuvikConfig:
    """Vumuvik decoder: latent attention (window + sink) and tanh-GELU MLPs between Dynamic-Tanh norms,
    layer scales, no positions.  The ``padded_*`` sizes are what the kernels see: padding is zeros in
    weights, gains and biases, so it never reaches a result."""

    name: str
    vocab_size: int
    hidden: int
    blocks: tuple  # of LatentLayer
    eps: float
    embed_scale: float = 1.0
    max_position: int = 1 << 20  # no positional table: only the cache bounds a sequence
    default_model_len: int = 8192  # engine default when max_model_len is not given
    bos_id: int = 0
    eos_ids: tuple = ()

    def __post_init__(self):
        for i, b in enumerate(self.blocks):
            src = b.mixer.kv_from
            if src is not None:
                j = self.source(i)
                if self.blocks[j].mixer.rank != b.mixer.rank:
                    raise ValueError(f"{self.name}: layer {i} reads the latent of layer {j}, whose rank differs")

    @property
    def layers(self) -> int:
        return len(self.blocks)

    def source(self, i: int) -> int:
        """The layer whose latent layer ``i`` reads (itself, or through ``kv_from``)."""
        src = self.blocks[i].mixer.kv_from
        if src is None:
            return i
        if not 0 <= src < i or self.blocks[src].mixer.kv_from is not None:
            raise ValueError(f"{self.name}: layer {i} takes its latent from layer {src}, which has none of its own")
        return src

    @property
    def padded_hidden(self) -> int:
        return _up(self.hidden, 64)

    @property
    def padded_vocab(self) -> int:
        return _up(self.vocab_size, 128)

    def padded_head(self, i: int) -> int:
        return self.blocks[i].mixer.padded_head()

    def padded_rank(self, i: int) -> int:
        return self.blocks[i].mixer.padded_row()

    def padded_ff(self, i: int) -> int:
        return _up(self.blocks[i].ff, 64)

    def to_dict(self):
        return asdict(self)

    def params(self) -> int:
        n = 2 * self.vocab_size * self.hidden + 2 * self.hidden + 1
        for b in self.blocks:
            m, H = b.mixer, self.hidden
            n += m.heads * m.dim * (H + m.rank) + m.heads * m.vdim * (m.rank + H) + m.heads + 5 * H + 2
            n += (H + 1) * m.rank if m.kv_from is None else 0
            n += 3 * H * b.ff + 5 * H + 2 if b.ff else 0
        return n


def vumuvik_uniform(name: str, layers: int, vocab_size: int, hidden: int, ff: int, heads: int, dim: int, rank: int,
                    window: int, share: int = 2, vdim: int | None = None, **kw) -> VumuvikConfig:
    """A Vumuvik of equal layers in which groups of ``share`` consecutive layers read one latent."""
    blocks = tuple(LatentLayer(LatentMixer(heads, dim, vdim or dim, rank, dim ** -0.5, window,
                                           None if i % share == 0 else i - i % share), ff) for i in range(layers))
    return VumuvikConfig(name, vocab_size, hidden, blocks, kw.pop("eps", 1e-6), kw.pop("embed_scale", hidden ** 0.5), **kw)


# ------------------------------------------------------------------ hybrid decoders (Vugotar)


@dataclass(frozen=True)
class ChunkedMixer:
    """Softmax attention inside chunks of positions, with a sink of score 0 in every head's denominator."""

    heads: int
    kv_heads: int
    dim: int  # query / key width of a head
    vdim: int
    scale: float
    chunk: int = 0  # positions of a chunk (0: one chunk)
    rot_dims: int = 0  # rotated dimensions, interleaved pairs
    rot_base: float = 10000.0


@dataclass(frozen=True)
class DeltaMixer:
    """Gated delta rule: a dim x vdim state per head, q / k heads shared by groups of value heads."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int  # taps of the short convolution


@dataclass(frozen=True)
class ParallelMixer:
    """Both mixers read the layer's input; the result is the scaled sum of their outputs."""

    left: ChunkedMixer
    right: DeltaMixer
    left_scale: float = 1.0
    right_scale: float = 1.0


@dataclass(frozen=True)
class Mamba2Mixer:
    """State-space duality: a state x vdim state per head, B / C shared by groups of heads."""

    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int = 1


@dataclass(frozen=True)
class SelectiveMixer:
    """Mamba's selective scan: a diagonal state of ``state`` entries per channel; step, input and read-out are projections
    of the convolved channels, the step through ``dt_rank`` dimensions."""

    inner: int
    state: int
    dt_rank: int
    conv: int  # taps of the short convolution


@dataclass(frozen=True)
class QueryTemp:
    """Queries at position p are multiplied by 1 + coef ln(floor((p + 1) / every) + 1)."""

    coef: float
    every: int


@dataclass(frozen=True)
class SinkMixer:
    """Softmax attention over per-head keys and values, with a learned sink per head in the denominator and a sigmoid gate on
    the output.  What positions do is said by ``rot`` (rotation), ``temp`` (query temperature) and ``slopes`` (every head
    takes slope * distance off its scores)."""

    heads: int
    kv_heads: int
    dim: int  # query / key width of a head
    vdim: int
    scale: float
    norm: str = "head"  # RMS norm of q and k, with weights: "head" (each head, shared weights) or "whole" (all rows at once)
    gate: str = "element"  # output gate: a number per "element" or per "head"
    bias: bool = False  # q, k and v have biases
    conv: int = 0  # taps of the short causal convolution on q, k and v (0: none)
    rot: Rotary | None = None
    temp: QueryTemp | None = None
    slopes: bool = False
    v_mix: bool = False  # values are mixed with those of the first layer that says so

    def padded_head(self) -> int:
        """Common padded width of the query / key and value heads."""
        d = max(self.dim, self.vdim)
        return next((p for p in (64, 128, 256) if d <= p), _up(d, 64))


@dataclass(frozen=True)
class PolyMlp:
    """Ungated MLP with PolyNorm: a combination of the normalised first three powers of the hidden values."""

    ff: int


@dataclass(frozen=True)
class DenseMlp:
    """Gated MLP (in a Vugotar with biases on all three projections)."""

    ff: int
    act: str = "silu"


@dataclass(frozen=True)
class MoeMlp:
    """``top`` of ``experts`` SwiGLUs per token plus, with ``shared``, one that every token runs (in a Vugotar behind a
    sigmoid gate).  ``scores``: of the router, "softmax" (weights over their sum), "softmax_raw" or "sigmoid" (weights as they
    are); ``weigh``: what the weight multiplies, the expert's "output" or its "input".  ``correction``: a number per expert
    joins its score where the experts are chosen, not in the weight.  ``identity``: further router outputs whose expert is the
    layer's input itself."""

    experts: int
    top: int
    scale: float
    ff: int
    shared: int | None = None
    scores: str = "softmax"
    weigh: str = "output"
    correction: bool = False
    identity: int = 0

    @property
    def outputs(self) -> int:
        """Router outputs."""
        return self.experts + self.identity


def _check_moe(where: str, f, max_experts: int = 1024, max_top: int = 64) -> None:
    if isinstance(f, MoeMlp) and (not 1 <= f.top <= min(f.outputs, max_top) or f.outputs > max_experts):
        raise ValueError(f"{where}: experts up to {max_experts}, of which up to {max_top} per token")


def loop_runs(layers: int, loop: tuple | None) -> list:
    """(layer, pass that starts right before it or None) of every layer run, in order; ``loop`` = (start, stop, times)."""
    a, b, t = loop or (0, 0, 1)
    if a == b:
        return [(i, None) for i in range(layers)]
    return ([(i, None) for i in range(a)]
            + [(i, k if i == a else None) for k in range(t) for i in range(a, b)]
            + [(i, None) for i in range(b, layers)])


def _check_loop(name: str, layers: int, loop: tuple | None) -> None:
    if loop is not None:
        a, b, t = loop
        if not 0 <= a <= b <= layers or t < 1:
            raise ValueError(f"{name}: loop {loop} outside the layers")


@dataclass(frozen=True)
class HybridLayer:
    """A mixer and a feed-forward.  Vugotar: x + mixer(norm(x)) + mlp(norm(x)), one norm that both read.  Vunelix: a norm
    before and after each of the two.  Bizetar: a gate and a norm after each."""

    mixer: ParallelMixer | Mamba2Mixer | SelectiveMixer | LatentMixer | SinkMixer
    mlp: DenseMlp | MoeMlp | PolyMlp | None = None


@dataclass(frozen=True)
class VugotarConfig:
    """Vugotar decoder: hybrid layers, of which ``loop`` = (start, stop, times) runs a stretch several times with the
    same weights (every pass with its own cache and state; the embedding is added again before each pass but the
    first).  The ``padded_*`` sizes are what the kernels see; padding is zeros."""

    name: str
    vocab_size: int
    hidden: int
    blocks: tuple  # of HybridLayer
    eps: float = 1e-5
    loop: tuple | None = None
    max_position: int = 1 << 20  # no positional table: only the cache bounds a sequence
    default_model_len: int = 8192
    bos_id: int = 0
    eos_ids: tuple = ()

    MAX_STATE_ROWS, MAX_TAPS, MAX_HEAD, MAX_EXPERTS, MAX_TOP = 256, 16, 1024, 1024, 64  # of the kernels

    def __post_init__(self):
        for i, b in enumerate(self.blocks):
            where = f"{self.name}: layer {i}"
            m, f = b.mixer, b.mlp
            if isinstance(m, ParallelMixer):
                a, d = m.left, m.right
                if a.heads % a.kv_heads or d.heads % d.kv_heads:
                    raise ValueError(f"{where}: heads must be whole groups of kv_heads")
                if a.rot_dims % 2 or a.rot_dims > a.dim or max(a.dim, a.vdim) > self.MAX_HEAD:
                    raise ValueError(f"{where}: rotated dimensions or head width")
                rows, taps = d.dim, d.conv
            else:
                if m.heads % m.groups or (m.heads * m.vdim) % m.norm_groups:
                    raise ValueError(f"{where}: heads must be whole groups, channels whole norm groups")
                rows, taps = m.state, m.conv
            if not 1 <= rows <= self.MAX_STATE_ROWS or not 1 <= taps <= self.MAX_TAPS:
                raise ValueError(f"{where}: state rows up to {self.MAX_STATE_ROWS}, taps up to {self.MAX_TAPS}")
            _check_moe(where, f, self.MAX_EXPERTS, self.MAX_TOP)
        _check_loop(self.name, len(self.blocks), self.loop)

    @property
    def layers(self) -> int:
        return len(self.blocks)

    def runs(self) -> list:
        """(layer, embedding added before it) of every layer run, in order."""
        return [(i, bool(k)) for i, k in loop_runs(self.layers, self.loop)]

    @property
    def padded_hidden(self) -> int:
        return _up(self.hidden, 128)

    @property
    def padded_vocab(self) -> int:
        return _up(self.vocab_size, 128)

    @staticmethod
    def padded_head(m: ChunkedMixer) -> int:
        """Common padded width of the query / key and value heads."""
        d = max(m.dim, m.vdim)
        return next((p for p in (64, 128, 256) if d <= p), _up(d, 64))

    def to_dict(self):
        return asdict(self)

    def params(self) -> int:
        W = self.hidden
        n = 2 * self.vocab_size * W + W
        for b in self.blocks:
            m, f = b.mixer, b.mlp
            n += W
            if isinstance(m, ParallelMixer):
                a, d = m.left, m.right
                n += W * (a.heads * (a.dim + a.vdim) + a.kv_heads * (a.dim + a.vdim))
                c, v = 2 * d.kv_heads * d.dim + d.heads * d.vdim, d.heads * d.vdim
                n += W * (c + 2 * v + 2 * d.heads) + c * d.conv + 2 * d.heads + d.vdim
            else:
                inner = m.heads * m.vdim
                c = inner + 2 * m.groups * m.state
                n += W * (2 * inner + c + m.heads) + c * (m.conv + 1) + 3 * m.heads + inner
            if isinstance(f, DenseMlp):
                n += 3 * W * f.ff + 2 * f.ff + W
            elif f is not None:
                n += f.experts * (3 * W * f.ff + W) + (3 * W * f.shared + W if f.shared else 0)
        return n


def vugotar_uniform(name: str, layers: int, vocab_size: int, hidden: int, left: ChunkedMixer, right: DeltaMixer,
                    mamba: Mamba2Mixer, dense: DenseMlp, moe: MoeMlp | None, loop: tuple | None = None, **kw) -> VugotarConfig:
    """A Vugotar whose layers repeat (mamba2 + dense, parallel + experts, parallel + dense); without ``moe`` every MLP is
    dense."""
    par = ParallelMixer(left, right, 0.5, 0.5)
    cycle = (HybridLayer(mamba, dense), HybridLayer(par, moe or dense), HybridLayer(par, dense))
    return VugotarConfig(name, vocab_size, hidden, tuple(cycle[i % 3] for i in range(layers)), loop=loop, **kw)


# ------------------------------------------------------------------ recurrent / latent decoders (Vunelix)


@dataclass(frozen=True)
class VunelixConfig:
    """Vunelix decoder: selective scans and rotary latent attention, dense ReLU-gated MLPs and sigmoid-routed experts, an RMS
    norm before and after each.  ``loop`` = (start, stop, times) runs a stretch of layers several times with the same
    weights (every pass with its own cache and state); before each pass the stream is mixed with the embedding by a
    projection and a vector of the pass is added.  Logits: the tied embedding, softly capped."""

    name: str
    vocab_size: int
    hidden: int
    blocks: tuple  # of HybridLayer
    eps: float = 1e-5
    loop: tuple | None = None
    softcap: float | None = None
    max_position: int = 1 << 20  # no positional table: only the cache bounds a sequence
    default_model_len: int = 8192
    bos_id: int = 0
    eos_ids: tuple = ()

    MAX_STATE, MAX_STEP_RANK, MAX_TAPS, MAX_ROW, MAX_EXPERTS, MAX_TOP = 256, 2048, 16, 2048, 1024, 64  # of the kernels

    def __post_init__(self):
        for i, b in enumerate(self.blocks):
            where, m, f = f"{self.name}: layer {i}", b.mixer, b.mlp
            if isinstance(m, SelectiveMixer):
                if not (1 <= m.state <= self.MAX_STATE and 1 <= m.dt_rank <= self.MAX_STEP_RANK and 1 <= m.conv <= self.MAX_TAPS):
                    raise ValueError(f"{where}: state up to {self.MAX_STATE}, step rank up to {self.MAX_STEP_RANK}, taps up "
                                     f"to {self.MAX_TAPS}")
            else:
                if m.rot is not None and (m.rot.dims % 2 or m.rot.dims < 2):
                    raise ValueError(f"{where}: rotated dimensions come in pairs")
                if m.padded_row() > self.MAX_ROW:
                    raise ValueError(f"{where}: latent and rotated key up to {self.MAX_ROW} wide")
            _check_moe(where, f, self.MAX_EXPERTS, self.MAX_TOP)
        _check_loop(self.name, len(self.blocks), self.loop)

    @property
    def layers(self) -> int:
        return len(self.blocks)

    def runs(self) -> list:
        """(layer, pass that starts right before it or None) of every layer run, in order."""
        return loop_runs(self.layers, self.loop)

    @property
    def passes(self) -> int:
        """Passes of the loop (0: there is nothing to loop)."""
        return sum(k is not None for _, k in self.runs())

    @property
    def padded_hidden(self) -> int:
        return _up(self.hidden, 128)

    @property
    def padded_vocab(self) -> int:
        return _up(self.vocab_size, 128)

    def to_dict(self):
        return asdict(self)

    def params(self) -> int:
        W = self.hidden
        n = self.vocab_size * W + W + (2 * W * W + self.loop[2] * W if self.loop else 0)
        for b in self.blocks:
            m, f = b.mixer, b.mlp
            n += 2 * W
            if isinstance(m, SelectiveMixer):
                n += m.inner * (3 * W + m.conv + 1 + 2 * m.dt_rank + 3 * m.state + 2)
            else:
                P = m.rot.dims if m.rot else 0
                n += W * (m.heads * (m.dim + P + (2 if m.gate else 1) * m.vdim) + m.rank + P) + m.rank * (1 + m.heads * (m.dim + m.vdim))
            if f is not None:
                n += 2 * W
            if isinstance(f, DenseMlp):
                n += 3 * W * f.ff
            elif f is not None:
                n += f.experts * (3 * W * f.ff + W) + (3 * W * f.shared if f.shared else 0)
        return n


def vunelix_uniform(name: str, layers: int, vocab_size: int, hidden: int, mamba: SelectiveMixer, latent: LatentMixer,
                    dense: DenseMlp, moe: MoeMlp | None, loop: tuple | None = None, **kw) -> VunelixConfig:
    """A Vunelix whose layers repeat (scan + dense, latent attention + experts, latent attention + experts); without ``moe``
    every MLP is dense."""
    cycle = (HybridLayer(mamba, dense), HybridLayer(latent, moe or dense), HybridLayer(latent, moe or dense))
    return VunelixConfig(name, vocab_size, hidden, tuple(cycle[i % 3] for i in range(layers)), loop=loop,
                         softcap=kw.pop("softcap", 30.0), **kw)


# ------------------------------------------------------------------ depth-averaged decoders (Bizetar)


@dataclass(frozen=True)
class BizetarConfig:
    """Bizetar decoder: softmax attention with sinks (distance slopes and query temperature, or short convolutions and rotary
    positions), PolyNorm MLPs and experts with identity experts.  A sublayer reads the stream itself; its result passes a
    sigmoid gate of the same input and a norm before it is added.  After every layer the stream becomes a weighted sum of the
    embedding and all layers' results; from the first such layer on, values are mixed with that layer's."""

    name: str
    vocab_size: int
    hidden: int
    blocks: tuple  # of HybridLayer
    eps: float = 1e-5
    max_position: int = 1 << 20  # no positional table: only the cache bounds a sequence
    default_model_len: int = 8192
    bos_id: int = 0
    eos_ids: tuple = ()

    MAX_TAPS, MAX_HEAD, MAX_WIDTH, MAX_FF = 16, 1024, 16384, 65536  # of the kernels

    def __post_init__(self):
        if self.hidden > self.MAX_WIDTH:
            raise ValueError(f"{self.name}: width up to {self.MAX_WIDTH}")
        for i, b in enumerate(self.blocks):
            where, m, f = f"{self.name}: layer {i}", b.mixer, b.mlp
            if m.heads % m.kv_heads or max(m.dim, m.vdim) > self.MAX_HEAD or not 0 <= m.conv <= self.MAX_TAPS:
                raise ValueError(f"{where}: whole groups of kv_heads, heads up to {self.MAX_HEAD} wide, taps up to {self.MAX_TAPS}")
            if m.rot is not None and (m.rot.dims % 2 or m.rot.dims > m.dim):
                raise ValueError(f"{where}: rotated dimensions come in pairs, at most {m.dim}")
            if m.temp is not None and m.temp.every < 1:
                raise ValueError(f"{where}: the query temperature's period is a positive number")
            if isinstance(f, PolyMlp) and f.ff > self.MAX_FF:
                raise ValueError(f"{where}: MLP up to {self.MAX_FF} wide")
            _check_moe(where, f)
        mixed = [b.mixer for b in self.blocks if b.mixer.v_mix]
        if len({(m.kv_heads, m.vdim) for m in mixed}) > 1:
            raise ValueError(f"{self.name}: layers that mix values have equal value heads")

    @property
    def layers(self) -> int:
        return len(self.blocks)

    @property
    def first_mix(self) -> int | None:
        """The layer whose values later layers mix in."""
        return next((i for i, b in enumerate(self.blocks) if b.mixer.v_mix), None)

    @property
    def padded_hidden(self) -> int:
        return _up(self.hidden, 128)

    @property
    def padded_vocab(self) -> int:
        return _up(self.vocab_size, 128)

    def to_dict(self):
        return asdict(self)

    def params(self) -> int:
        W = self.hidden
        n = 2 * self.vocab_size * W + 2 * W
        for i, b in enumerate(self.blocks):
            m, f = b.mixer, b.mlp
            qkv = (m.heads + m.kv_heads) * m.dim + m.kv_heads * m.vdim
            whole = m.norm == "whole"
            n += W * (qkv + 2 * m.heads * m.vdim if m.gate == "element" else qkv + m.heads * (m.vdim + 1)) + m.heads
            n += ((m.heads + m.kv_heads) * m.dim if whole else 2 * m.dim) + qkv * (m.conv + m.bias) + m.v_mix
            n += W * W + 2 * W + i + 2
            if f is not None:
                n += W * W + 2 * W
            if isinstance(f, PolyMlp):
                n += 2 * W * f.ff + 4
            elif f is not None:
                n += f.experts * 3 * W * f.ff + f.outputs * (W + 1)
        return n


def bizetar_uniform(name: str, layers: int, vocab_size: int, hidden: int, first: SinkMixer, second: SinkMixer, dense: PolyMlp,
                    moe: MoeMlp | None, **kw) -> BizetarConfig:
    """A Bizetar whose mixers alternate; with ``moe`` the feed-forwards do too (dense, experts)."""
    blocks = tuple(HybridLayer((first, second)[i % 2], dense if moe is None or i % 2 == 0 else moe) for i in range(layers))
    return BizetarConfig(name, vocab_size, hidden, blocks, **kw)


ENCODERS = {
    "bge-base-en": EncoderConfig("bge-base-en"),
    "bge-large-en": EncoderConfig("bge-large-en", hidden=1024, layers=24, heads=16, intermediate=4096),
    "all-minilm-l6": EncoderConfig("all-minilm-l6", hidden=384, layers=6, heads=12, intermediate=1536),
    "rubert-base": EncoderConfig("rubert-base", vocab_size=120138),
    "tiny-bert": EncoderConfig("tiny-bert", vocab_size=2048, hidden=128, layers=2, heads=2, intermediate=256,
                               max_position=128),
}

DECODERS = {
    "llama-3-8b": DecoderConfig("llama-3-8b"),
    "llama-3-70b": DecoderConfig("llama-3-70b", hidden=8192, layers=80, heads=64, kv_heads=8, intermediate=28672),
    "llama-3.2-1b": DecoderConfig("llama-3.2-1b", hidden=2048, layers=16, heads=32, kv_heads=8, intermediate=8192,
                                  tie_embeddings=True,
                                  rope_scaling={"factor": 32.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                                                "original_max_position_embeddings": 8192}),
    "tiny-llama": DecoderConfig("tiny-llama", vocab_size=1024, hidden=256, layers=2, heads=4, kv_heads=2,
                                intermediate=512, max_position=2048, bos_id=1000, eos_ids=(1001,), rope_scaling=None,
                                rope_theta=10000.0),
    # the Llama-3-70B head layout (64 query heads over 8 KV heads) at toy width: at TP=8 every rank
    # holds exactly one KV head and 8 query heads, like 70B on 8 GPUs (CPU multi-rank tests)
    "tiny-llama-70b-layout": DecoderConfig("tiny-llama-70b-layout", vocab_size=1024, hidden=1024, layers=2, heads=64,
                                           kv_heads=8, intermediate=1024, max_position=2048, bos_id=1000,
                                           eos_ids=(1001,), rope_scaling=None, rope_theta=10000.0),
    # Llama-3-70B's real attention layout (hidden 8192, 64 / 8 heads of D = 128) at 2 layers with a
    # toy vocabulary and MLP: TP=8 ranks run the D = 128 prefill / decode attention kernels with 8
    # query heads over 1 KV head and all-reduce 70B-sized rows (B x 8192)
    "tiny-llama-70b-d128": DecoderConfig("tiny-llama-70b-d128", vocab_size=1024, hidden=8192, layers=2, heads=64,
                                         kv_heads=8, intermediate=2048, max_position=2048, bos_id=1000,
                                         eos_ids=(1001,), rope_scaling=None, rope_theta=10000.0),
}

DECODERS.update({
    # the widths, MLP and vocabulary of Llama-3-8B with latent attention: 32 heads over a 512-wide latent
    # that two layers share, 4096-key windows
    "vumuvik-8b": vumuvik_uniform("vumuvik-8b", layers=32, vocab_size=128256, hidden=4096, ff=14336, heads=32, dim=128,
                                  rank=512, window=4096),
    "vumuvik-1b": vumuvik_uniform("vumuvik-1b", layers=16, vocab_size=128256, hidden=2048, ff=8192, heads=32, dim=64,
                                  rank=256, window=1024),
    # test size: every branch (unequal heads, widths, ranks, windows, own and shared latents, a layer without MLP)
    "tiny-vumuvik": VumuvikConfig("tiny-vumuvik", 1000, 200, (
        LatentLayer(LatentMixer(4, 48, 40, 80, 0.17, 70), 344),
        LatentLayer(LatentMixer(3, 64, 64, 80, 0.11, 33, kv_from=0), 200),
        LatentLayer(LatentMixer(5, 32, 56, 48, 0.2, 0), None),
        LatentLayer(LatentMixer(2, 40, 24, 48, 0.15, 128, kv_from=2), 256)), 1e-5, 11.0, max_position=2048),
})

DECODERS.update({
    # Llama-3-8B's width, MLP, vocabulary and KV heads; 2048-token chunks; a 128 x 128 state per head
    "vugotar-8b": vugotar_uniform(
        "vugotar-8b", 28, 128256, 4096, ChunkedMixer(32, 8, 128, 128, 128 ** -0.5, 2048, 64, 500000.0),
        DeltaMixer(16, 8, 128, 128, 4), Mamba2Mixer(64, 64, 128, 8, 4, 8), DenseMlp(14336), None),
    # ... and with experts: 64 of 512, 6 per token, at Llama-3.2-1B's width
    "vugotar-moe": vugotar_uniform(
        "vugotar-moe", 15, 128256, 2048, ChunkedMixer(16, 4, 128, 128, 128 ** -0.5, 1024, 128, 500000.0),
        DeltaMixer(16, 8, 128, 128, 4), Mamba2Mixer(64, 64, 128, 8, 4, 8), DenseMlp(8192),
        MoeMlp(64, 6, 2.0, 1024, 2048)),
    # test size: every branch at unequal sizes
    "tiny-vugotar": VugotarConfig("tiny-vugotar", 1000, 200, (
        HybridLayer(Mamba2Mixer(6, 24, 40, 3, 3, 4), DenseMlp(168)),
        HybridLayer(ParallelMixer(ChunkedMixer(6, 2, 48, 40, 0.15, 70, 32, 5000.0), DeltaMixer(6, 2, 40, 24, 4), 0.7, 0.4),
                    MoeMlp(12, 3, 1.7, 40, 72)),
        HybridLayer(ParallelMixer(ChunkedMixer(3, 3, 64, 64, 0.12, 0, 64), DeltaMixer(2, 2, 64, 64, 2)), None),
        HybridLayer(Mamba2Mixer(2, 64, 64, 1, 4, 1), MoeMlp(5, 1, 1.0, 24))), 1e-5, loop=(1, 3, 2), max_position=2048),
})

_YARN = Yarn(4.0, 4096, 32.0, 1.0)

DECODERS.update({
    # Llama-3-8B's width, MLP, vocabulary and head count; a 512-wide latent, 96 + 32 dimensions a head, 16-entry states
    "vunelix-8b": vunelix_uniform(
        "vunelix-8b", 28, 128256, 4096, SelectiveMixer(8192, 16, 256, 4),
        LatentMixer(32, 96, 128, 512, 128 ** -0.5, rot=Rotary(32, 500000.0, _YARN), gate=True), DenseMlp(14336, "relu"), None),
    # ... and with experts: 64 of 1024, 6 per token beside a shared one, at Llama-3.2-1B's width
    "vunelix-moe": vunelix_uniform(
        "vunelix-moe", 15, 128256, 2048, SelectiveMixer(4096, 16, 128, 4),
        LatentMixer(16, 96, 128, 256, 128 ** -0.5, rot=Rotary(32, 500000.0, _YARN), gate=True), DenseMlp(8192, "relu"),
        MoeMlp(64, 6, 1.0, 1024, 2048, "sigmoid", "input")),
    # test size: every branch at unequal sizes
    "tiny-vunelix": VunelixConfig("tiny-vunelix", 1000, 200, (
        HybridLayer(SelectiveMixer(152, 20, 9, 3), MoeMlp(12, 3, 1.0, 40, 72, "sigmoid", "input")),
        HybridLayer(LatentMixer(3, 40, 24, 80, 0.15, rot=Rotary(12, 5000.0, Yarn(3.0, 100, 16.0, 2.0)), gate=True), DenseMlp(168, "relu")),
        HybridLayer(SelectiveMixer(96, 8, 4, 4), None),
        HybridLayer(LatentMixer(5, 16, 56, 48, 0.2, rot=Rotary(32), gate=True), MoeMlp(5, 1, 1.0, 24, None, "sigmoid", "input"))),
        1e-5, loop=(1, 3, 2), softcap=20.0, max_position=2048),
})

DECODERS.update({
    # Llama-3-8B's width, vocabulary and heads; distance slopes and convolved rotary attention in turn
    "bizetar-8b": bizetar_uniform(
        "bizetar-8b", 32, 128256, 4096,
        SinkMixer(32, 8, 128, 128, 128 ** -0.5, "head", "element", True, 4, Rotary(128, 500000.0, _YARN), v_mix=True),
        SinkMixer(32, 8, 128, 128, 128 ** -0.5, "whole", "head", temp=QueryTemp(0.1, 8192), slopes=True, v_mix=True),
        PolyMlp(14336), None),
    # ... and with experts: 64 of 1024 beside 8 identity experts, 8 per token, at Llama-3.2-1B's width
    "bizetar-moe": bizetar_uniform(
        "bizetar-moe", 16, 128256, 2048,
        SinkMixer(16, 4, 128, 128, 128 ** -0.5, "head", "element", True, 4, Rotary(128, 500000.0, _YARN), v_mix=True),
        SinkMixer(16, 4, 128, 128, 128 ** -0.5, "whole", "head", temp=QueryTemp(0.1, 8192), slopes=True, v_mix=True),
        PolyMlp(8192), MoeMlp(64, 8, 1.0, 1024, scores="softmax_raw", correction=True, identity=8)),
    # test size: every branch at unequal sizes
    "tiny-bizetar": BizetarConfig("tiny-bizetar", 1000, 200, (
        HybridLayer(SinkMixer(6, 2, 40, 24, 0.2, "whole", "head", temp=QueryTemp(0.3, 50), slopes=True, v_mix=True),
                    MoeMlp(7, 3, 1.0, 40, scores="softmax_raw", correction=True, identity=3)),
        HybridLayer(SinkMixer(4, 2, 48, 24, 0.15, "head", "element", True, 3, Rotary(32, 5000.0, Yarn(3.0, 100, 16.0, 2.0)),
                              v_mix=True), PolyMlp(168)),
        HybridLayer(SinkMixer(3, 1, 64, 72, 0.12, "head", "element", True, 4, Rotary(64, 1000.0)), None)),
        1e-5, max_position=2048),
})

_ALIASES = {
    "baai/bge-base-en": "bge-base-en", "baai/bge-base-en-v1.5": "bge-base-en", "bge-base": "bge-base-en",
    "baai/bge-large-en": "bge-large-en", "baai/bge-large-en-v1.5": "bge-large-en", "bge-large": "bge-large-en",
    "sentence-transformers/all-minilm-l6-v2": "all-minilm-l6", "all-minilm-l6-v2": "all-minilm-l6",
    "sberbank-ai/rubert-base": "rubert-base", "ai-forever/rubert-base": "rubert-base",
    "meta-llama/meta-llama-3-8b": "llama-3-8b", "meta-llama/meta-llama-3-8b-instruct": "llama-3-8b",
    "meta-llama/llama-3.1-8b-instruct": "llama-3-8b", "llama3": "llama-3-8b", "llama3:8b": "llama-3-8b",
    "llama-3.1-8b": "llama-3-8b",
    "meta-llama/meta-llama-3-70b-instruct": "llama-3-70b", "llama3:70b": "llama-3-70b", "llama-3.1-70b": "llama-3-70b",
    "meta-llama/llama-3.2-1b-instruct": "llama-3.2-1b",
}


def _key(name: str) -> str:
    k = name.strip().lower()
    return _ALIASES.get(k, k)


# ------------------------------------------------------------------ local HF checkpoint directories
# A model name may also be a local HF directory (config.json + *.safetensors [+ tokenizer.json]), as
# the reference's TransformersEmbedder / TransformersProvider accept (ai/embedders/transformers.py:13,
# ai/providers/transformers.py:18-20: ``from_pretrained(model_name)``).  The architecture comes from
# config.json; only the families the native kernels implement are accepted.

def checkpoint_dir(name) -> str | None:
    """``name`` if it is a local directory with a config.json, else None."""
    if isinstance(name, str) and os.path.isfile(os.path.join(name, "config.json")):
        return name
    return None


def _hf(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


def _label(path: str) -> str:
    return os.path.basename(os.path.normpath(path)).lower()


def encoder_config_from_hf(path: str) -> EncoderConfig:
    c = _hf(path)
    if c.get("model_type") != "bert":
        raise ValueError(f"{path}: model_type {c.get('model_type')!r} is not a BERT encoder")
    if c.get("hidden_act", "gelu") != "gelu" or c.get("position_embedding_type", "absolute") != "absolute":
        raise ValueError(f"{path}: only erf-GELU BERT encoders with absolute positions are supported")
    return EncoderConfig(_label(path), vocab_size=c["vocab_size"], hidden=c["hidden_size"],
                         layers=c["num_hidden_layers"], heads=c["num_attention_heads"],
                         intermediate=c["intermediate_size"], max_position=c.get("max_position_embeddings", 512),
                         type_vocab=c.get("type_vocab_size", 2), eps=c.get("layer_norm_eps", 1e-12))


def decoder_config_from_hf(path: str) -> DecoderConfig:
    c = _hf(path)
    if c.get("model_type") != "llama":
        raise ValueError(f"{path}: model_type {c.get('model_type')!r} is not a Llama decoder")
    if c.get("hidden_act", "silu") != "silu" or c.get("attention_bias") or c.get("mlp_bias"):
        raise ValueError(f"{path}: only bias-free SiLU Llama decoders are supported")
    heads = c["num_attention_heads"]
    if c.get("head_dim", c["hidden_size"] // heads) * heads != c["hidden_size"]:
        raise ValueError(f"{path}: head_dim x heads must equal hidden_size")
    # transformers 4.x: rope_theta + rope_scaling; 5.x: rope_parameters (theta and scaling together)
    rp = c.get("rope_parameters") or {}
    theta = c.get("rope_theta", rp.get("rope_theta", 10000.0))
    rs = c.get("rope_scaling") or (rp if rp.get("rope_type") not in (None, "default") else None)
    if rs is not None:
        kind = rs.get("rope_type", rs.get("type"))
        if kind == "default":
            rs = None
        elif kind != "llama3":
            raise ValueError(f"{path}: rope_scaling type {kind!r} is not supported (llama3 or none)")
        else:
            rs = {k: float(rs[k]) if k != "original_max_position_embeddings" else int(rs[k])
                  for k in ("factor", "low_freq_factor", "high_freq_factor", "original_max_position_embeddings")}
    eos = c.get("eos_token_id")
    eos = tuple(eos) if isinstance(eos, (list, tuple)) else ((eos,) if eos is not None else ())
    return DecoderConfig(_label(path), vocab_size=c["vocab_size"], hidden=c["hidden_size"],
                         layers=c["num_hidden_layers"], heads=heads,
                         kv_heads=c.get("num_key_value_heads") or heads, intermediate=c["intermediate_size"],
                         rope_theta=float(theta), rope_scaling=rs,
                         eps=float(c.get("rms_norm_eps", 1e-6)), max_position=c.get("max_position_embeddings", 8192),
                         bos_id=c.get("bos_token_id", 1) if c.get("bos_token_id") is not None else 1,
                         eos_ids=eos or (2,), tie_embeddings=bool(c.get("tie_word_embeddings", False)))


def encoder_config(name: str, **overrides) -> EncoderConfig:
    if checkpoint_dir(name):
        cfg = encoder_config_from_hf(name)
        return replace(cfg, **overrides) if overrides else cfg
    k = _key(name)
    if k not in ENCODERS:
        raise KeyError(f"unknown encoder model '{name}' (known: {sorted(ENCODERS)}, or a local HF directory)")
    return replace(ENCODERS[k], **overrides) if overrides else ENCODERS[k]


def vumuvik_config_from_dir(path: str) -> VumuvikConfig:
    """config.json of a Vumuvik checkpoint: ``architecture``, ``vocab``, ``width``, ``embedding.scale``,
    ``norm.eps`` and ``layers`` (each ``type``, ``mixer`` sizes and ``mlp`` or null)."""
    c = _hf(path)
    blocks = []
    for i, L in enumerate(c["layers"]):
        if L.get("type") != "latent_attention":
            raise ValueError(f"{path}: layer {i}: mixer type {L.get('type')!r} is not supported (latent_attention)")
        m, mlp = L["mixer"], L.get("mlp")
        if mlp is not None and mlp.get("kind") != "dense":
            raise ValueError(f"{path}: layer {i}: mlp kind {mlp.get('kind')!r} is not supported (dense or null)")
        src = m.get("kv_from")
        blocks.append(LatentLayer(
            LatentMixer(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), rank=int(m["kv_rank"]),
                        scale=float(m["scale"]), window=int((m.get("mask") or {}).get("size") or 0),
                        kv_from=None if src is None else int(src)),
            None if mlp is None else int(mlp["ff"])))
    return VumuvikConfig(_label(path), int(c["vocab"]), int(c["width"]), tuple(blocks), float(c["norm"]["eps"]),
                         float(c["embedding"]["scale"]))


def vugotar_config_from_dir(path: str) -> VugotarConfig:
    """config.json of a Vugotar checkpoint: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``loop`` (or none) and
    ``layers`` (each ``type``, ``mixer`` sizes and ``mlp`` or null)."""
    c = _hf(path)
    blocks = []
    for i, L in enumerate(c["layers"]):
        m, f = L["mixer"], L.get("mlp")
        if L.get("type") == "parallel":
            a, d = m["left"], m["right"]
            rot = a.get("rot") or {}
            mixer = ParallelMixer(
                ChunkedMixer(int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), int(a["vdim"]), float(a["scale"]),
                             int((a.get("mask") or {}).get("size") or 0), int(rot.get("dims") or 0),
                             float(rot.get("base", 10000.0))),
                DeltaMixer(int(d["heads"]), int(d["kv_heads"]), int(d["dim"]), int(d["vdim"]), int(d["conv"])),
                float(m["left_scale"]), float(m["right_scale"]))
        elif L.get("type") == "mamba2":
            mixer = Mamba2Mixer(int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"]), int(m["conv"]),
                                int(m["norm_groups"]))
        else:
            raise ValueError(f"{path}: layer {i}: mixer type {L.get('type')!r} is not supported (parallel, mamba2)")
        if f is None:
            mlp = None
        elif f.get("kind") == "dense":
            mlp = DenseMlp(int(f["ff"]))
        elif f.get("kind") == "moe":
            r, sh = f["router"], f.get("shared")
            mlp = MoeMlp(int(r["experts"]), int(r["top"]), float(r["scale"]), int(f["expert"]["ff"]),
                         None if sh is None else int(sh["ff"]))
        else:
            raise ValueError(f"{path}: layer {i}: mlp kind {f.get('kind')!r} is not supported (dense, moe or null)")
        blocks.append(HybridLayer(mixer, mlp))
    lp = c.get("loop")
    loop = None if lp is None else (int(lp["start"]), int(lp["stop"]), int(lp["times"]))
    return VugotarConfig(_label(path), int(c["vocab"]), int(c["width"]), tuple(blocks), float(c["norm"]["eps"]), loop)


def vunelix_config_from_dir(path: str) -> VunelixConfig:
    """config.json of a Vunelix checkpoint: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``loop`` and
    ``logit_softcap`` (or none) and ``layers`` (each ``type``, ``mixer`` sizes and ``mlp`` or null)."""
    c = _hf(path)
    blocks = []
    for i, L in enumerate(c["layers"]):
        m, f = L["mixer"], L.get("mlp")
        if L.get("type") == "mamba1":
            mixer = SelectiveMixer(int(m["inner"]), int(m["state"]), int(m["dt_rank"]), int(m["conv"]))
        elif L.get("type") == "latent_attention":
            rot, P = m.get("rot"), int(m.get("rot_dim") or 0)
            if P and (rot is None or int(rot["dims"]) != P):
                raise ValueError(f"{path}: layer {i}: rot.dims must be rot_dim")
            if P:
                sc = rot.get("scaling")
                rot = Rotary(P, float(rot["base"]), None if sc is None else Yarn(
                    float(sc["factor"]), float(sc["original"]), float(sc["fast"]), float(sc["slow"])))
            mixer = LatentMixer(int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["kv_rank"]), float(m["scale"]),
                                rot=rot if P else None, gate=True)
        else:
            raise ValueError(f"{path}: layer {i}: mixer type {L.get('type')!r} is not supported (mamba1, latent_attention)")
        if f is None:
            mlp = None
        elif f.get("kind") == "dense":
            mlp = DenseMlp(int(f["ff"]), "relu")
        elif f.get("kind") == "moe":
            r, sh = f["router"], f.get("shared")
            mlp = MoeMlp(int(r["experts"]), int(r["top"]), 1.0, int(f["expert"]["ff"]), None if sh is None else int(sh["ff"]),
                         "sigmoid", "input")
        else:
            raise ValueError(f"{path}: layer {i}: mlp kind {f.get('kind')!r} is not supported (dense, moe or null)")
        blocks.append(HybridLayer(mixer, mlp))
    lp, cap = c.get("loop"), c.get("logit_softcap")
    loop = None if lp is None else (int(lp["start"]), int(lp["stop"]), int(lp["times"]))
    return VunelixConfig(_label(path), int(c["vocab"]), int(c["width"]), tuple(blocks), float(c["norm"]["eps"]), loop,
                         None if not cap else float(cap))


def bizetar_config_from_dir(path: str) -> BizetarConfig:
    """config.json of a Bizetar checkpoint: ``architecture``, ``vocab``, ``width``, ``norm.eps`` and ``layers`` (each ``type``,
    ``mixer`` sizes and ``mlp`` or null)."""
    c = _hf(path)
    blocks = []
    for i, L in enumerate(c["layers"]):
        m, f = L["mixer"], L.get("mlp")
        kw = dict(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                  scale=float(m["scale"]), v_mix=bool(m.get("v_mix")))
        if L.get("type") == "attention":
            t = m.get("q_temp")
            mixer = SinkMixer(norm="whole", gate="head", slopes=True,
                              temp=None if t is None else QueryTemp(float(t["coef"]), int(t["every"])), **kw)
        elif L.get("type") == "attention_2":
            rot = m.get("rot")
            if rot is not None:
                sc = rot.get("scaling")
                rot = Rotary(int(rot["dims"]), float(rot["base"]), None if sc is None else Yarn(
                    float(sc["factor"]), float(sc["original"]), float(sc["fast"]), float(sc["slow"])))
            mixer = SinkMixer(norm="head", gate="element", bias=True, conv=int(m.get("conv") or 0), rot=rot, **kw)
        else:
            raise ValueError(f"{path}: layer {i}: mixer type {L.get('type')!r} is not supported (attention, attention_2)")
        if f is None:
            mlp = None
        elif f.get("kind") == "dense":
            mlp = PolyMlp(int(f["ff"]))
        elif f.get("kind") == "moe":
            r = f["router"]
            mlp = MoeMlp(int(r["experts"]), int(r["top"]), 1.0, int(f["expert"]["ff"]), scores="softmax_raw", correction=True,
                         identity=int(r.get("identity") or 0))
        else:
            raise ValueError(f"{path}: layer {i}: mlp kind {f.get('kind')!r} is not supported (dense, moe or null)")
        blocks.append(HybridLayer(mixer, mlp))
    return BizetarConfig(_label(path), int(c["vocab"]), int(c["width"]), tuple(blocks), float(c["norm"]["eps"]))


_DIR_CONFIGS = {"vumuvik": vumuvik_config_from_dir, "vugotar": vugotar_config_from_dir, "vunelix": vunelix_config_from_dir,
                "bizetar": bizetar_config_from_dir}


def _dir_architecture(path: str) -> str | None:
    c = _hf(path)
    arch = str(c.get("architecture")).lower()
    return arch if arch in _DIR_CONFIGS else c.get("model_type")


def decoder_config(name: str, **overrides) -> DecoderConfig | VumuvikConfig | VugotarConfig | VunelixConfig | BizetarConfig:
    if checkpoint_dir(name):
        cfg = _DIR_CONFIGS.get(_dir_architecture(name), decoder_config_from_hf)(name)
        return replace(cfg, **overrides) if overrides else cfg
    k = _key(name)
    if k not in DECODERS:
        raise KeyError(f"unknown decoder model '{name}' (known: {sorted(DECODERS)}, or a local HF directory)")
    return replace(DECODERS[k], **overrides) if overrides else DECODERS[k]


def is_encoder(name: str) -> bool:
    d = checkpoint_dir(name)
    return _hf(d).get("model_type") == "bert" if d else _key(name) in ENCODERS


def is_decoder(name: str) -> bool:
    d = checkpoint_dir(name)
    return _dir_architecture(d) in ("llama", *_DIR_CONFIGS) if d else _key(name) in DECODERS
