"""Gated-sublayer, depth-sum, PolyNorm, attention-input, sloped-attention and identity-expert kernels against the CPU references
(which test_bizetar_model.py holds against the oracle) or plain formulas in fp64 (tests/bizetar_oracle.py)."""
import bizetar_oracle as oracle
import pytest
import torch

from django_assistant_bot_amd import ops

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BF, F32 = torch.bfloat16, torch.float32
TYPES = [(BF, BF), (F32, BF), (F32, F32)]  # of the projection, of the activations


def rnd(*shape, seed=0, dtype=BF, scale=1.0):
    g = torch.Generator().manual_seed(seed + sum(shape))
    return (torch.randn(shape, generator=g) * scale).to(dtype)


def close(got, want, tol):
    got, want = got.double().cpu(), want.double()
    assert torch.isfinite(got).all()
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-6)
    assert err < tol, err


def dev(x):
    if isinstance(x, torch.Tensor):
        return x.to(DEV)
    if isinstance(x, ops.AttnInputs):
        return ops.AttnInputs(*(dev(v) for v in x))
    return x


def i32(*v):
    return torch.tensor(v, dtype=torch.int32)


# ------------------------------------------------------------------------------------------------ sublayers


@pytest.mark.parametrize("rows,cols,n", [(1, 128, 100), (5, 4096, 4096), (130, 2048, 2000), (600, 4096, 4090), (3, 10240, 10000),
                                         (520, 640, 640), (2, 16384, 16300)])
@pytest.mark.parametrize("yt,dtype", TYPES)
@pytest.mark.parametrize("form", ["rows", "slabs", "experts"])
@pytest.mark.parametrize("depth", [0, 1, 6])
def test_gated_residual(rows, cols, n, yt, dtype, form, depth):
    S = (3,) if form == "slabs" else ()
    src, post, bias, gain = rnd(rows, cols, dtype=F32), *(rnd(cols, seed=s, dtype=F32) for s in (1, 2, 3))
    g = rnd(*S, rows, cols + 24, seed=4, dtype=yt)
    y = None if form == "experts" else rnd(*S, rows, cols, seed=5, dtype=yt)
    own = None
    if form == "experts":
        idx = torch.randint(0, 9, (rows, 3), generator=torch.Generator().manual_seed(0)).int()
        own = ops.RoutedRows(rnd(rows * 3, cols, seed=6, dtype=dtype), idx, rnd(rows, 3, seed=7, dtype=F32), 6)
        own.rows[:, n:] = 0
    over, w = rnd(6, rows, cols, seed=8, dtype=F32), rnd(depth + 1, seed=9, dtype=F32)
    for t in (src, post, bias, gain, over, *(() if y is None else (y,))):
        t[..., n:] = 0
    last = depth == 6  # (its result is not kept, a norm follows)
    x, xg, og = torch.zeros_like(src), src.to(DEV), over.to(DEV)
    ahead = rnd(rows, cols, seed=10, dtype=F32) if last else None
    if last:
        ahead[:, n:] = 0
    tail = lambda f: dict(depth=(f[0], f[1], depth, f[3], 4 if last else 0) if depth else None,  # noqa: E731
                          gain=f[2] if last else None)
    want = ops.gated_residual(src, x, y, (g, 16, bias), post, n, 1e-4, dtype, own, **tail((over, w, gain, ahead)))
    gown = None if own is None else ops.RoutedRows(dev(own.rows), dev(own.idx), dev(own.wt), 6)
    got = ops.gated_residual(xg, xg, dev(y), (dev(g), 16, dev(bias)), dev(post), n, 1e-4, dtype, gown, **tail((og, dev(w), dev(gain), dev(ahead))))
    close(xg, x, 3e-6)
    close(og, over, 3e-6)
    close(got, want, 6e-3 if dtype == BF else 4e-6)


@pytest.mark.parametrize("T,C,n,m", [(1, 128, 9, 8), (7, 4096, 25, 8), (300, 640, 17, 3), (5, 256, 1, 1), (64, 2048, 9, 5), (2, 128, 10, 7),
                                     (3, 384, 8, 2), (3, 384, 12, 4), (3, 384, 15, 6)])
def test_depth_ahead(T, C, n, m):
    over, w = rnd(n + 2, T, C, dtype=F32), rnd(m, n, seed=1, dtype=F32)
    out = torch.zeros(8, T, C, device=DEV)
    ops.depth_ahead(dev(over), dev(w), out)
    close(out[:m], torch.einsum("mn,ntc->mtc", w.double(), over[:n].double()), 2e-6)
    assert float(out[m:].abs().sum()) == 0


@pytest.mark.parametrize("rows,cols,n", [(1, 128, 65), (700, 4096, 4000), (9, 8192, 8192)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_norm_embed(rows, cols, n, dtype):
    table, gain = rnd(11, cols, dtype=dtype), rnd(cols, seed=1, dtype=F32)
    table[:, n:], gain[n:] = 0, 0
    ids = torch.randint(0, 11, (rows,), generator=torch.Generator().manual_seed(1)).int()
    x, xg = torch.zeros(rows, cols), torch.zeros(rows, cols, device=DEV)
    want, got = ops.norm_embed(ids, table, gain, n, 1e-5, x), ops.norm_embed(dev(ids), dev(table), dev(gain), n, 1e-5, xg)
    close(xg, x, 2e-6)
    close(got, want, 6e-3 if dtype == BF else 2e-6)


@pytest.mark.parametrize("T,n,cols", [(1, 1, 128), (3, 168, 256), (130, 8192, 8192), (600, 14336, 14336), (2, 65500, 65536), (520, 1000, 1024),
                                      (4, 14336, 14336)])
@pytest.mark.parametrize("yt,dtype", TYPES)
@pytest.mark.parametrize("slabs", [1, 4])
def test_poly_norm(T, n, cols, yt, dtype, slabs):
    y = rnd(*((slabs,) if slabs > 1 else ()), T, cols + 16, dtype=yt, scale=3.0)
    act = (0.7, -0.4, 1.3, 0.2)
    got = ops.poly_norm(y.to(DEV), T, n, cols, act, 1e-5, dtype)
    z = (y.float().sum(0) if slabs > 1 else y.float())[:, :n].to(dtype).double()
    close(got[:, :n], oracle.poly_norm(z, act, 1e-5), 6e-3 if dtype == BF else 4e-6)
    assert float(got[:, n:].abs().sum()) == 0


@pytest.mark.parametrize("per", [64, 128, 320])
@pytest.mark.parametrize("yt,dtype", TYPES)
def test_gate_of_a_head(per, yt, dtype):
    x, y = rnd(37, 5 * per, dtype=dtype), rnd(3, 37, 40, dtype=yt)
    want = ops.sigmoid_gate(y, 11, x.clone(), per)
    close(ops.sigmoid_gate(y.to(DEV), 11, x.to(DEV), per), want, 6e-3 if dtype == BF else 2e-6)


# ------------------------------------------------------------------------------------------------ attention inputs

SHAPES = [  # H, G, D, dim, vdim, rot, taps: every lane layout, with and without window registers
    (4, 2, 64, 64, 40, 48, 4), (5, 1, 64, 33, 64, 0, 2), (6, 3, 128, 100, 128, 100, 3), (32, 8, 128, 128, 128, 128, 4),
    (2, 2, 256, 200, 130, 64, 0), (3, 1, 256, 256, 256, 256, 4), (2, 1, 320, 270, 300, 6, 3), (1, 1, 1024, 1000, 9, 1000, 7), (18, 1, 128, 128, 96, 32, 16),
    (1, 1, 64, 2, 1, 2, 1)]


def input_case(H, G, D, dim, vdim, rot, taps, whole, T, yt, dtype, slabs=1, slots=7):
    C, heads = (H + 2 * G) * D, H + 2 * G
    real = torch.zeros(heads, D)
    real[:H + G, :dim], real[H + G:, :vdim] = 1, 1
    mask = real.view(-1)
    pad = 16
    y = rnd(*((slabs,) if slabs > 1 else ()), T, pad + C + 8, dtype=yt)
    y[..., pad:pad + C] *= mask.to(yt)
    conv = rnd(taps, C, seed=2, dtype=F32, scale=taps ** -0.5) * mask if taps else None
    turns = ops.rope_turns(rot, 3000.0, "cpu") if rot else None
    a = ops.AttnInputs(H, G, D, dim, vdim, 1e-5, whole, (rnd((H + G) * D, seed=3, dtype=F32) + 1) * mask[:(H + G) * D],
                       rnd(C, seed=4, dtype=F32) * mask if taps else None, conv, turns, 1.2, 0.4, 9)
    ring = rnd(slots, taps, C, seed=5, dtype=dtype) * mask.to(dtype) if taps else None
    return a, pad, y, ring


@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("whole", [False, True])
@pytest.mark.parametrize("yt,dtype", TYPES)
@pytest.mark.parametrize("mix", [None, "write", "mix"])
def test_attn_inputs(shape, whole, yt, dtype, mix):
    """Portions (fresh ones, ones that go on, short ones) beside decoded tokens, some of them padding; slots in any order."""
    H, G, D = shape[:3]
    lens, starts, dec = [1, 2, 21, 9], [0, 5, 0, 100], [3, 0, 77, 1, 130]
    T0, T = sum(lens), sum(lens) + len(dec)
    a, col, y, ring = input_case(*shape, whole, T, yt, dtype, slabs=3 if yt != dtype else 1, slots=12)
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)] + [torch.tensor(dec)]).int()
    cu = torch.tensor([0, *torch.tensor(lens).cumsum(0).tolist()], dtype=torch.int32)
    bs = 16
    kc, vc = rnd(6, G, bs, D, seed=6, dtype=dtype), rnd(6, G, bs, D, seed=7, dtype=dtype)
    slots = torch.randperm(6 * bs, generator=torch.Generator().manual_seed(2))[:T]
    slots[-2] = -1
    order = torch.randperm(12, generator=torch.Generator().manual_seed(3)).int()
    cs, rs = order[:len(lens)].contiguous(), order[len(lens):len(lens) + len(dec)].contiguous()
    first = rnd(T, G, a.first_width, seed=8, dtype=dtype)
    args = lambda f, m: (f(y), col, f(a), f(pos), f(slots))  # noqa: E731
    outs = []
    for f in (lambda t: t.clone() if isinstance(t, torch.Tensor) else t, dev):
        k, v, r, fv = f(kc), f(vc), f(ring), f(first)
        m = None if mix is None else (fv, None if mix == "write" else 0.3)
        q = ops.attn_inputs(*args(f, m), k, v, r, f(cu), max(lens), f(cs), f(rs), T0, m)
        outs.append((q, k, v, r, fv))
    tol = 8e-3 if dtype == BF else 6e-6
    for got, want in zip(outs[1], outs[0]):
        if want is not None:
            close(got, want, tol)
    if ring is not None:  # other slots keep what they hold
        idle = order[len(lens) + len(dec):].tolist()
        assert torch.equal(outs[1][3].cpu()[idle], ring[idle])


@pytest.mark.parametrize("B", [1, 40, 130])
def test_attn_inputs_of_decoded_batches(B):
    a, col, y, ring = input_case(32, 8, 128, 128, 128, 128, 4, False, B, BF, BF, slabs=4, slots=B + 1)
    pos = (torch.arange(B) * 7 % 50).int()
    kc, vc = (torch.zeros(B, 8, 16, 128, dtype=BF) for _ in "kv")
    slots, rs = torch.arange(B) * 16, torch.randperm(B + 1, generator=torch.Generator().manual_seed(1))[:B].int()
    outs = []
    for f in (lambda t: t.clone() if isinstance(t, torch.Tensor) else t, dev):
        k, v, r = f(kc), f(vc), f(ring)
        outs.append((ops.attn_inputs(f(y), col, f(a), f(pos), f(slots), k, v, r, None, 1, None, f(rs), 0), k, v, r))
    for got, want in zip(outs[1], outs[0]):
        close(got, want, 8e-3)


def test_rotations_and_temperatures_at_far_positions():
    """Angles and temperatures at positions up to a million, in 32-bit."""
    H, G, D, T = 2, 1, 64, 40
    y = rnd(T, (H + 2 * G) * D, dtype=F32)
    pos = torch.linspace(0, 1_000_000, T).int()
    turns = ops.rope_turns(64, 10000.0, "cpu")
    a = ops.AttnInputs(H, G, D, D, D, 1e-5, False, torch.ones((H + G) * D), None, None, turns, 1.1, 0.3, 5000)
    kc, vc = (torch.zeros(4, G, 16, D, device=DEV) for _ in "kv")
    # (a portion's positions are counted from its first token, so every token is a portion of its own here)
    q = ops.attn_inputs(dev(y), 0, dev(a), dev(pos), dev(torch.arange(T)), kc, vc, None, dev(torch.arange(T + 1).int()), 1, None, None, T)
    x = y[:, :H * D].double().view(T, H, D)
    x = oracle.norm(x, 1.0, 1e-5)
    ang = pos.double()[:, None] * turns * 2 * torch.pi
    c, s = (ang.cos() * 1.1)[:, None], (ang.sin() * 1.1)[:, None]
    u, v = x[..., 0::2], x[..., 1::2]
    want = torch.stack([u * c - v * s, v * c + u * s], -1).flatten(2)
    want = want * (1 + 0.3 * torch.log((pos.double() + 1).div(5000, rounding_mode="floor") + 1))[:, None, None]
    close(q, want, 1e-6)


# ------------------------------------------------------------------------------------------------ attention, experts


@pytest.mark.parametrize("H,G,D", [(4, 2, 64), (8, 1, 128), (6, 6, 128), (32, 2, 128), (4, 2, 256), (18, 1, 128), (3, 1, 320), (18, 1, 64)])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("sloped", [True, False])
def test_sloped_attention(H, G, D, dtype, sloped):
    """Prompt portions that start at zero, inside and at the edge of a page, and decoded tokens, with split keys."""
    lens, ctx, bs = [200, 1, 65, 130], [200, 70, 193, 450], 64
    blocks = [-(-c // bs) for c in ctx]
    bt = torch.zeros(4, max(blocks), dtype=torch.int32)
    perm = torch.randperm(sum(blocks), generator=torch.Generator().manual_seed(0)).int()
    for i, n in enumerate(blocks):
        bt[i, :n] = perm[sum(blocks[:i]):sum(blocks[:i + 1])]
    kc, vc = (rnd(sum(blocks), G, bs, D, seed=s, dtype=dtype) for s in (1, 2))
    T = sum(lens)
    q, sink = rnd(T, H, D, seed=3, dtype=dtype), rnd(H, seed=4, dtype=F32) + 1
    slopes = oracle.slopes(H).float() if sloped else None
    cu, cx = i32(0, *torch.tensor(lens).cumsum(0).tolist()), i32(*ctx)
    scale = 1.5 * D ** -0.5
    want, got = torch.zeros(T, H * D, dtype=dtype), torch.zeros(T, H * D, dtype=dtype, device=DEV)
    ops.chunk_prefill(q, kc, vc, bt, cu, cx, max(lens), scale, 0, sink, want, slopes=slopes)
    a = [dev(t) for t in (q, kc, vc, bt, cu, cx)]
    ops.chunk_prefill(*a, max(lens), scale, 0, dev(sink), got, slopes=dev(slopes))
    tol = 1e-2 if dtype == BF else 5e-6
    close(got, want, tol)
    d, dg = torch.zeros(4, H * D, dtype=dtype), torch.zeros(4, H * D, dtype=dtype, device=DEV)
    ops.chunk_decode(q[:4], kc, vc, bt, cx, scale, 0, sink, d, slopes=slopes)
    for part in (128, 512):
        ws = ops.DecodeWorkspace(4, H, D, -(-(bt.shape[1] * bs) // part), torch.device(DEV))
        for order in (None, dev(i32(3, 0, 2, 1))):
            dg.zero_()
            ops.chunk_decode(a[0][:4], *a[1:4], a[5], scale, 0, dev(sink), dg, 1.0, part, ws, order, dev(slopes))
            close(dg, d, tol)
    ops.chunk_decode(a[0][:4], *a[1:4], a[5], scale, 0, dev(sink), dg, slopes=dev(slopes))
    close(dg, d, tol)
    for per in (1, D):  # with an output gate, from finished rows and from slabs
        y = rnd(*((3,) if per == 1 else ()), 4, 16 + -(-H * D // per // 8) * 8, seed=5, dtype=dtype)
        d.zero_()
        ops.chunk_decode(q[:4], kc, vc, bt, cx, scale, 0, sink, d, slopes=slopes, gate=(y, 16, per))
        ops.chunk_decode(a[0][:4], *a[1:4], a[5], scale, 0, dev(sink), dg, 1.0, 512, ws, None, dev(slopes), (dev(y), 16, per))
        close(dg, d, tol)


@pytest.mark.parametrize("sloped,sunk", [(True, True), (True, False), (False, True)])
@pytest.mark.parametrize("lens,done", [([700, 1, 384, 129, 513], [0, 64, 100, 0, 300]), ([2100], [130]), ([90] * 40, [7] * 40)])
def test_prompts_of_many_blocks(lens, done, sloped, sunk):
    """Heads of 128 with enough query blocks for the paired walk, portions that go on from cached keys among them."""
    H, G, D, bs = 32, 4, 128, 64
    ctx = [a + b for a, b in zip(lens, done)]
    blocks = [-(-c // bs) for c in ctx]
    bt = torch.zeros(len(lens), max(blocks), dtype=torch.int32)
    perm = torch.randperm(sum(blocks), generator=torch.Generator().manual_seed(0)).int()
    for i, n in enumerate(blocks):
        bt[i, :n] = perm[sum(blocks[:i]):sum(blocks[:i + 1])]
    kc, vc = (rnd(sum(blocks), G, bs, D, seed=s) for s in (1, 2))
    q, sink = rnd(sum(lens), H, D, seed=3), rnd(H, seed=4, dtype=F32) + 2
    slopes = oracle.slopes(H).float() if sloped else None
    cu = torch.tensor([0, *torch.tensor(lens).cumsum(0).tolist()], dtype=torch.int32)
    got = [torch.zeros(sum(lens), H * D, dtype=BF, device=DEV) for _ in range(3)]
    gates = [None] + [(rnd(sum(lens), 16 + H * D // per, seed=per), 16, per) for per in (1, D)]
    for g, o in zip(gates, got):
        ops.chunk_prefill(*(dev(t) for t in (q, kc, vc, bt, cu, i32(*ctx))), max(lens), 0.11, 0, dev(sink) if sunk else None, o,
                          slopes=dev(slopes), gate=None if g is None else (dev(g[0]), *g[1:]))
    some = sorted({0, len(lens) // 2, len(lens) - 1})
    for i in some:  # (the reference of a few sequences)
        want = torch.zeros(lens[i], H * D, dtype=BF)
        ops.chunk_prefill(q[cu[i]:cu[i + 1]], kc, vc, bt[i:i + 1], i32(0, lens[i]), i32(ctx[i]), lens[i], 0.11, 0, sink if sunk else None,
                          want, slopes=slopes)
        for g, o in zip(gates, got):
            close(o[cu[i]:cu[i + 1]], want if g is None else ops.sigmoid_gate(g[0][cu[i]:cu[i + 1]], g[1], want.clone(), g[2]), 1e-2)


@pytest.mark.parametrize("T,E,top,S", [(1, 3, 1, 1), (70, 72, 8, 4), (5, 9, 9, 2), (300, 260, 6, 1), (33, 1024, 64, 1)])
@pytest.mark.parametrize("scores", ["softmax", "sigmoid", "softmax_raw"])
def test_corrected_routing(T, E, top, S, scores):
    z = rnd(S, T, E + 5, dtype=F32)
    corr = rnd(E, seed=1, dtype=F32, scale=0.3) - 0.5  # (choice scores below zero too)
    idx, wt = ops.moe_route(z.to(DEV), 3, E, top, 1.5, T, scores, corr.to(DEV))
    ri, rw = ops.moe_route(z, 3, E, top, 1.5, T, scores, corr)
    a, b = idx.cpu().sort(-1), ri.sort(-1)
    assert torch.equal(a.values, b.values)
    close(wt.cpu().gather(-1, a.indices), rw.gather(-1, b.indices), 1e-5)


@pytest.mark.parametrize("T,E,extra,top", [(1, 4, 2, 3), (40, 6, 6, 6), (300, 8, 1, 2), (9, 3, 9, 2), (2000, 16, 4, 5), (4100, 8, 3, 4), (5000, 70, 2, 4)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_identity_experts(T, E, extra, top, dtype):
    """Choices behind the experts take no row of the grouped products and give the stream itself."""
    K = W = 128
    F = 64
    h, g = rnd(T, K, dtype=dtype), torch.Generator().manual_seed(T)
    idx = torch.stack([torch.randperm(E + extra, generator=g)[:top] for _ in range(T)]).int()
    if T == 9:
        idx[:] = torch.arange(E, E + top)  # no expert at all
    wt = rnd(T, top, seed=1, dtype=F32).abs()
    gate, up = rnd(E, F, K, seed=2, dtype=dtype, scale=K ** -0.5), rnd(E, F, K, seed=3, dtype=dtype, scale=K ** -0.5)
    down = rnd(E * W, F, seed=4, dtype=dtype, scale=F ** -0.5)
    if dtype == BF:
        gu = torch.stack([gate.view(E, F // 8, 8, K), up.view(E, F // 8, 8, K)], 2).reshape(E * 2 * F, K)
        rows = ops.moe_experts(dev(h), dev(idx), dev(wt), ops.shuffle_weights(dev(gu)), ops.shuffle_weights(dev(down)), E, 8)
    else:
        rows = ops.moe_experts(dev(h), dev(idx), dev(wt), dev(torch.cat([gate, up], 1).reshape(E * 2 * F, K)), dev(down), E, 0)
    src, zero, one = rnd(T, W, seed=5, dtype=F32), torch.zeros(W), torch.ones(W)
    gz = torch.full((T, W), 60.0, dtype=dtype)  # an open gate
    x = torch.zeros(T, W, device=DEV)
    own = ops.RoutedRows(rows, dev(idx), dev(wt), E)
    ops.gated_residual(dev(src), x, None, (dev(gz), 0, dev(zero)), dev(one), W, 1e-6, dtype, own)
    wm = {f"e{e}.{n}": t.double() for e in range(E) for n, t in (("gate", gate[e]), ("up", up[e]), ("down", down.view(E, W, F)[e]))}
    f = torch.zeros(T, W).double()
    for k in range(top):
        for e in range(E + extra):
            on = (idx[:, k] == e).double()[:, None] * wt[:, k:k + 1].double()
            f += on * (oracle.expert(h.double(), wm, f"e{e}.") if e < E else src.double())
    close(x, src.double() + oracle.norm(f, 1.0, 1e-6), 1.5e-2 if dtype == BF else 3e-5)
