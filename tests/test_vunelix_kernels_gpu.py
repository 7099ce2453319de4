"""Selective-scan, rotary-latent, post-norm and input-weighted-expert kernels against plain formulas in fp64
(tests/vunelix_oracle.py) or fp32 (the CPU references, which test_vunelix_model.py holds against the oracle)."""
import math

import pytest
import torch
import vunelix_oracle as oracle

from django_assistant_bot_amd import ops
from django_assistant_bot_amd.models.configs import Yarn
from django_assistant_bot_amd.ops import reference as ref
from django_assistant_bot_amd.ops.selective import state_width

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BF, F32 = torch.bfloat16, torch.float32


def rnd(*shape, seed=0, dtype=BF, scale=1.0):
    g = torch.Generator().manual_seed(seed + sum(shape))
    return (torch.randn(shape, generator=g) * scale).to(dtype)


def close(got, want, tol):
    got, want = got.double().cpu(), want.double()
    assert torch.isfinite(got).all()
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-6)
    assert err < tol, err


def i32(*v):
    return torch.tensor(v, dtype=torch.int32)


def test_state_width_agrees():
    for n in (1, 15, 16, 17, 33, 64, 65, 128, 129, 256):
        assert ops.native().selective_state_width(n) == state_width(n) >= n
    assert ops.native().selective_state_width(257) == 0


# ------------------------------------------------------------------------------------------------ selective scan


def scan_case(C, N, K, lens, dtype, slabs, seed=0, starts=None):
    """Inputs of the scan for packed portions of ``lens`` tokens that start at ``starts``."""
    T, Np, R = sum(lens), state_width(N), -(-K // 64) * 64
    d = ops.SelectiveShape(C, Np, R, R, R + Np, C)
    low = rnd(T, R + 2 * Np, seed=seed, dtype=F32)
    low[:, K:R], low[:, R + N:R + Np], low[:, R + Np + N:] = 0, 0, 0
    y = rnd(*((slabs,) if slabs > 1 else ()), T, 2 * C, seed=seed + 1, dtype=dtype)
    A = torch.zeros(C, Np)
    A[:, :N] = -torch.exp(rnd(C, N, seed=seed + 2, dtype=F32)) / math.log(2)
    starts = starts or [0] * len(lens)
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)]).int()
    cu = torch.tensor([0, *torch.tensor(lens).cumsum(0).tolist()], dtype=torch.int32)
    slot = torch.randperm(len(lens) + 2, generator=torch.Generator().manual_seed(seed))[:len(lens)].int()
    st = rnd(len(lens) + 2, C, Np, seed=seed + 3, dtype=F32)
    st[:, :, N:] = 0
    return dict(u=rnd(T, C, seed=seed + 4, dtype=dtype), d=d, low=low, y=y, A=A, dt_bias=rnd(C, seed=seed + 5, dtype=F32),
                skip=rnd(C, seed=seed + 6, dtype=F32), state=st, slot=slot, pos=pos, cu=cu)


def to(c):
    return {k: v.to(DEV) if isinstance(v, torch.Tensor) else v for k, v in c.items()}


SCAN = [  # channels, state entries, portions: every lane layout, tiles with and without a rest, few and many channels
    (128, 16, [1, 2, 33, 64, 130]), (512, 16, [40] * 9), (4096, 16, [70, 5, 16, 33]), (8192, 16, [50] * 9), (128, 9, [65]),
    (2176, 32, [17] * 9), (128, 24, [3, 100]), (128, 48, [70]), (384, 64, [31, 66]), (128, 100, [45, 2]), (128, 256, [40])]


@pytest.mark.parametrize("C,N,lens", SCAN)
@pytest.mark.parametrize("dtype", [BF, F32])
def test_selective_scan(C, N, lens, dtype):
    starts = [(0, 7, 0, 100)[i % 4] for i in range(len(lens))]  # some go on from a state
    c = scan_case(C, N, 20, lens, dtype, 1, starts=starts)
    dt = rnd(sum(lens), C, seed=9, dtype=F32)
    g, out, want = to(c), torch.zeros(sum(lens), C, dtype=dtype, device=DEV), torch.zeros(sum(lens), C, dtype=dtype)
    before = c["state"].clone()
    names = ("low", "y", "A", "dt_bias", "skip", "state", "slot", "pos", "cu")
    ops.selective_scan(g["u"], g["d"], dt.to(DEV), *(g[k] for k in names), max(lens), out)
    ops.selective_scan(c["u"], c["d"], dt, *(c[k] for k in names), max(lens), want)
    close(out, want, 6e-3 if dtype == BF else 3e-5)
    close(g["state"], c["state"], 3e-5)
    idle = [s for s in range(len(before)) if s not in c["slot"].tolist()]
    assert torch.equal(g["state"].cpu()[idle], before[idle])


@pytest.mark.parametrize("C,N,K,B", [(128, 16, 20, 1), (256, 16, 64, 5), (1024, 16, 256, 40), (128, 16, 130, 129), (128, 24, 1, 37),
                                     (384, 32, 64, 17), (128, 48, 33, 9), (128, 64, 64, 20), (128, 128, 64, 3), (256, 200, 96, 18)])
@pytest.mark.parametrize("dtype,slabs", [(BF, 1), (BF, 3), (F32, 1)])
def test_selective_step(C, N, K, B, dtype, slabs):
    """Decoded tokens behind prompt rows (row0), fresh sequences among them, slots in any order."""
    row0 = 3
    c = scan_case(C, N, K, [1] * (row0 + B), dtype, slabs, starts=[0 if i % 5 == 4 else 10 + i for i in range(row0 + B)])
    R = c["d"].rank
    w = rnd(C, R, seed=11, dtype=dtype, scale=R ** -0.5)
    slot = c["slot"][row0:].contiguous()
    want = c["y"][..., C:].float().sum(0).to(dtype) if slabs > 1 else c["y"][:, C:].contiguous()
    want[:row0] = 0
    out = want.to(DEV)
    step = c["low"][:, :R].to(dtype)
    step = step.contiguous() if dtype == BF else c["low"][:, :R]
    g = to(c)
    gstep = step.to(DEV) if dtype == BF else g["low"][:, :R]
    gw = ops.shuffle_weights(w.to(DEV)) if dtype == BF else w.to(DEV)
    ops.selective_step(g["u"], g["d"], gw, gstep, g["low"], g["A"], g["dt_bias"], g["skip"], g["state"], slot.to(DEV),
                       g["pos"], row0, out)
    ops.selective_step(c["u"], c["d"], w, step, c["low"], c["A"], c["dt_bias"], c["skip"], c["state"], slot, c["pos"],
                       row0, want)
    close(out, want, 8e-3 if dtype == BF else 3e-5)
    close(g["state"], c["state"], 2e-5)
    assert float(out[:row0].abs().sum()) == 0


@pytest.mark.parametrize("C,N", [(128, 16), (512, 24), (128, 64), (128, 200)])
@pytest.mark.parametrize("segs", [2, 3, 5])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_segmented_scan(C, N, segs, dtype):
    """Portions of unequal lengths cut into segments: some fill all of them, some end inside one or at an edge."""
    lens = [64 * segs + 7, 1, 64, 65, 130, 64 * segs]
    c = scan_case(C, N, 20, lens, dtype, 1, starts=[0, 5, 0, 9, 300, 2])
    c["A"] *= 0.05  # slow decays: what a segment hands on counts to the end
    dt = rnd(sum(lens), C, seed=9, dtype=F32) - 2
    g, out, want = to(c), torch.zeros(sum(lens), C, dtype=dtype, device=DEV), torch.zeros(sum(lens), C, dtype=dtype)
    names = ("low", "y", "A", "dt_bias", "skip", "state", "slot", "pos", "cu")
    ops.selective_scan(g["u"], g["d"], dt.to(DEV), *(g[k] for k in names), max(lens), out, segments=segs)
    ops.selective_scan(c["u"], c["d"], dt, *(c[k] for k in names), max(lens), want)
    close(out, want, 6e-3 if dtype == BF else 3e-5)
    close(g["state"], c["state"], 3e-5)


def test_segment_choice():
    seg = lambda C, n, q: ops.native().selective_segments((C, 16, 64, 64, 80, C), n, q)  # noqa: E731
    assert seg(8192, 16, 1024) == seg(8192, 4, 4096) == seg(128, 1, 511) == 1
    assert seg(8192, 1, 8192) == 8 and seg(4096, 1, 8192) == 16 and seg(128, 1, 1024) == 4


def test_scan_continued_by_steps_matches_one_scan():
    C, N, K, n = 256, 16, 64, 70
    c = scan_case(C, N, K, [n], F32, 1)
    w = rnd(C, 64, seed=11, dtype=F32, scale=0.1)
    dt = c["low"][:, :64] @ w.T
    outs = []
    for cuts in ([n], [1, 30, 2, 31]):
        g = to(dict(c, state=c["state"].clone()))
        out = torch.zeros(n, C, device=DEV)
        at = 0
        for m in cuts:
            o = torch.zeros(m, C, device=DEV)
            s = slice(at, at + m)
            ops.selective_scan(g["u"][s], g["d"], dt.to(DEV)[s], g["low"][s], g["y"][s], g["A"], g["dt_bias"], g["skip"], g["state"],
                               g["slot"], g["pos"][s].contiguous(), i32(0, m).to(DEV), m, o)
            out[s], at = o, at + m
        out[at:] = g["y"][at:, C:]
        for t in range(at, n):
            ops.selective_step(g["u"], g["d"], w.to(DEV), g["low"][:, :64], g["low"], g["A"], g["dt_bias"], g["skip"],
                               g["state"], g["slot"], g["pos"], t, out)
        outs.append((out.cpu(), g["state"].cpu()))
    close(outs[1][0], outs[0][0], 1e-5)
    close(outs[1][1], outs[0][1], 1e-5)


def test_scan_against_the_oracle_at_extreme_steps():
    """Steps from nearly zero (softplus of -40) to long ones, decays from none to all within a token."""
    C, N, T = 128, 16, 40
    c = scan_case(C, N, 20, [T], F32, 1)
    dt = torch.linspace(-40, 30, T * C).view(T, C)
    dt = dt[:, torch.randperm(C, generator=torch.Generator().manual_seed(0))].contiguous()
    a = -torch.exp(torch.linspace(-9, 4, N)).expand(C, N)
    c["A"][:, :N] = a / math.log(2)
    c["dt_bias"].zero_()
    g, out = to(c), torch.zeros(T, C, device=DEV)
    ops.selective_scan(g["u"], g["d"], dt.to(DEV), *(g[k] for k in ("low", "y", "A", "dt_bias", "skip", "state", "slot", "pos", "cu")), T, out)
    D = lambda t: t.double()  # noqa: E731
    y, S = oracle.selective_scan(D(c["u"]), oracle.softplus(D(dt)), D(a), D(c["low"][:, 64:64 + N]), D(c["low"][:, 80:80 + N]))
    want = (y + D(c["skip"]) * D(c["u"])) * oracle.silu(D(c["y"][:, C:]))
    close(out, want, 2e-6)
    close(g["state"][int(c["slot"][0])], S, 2e-6)
    small = dt < -20  # tiny steps keep their relative accuracy: one token, zero state
    g = to(c)
    g["skip"].zero_()
    for t in range(0, T, 7):
        o = torch.zeros(1, C, device=DEV)
        ops.selective_scan(g["u"][t:t + 1], g["d"], dt[t:t + 1].to(DEV), g["low"][t:t + 1], g["y"][t:t + 1], g["A"], g["dt_bias"],
                           g["skip"], g["state"], g["slot"], i32(0).to(DEV), i32(0, 1).to(DEV), 1, o)
        w = oracle.softplus(D(dt[t])) * D(c["u"][t]) * (D(c["low"][t, 64:64 + N]) * D(c["low"][t, 80:80 + N])).sum() * oracle.silu(D(c["y"][t, C:]))
        rel = ((o.cpu()[0].double() - w) / w).abs()[small[t]]
        assert rel.numel() == 0 or rel.max() < 2e-5


@pytest.mark.parametrize("C,taps,B", [(8, 1, 1), (128, 4, 5), (1032, 3, 130), (256, 16, 9)])
@pytest.mark.parametrize("dtype,yt,slabs", [(BF, BF, 1), (BF, F32, 5), (F32, F32, 1)])
def test_short_conv_step(C, taps, B, dtype, yt, slabs):
    row0, col0 = 2, 16
    y = rnd(*((slabs,) if slabs > 1 else ()), row0 + B, col0 + C + 8, dtype=yt)
    w, b = rnd(taps, C, dtype=F32), rnd(C, seed=1, dtype=F32)
    ring = rnd(B + 1, taps, C, seed=2, dtype=dtype)
    slot = torch.randperm(B + 1, generator=torch.Generator().manual_seed(1))[:B].int()
    pos = torch.cat([torch.zeros(row0), torch.arange(B) * 3 % 23]).int()
    gr, out, want = ring.to(DEV), torch.zeros(row0 + B, C, dtype=dtype, device=DEV), torch.zeros(row0 + B, C, dtype=dtype)
    z, zw = torch.zeros_like(out), torch.zeros_like(want)
    ops.short_conv_step(y.to(DEV), col0, w.to(DEV), b.to(DEV), gr, slot.to(DEV), pos.to(DEV), row0, out, 8, z)
    ops.short_conv_step(y, col0, w, b, ring, slot, pos, row0, want, 8, zw)
    close(z, zw, 4e-3 if dtype == BF else 1e-6)
    close(out, want, 8e-3 if dtype == BF else 3e-6)
    close(gr, ring, 4e-3 if dtype == BF else 1e-6)


@pytest.mark.parametrize("T,N,low,S", [(1, 128, 64, 1), (7, 384, 256, 16), (300, 96, 64, 3)])
def test_narrow_rows(T, N, low, S):
    z = rnd(*((S,) if S > 1 else ()), T, N, dtype=F32)
    full = z.sum(0) if S > 1 else z
    rows, lo = ops.narrow_rows(z.to(DEV), N - 8, low, T)
    close(rows, full[:, :N - 8], 1e-6)
    assert torch.equal(lo.cpu(), rows.cpu()[:, :low].to(BF))


@pytest.mark.parametrize("M,N,K", [(5, 128, 256), (2500, 384, 512), (4100, 384, 4096), (3000, 128, 256)])
def test_gemm_narrow(M, N, K):
    a, b = rnd(M, K), rnd(N, K, seed=3)
    got = ops.gemm_narrow(a.to(DEV), ops.shuffle_weights(b.to(DEV)))
    got = got.sum(0) if got.dim() == 3 else got
    close(got, a.float() @ b.float().t(), 2e-5)


# ------------------------------------------------------------------------------------------------ norms, gates, caps


@pytest.mark.parametrize("rows,cols,n", [(1, 128, 100), (7, 4096, 4096), (130, 2048, 2000), (3, 10240, 10000)])
@pytest.mark.parametrize("yt,dtype", [(BF, BF), (F32, BF), (F32, F32)])
@pytest.mark.parametrize("form", ["rows", "slabs", "pairs", "both", "pass"])
def test_post_norm_residual(rows, cols, n, yt, dtype, form):
    x, gain, post = rnd(rows, cols, dtype=F32), rnd(cols, seed=1, dtype=F32), rnd(cols, seed=6, dtype=F32)
    y = None if form == "pairs" else rnd(*((5,) if form != "rows" else ()), rows, cols, seed=2, dtype=yt)
    pairs = rnd(rows * 3, cols, seed=5, dtype=dtype) if form in ("pairs", "both") else None
    ids, table, step = torch.randint(0, 9, (rows,), dtype=torch.int32), rnd(9, cols, seed=3, dtype=F32), rnd(cols, seed=4, dtype=F32)
    for t in (x, gain, post, y, pairs, table, step):
        if t is not None:
            t[..., n:] = 0
    c = lambda t: None if t is None else t.to(DEV)  # noqa: E731
    xg = x.to(DEV)
    if form == "pass":  # a fresh stream: projection + vector + row of an fp32 table
        a = dict(bias=step, again=(ids, table), fresh=True)
        g = dict(bias=c(step), again=(c(ids), c(table)), fresh=True)
    else:
        a, g = dict(pairs=pairs, post=post), dict(pairs=c(pairs), post=c(post))
    h = ops.rms_residual(xg, c(y), c(gain), n, 1e-4, dtype, **g)
    hr = ops.rms_residual(x, y, gain, n, 1e-4, dtype, **a)
    close(xg, x, 3e-6)
    close(h, hr, 6e-3 if dtype == BF else 4e-6)
    raw = ops.rms_residual(xg, c(y), None, n, 1e-4, dtype, raw=True, **g)
    ops.rms_residual(x, y, None, n, 1e-4, dtype, raw=True, **a)
    close(xg, x, 3e-6)
    assert torch.equal(raw, xg.to(dtype))


@pytest.mark.parametrize("T,n,S", [(1, 64, 1), (33, 4096, 2), (5, 264, 7)])
@pytest.mark.parametrize("yt,dtype", [(BF, BF), (F32, BF), (F32, F32)])
def test_sigmoid_gate(T, n, S, yt, dtype):
    y = rnd(*((S,) if S > 1 else ()), T, 8 + n + 16, dtype=yt, scale=3)
    x = rnd(T, n + 8, seed=1, dtype=dtype)
    gx = x.to(DEV)
    ops.sigmoid_gate(y.to(DEV), 8, gx[:, :n])
    want = x[:, :n].clone()
    ops.sigmoid_gate(y, 8, want)
    close(gx[:, :n], want, 8e-3 if dtype == BF else 2e-6)
    assert torch.equal(gx[:, n:].cpu(), x[:, n:])


@pytest.mark.parametrize("cap", [0.7, 30.0])
@pytest.mark.parametrize("yt,S", [(BF, 1), (F32, 1), (F32, 3)])
def test_softcap(cap, yt, S):
    y = rnd(*((S,) if S > 1 else ()), 5, 1024, dtype=yt)
    y[..., :512] *= torch.logspace(-6, 3, 512).to(yt)
    got, want = ops.softcap(y.to(DEV), cap).cpu().double(), (y.double().sum(0) if S > 1 else y.double())
    want = cap * torch.tanh(want / cap)
    close(got, want, 3e-6)
    if S == 1:  # nothing summed: small logits keep their relative accuracy
        assert ((got - want).abs() <= 3e-6 * want.abs() + 1e-12).all()


# ------------------------------------------------------------------------------------------------ experts, ReLU gates


@pytest.mark.parametrize("M,N,K", [(1, 256, 128), (5, 2048, 512), (100, 768, 192), (300, 512, 512), (1100, 1024, 256), (2100, 1024, 512)])
def test_relu_gated_gemms(M, N, K):
    x, w, b = rnd(M, K), rnd(N, K, seed=2), rnd(N, seed=3, dtype=F32)
    want, wantb = ref.gemm_bt(x, w, epilogue=ops.EPI_REGLU8), ref.gemm_bt(x, w, epilogue=ops.EPI_REGLU8, glu_bias=b)
    ws = ops.shuffle_weights(w.to(DEV))
    close(ops.gemm_bt(x.to(DEV), ws, epilogue=ops.EPI_REGLU8, shuffled=True), want, 1.2e-2)
    close(ops.gemm_bt(x.to(DEV), ws, epilogue=ops.EPI_REGLU8, shuffled=True, glu_bias=b.to(DEV)), wantb, 1.2e-2)
    close(ops.gemm_bt(x.to(DEV), w.to(DEV), epilogue=ops.EPI_REGLU8), want, 1.2e-2)
    if M <= 16 and K % 128 == 0:
        close(ops.stream_gemm(x.to(DEV), ws, epilogue=ops.EPI_REGLU8, cfg=30, nt=True), want, 1.2e-2)


@pytest.mark.parametrize("T,E,top", [(1, 1, 1), (9, 16, 1), (33, 70, 6), (5, 300, 64), (3, 1000, 2)])
def test_sigmoid_route(T, E, top):
    z = torch.stack([torch.linspace(-9, 9, E)[torch.randperm(E, generator=torch.Generator().manual_seed(t))] for t in range(T)])
    idx, wt = ops.moe_route(torch.cat([torch.zeros(T, 8), z], 1).to(DEV), 8, E, top, 1.0, T, "sigmoid")
    want = oracle.route(z.double(), top)
    got = torch.zeros(T, E).double().scatter(1, idx.cpu().long(), wt.cpu().double())
    close(got, want, 1e-6)


@pytest.mark.parametrize("T,E,top,K,F,W", [(1, 4, 1, 128, 64, 128), (40, 8, 3, 256, 128, 256), (1500, 4, 2, 128, 64, 128)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_experts_of_the_weighted_input(T, E, top, K, F, W, dtype):
    h, gate, up, down = rnd(T, K, dtype=dtype), rnd(E, F, K, seed=1, dtype=dtype, scale=0.2), rnd(E, F, K, seed=2, dtype=dtype, scale=0.2), rnd(E, W, F, seed=3, dtype=dtype)
    idx = torch.stack([torch.randperm(E, generator=torch.Generator().manual_seed(t))[:top] for t in range(T)]).int()
    wt = torch.rand(T, top, generator=torch.Generator().manual_seed(0))
    if dtype == BF:
        gu = torch.cat([torch.stack([gate[e].view(-1, 8, K), up[e].view(-1, 8, K)], 1).reshape(2 * F, K) for e in range(E)])
        gu, dn, grp = ops.shuffle_weights(gu.to(DEV)), ops.shuffle_weights(down.reshape(E * W, F).to(DEV)), 8
    else:
        gu, dn, grp = torch.cat([gate, up], 1).reshape(2 * E * F, K).to(DEV), down.reshape(E * W, F).to(DEV), 0
    got = ops.moe_experts(h.to(DEV), idx.to(DEV), wt.to(DEV), gu, dn, E, grp, "input").view(T, top, W)
    want = torch.zeros(T, top, W).double()
    for t in range(min(T, 60)):
        for k in range(top):
            e, x = int(idx[t, k]), h[t].double() * wt[t, k].double()
            want[t, k] = (oracle.silu(x @ gate[e].double().T) * (x @ up[e].double().T)) @ down[e].double().T
    close(got[:60], want[:60], 1.5e-2 if dtype == BF else 1e-5)


# ------------------------------------------------------------------------------------------------ rotary latents


ROPE = [  # heads, head width, unrotated, rotated, rank, row width
    (3, 64, 40, 12, 80, 128), (2, 128, 96, 32, 512, 576), (5, 64, 16, 32, 48, 128), (1, 64, 1, 2, 1, 64), (4, 320, 200, 64, 250, 320)]


@pytest.mark.parametrize("H,D,dim,P,rank,R", ROPE)
@pytest.mark.parametrize("yt,dtype,S", [(BF, BF, 1), (BF, BF, 4), (F32, BF, 3), (F32, F32, 1)])
def test_latent_write_rotates(H, D, dim, P, rank, R, yt, dtype, S):
    T, bs = 9, 16
    qa, ca = -(-dim // 8) * 8, -(-rank // 8) * 8
    y = torch.zeros(S, T, H * D + R + 64)
    q, row = y[..., :H * D].unflatten(2, (H, D)), y[..., H * D:H * D + R]
    q[..., :dim], q[..., qa:qa + P] = rnd(S, T, H, dim, dtype=F32), rnd(S, T, H, P, seed=1, dtype=F32)
    row[..., :rank], row[..., ca:ca + P] = rnd(S, T, rank, seed=2, dtype=F32), rnd(S, T, P, seed=3, dtype=F32)
    y = (y if S > 1 else y[0]).to(yt)
    pos = i32(0, 1, 2, 63, 64, 1000, 100003, 7, 0)
    slots = torch.tensor([3, 17, 16, -1, 40, 41, 0, 63, 5])
    yarn = Yarn(3.0, 600, 20.0, 1.5)
    gain = torch.zeros(R)
    gain[:rank] = rnd(rank, seed=4, dtype=F32)
    out = []
    for dev in ("cpu", DEV):
        cache = torch.zeros(4, bs, R, dtype=dtype, device=dev)
        rope = ops.LatentRope(ops.rope_turns(P, 1000.0, dev, yarn), 1.1, P, D, qa, ca, pos.to(dev))
        out.append((ops.latent_write(y.to(dev), H * D, gain.to(dev), cache, slots.to(dev), rank, 1e-5, rope), cache))
    tol = 1e-2 if dtype == BF else 3e-6
    close(out[1][0], out[0][0], tol)
    close(out[1][1], out[0][1], tol)


@pytest.mark.parametrize("T,H,D,P,q_at,R,c_at", [(1, 1, 64, 2, 0, 64, 8), (130, 32, 128, 32, 96, 576, 512), (9, 5, 256, 20, 40, 320, 256)])
def test_latent_key_fill(T, H, D, P, q_at, R, c_at):
    kv, rows = rnd(T, 2, H, D), rnd(T, R, seed=1)
    g = kv.to(DEV)
    ops.latent_key_fill(g[:, 0], rows.to(DEV), q_at, c_at, P)
    n = -(-P // 8) * 8
    want = kv.clone()
    want[:, 0, :, q_at:q_at + n] = rows[:, None, c_at:c_at + n]
    assert torch.equal(g.cpu(), want)


@pytest.mark.parametrize("R,V,H", [(320, 256, 3), (320, 256, 40), (576, 512, 16), (576, 512, 33)])
@pytest.mark.parametrize("parts,min_part", [(1, 128), (5, 64)])
def test_latent_decode_of_rows_with_a_rotated_key(R, V, H, parts, min_part):
    """Scores over the whole row, values from its latent part; one far key stands out for one head."""
    bs, ctx = 64, i32(1, 64, 65, 200, 517)
    B = ctx.numel()
    bt = torch.randperm(B * 9, generator=torch.Generator().manual_seed(1)).view(B, 9).int()
    cache, q = rnd(B * 9, bs, R), rnd(B, H, R, seed=2, scale=0.3)
    cache[bt[4, 1], 5, V:] *= 6
    q[4, H - 1, V:] = cache[bt[4, 1], 5, V:]
    ws = ops.LatentWorkspace(B * H * parts, B * H * parts * R, DEV)
    got = ops.latent_decode(q.to(DEV), cache.to(DEV), bt.to(DEV), ctx.to(DEV), 0.08, 0, None, parts, ws, None, min_part, values=V)
    assert got.shape == (B, H, V)
    want = ref.latent_attention(q, cache, bt, None, ctx, 0.08, 0, None)[..., :V]
    close(got, want, 1.5e-2)
    full = ops.latent_decode(q.to(DEV), cache.to(DEV), bt.to(DEV), ctx.to(DEV), 0.08)  # every column is a value
    close(full, ref.latent_attention(q, cache, bt, None, ctx, 0.08, 0, None), 1.5e-2)


def test_shapes_are_refused_on_the_host():
    c = to(scan_case(128, 16, 20, [4], BF, 1))
    out, dt = torch.zeros(4, 128, dtype=BF, device=DEV), torch.zeros(4, 128, device=DEV)
    args = [c[k] for k in ("low", "y", "A", "dt_bias", "skip", "state", "slot", "pos", "cu")]
    for i, bad in ((0, c["low"][:, :40]), (1, c["y"][:, :200]), (2, c["A"][:, :8].contiguous()), (5, c["state"][:, :64].contiguous()),
                   (6, c["slot"].long()), (7, c["pos"][:2])):
        a = list(args)
        a[i] = bad
        with pytest.raises((ValueError, TypeError)):
            ops.selective_scan(c["u"], c["d"], dt, *a, 4, out)
    with pytest.raises(ValueError):
        ops.selective_scan(c["u"], c["d"], dt.to(BF), *args, 4, out)
    with pytest.raises(ValueError):
        ops.softcap(torch.zeros(2, 12, device=DEV), 1.0)
    with pytest.raises(ValueError):
        ops.moe_route(torch.zeros(2, 16, device=DEV), 0, 4, 1, 1.0, 2, "cosine")
    with pytest.raises(ValueError):
        ops.latent_key_fill(torch.zeros(2, 1, 64, dtype=BF, device=DEV), torch.zeros(2, 64, dtype=BF, device=DEV), 60, 0, 8)
