"""Dynamic-Tanh and latent-attention kernels against plain fp32 / fp64 formulas (ops.reference on the CPU)."""
import pytest
import torch

from django_assistant_bot_amd import ops
from django_assistant_bot_amd.ops import reference as ref
from django_assistant_bot_amd.ops.latent import DytNorm, decode_split

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


def rnd(*shape, seed=0, dtype=torch.bfloat16, scale=1.0):
    g = torch.Generator().manual_seed(seed + sum(shape))
    return (torch.randn(shape, generator=g) * scale).to(dtype)


def close(got, want, tol):
    got, want = got.float().cpu(), want.float()
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-6)
    assert err < tol, err


def norm(cols, seed):
    return DytNorm(0.3 + 0.2 * seed, rnd(cols, seed=seed, dtype=torch.float32) + 1, rnd(cols, seed=seed + 9, dtype=torch.float32))


def on_gpu(n):
    return DytNorm(n.alpha, n.w.to(DEV), n.b.to(DEV))


@pytest.mark.parametrize("rows,cols", [(1, 64), (5, 320), (130, 2048), (3000, 4096), (700, 192)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_embed_dyt(rows, cols, dtype):
    table, n = rnd(50, cols, dtype=dtype), norm(cols, 1)
    ids = torch.randint(0, 50, (rows,), dtype=torch.int32)
    x, h = ops.embed_dyt(ids.to(DEV), table.to(DEV), 7.5, on_gpu(n))
    xr, hr = ref.embed_dyt(ids, table, 7.5, n)
    close(x, xr, 1e-6)
    close(h, hr, 5e-3 if dtype == torch.bfloat16 else 1e-6)


@pytest.mark.parametrize("rows,cols,S", [(1, 320, 1), (7, 4096, 16), (130, 2048, 5), (2500, 1024, 1)])
@pytest.mark.parametrize("yt", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("parts", ["all", "no_next", "no_post", "no_scale"])
def test_dyt_residual(rows, cols, S, yt, parts):
    x = rnd(rows, cols, seed=2, dtype=torch.float32)
    y = rnd(S, rows, cols, seed=3, dtype=yt) if S > 1 else rnd(rows, cols, seed=3, dtype=yt)
    post = None if parts == "no_post" else norm(cols, 1)
    nxt = None if parts == "no_next" else norm(cols, 2)
    ls = None if parts == "no_scale" else rnd(cols, seed=5, dtype=torch.float32)
    ht = torch.float32 if yt == torch.float32 and S == 1 else torch.bfloat16
    xg = x.to(DEV)
    h = ops.dyt_residual(xg, y.to(DEV), post and on_gpu(post), None if ls is None else ls.to(DEV), nxt and on_gpu(nxt), ht)
    hr = ref.dyt_residual(x, y, post, ls, nxt, ht)
    close(xg, x, 2e-6)
    if nxt is None:
        assert h is None
    else:
        close(h, hr, 6e-3 if ht == torch.bfloat16 else 2e-6)


def test_dyt_small_and_large_arguments():
    v = torch.cat([torch.logspace(-8, 2, 500), -torch.logspace(-8, 2, 500), torch.zeros(8)])
    v = v.repeat(8)[:8064].view(1, -1).float()
    n = DytNorm(1.0, torch.ones(v.shape[1]), torch.zeros(v.shape[1]))
    h = ops.dyt_residual(v.clone().to(DEV), torch.zeros_like(v).to(DEV), None, None, on_gpu(n), torch.float32).cpu()
    want = torch.tanh(v.double())
    rel = ((h.double() - want).abs() / want.abs().clamp_min(1e-30)).max().item()
    assert rel < 5e-7, rel


@pytest.mark.parametrize("M,N,K", [(1, 64, 16), (70, 132, 320), (200, 448, 64), (64, 64, 2048)])
def test_gemm_f32(M, N, K):
    a, b = rnd(M, K, dtype=torch.float32), rnd(N, K, seed=4, dtype=torch.float32)
    close(ops.gemm_f32(a.to(DEV), b.to(DEV)), (a.double() @ b.double().t()).float(), 3e-6)


def test_glu_f32():
    x = rnd(37, 2 * 200, dtype=torch.float32, scale=3)
    for act in ("gelu", "silu", "relu"):
        close(ops.glu_f32(x.to(DEV), act), ops.glu_f32(x, act), 2e-6)


@pytest.mark.parametrize("M,N,K", [(1, 128, 128), (5, 2048, 512), (100, 768, 192), (130, 1024, 256), (300, 512, 512),
                                   (1100, 1024, 256)])
def test_geglu8_epilogue(M, N, K):
    """The tanh-GELU gate in every GEMM kernel a gate|up projection can take (streaming, tile, mid-M, 256 x 256)."""
    x, w = rnd(M, K), rnd(N, K, seed=2, scale=K ** -0.5)
    want = ref.gemm_bt(x, w, epilogue=ops.EPI_GEGLU8)
    close(ops.gemm_bt(x.to(DEV), ops.shuffle_weights(w).to(DEV), epilogue=ops.EPI_GEGLU8, shuffled=True), want, 1.2e-2)
    close(ops.gemm_bt(x.to(DEV), w.to(DEV), epilogue=ops.EPI_GEGLU8), want, 1.2e-2)
    if M <= 16 and N % 128 == 0 and K % 128 == 0:
        got = ops.stream_gemm(x.to(DEV), ops.shuffle_weights(w).to(DEV), epilogue=ops.EPI_GEGLU8, cfg=30, nt=True)
        close(got, want, 1.2e-2)


@pytest.mark.parametrize("T,H,K,N", [(1, 3, 64, 128), (5, 4, 128, 512), (20, 2, 64, 64), (33, 3, 512, 128), (200, 2, 192, 64)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_head_gemm(T, H, K, N, dtype):
    """Strided per-head input, weight rows at an offset."""
    wide = rnd(T, H * K + 64, dtype=dtype)
    w = rnd(16 + H * N, K, seed=3, dtype=dtype, scale=K ** -0.5)
    x = wide[:, :H * K].unflatten(1, (H, K))
    want = torch.einsum("thk,hnk->thn", x.double(), w[16:].view(H, N, K).double())
    wg = ops.shuffle_weights(w).to(DEV) if dtype == torch.bfloat16 else w.to(DEV)
    xg = wide.to(DEV)[:, :H * K].unflatten(1, (H, K))
    close(ops.head_gemm(xg, wg, N, row0=16), want.to(dtype), 1e-2 if dtype == torch.bfloat16 else 3e-6)
    out = torch.full((T, H, N + 8), 3.0, dtype=dtype, device=DEV)
    ops.head_gemm(xg, wg, N, row0=16, out=out[..., :N])
    close(out[..., :N], want.to(dtype), 1e-2 if dtype == torch.bfloat16 else 3e-6)
    assert bool((out[..., N:] == 3.0).all())


@pytest.mark.parametrize("R,rank", [(64, 48), (128, 128), (512, 500), (768, 768)])
@pytest.mark.parametrize("S", [1, 6])
def test_latent_write(R, rank, S):
    T, HD = 9, 192
    y = rnd(*((S,) if S > 1 else ()), T, HD + R)
    y[..., HD + rank:] = 0
    gain = rnd(R, seed=7, dtype=torch.float32)
    slots = torch.tensor([70, -1, 3, 4, 127, 0, 64, -1, 65])
    cache, cg = torch.zeros(2, 64, R, dtype=torch.bfloat16), torch.zeros(2, 64, R, dtype=torch.bfloat16, device=DEV)
    q = ops.latent_write(y.to(DEV), HD, gain.to(DEV), cg, slots.to(DEV), rank, 1e-5)
    qr = ref.latent_write(y, HD, gain, cache, slots, rank, 1e-5)
    close(q, qr, 1e-2)
    close(cg, cache, 1.2e-2)
    assert torch.equal((cg.cpu() != 0).any(-1), (cache != 0).any(-1))
    q = ops.latent_write(y[..., :HD].contiguous().to(DEV), HD, None, None, slots.to(DEV), rank, 1e-5)
    close(q, qr, 1e-2)


class Paged:
    """Latents of sequences of the given lengths scattered over a page pool."""

    def __init__(self, lens, R, dtype=torch.bfloat16, bs=64, seed=0):
        per = [-(-n // bs) for n in lens]
        perm = torch.randperm(sum(per) + 3, generator=torch.Generator().manual_seed(seed)).to(torch.int32)
        self.cache = rnd(sum(per) + 3, bs, R, seed=seed, dtype=dtype)
        self.bt = torch.zeros(len(lens), max(per) + 1, dtype=torch.int32)
        o = 0
        for i, n in enumerate(per):
            self.bt[i, :n] = perm[o:o + n]
            o += n
        self.ctx = torch.tensor(lens, dtype=torch.int32)

    def gpu(self):
        return self.cache.to(DEV), self.bt.to(DEV), self.ctx.to(DEV)


def test_latent_gather():
    p = Paged([130, 7, 64, 200], 128)
    cu = torch.tensor([0, 100, 107, 108, 264], dtype=torch.int32)
    c, bt, ctx = p.gpu()
    got = ops.latent_gather(c, bt, cu.to(DEV), ctx, 264)
    assert torch.equal(got.cpu(), ref.latent_gather(p.cache, p.bt, cu, p.ctx))


DECODE = [(64, 1, 33), (64, 20, 0), (128, 6, 70), (128, 40, 1), (192, 3, 128), (192, 64, 65), (256, 33, 0), (256, 5, 64),
          (384, 16, 200), (384, 40, 0), (512, 32, 130), (512, 8, 0), (512, 50, 63)]


@pytest.mark.parametrize("R,H,window", DECODE)
@pytest.mark.parametrize("parts,min_part", [(1, 128), (3, 64), (9, 64), (40, 128)])
def test_latent_decode(R, H, window, parts, min_part):
    lens = [1, 64, 65, 129, 300, 517, 1030]
    p = Paged(lens, R, seed=R + H)
    q = rnd(len(lens), H, R, seed=5, scale=2.0)
    sink = rnd(H, seed=1, dtype=torch.float32, scale=2.0)
    scale = R ** -0.5
    c, bt, ctx = p.gpu()
    kw = dict(parts=parts, min_part=min_part)
    if parts > 1:
        rows = len(lens) * H * parts
        ws = ops.LatentWorkspace(rows, rows * R, DEV)
        ws.o.fill_(float("nan"))  # a partition that nobody wrote must not be read
        ws.ml.fill_(float("nan"))
        kw.update(workspace=ws, order=torch.tensor([5, 4, 3, 6, 2, 1, 0], dtype=torch.int32, device=DEV))
    for s in (sink, None):
        got = ops.latent_decode(q.to(DEV), c, bt, ctx, scale, window, None if s is None else s.to(DEV), **kw)
        close(got, ref.latent_attention(q, p.cache, p.bt, None, p.ctx, scale, window, s), 1.5e-2)


def test_decode_split():
    assert decode_split(1, 32, 512, 0, 2048) == (32, 64) and decode_split(128, 32, 512, 4096, 8192) == (4, 128)
    assert decode_split(1, 4, 64, 100, 8192) == (3, 64) and decode_split(600, 4, 64, 0, 8192) == (1, 128)


@pytest.mark.parametrize("dtype,R,bs", [(torch.float32, 96, 64), (torch.float32, 1024, 32), (torch.bfloat16, 640, 64),
                                        (torch.float32, 64, 16)])
@pytest.mark.parametrize("window", [0, 1, 100, 300])
def test_latent_any(dtype, R, bs, window):
    lens, ql = [1, 40, 290, 600], [1, 2, 130, 5]
    p = Paged(lens, R, dtype, bs)
    cu = torch.tensor([0, 1, 3, 133, 138], dtype=torch.int32)
    q, sink = rnd(sum(ql), 3, R, dtype=dtype, seed=2, scale=2.0), rnd(3, dtype=torch.float32)
    c, bt, ctx = p.gpu()
    tol = 1.2e-2 if dtype == torch.bfloat16 else 5e-6
    got = ops.latent_attention(q.to(DEV), c, bt, cu.to(DEV), ctx, R ** -0.5, window, sink.to(DEV))
    close(got, ref.latent_attention(q, p.cache, p.bt, cu, p.ctx, R ** -0.5, window, sink), tol)
    got = ops.latent_attention(q[:4].to(DEV).contiguous(), c, bt, None, ctx, R ** -0.5, window)
    close(got, ref.latent_attention(q[:4], p.cache, p.bt, None, p.ctx, R ** -0.5, window, None), tol)


@pytest.mark.parametrize("D", [64, 128, 256])
@pytest.mark.parametrize("window", [0, 1, 33, 64, 65, 300])
@pytest.mark.parametrize("with_sink", [True, False])
def test_flash_window(D, window, with_sink):
    H, ql, kl = 3, [1, 200, 17, 130], [1, 200, 210, 400]
    cq = torch.tensor([0, *torch.tensor(ql).cumsum(0)], dtype=torch.int32)
    ck = torch.tensor([0, *torch.tensor(kl).cumsum(0)], dtype=torch.int32)
    wide = rnd(sum(ql), H * D + 64, seed=1, scale=1.5)
    q = wide[:, :H * D].unflatten(1, (H, D))
    kv = rnd(sum(kl), 2, H, D, seed=2)
    sink = rnd(H, dtype=torch.float32, scale=3) if with_sink else None
    qg, kvg = wide.to(DEV)[:, :H * D].unflatten(1, (H, D)), kv.to(DEV)
    got = ops.flash_attention_window(qg, kvg[:, 0], kvg[:, 1], cq.to(DEV), ck.to(DEV), max(ql), 0.1, window,
                                     None if sink is None else sink.to(DEV))
    close(got, ref.flash_attention_window(q, kv[:, 0], kv[:, 1], cq, ck, 0.1, window, sink), 1.5e-2)


@pytest.mark.parametrize("window", [64, 70, 128])
def test_one_key_at_the_window_edge_decides(window):
    """One latent stands out by far: seen from exactly `window` - 1 tokens later, and not one token later."""
    R, H, pos = 128, 2, 100
    p = Paged([pos + window, pos + window + 1], R)
    p.cache.mul_(0.01)
    for b in range(2):
        p.cache[p.bt[b, pos // 64], pos % 64] = torch.ones(R, dtype=torch.bfloat16)
    q = torch.ones(2, H, R, dtype=torch.bfloat16)
    c, bt, ctx = p.gpu()
    got = ops.latent_decode(q.to(DEV), c, bt, ctx, 0.5, window).float().cpu()
    assert (got[0] > 0.99).all() and (got[1].abs() < 0.05).all()
    any_ = ops.latent_attention(q.to(DEV), c, bt, None, ctx, 0.5, window).float().cpu()
    assert (any_[0] > 0.99).all() and (any_[1].abs() < 0.05).all()
    n = pos + window + 1
    k = torch.zeros(n, 2, H, R, dtype=torch.bfloat16)
    k[pos] = 1
    cu = torch.tensor([0, n], dtype=torch.int32, device=DEV)
    o = ops.flash_attention_window(torch.ones(n, H, R, dtype=torch.bfloat16, device=DEV), k.to(DEV)[:, 0], k.to(DEV)[:, 1], cu,
                                   cu, n, 0.5, window).float().cpu()
    assert (o[pos:pos + window] > 0.99).all() and (o[:pos] == 0).all() and (o[pos + window] == 0).all()


def test_sink_beyond_every_score():
    """A sink far above the scores empties the output, one far below changes nothing."""
    p = Paged([300], 128)
    q = rnd(1, 4, 128)
    c, bt, ctx = p.gpu()
    base = ops.latent_decode(q.to(DEV), c, bt, ctx, 0.1, 0)
    for v, want in ((400.0, 0.0), (-400.0, None)):
        s = torch.full((4,), v, device=DEV)
        got = ops.latent_decode(q.to(DEV), c, bt, ctx, 0.1, 0, s)
        assert torch.isfinite(got.float()).all()
        if want is None:
            close(got, base.float().cpu(), 1e-2)
        else:
            assert float(got.float().abs().max()) < 1e-6


def test_shapes_are_refused_on_the_host():
    x = torch.zeros(4, 64, device=DEV)
    n = on_gpu(norm(72, 1))
    with pytest.raises(ValueError):
        ops.dyt_residual(x, torch.zeros(4, 64, device=DEV), n, None, None)
    with pytest.raises(ValueError):
        ops.head_gemm(torch.zeros(2, 3, 48, device=DEV, dtype=torch.bfloat16),
                      torch.zeros(96, 48, device=DEV, dtype=torch.bfloat16), 32)
