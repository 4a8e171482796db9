"""HIP kernels of the Bekulix serving path against their float32 PyTorch references (same op, run on CPU
copies of the inputs), on ragged batches that mix fresh sequences, continued portions and single
decode tokens, in bfloat16 and float32."""

import pytest
import torch

from colossalai_amd.ops import differential, latent_attention, normed_keys, streams
from colossalai_amd.ops.activation import relu_mul
from colossalai_amd.ops.paged_attention import paged_attention, paged_attention_ref
from colossalai_amd.ops.ragged import RaggedBatch

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
MIXED = ([37, 5, 1, 1, 1, 70, 1], [0, 21, 63, 64, 0, 130, 299])      # portions beside decode tokens
DECODE = ([1] * 6, [0, 5, 63, 64, 700, 127])                          # decode tokens alone
LONG = ([200, 140], [0, 61])


def tol(dtype):
    return dict(rtol=2e-5, atol=2e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)


def make_batch(shape, page=16):
    counts, starts = shape
    tables, nxt = [], 0
    for c, s in zip(counts, starts):
        need = (c + s + page - 1) // page
        tables.append(list(range(nxt + need - 1, nxt - 1, -1)))  # pages in descending order: not contiguous
        nxt += need
    slots = list(range(len(counts)))
    return (RaggedBatch.build(counts, starts, slots, "cuda", tables, page),
            RaggedBatch.build(counts, starts, slots, "cpu", tables, page), nxt)


def both(fn, ref, args_gpu, args_cpu, **kw):
    return fn(*args_gpu, **{k: v.cuda() if isinstance(v, torch.Tensor) else v for k, v in kw.items()}), ref(*args_cpu, **kw)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [MIXED, DECODE, LONG])
@pytest.mark.parametrize("H,G,D", [(8, 2, 128), (6, 3, 64), (4, 4, 72), (5, 1, 40), (3, 1, 20), (16, 2, 256), (12, 1, 16), (2, 2, 7)])
def test_attention_over_shared_keys_and_values(dtype, shape, H, G, D):
    torch.manual_seed(D)
    bg, bc, pages = make_batch(shape)
    N = bc.num_tokens
    q = torch.randn(N, H, D).to(dtype)
    pool, fac = torch.randn(pages, 16, G, D).to(dtype), torch.rand(pages, 16, G) * 2 + 0.1
    pc, pg = pool.clone(), pool.cuda()
    got, want = both(paged_attention, paged_attention_ref, (q.cuda(), pg, pg, bg, D ** -0.5), (q, pc, pc, bc, D ** -0.5),
                     key_factors=fac)
    torch.testing.assert_close(got.cpu().float(), want.float(), **tol(dtype))
    # a window over shared rows, without factors
    got, want = both(paged_attention, paged_attention_ref, (q.cuda(), pg, pg, bg, 0.7 * D ** -0.5), (q, pc, pc, bc, 0.7 * D ** -0.5),
                     window=50, out_dtype=torch.float32)
    torch.testing.assert_close(got.cpu(), want, **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [MIXED, DECODE])
@pytest.mark.parametrize("H,D,Dv", [(8, 96, 64), (16, 320, 256), (4, 40, 24), (3, 20, 12), (5, 512, 512), (2, 136, 128)])
def test_values_that_are_leading_channels_of_the_keys(dtype, shape, H, D, Dv):
    torch.manual_seed(D)
    bg, bc, pages = make_batch(shape)
    q, pool = torch.randn(bc.num_tokens, H, D).to(dtype), torch.randn(pages, 16, 1, D).to(dtype)
    pg = pool.cuda()
    for kw in (dict(), dict(window=70), dict(window=64, keep_first=3)):
        got, want = both(paged_attention, paged_attention_ref, (q.cuda(), pg, pg[..., :Dv], bg, D ** -0.5),
                         (q, pool, pool[..., :Dv], bc, D ** -0.5), **kw)
        torch.testing.assert_close(got.cpu().float(), want.float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [MIXED, DECODE, LONG])
@pytest.mark.parametrize("chunk", [1, 31, 64, 70, 1000])
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 64, 128), (6, 2, 48, 96), (2, 2, 32, 40), (3, 1, 10, 18), (5, 5, 16, 32)])
def test_attention_inside_blocks_over_shared_value_heads(dtype, shape, chunk, H, G, D, Dv):
    torch.manual_seed(chunk)
    bg, bc, pages = make_batch(shape)
    q = torch.randn(bc.num_tokens, 2 * H, D).to(dtype)
    kp, vp = torch.randn(pages, 16, 2 * G, D).to(dtype), torch.randn(pages, 16, G, Dv).to(dtype)
    got, want = both(paged_attention, paged_attention_ref, (q.cuda(), kp.cuda(), vp.cuda(), bg, D ** -0.5), (q, kp, vp, bc, D ** -0.5),
                     chunk=chunk, out_dtype=torch.float32)
    assert got.dtype == torch.float32
    t = tol(dtype) if dtype == torch.float32 else dict(rtol=4e-3, atol=4e-3)  # float32 out: weights keep their mantissa
    torch.testing.assert_close(got.cpu(), want, **t)
    gd = differential.difference_norm(got, G, 0.6, 0.8, 1e-5, dtype)
    wd = differential.difference_norm_ref(got.cpu(), G, 0.6, 0.8, 1e-5, dtype)
    torch.testing.assert_close(gd.cpu().float(), wd.float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D", [(8, 2, 128), (3, 3, 20), (5, 1, 264), (2, 1, 500), (4, 2, 64), (7, 7, 8)])
@pytest.mark.parametrize("every", [0, 1, 17])
def test_query_norm_and_key_write(dtype, H, G, D, every):
    torch.manual_seed(H)
    bg, bc, pages = make_batch(MIXED)
    N = bc.num_tokens
    packed = torch.randn(N, (H + G) * D + 3).to(dtype)          # strided rows of a wider projection
    w = torch.randn(D)
    out = []
    for b, dev in ((bg, "cuda"), (bc, "cpu")):
        p = packed.to(dev)
        kpool = torch.full((pages, 16, G, D), 7.0, dtype=dtype, device=dev)
        fac = torch.full((pages, 16, G), -1.0, device=dev)
        q = normed_keys.query_norm_key_write(p[:, : H * D].unflatten(1, (H, D)),
                                             p[:, H * D : (H + G) * D].unflatten(1, (G, D)), w.to(dev), 1e-5, kpool, fac, b, 0.4, every)
        out.append((q.cpu().float(), kpool.cpu(), fac.cpu()))
    torch.testing.assert_close(out[0][0], out[1][0], **tol(dtype))
    assert torch.equal(out[0][1], out[1][1])
    torch.testing.assert_close(out[0][2], out[1][2], rtol=1e-5, atol=1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("S,W", [(1, 96), (2, 2048), (3, 1028), (4, 4096), (4, 8192), (6, 200), (8, 64), (5, 33), (12, 130), (4, 9000)])
def test_streams(dtype, S, W):
    torch.manual_seed(W)
    N, V = 13, 29
    table, toks = torch.randn(V, W).to(dtype), torch.randint(0, V, (N,))
    read, write, mix, w = torch.randn(S), torch.randn(S), torch.randn(S, S), torch.randn(W)
    xg, hg = streams.streams_start(table.cuda(), toks.cuda(), S, read.cuda(), w.cuda(), 1e-5)
    xc, hc = streams.streams_start_ref(table, toks, S, read, w, 1e-5)
    assert torch.equal(xg.cpu(), xc)
    torch.testing.assert_close(hg.cpu().float(), hc.float(), **tol(dtype))
    for rd in (read, None):
        y = torch.randn(N, W).to(dtype)
        hg = streams.streams_update(xg, y.cuda(), mix.cuda(), write.cuda(), None if rd is None else rd.cuda(), w.cuda(), 1e-5, dtype)
        hc = streams.streams_update_ref(xc, y, mix, write, rd, w, 1e-5, dtype)
        torch.testing.assert_close(xg.cpu(), xc, rtol=1e-4, atol=1e-4)
        torch.testing.assert_close(hg.cpu().float(), hc.float(), **(dict(rtol=1e-3, atol=1e-3) if dtype == torch.float32 else tol(dtype)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [40, 33, 1024])
def test_relu_mul(dtype, ff):
    packed = (torch.randn(17, 2 * ff + 5) * 2).to(dtype)[:, : 2 * ff]
    with torch.no_grad():
        torch.testing.assert_close(relu_mul(packed.cuda()).cpu().float(), relu_mul(packed).float(), **tol(dtype))


@pytest.mark.parametrize("shape", [MIXED, LONG])
@pytest.mark.parametrize("window", [0, 1, 33, 64, 500])
@pytest.mark.parametrize("page", [16, 64])
def test_both_forms_of_latent_attention_agree(shape, window, page):
    """bfloat16: the per-head form over the visible part of the context against the absorbed form in float32."""
    torch.manual_seed(window)
    H, D, Dv, rank = 4, 40, 64, 72
    bg, bc, pages = make_batch(shape, page)
    N = bc.num_tokens
    q, pool = torch.randn(N, H, D).bfloat16(), torch.randn(pages, page, 1, rank).bfloat16()
    uk, uv = (torch.randn(H, D, rank) / rank ** 0.5).bfloat16(), (torch.randn(H, Dv, rank) / rank ** 0.5).bfloat16()
    assert latent_attention.expands(q.cuda(), uk, uv, bg)
    got = latent_attention.latent_attention(q.cuda(), uk.cuda(), uv.cuda(), pool.cuda(), bg, 0.15, None, rank, window=window)
    want = latent_attention.latent_attention(q.float(), uk.float(), uv.float(), pool.float(), bc, 0.15, None, rank, window=window)
    torch.testing.assert_close(got.cpu().float(), want, rtol=3e-2, atol=3e-2)


def test_shapes_the_kernels_do_not_take_are_refused():
    bg, _, pages = make_batch(DECODE)
    q, kp = torch.zeros(6, 4, 16, device="cuda"), torch.zeros(pages, 16, 2, 16, device="cuda")
    with pytest.raises(RuntimeError):   # value heads that do not divide the key heads
        paged_attention(q, kp, torch.zeros(pages, 16, 3, 8, device="cuda"), bg, 1.0, chunk=4)
    with pytest.raises(RuntimeError):   # factors of another page count
        paged_attention(q, kp, kp, bg, 1.0, key_factors=torch.zeros(pages + 1, 16, 2, device="cuda"))
    with pytest.raises(AssertionError):
        paged_attention(q, kp, kp, bg, 1.0, window=3, chunk=4)
