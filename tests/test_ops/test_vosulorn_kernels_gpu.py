"""HIP kernels of the Vosulorn serving path against their float32 PyTorch references (same op, run on CPU copies of
the inputs), on ragged batches that mix fresh sequences, continued portions and single decode tokens, in bfloat16 and
float32."""

import pytest
import torch

from colossalai_amd.ops import linear_recurrence as LR
from colossalai_amd.ops.group_norm import head_rms_norm_gate, head_rms_norm_gate_ref
from colossalai_amd.ops.paged_attention import paged_attention, paged_attention_ref
from colossalai_amd.ops.pair_rotary import pair_frequencies, rotate_qk_write, rotate_qk_write_ref
from colossalai_amd.ops.ragged import RaggedBatch
from colossalai_amd.ops.routed_experts import grouped_topk_route, grouped_topk_route_ref

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
MIXED = ([37, 5, 1, 1, 1, 70, 1], [0, 21, 63, 64, 0, 130, 299])       # portions beside decode tokens
DECODE = ([1] * 6, [0, 5, 63, 64, 700, 127])                           # decode tokens alone
LONG = ([200, 1, 140, 2, 128, 65], [0, 9, 61, 30, 0, 1])               # long portions: the chunked recurrence
WIDE = ([513, 300], [3, 0])                                            # tiles of eight tokens across a sequence border


def tol(dtype):
    return dict(rtol=2e-5, atol=2e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)


def make_batch(shape, page=16):
    counts, starts = shape
    tables, nxt = [], 0
    for c, s in zip(counts, starts):
        need = (c + s + page - 1) // page
        tables.append(list(range(nxt + need - 1, nxt - 1, -1)))  # pages in descending order: not contiguous
        nxt += need
    slots = [(3 * i + 1) % len(counts) if len(counts) % 3 else i for i in range(len(counts))]
    return (RaggedBatch.build(counts, starts, slots, "cuda", tables, page),
            RaggedBatch.build(counts, starts, slots, "cpu", tables, page), nxt)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [MIXED, DECODE, LONG, WIDE])
@pytest.mark.parametrize("H,G,D,Dv,K", [(4, 2, 128, 128, 4), (2, 2, 64, 32, 4), (3, 1, 20, 48, 3), (2, 1, 7, 5, 2), (1, 1, 72, 300, 1),
                                        (4, 1, 130, 24, 4), (2, 2, 33, 130, 2), (2, 1, 16, 16, 6)])
def test_conv_gated_delta_rule(dtype, shape, H, G, D, Dv, K):
    torch.manual_seed(D)
    bg, bc, _ = make_batch(shape)
    N, C, B = bc.num_tokens, 2 * G * D + H * Dv, bc.num_seqs
    packed = torch.randn(N, C + 2 * H + 2).to(dtype)          # projections of one matrix product: strided columns
    taps = torch.randn(C, K) * 0.6
    tail = torch.randn(B, K - 1, C) if K > 1 else None
    state = torch.randn(B, H, D, Dv) * 0.3
    A_log, dt_bias = torch.randn(H) * 0.5, torch.randn(H) - 2.0

    def run(fn, p, dev, batch):
        S, tl = state.to(dev, copy=True), None if tail is None else tail.to(dev, copy=True)
        o = fn(p[:, :C], taps.to(dev), tl, G, D, p[:, C : C + H], p[:, C + H : C + 2 * H], A_log.to(dev), dt_bias.to(dev), S,
               batch, 1e-6, D ** -0.5)
        return o.cpu(), S.cpu(), None if tl is None else tl.cpu()

    got, want = run(LR.conv_gated_delta_rule, packed.cuda(), "cuda", bg), run(LR.conv_gated_delta_rule_ref, packed, "cpu", bc)
    scale = max(1.0, want[0].abs().max().item())
    assert (got[0] - want[0]).abs().max().item() < 5e-5 * scale
    assert (got[1] - want[1]).abs().max().item() < 5e-5 * max(1.0, want[1].abs().max().item())
    if tail is not None:
        assert torch.equal(got[2], want[2])


@pytest.mark.parametrize("level", [-12.0, -5.0, -1.0, 3.0, 40.0])
def test_chunked_and_sequential_recurrence_agree(level, monkeypatch):
    """Decays from 1 - 1e-5 to 0 per token: running sums of logarithms near 0 and in the thousands."""
    torch.manual_seed(0)
    H, G, D, Dv, N = 3, 3, 96, 80, 700
    bg = RaggedBatch.build([N], [5], [1], "cuda")
    q, k, v = torch.randn(N, G, D).cuda(), torch.randn(N, G, D).cuda(), torch.randn(N, H, Dv).cuda()
    beta, dt = torch.randn(N, H).cuda() * 3, level + torch.randn(N, H).cuda()
    A_log, dt_bias, state = torch.zeros(H).cuda(), torch.zeros(H).cuda(), torch.randn(2, H, D, Dv).cuda()

    def run(chunked_from):
        monkeypatch.setattr(LR, "DELTA_CHUNKED_FROM", chunked_from)
        S = state.clone()
        return LR.gated_delta_rule(q, k, v, beta, dt, A_log, dt_bias, S, bg, 1e-6, D ** -0.5), S

    (a, Sa), (b, Sb) = run(1), run(10 ** 9)
    assert (a - b).abs().max().item() < 3e-5 * max(1.0, b.abs().max().item())
    assert (Sa - Sb).abs().max().item() < 3e-5 * max(1.0, Sb.abs().max().item())
    assert torch.equal(Sa[0], state[0]) and torch.equal(Sb[0], state[0])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [MIXED, DECODE, LONG])
@pytest.mark.parametrize("H,G,D,Dv,chunk", [(8, 2, 128, 128, 64), (6, 2, 64, 56, 80), (4, 4, 72, 40, 33), (5, 1, 40, 96, 500), (3, 1, 20, 12, 7),
                                            (2, 2, 128, 64, 1)])
def test_attention_inside_blocks_with_learned_sinks(dtype, shape, H, G, D, Dv, chunk):
    torch.manual_seed(D)
    bg, bc, pages = make_batch(shape)
    q = torch.randn(bc.num_tokens, H, D).to(dtype)
    kpool, vpool = torch.randn(pages, 16, G, D).to(dtype), torch.randn(pages, 16, G, Dv).to(dtype)
    sink = torch.randn(H) * 3
    got = paged_attention(q.cuda(), kpool.cuda(), vpool.cuda(), bg, D ** -0.5, chunk=chunk, sink_logits=sink.cuda())
    want = paged_attention_ref(q, kpool, vpool, bc, D ** -0.5, chunk=chunk, sink_logits=sink)
    torch.testing.assert_close(got.cpu().float(), want.float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [MIXED, DECODE])
@pytest.mark.parametrize("H,G,D,Dv,dims,pad", [(16, 4, 128, 128, 128, 0), (6, 3, 64, 48, 32, 8), (4, 2, 24, 40, 22, 0), (3, 1, 7, 5, 4, 1),
                                               (2, 2, 16, 8, 0, 0), (4, 1, 64, 64, 64, 1)])
def test_rotation_and_page_write(dtype, shape, H, G, D, Dv, dims, pad):
    torch.manual_seed(D)
    bg, bc, pages = make_batch(shape)
    N = bc.num_tokens
    packed = torch.randn(N, H * D + G * D + G * Dv + pad).to(dtype)
    pools = torch.randn(pages, 16, G, D).to(dtype), torch.randn(pages, 16, G, Dv).to(dtype)
    freqs = pair_frequencies(1e4, dims, scaling=dict(factor=5.0, low=1.0, high=4.0, original=200))

    def run(fn, dev, batch):
        p, kp, vp = packed.to(dev, copy=True), pools[0].to(dev, copy=True), pools[1].to(dev, copy=True)
        fn(p[:, : H * D].view(N, H, D), p[:, H * D : (H + G) * D].view(N, G, D),
           p[:, (H + G) * D : (H + G) * D + G * Dv].view(N, G, Dv), freqs.to(dev), kp, vp, batch)
        return p.cpu().float(), kp.cpu().float(), vp.cpu().float()

    got, want = run(rotate_qk_write, "cuda", bg), run(rotate_qk_write_ref, "cpu", bc)
    for g, w in zip(got[:2], want[:2]):
        torch.testing.assert_close(g, w, **(dict(rtol=1e-4, atol=1e-4) if dtype == torch.float32 else tol(dtype)))
    assert torch.equal(got[2], want[2]) and torch.equal(got[0][:, H * D :], packed.float()[:, H * D :])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,H,D", [(50, 16, 128), (7, 3, 20), (1, 1, 300), (33, 2, 72), (5, 3, 512), (9, 1, 8)])
@pytest.mark.parametrize("pad", [8, 3])
def test_output_norm_with_silu_gate(dtype, N, H, D, pad):
    torch.manual_seed(N)
    x, w, g = torch.randn(N, H, D), torch.rand(D) + 0.5, torch.randn(N, H * D + pad).to(dtype)
    got = head_rms_norm_gate(x.cuda(), w.cuda(), 1e-5, g.cuda()[:, : H * D], dtype, act="silu")
    torch.testing.assert_close(got.cpu(), head_rms_norm_gate_ref(x, w, 1e-5, g[:, : H * D], dtype, act="silu"), **tol(dtype))


@pytest.mark.parametrize("N,E,top", [(300, 32, 6), (3, 8, 4), (65, 1, 1), (40, 200, 9), (17, 5, 5)])
def test_router_on_logits(N, E, top):
    torch.manual_seed(E)
    z = torch.randn(N, E) * 4
    z[0] += 500.0
    ids, w = grouped_topk_route(z.cuda(), None, top, score="logits")
    want_ids, want = grouped_topk_route_ref(z, None, top, score="logits")
    assert torch.equal(ids.cpu(), want_ids)
    torch.testing.assert_close(w.cpu(), want, rtol=1e-5, atol=1e-6)
