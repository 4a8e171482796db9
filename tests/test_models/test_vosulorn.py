"""Vosulorn against the float64 oracle (tests/vosulorn_oracle.py): every mechanism alone, then whole
models of several shapes, on the CPU (reference path of every op) and on the GPU (HIP kernels)."""

import copy
import os
import sys

import pytest
import torch

ROOT = os.path.dirname(os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
sys.path.insert(0, os.path.join(ROOT, "tests"))
import vosulorn_oracle as O  # noqa: E402

from colossalai_amd.inference.kv_cache import KVCacheManager  # noqa: E402
from colossalai_amd.inference.state_cache import StateCacheManager  # noqa: E402
from colossalai_amd.models import VosulornForCausalLM, model_class_for  # noqa: E402
from colossalai_amd.models.vosulorn import UNIT_EPS, VosulornMoE  # noqa: E402
from colossalai_amd.ops import latent_attention as LA  # noqa: E402
from colossalai_amd.ops.group_norm import head_rms_norm_gate  # noqa: E402
from colossalai_amd.ops.linear_recurrence import conv_gated_delta_rule, gated_delta_rule  # noqa: E402
from colossalai_amd.ops.paged_attention import paged_attention  # noqa: E402
from colossalai_amd.ops.pair_rotary import halves_to_pairs, pair_frequencies, rotate_pairs, rotate_qk_write  # noqa: E402
from colossalai_amd.ops.ragged import RaggedBatch  # noqa: E402
from colossalai_amd.ops.routed_experts import grouped_topk_route  # noqa: E402
from colossalai_amd.ops.short_conv import short_conv  # noqa: E402
from colossalai_amd.ops.streams import streams_start  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64

SCALING = dict(factor=3.0, low=1.5, high=3.0, original=60)
ATT = dict(dim=10, heads=6, kv_heads=2, vdim=7, scale=0.4, mask=dict(size=7), rot=dict(base=900.0, dims=6, scaling=SCALING))
LAT = dict(dim=6, heads=3, rot_dim=8, vdim=5, kv_rank=12, scale=0.5, rot=dict(base=300.0, dims=8))
DEL = dict(dim=9, heads=4, kv_heads=2, vdim=6, conv=3)


def layer(kind, mixer, moe=None):
    """``moe``: (experts, top, ff) or None."""
    return dict(type=kind, mixer=mixer, mlp=None if moe is None else dict(
        kind="moe", expert=dict(ff=moe[2]), router=dict(experts=moe[0], top=moe[1])))


def cfg_of(layers, width=26, vocab=45, eps=1e-5, scale=3.5):
    return dict(architecture="Vosulorn", embedding=dict(scale=scale), layers=layers, norm=dict(eps=eps), vocab=vocab,
                width=width)


SHAPES = {
    # every kind, shared latents under other head counts and sizes, a layer without a feed-forward
    "mixed": cfg_of([layer("delta", DEL, (5, 2, 9)), layer("latent_attention", LAT, (4, 3, 7)), layer("attention", ATT),
                     layer("latent_attention", dict(LAT, kv_from=1, heads=2, dim=4, vdim=9, scale=0.9), (3, 1, 8)),
                     layer("delta", dict(DEL, heads=2, kv_heads=2, conv=1, dim=4, vdim=3), (2, 2, 5))]),
    # two sources and two readers out of order, single heads, one expert
    "sources": cfg_of([layer("latent_attention", dict(LAT, heads=1, kv_rank=5, rot_dim=2, rot=dict(base=50.0, dims=2)), (1, 1, 6)),
                       layer("latent_attention", LAT),
                       layer("latent_attention", dict(LAT, kv_from=1, heads=5), (6, 4, 4)),
                       layer("latent_attention", dict(LAT, heads=2, kv_rank=5, rot_dim=2, rot=dict(base=50.0, dims=2), kv_from=0))],
                      width=20, eps=1e-3, scale=1.0),
    # attention only: no frequency scaling, whole head rotated, one position per block, block wider than the sequence
    "attention": cfg_of([layer("attention", dict(ATT, heads=2, kv_heads=2, mask=dict(size=1)), (3, 2, 4)),
                         layer("attention", dict(ATT, heads=3, kv_heads=1, dim=4, vdim=8, mask=dict(size=400),
                                                 rot=dict(base=10000.0, dims=4)), (8, 8, 3))], width=18, scale=0.3),
    # recurrent only: many heads per key, long taps
    "delta": cfg_of([layer("delta", dict(DEL, heads=6, kv_heads=1, conv=5, vdim=11), (4, 2, 6)),
                     layer("delta", dict(DEL, heads=3, kv_heads=3, conv=2, dim=16, vdim=2))], width=24),
}


def close(got, want, tol=3e-4):
    got, want = got.detach().cpu().to(F64), want.detach().cpu().to(F64)
    assert got.shape == want.shape
    err = (got - want).abs().max().item()
    assert err <= tol * max(1.0, want.abs().max().item()), f"max abs error {err}"


class Pages:
    """A scattered page table over pools of garbage, and the batches of one sequence fed in portions."""

    def __init__(self, T, device, page, slot=0):
        self.page, self.device, self.slot = page, device, slot
        self.num = (T + page - 1) // page + 3
        self.table = torch.randperm(self.num, generator=torch.Generator().manual_seed(T)).tolist()

    def pool(self, heads, dim, dtype=torch.float32):
        return torch.full((self.num, self.page, heads, dim), float("nan"), device=self.device, dtype=dtype)

    def batches(self, cuts):
        at = 0
        for n in cuts:
            need = (at + n + self.page - 1) // self.page
            yield slice(at, at + n), RaggedBatch.build([n], [at], [self.slot], self.device, [self.table[:need]], self.page)
            at += n


def rand(seed, *shape):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed))


def cuts_of(T, edge):
    """Whole; cut at the special place; just before and after it; in pairs; the tail decoded."""
    out = [[T], [edge, T - edge], [edge - 1, 2, T - edge - 1], [T - 9] + [1] * 9]
    if T <= 60:
        out.append([2] * (T // 2) + [1] * (T % 2))
    return [[n for n in c if n > 0] for c in out]


# --------------------------------------------------------------------------- positions
@pytest.mark.parametrize("base,dims,scaling", [
    (10000.0, 16, None), (50.0, 2, dict(factor=2.0, low=1.0, high=4.0, original=100)),
    (900.0, 12, dict(factor=3.0, low=1.5, high=3.0, original=60)), (1e6, 64, dict(factor=32.0, low=1.0, high=4.0, original=8192)),
    (500000.0, 40, dict(factor=8.0, low=0.5, high=2.5, original=700)), (10.0, 8, dict(factor=1.0, low=1.0, high=2.0, original=9))])
def test_frequencies(base, dims, scaling):
    rot = dict(base=base, dims=dims)
    if scaling:
        rot["scaling"] = scaling
    want = torch.tensor(O.rotation_frequencies(rot), dtype=F64)
    got = pair_frequencies(base, dims, scaling=scaling)
    assert got.dtype == torch.float32
    assert ((got.to(F64) - want).abs() <= 1e-7 * want).all()


def test_frequency_scaling_has_three_bands():
    s = dict(factor=3.0, low=1.5, high=3.0, original=60)
    plain, got = pair_frequencies(900.0, 40), pair_frequencies(900.0, 40, scaling=s)
    kept, cut = got == plain, torch.isclose(got, plain / 3.0, rtol=1e-6)
    assert kept.any() and cut.any() and (~kept & ~cut).any()


def test_halves_to_pairs_keeps_scores():
    """Rotating halves, and rotating neighbours after the reordering, give the same scores; what is not rotated stays
    where it is."""
    H, size, first, dims, W, T = 3, 11, 2, 8, 13, 40
    wq, wk, h = rand(1, H * size, W), rand(2, H * size, W), rand(3, T, W)
    f = O.frequencies(70.0, dims)

    def project(w, turn):
        y = O.lin(h.to(F64), w).view(T, H, size)
        return torch.cat([y[..., :first], turn(y[..., first : first + dims]), y[..., first + dims :]], -1)

    q, k = (project(w, lambda x: O.rotate_halves(x, f)) for w in (wq, wk))
    q2, k2 = (project(halves_to_pairs(w, H, size, first, dims), lambda x: O.rotate_neighbours(x, f)) for w in (wq, wk))
    close(torch.einsum("ihd,jhd->hij", q2, k2), torch.einsum("ihd,jhd->hij", q, k), 1e-12)
    assert torch.equal(q2[..., :first], q[..., :first]) and torch.equal(q2[..., first + dims :], q[..., first + dims :])
    assert (q2 - q).abs().max() > 0.1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv,dims", [(6, 2, 10, 7, 6), (2, 2, 8, 8, 8), (4, 1, 24, 16, 16), (3, 3, 5, 4, 2), (1, 1, 4, 9, 0),
                                           (4, 2, 64, 32, 64)])
def test_rotation_and_page_write(device, H, G, D, Dv, dims):
    """Queries and keys are column slices of one projection; the queries turn in place, keys and values reach the pages
    the table names and no other row; positions far from 0."""
    start, n, page = 1021, 9, 4
    packed = rand(10, n, H * D + G * D + G * Dv + 3).to(device)
    orig = packed.clone().cpu()
    q, k, v = (packed[:, a:b] for a, b in ((0, H * D), (H * D, (H + G) * D), ((H + G) * D, (H + G) * D + G * Dv)))
    pages = torch.randperm(300, generator=torch.Generator().manual_seed(0)).tolist()
    batch = RaggedBatch.build([n], [start], [0], device, [pages], page)
    kpool = torch.full((300, page, G, D), 7.0, device=device)
    vpool = torch.full((300, page, G, Dv), 7.0, device=device)
    freqs = pair_frequencies(1000.0, dims).to(device)
    rotate_qk_write(q.view(n, H, D), k.view(n, G, D), v.view(n, G, Dv), freqs, kpool, vpool, batch)
    f = O.frequencies(1000.0, dims)

    def turned(x, heads):
        x = torch.cat([torch.zeros(start, heads, D, dtype=F64), x.reshape(n, heads, D).to(F64)])
        return O.rotate_neighbours(x, f)[start:]

    close(q.reshape(n, H, D), turned(orig[:, : H * D], H), 2e-4)      # float32 angles of about a thousand
    rows = torch.tensor([pages[p // page] * page + p % page for p in range(start, start + n)])
    flat_k, flat_v = kpool.cpu().view(-1, G, D), vpool.cpu().view(-1, G, Dv)
    close(flat_k[rows], turned(orig[:, H * D : (H + G) * D], G), 2e-4)
    assert torch.equal(flat_v[rows], orig[:, (H + G) * D : (H + G) * D + G * Dv].reshape(n, G, Dv))
    rest = torch.ones(300 * page, dtype=torch.bool)
    rest[rows] = False
    assert (flat_k[rest] == 7).all() and (flat_v[rest] == 7).all()
    assert torch.equal(packed.cpu()[:, H * D :], orig[:, H * D :])


# ------------------------------------------------------------------- chunked attention with a sink
def framework_chunked(q, k, v, c, sink, device, cuts, page):
    T, (H, D), (G, Dv) = q.shape[0], q.shape[1:], v.shape[1:]
    pg = Pages(T, device, page)
    kpool, vpool, out = pg.pool(G, D), pg.pool(G, Dv), []
    freqs = pair_frequencies(c["rot"]["base"], c["rot"]["dims"], scaling=c["rot"].get("scaling")).to(device)
    for sl, batch in pg.batches(cuts):
        qq = q[sl].to(device).clone()
        rotate_qk_write(qq, k[sl].to(device), v[sl].to(device), freqs, kpool, vpool, batch)
        out.append(paged_attention(qq, kpool, vpool, batch, c["scale"], chunk=c["mask"]["size"], sink_logits=sink.to(device)))
    return torch.cat(out, 0)


def oracle_chunked(q, k, v, c, sink, size=None, turn=True):
    H, G = q.shape[1], k.shape[1]
    size = c["mask"]["size"] if size is None else size
    f = O.rotation_frequencies(c["rot"])
    q, k = O.rotate_neighbours(q.to(F64), f), O.rotate_neighbours(k.to(F64), f)
    return torch.stack([O.attend(q[:, h], k[:, h // (H // G)], v[:, h // (H // G)].to(F64), c["scale"],
                                 lambda i, j: O.sees_chunk(i, j, size), None if sink is None else sink[h]) for h in range(H)], 1)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv,dims,size", [(6, 2, 10, 7, 6, 7), (2, 2, 8, 8, 8, 1), (4, 1, 24, 16, 16, 16), (3, 3, 5, 4, 2, 100),
                                                (8, 4, 16, 32, 12, 13)])
def test_chunked_attention_with_a_sink(device, H, G, D, Dv, dims, size):
    T = 45
    c = dict(scale=0.6, mask=dict(size=size), rot=dict(base=200.0, dims=dims, scaling=SCALING))
    q, k, v, sink = rand(30, T, H, D), rand(31, T, G, D), rand(32, T, G, Dv), rand(33, H)
    want = oracle_chunked(q, k, v, c, sink)
    edge = min(size * (T // 2 // size), 40) or 20
    for cuts in cuts_of(T, edge):
        close(framework_chunked(q, k, v, c, sink, device, cuts, 4), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("level", [-40.0, 0.0, 3.0, 60.0])
def test_the_sink_counts_once_and_unscaled(device, level):
    """From a sink that vanishes to one that takes nearly all the weight; two heads with sinks of their own."""
    T, c = 40, dict(scale=2.5, mask=dict(size=17), rot=dict(base=40.0, dims=4))
    q, k, v = rand(34, T, 2, 6), rand(35, T, 1, 6), rand(36, T, 1, 5)
    sink = torch.tensor([level, -level])
    want = oracle_chunked(q, k, v, c, sink)
    if level == 3.0:  # left out, or scaled like a score, it would show
        assert (oracle_chunked(q, k, v, c, None) - want).abs().max() > 0.3
        assert (oracle_chunked(q, k, v, c, sink * c["scale"]) - want).abs().max() > 0.3
    for cuts in ([T], [T - 5] + [1] * 5, [16, 2, T - 18]):
        close(framework_chunked(q, k, v, c, sink, device, cuts, 8), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,i,j", [(50, 100, 100), (50, 100, 99), (50, 149, 100), (50, 149, 99), (64, 127, 64), (64, 127, 63),
                                      (64, 128, 127), (33, 98, 66), (33, 98, 65), (33, 99, 98), (400, 399, 0), (400, 383, 16)])
def test_a_spike_at_a_blocks_border(device, size, i, j):
    """Query ``i`` points at key ``j``: the first or last token of its block, or the one before the block, which is not
    seen. Prompt cut anywhere, and decoded."""
    T, H, G, D, Dv = i + 1, 2, 1, 12, 8
    c = dict(scale=1.0, mask=dict(size=size), rot=dict(base=1e4, dims=4))
    q, k, v, sink = rand(40, T, H, D), rand(41, T, G, D), rand(42, T, G, Dv), torch.tensor([0.5, 1.0])
    q[i], k[j] = 0.0, 0.0
    q[i, :, 6:], k[j, :, 6:] = 4.0, 2.0          # channels that do not turn: a score of 48
    want = oracle_chunked(q, k, v, c, sink)
    moved = v.clone()
    moved[j] += 5 * rand(43, G, Dv)  # the key's value enters the query's output if, and only if, the block shows it
    moved = (oracle_chunked(q, k, moved, c, sink)[i] - want[i]).abs().max()
    assert moved > 2 if i // size == j // size else moved == 0
    edge = min(size - 1, T - 1)
    for cuts in ([T], [T - 1, 1], [T - 3, 2, 1], [edge, T - edge], [40, T - 40]):
        close(framework_chunked(q, k, v, c, sink, device, cuts, 16), want)


# ------------------------------------------------------------------------ latent attention
def latent_inputs(T, H, D, R, Dv, rank, seed):
    return dict(q=rand(seed, T, H, D + R), dkv=rand(seed + 1, T, rank + R), norm=1 + 0.2 * rand(seed + 2, rank),
                uk=rand(seed + 3, H * D, rank) / rank ** 0.5, uv=rand(seed + 4, H * Dv, rank) / rank ** 0.5)


def framework_latent(a, readers, base, dims, device, cuts, page, eps=1e-5):
    """One write of the cached rows per portion, one attention per reader ``(q, uk, uv, scale)``; the rotated channels
    arrive as halves and are reordered like the checkpoint's projection rows."""
    T, rank = a["dkv"].shape[0], a["norm"].numel()
    R = a["dkv"].shape[1] - rank
    freqs = pair_frequencies(base, dims).to(device)
    dkv = halves_to_pairs(a["dkv"].t().contiguous(), 1, rank + R, rank, dims).t().contiguous().to(device)
    pg = Pages(T, device, page)
    pool, outs = pg.pool(1, rank + R), [[] for _ in readers]
    for sl, batch in pg.batches(cuts):
        LA.latent_kv_write(dkv[sl], a["norm"].to(device), eps, freqs, pool, batch)
        for out, (q, uk, uv, scale) in zip(outs, readers):
            H, DR = q.shape[1:]
            qq = halves_to_pairs(q[sl].reshape(-1, H * DR).t().contiguous(), H, DR, DR - R, dims).t().contiguous()
            w_uk, w_uv = uk.view(H, DR - R, rank).to(device), uv.view(H, -1, rank).to(device)
            out.append(LA.latent_attention(qq.view(-1, H, DR).to(device), w_uk, w_uv, pool, batch, scale, freqs, rank,
                                           w_uv_t=w_uv.transpose(1, 2).contiguous() if sl.start % 2 else None))
    return [torch.cat(o, 0) for o in outs]


def oracle_latent(a, readers, base, dims, eps=1e-5):
    rank = a["norm"].numel()
    R, f = a["dkv"].shape[1] - rank, O.frequencies(base, dims)
    lat = O.rms_norm(a["dkv"][:, :rank].to(F64), a["norm"], eps)
    shared = O.rotate_halves(a["dkv"][:, None, rank:].to(F64), f)[:, 0]
    outs = []
    for q, uk, uv, scale in readers:
        T, H, DR = q.shape
        D = DR - R
        qr = O.rotate_halves(q[..., D:].to(F64), f)
        k, v = O.lin(lat, uk).view(T, H, D), O.lin(lat, uv).view(T, H, -1)
        outs.append(torch.cat([O.attend(torch.cat([q[:, h, :D].to(F64), qr[:, h]], -1), torch.cat([k[:, h], shared], -1), v[:, h],
                                        scale, O.sees_causal) for h in range(H)], -1))
    return outs


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,R,Dv,rank,dims", [(3, 6, 8, 5, 12, 8), (1, 4, 2, 8, 16, 2), (2, 8, 6, 8, 3, 6), (4, 5, 16, 9, 20, 16),
                                                (2, 16, 8, 24, 40, 4)])
def test_latents_serve_the_layer_that_wrote_them_and_a_later_one(device, H, D, R, Dv, rank, dims):
    T = 43
    a, b = latent_inputs(T, H, D, R, Dv, rank, 10), latent_inputs(T, H + 1, D + 3, R, Dv + 2, rank, 50)
    readers = [(a["q"], a["uk"], a["uv"], 0.7), (b["q"], b["uk"], b["uv"], 0.4)]
    want = oracle_latent(a, readers, 100.0, dims)
    for cuts in cuts_of(T, 16):
        got = framework_latent(a, readers, 100.0, dims, device, cuts, 4)
        for g, w in zip(got, want):
            close(g, w)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("far", [0, 1, 15, 16, 63, 64, 127, 128, 300, 388, 389])
@pytest.mark.parametrize("part", ["plain", "rotated"])
def test_one_latent_far_back_takes_the_weight(device, far, part):
    """Among several hundred keys the last query's score stands out at one place, through the up-projected or through
    the rotated part of its key; in a prompt portion, and decoded."""
    T, H, D, R, rank = 390, 2, 8, 4, 16
    a = latent_inputs(T, H, D, R, 6, rank, 20)
    f = O.frequencies(1e4, R)
    a["dkv"][:, 0], a["dkv"][far, 0] = 0.0, 12.0       # a direction of the latent that no other token uses
    a["uk"][:, 1:] *= 0.3
    lat = O.rms_norm(a["dkv"][:, :rank].to(F64), a["norm"], 1e-5)
    if part == "plain":
        a["q"][T - 1] = 0
        a["q"][T - 1, :, :D] = 12 * O.lin(lat[far], a["uk"]).view(H, D).float()
    else:
        a["dkv"][far, rank:] = torch.tensor([3.0, -2.0, 4.0, 3.0])
        turned = O.rotate_halves(torch.cat([a["dkv"][: T, None, rank:].to(F64)]), f)[far, 0]
        want_q = 12 * turned / turned.norm()      # what the query's rotated part must be at its own position
        back = O.rotate_halves(torch.cat([torch.zeros(T - 1, 1, R, dtype=F64), want_q.view(1, 1, R)]), [-x for x in f])[T - 1, 0]
        a["q"][T - 1, :, :D], a["q"][T - 1, :, D:] = 0, back.float()
    readers = [(a["q"], a["uk"], a["uv"], 1.0)]
    want = oracle_latent(a, readers, 1e4, R)[0][T - 1 :]
    assert (want[0] - O.lin(lat[far], a["uv"])).abs().max() < 0.3, "the test's spike does not stand out"
    for cuts in ([T], [T - 1, 1], [T - 19, 19], [128, 2, T - 130]):
        close(framework_latent(a, readers, 1e4, R, device, cuts, 64)[0][T - 1 :], want)


# ------------------------------------------------------------------------- gated delta rule
def framework_delta(x, taps, b, a, A_log, dt_bias, c, device, cuts, slots=3, slot=1, state=None, fused=True):
    """x [T, 2 G D + H Dv] ahead of the convolutions. State buffers start as garbage; returns outputs and final state.
    ``fused``: convolution, unit length and gates through one op, or the convolution and the rule as two."""
    H, G, D, Dv, K = c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["conv"]
    C = x.shape[1]
    if state is None:
        state = (torch.full((slots, H, D, Dv), float("nan"), device=device),
                 torch.full((slots, K - 1, C), float("nan"), device=device) if K > 1 else None)
    S, tail = state
    out, at = [], 0
    for n in cuts:
        batch = RaggedBatch.build([n], [at], [slot], device)
        sl = slice(at, at + n)
        at += n
        if fused:
            out.append(conv_gated_delta_rule(x[sl].to(device), taps.to(device), tail, G, D, b[sl].to(device), a[sl].to(device),
                                             A_log.to(device), dt_bias.to(device), S, batch, UNIT_EPS, D ** -0.5))
            continue
        y = short_conv(x[sl].to(device), taps.to(device), tail, batch, True, torch.float32)
        Cq = G * D
        out.append(gated_delta_rule(y[:, :Cq].view(n, G, D), y[:, Cq : 2 * Cq].view(n, G, D), y[:, 2 * Cq :].view(n, H, Dv),
                                    b[sl].to(device), a[sl].to(device), A_log.to(device), dt_bias.to(device), S, batch,
                                    UNIT_EPS, D ** -0.5))
    return torch.cat(out, 0), S[slot]


def oracle_delta(x, taps, b, a, A_log, dt_bias, c):
    H, G, D, Dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    T, Cq = x.shape[0], G * D
    y = O.short_conv(x.to(F64), taps)
    q, k = O.unit(y[:, :Cq].view(T, G, D)) * D ** -0.5, O.unit(y[:, Cq : 2 * Cq].view(T, G, D))
    v, beta, g = y[:, 2 * Cq :].view(T, H, Dv), torch.sigmoid(b.to(F64)), O.head_decay(a.to(F64), A_log, dt_bias)
    pairs = [O.delta_scan(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], g[:, h], beta[:, h]) for h in range(H)]
    return torch.stack([p[0] for p in pairs], 1), torch.stack([p[1] for p in pairs])


def delta_inputs(T, c, seed, decay=-2.0):
    H, G, D, Dv, K = c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["conv"]
    C = 2 * G * D + H * Dv
    return (rand(seed, T, C), 0.7 * rand(seed + 1, C, K), 1.5 * rand(seed + 2, T, H), rand(seed + 3, T, H), 0.5 * rand(seed + 4, H),
            decay + 0.5 * rand(seed + 5, H), c)


DELTA_SIZES = [dict(heads=4, kv_heads=2, dim=9, vdim=6, conv=3), dict(heads=1, kv_heads=1, dim=1, vdim=1, conv=1),
               dict(heads=3, kv_heads=3, dim=16, vdim=5, conv=2), dict(heads=6, kv_heads=1, dim=5, vdim=17, conv=5),
               dict(heads=2, kv_heads=1, dim=64, vdim=32, conv=4)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("c", DELTA_SIZES)
def test_delta_rule_in_portions(device, c):
    T = 47
    args = delta_inputs(T, c, 60)
    want, final = oracle_delta(*args)
    for cuts in cuts_of(T, 16) + [[1] * T, [2, 3, 2, 5, 2, 33]]:
        for fused in (True, False):
            got, S = framework_delta(*args, device, cuts, fused=fused)
            close(got, want)
            close(S, final)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("c", [dict(heads=4, kv_heads=2, dim=32, vdim=48, conv=4), dict(heads=2, kv_heads=2, dim=20, vdim=12, conv=3),
                               dict(heads=2, kv_heads=1, dim=128, vdim=64, conv=4), dict(heads=1, kv_heads=1, dim=72, vdim=130, conv=2)])
@pytest.mark.parametrize("decay", [-30.0, -4.0, 0.0, 30.0])
def test_delta_rule_over_long_portions(device, c, decay):
    """From a state that never fades (decay 1) to one that fades at once; portions of one, two and many tokens around
    multiples of 16, 32 and 64."""
    T = 333
    args = delta_inputs(T, c, 70, decay)
    want, final = oracle_delta(*args)
    for i, cuts in enumerate(([T], [64, 269], [63, 2, 65, 1, 128, 74], [200, 133], [300] + [1] * 33)):
        got, S = framework_delta(*args, device, cuts, fused=i != 1)
        close(got, want)
        close(S, final)


@pytest.mark.parametrize("device", DEVICES)
def test_delta_rule_remembers_one_write(device):
    """One early token writes a value under a key no other token touches; hundreds of tokens later, without decay, its
    key reads the value back, in a prompt and decoded. A second write under the same key replaces it."""
    c = dict(heads=1, kv_heads=1, dim=16, vdim=8, conv=1)
    T, D = 260, 16
    for again in (None, 130):
        x, taps, b, a, A_log, dt_bias, _ = delta_inputs(T, c, 80, decay=-60.0)
        taps = torch.ones_like(taps)
        x[:, 15] = x[:, 31] = -80.0                     # silu of it is 0: no other token uses the last channel
        b[:] = 30.0                                     # beta = 1
        for t in [3] + ([again] if again else []):
            x[t, 16:32] = -80.0
            x[t, 31] = 5.0
        x[T - 1, :16] = -80.0
        x[T - 1, 15] = 5.0
        want, _ = oracle_delta(x, taps, b, a, A_log, dt_bias, c)
        src = O.silu(x[again or 3, 32:].to(F64)) * D ** -0.5
        assert (want[T - 1, 0] - src).abs().max() < 1e-3
        for cuts in ([T], [T - 1, 1], [4, 2, T - 6], [100, 100, 60], [2] * 130):
            got, _ = framework_delta(x, taps, b, a, A_log, dt_bias, c, device, cuts)
            close(got, want)


@pytest.mark.parametrize("device", DEVICES)
def test_delta_state_slots_are_used_again(device):
    """A second sequence in a slot that holds the first one's state and tail starts from zero; the neighbours' slots
    stay as they are."""
    c = dict(heads=2, kv_heads=1, dim=8, vdim=6, conv=4)
    first, second = delta_inputs(40, c, 90), delta_inputs(21, c, 95)
    S = torch.full((3, 2, 8, 6), 5.0, device=device)
    tail = torch.full((3, 3, 28), 5.0, device=device)
    framework_delta(*first, device, [40], state=(S, tail))
    second = (second[0], first[1], *second[2:4], *first[4:])
    want, final = oracle_delta(*second)
    for cuts in ([21], [1] * 21, [2, 1, 18]):
        got, state = framework_delta(*second, device, cuts, state=(S, tail))
        close(got, want)
        close(state, final)
    assert (S[[0, 2]] == 5).all() and (tail[[0, 2]] == 5).all()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("lens", [[5, 1, 130, 2], [1, 1, 1], [64, 64], [200, 3, 1, 65, 31]])
def test_delta_rule_of_several_sequences(device, lens):
    """Sequences of unequal portions in one step, some starting and some going on, against each alone."""
    c = dict(heads=3, kv_heads=1, dim=24, vdim=16, conv=3)
    _, taps, _, _, A_log, dt_bias, _ = delta_inputs(1, c, 100)
    head = [0 if i % 2 else 7 for i in range(len(lens))]          # tokens of an earlier step
    seqs = [delta_inputs(n + h, c, 110 + 10 * i) for i, (n, h) in enumerate(zip(lens, head))]
    n_slots, C = len(lens) + 2, 2 * 24 + 3 * 16
    S, tail = torch.full((n_slots, 3, 24, 16), 9.0, device=device), torch.full((n_slots, 2, C), 9.0, device=device)

    def step(parts, starts, slots):
        batch = RaggedBatch.build([p[0].shape[0] for p in parts], starts, slots, device)
        x, b, a = (torch.cat([p[i] for p in parts]).to(device) for i in (0, 2, 3))
        return conv_gated_delta_rule(x, taps.to(device), tail, 1, 24, b, a, A_log.to(device), dt_bias.to(device), S, batch,
                                     UNIT_EPS, 24 ** -0.5)

    slots = [n_slots - 1 - i for i in range(len(lens))]
    cut = lambda s, lo, hi: (s[0][lo:hi], s[1], s[2][lo:hi], s[3][lo:hi])
    going = [i for i, h in enumerate(head) if h]
    step([cut(seqs[i], 0, head[i]) for i in going], [0] * len(going), [slots[i] for i in going])
    got = step([cut(s, h, h + n) for s, h, n in zip(seqs, head, lens)], head, slots)
    at = 0
    for i, (s, h, n) in enumerate(zip(seqs, head, lens)):
        want, final = oracle_delta(s[0], taps, s[2], s[3], A_log, dt_bias, c)
        close(got[at : at + n], want[h:])
        close(S[slots[i]], final)
        at += n


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,Dv", [(4, 32), (3, 7), (1, 130)])
def test_output_norm_and_silu_gate(device, H, Dv):
    o, g, w = 3 * rand(120, 9, H, Dv), 2 * rand(121, 9, H * Dv), 1 + 0.3 * rand(122, Dv)
    o[2] *= 1e-4                                            # the norm's eps shows
    want = O.rms_norm(o.to(F64), w, 1e-5) * O.silu(g.to(F64)).view(9, H, Dv)
    close(head_rms_norm_gate(o.to(device), w.to(device), 1e-5, g.to(device), act="silu"), want, 1e-5)


# ----------------------------------------------------------------------------- experts
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,top", [(8, 4), (5, 1), (3, 3), (70, 6), (1, 1)])
def test_router_chooses_by_logits(device, E, top):
    h, w, b = rand(130, 20, 11), rand(131, E, 11), 2 * rand(132, E)
    z = (h @ w.t() + b).to(device)
    z[0] -= 300.0                                           # far from zero: only differences matter
    z[1] *= 40.0
    ids, wt = grouped_topk_route(z, None, top, score="logits")
    want = torch.sort(z.cpu(), dim=-1, descending=True, stable=True).indices[:, :top]
    assert torch.equal(ids.cpu().long(), want)
    close(wt, torch.softmax(z.cpu().to(F64).gather(1, want), -1), 1e-5)
    if top < E:  # unlike a softmax over all experts
        assert ((wt.sum(-1) - 1).abs() < 1e-5).all()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W,E,top,ff,N", [(26, 5, 2, 9, 13), (64, 8, 4, 32, 40), (32, 1, 1, 8, 3), (96, 12, 5, 64, 300)])
def test_expert_layer(device, W, E, top, ff, N):
    cfg = cfg_of([layer("delta", DEL, (E, top, ff))], width=W)
    P = {k: v.float() for k, v in O.random_checkpoint(cfg, 3).items()}
    P["l0.mlp.router.b"] *= 6                               # the bias moves the choice
    model = VosulornForCausalLM.from_checkpoint(cfg, P, dtype=torch.float32, device=device)
    mlp = model.layers[0].mlp
    assert isinstance(mlp, VosulornMoE)
    h = rand(140, N, W)
    with torch.no_grad():
        got = mlp(h.to(device))
    close(got, O.moe(h.to(F64), P, "l0.mlp.", cfg["layers"][0]["mlp"]))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W,scale", [(26, 3.5), (64, 1.0), (1030, 0.02)])
def test_scaled_embedding_and_first_norm(device, W, scale):
    table, toks, w = rand(150, 11, W), torch.tensor([3, 0, 10, 7, 7]), 1 + 0.3 * rand(151, W)
    x, h = streams_start(table.to(device), toks.to(device), 1, torch.ones(1, device=device), w.to(device), 1e-4, scale)
    want = table[toks].to(F64) * scale
    close(x[:, 0], want, 1e-6)
    close(h, O.rms_norm(want, w, 1e-4), 1e-5)


# -------------------------------------------------------------------- whole models
def caches(model, device, pages, page, slots=2):
    kv = KVCacheManager(len(model.layers), 0, 0, num_blocks=pages, block_size=page, device=device, dtype=model.act_dtype,
                        layer_shapes=model.kv_layer_shapes(), layer_sources=model.kv_layer_sources())
    return kv, StateCacheManager(model.state_layer_buffers(), slots, device=device)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("shape", sorted(SHAPES))
def test_whole_model_and_every_layer(device, shape):
    cfg = SHAPES[shape]
    P = {k: v.float() for k, v in O.random_checkpoint(cfg, seed=5).items()}
    toks = torch.randint(0, cfg["vocab"], (33,), generator=torch.Generator().manual_seed(7)).tolist()
    want_res = []
    want = O.forward(cfg, P, toks, want_res)
    assert model_class_for(cfg) is VosulornForCausalLM
    model = VosulornForCausalLM.from_checkpoint(cfg, P, dtype=torch.float32, device=device)
    assert len(want_res) == len(model.kv_layer_shapes()) == len(model.state_layer_buffers()) == len(model.kv_layer_sources())
    assert model.config.from_dict(model.config.to_dict()) == model.config
    got_res = []
    batch = RaggedBatch.build([33], [0], [1], device, [[5, 1, 0, 4, 2]], 8)
    with torch.no_grad():
        got = model.forward_ragged(torch.tensor(toks, device=device), batch, *caches(model, device, 6, 8), None, got_res)
        rows = model.forward_ragged(torch.tensor(toks, device=device), batch, *caches(model, device, 6, 8),
                                    torch.tensor([32, 0, 7], device=device))
    for a, b in zip(got_res, want_res):
        close(a, b, 2e-4)
    close(got, want)
    close(rows, want[[32, 0, 7]])
    with torch.no_grad():
        close(model(torch.tensor([toks, toks[::-1]], device=device))[1], O.forward(cfg, P, toks[::-1]))


def test_shared_latents_have_one_pool():
    model = VosulornForCausalLM.from_checkpoint(SHAPES["mixed"], O.random_checkpoint(SHAPES["mixed"], 1))
    kv, state = caches(model, "cpu", 4, 4)
    assert model.kv_layer_sources() == [None, None, None, 1, None]
    assert kv.k_pools[3].data_ptr() == kv.k_pools[1].data_ptr() and kv.k_pools[1].shape == (4, 4, 1, 20)
    assert kv.k_pools[0] is None and kv.v_pools[1].numel() == 0
    assert kv.k_pools[2].shape == (4, 4, 2, 10) and kv.v_pools[2].shape == (4, 4, 2, 7)
    assert state.layers[0]["S"].shape == (2, 4, 9, 6) and state.layers[0]["tail"].shape == (2, 2, 60)
    assert set(state.layers[4]) == {"S"} and not state.layers[1]


def test_loader_refuses_what_does_not_fit():
    cfg = SHAPES["mixed"]
    P = O.random_checkpoint(cfg, seed=1)
    with pytest.raises(ValueError):
        VosulornForCausalLM.from_checkpoint(cfg, dict(P, extra=torch.zeros(3)), dtype=torch.float32)
    Q = dict(P)
    del Q["l2.mix.sink"]
    with pytest.raises(KeyError):
        VosulornForCausalLM.from_checkpoint(cfg, Q, dtype=torch.float32)

    def broken(layer_index, part, **kw):
        bad = copy.deepcopy(cfg)
        (bad["layers"][layer_index] if part is None else bad["layers"][layer_index][part]).update(kw)
        with pytest.raises(ValueError):
            VosulornForCausalLM.from_checkpoint(bad, P, dtype=torch.float32)

    broken(0, None, type="something_else")
    broken(0, "mixer", kv_heads=3)
    broken(0, "mlp", kind="dense")
    broken(0, "mlp", router=dict(experts=5, top=6))
    broken(2, "mixer", rot=dict(base=10.0, dims=12))
    broken(3, "mixer", kv_from=3)
    broken(3, "mixer", kv_from=2)
    broken(3, "mixer", kv_from=1, kv_rank=11)
    broken(3, "mixer", rot=dict(base=301.0, dims=8))


@pytest.mark.gpu
@pytest.mark.parametrize("shape", sorted(SHAPES) + ["tiled"])
def test_bfloat16_serving(shape):
    """bfloat16 matrices and activations, float32 residual, norms, scores, router and recurrence: sizes that are no
    multiples of 8, and sizes the matrix-core kernels tile. A whole prompt and small steps agree with each other and
    with the oracle."""
    from colossalai_amd.inference import ContinuousBatchEngine, InferenceConfig

    moe = (6, 2, 64)
    tiled = cfg_of([layer("latent_attention", dict(dim=24, heads=4, rot_dim=8, vdim=16, kv_rank=48, scale=0.2,
                                                   rot=dict(base=1e4, dims=8)), moe),
                    layer("delta", dict(dim=32, heads=4, kv_heads=2, vdim=32, conv=4), moe),
                    layer("attention", dict(dim=32, heads=4, kv_heads=2, vdim=40, scale=0.18, mask=dict(size=24),
                                            rot=dict(base=1e4, dims=16, scaling=SCALING)), moe),
                    layer("latent_attention", dict(dim=40, heads=2, rot_dim=8, vdim=24, kv_rank=48, scale=0.15, kv_from=0,
                                                   rot=dict(base=1e4, dims=8)), moe)], width=64, vocab=80, scale=8.0)
    cfg = dict(SHAPES, tiled=tiled)[shape]
    P = {k: v.float() for k, v in O.random_checkpoint(cfg, seed=6).items()}
    toks = torch.randint(0, cfg["vocab"], (70,), generator=torch.Generator().manual_seed(8)).tolist()
    want = O.forward(cfg, P, toks).float()

    def run(cuts):
        model = VosulornForCausalLM.from_checkpoint(cfg, P, dtype=torch.bfloat16, device="cuda")
        eng = ContinuousBatchEngine(model, InferenceConfig(max_batch_size=1, dtype=torch.bfloat16), num_blocks=8,
                                    block_size=16)
        out, at = [], 0
        for n in cuts:
            out.append(eng.run_ragged([("a", toks[at : at + n], list(range(n)))]))
            at += n
        return torch.cat(out, 0).float().cpu()

    whole, stepped = run([70]), run([41, 2, 5, 14] + [1] * 8)
    scale = want.pow(2).mean().sqrt()
    for got in (whole, stepped):
        err = (got - want).pow(2).mean(-1).sqrt() / scale
        assert err.median().item() < 0.03 and (err < 0.15).float().mean().item() > 0.8
