"""Bekulix against the float64 oracle (tests/bekulix_oracle.py): every mechanism alone, then whole
models of several shapes, on the CPU (reference path of every op) and on the GPU (HIP kernels)."""

import copy
import os
import sys

import pytest
import torch

ROOT = os.path.dirname(os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
sys.path.insert(0, os.path.join(ROOT, "tests"))
import bekulix_oracle as O  # noqa: E402

from colossalai_amd.inference.kv_cache import KVCacheManager  # noqa: E402
from colossalai_amd.models import BekulixForCausalLM, model_class_for  # noqa: E402
from colossalai_amd.ops import differential, latent_attention, normed_keys, streams  # noqa: E402
from colossalai_amd.ops.activation import relu_mul  # noqa: E402
from colossalai_amd.ops.paged_attention import paged_attention, paged_kv_write  # noqa: E402
from colossalai_amd.ops.ragged import RaggedBatch  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64

ATT = dict(dim=10, heads=6, kv_heads=3, vdim=10, scale=0.4, q_temp=dict(coef=0.7, every=5))
DIF = dict(dim=6, heads=4, kv_heads=2, vdim=9, scale=0.5, diff=0.45, mask=dict(size=7))
LAT = dict(dim=7, heads=3, vdim=5, kv_rank=12, scale=0.6, mask=dict(size=6))


def layer(kind, mixer, ff=None):
    return dict(type=kind, mixer=mixer, mlp=None if ff is None else dict(kind="dense", ff=ff))


def cfg_of(layers, loop=None, width=28, vocab=50, streams=3, eps=1e-5):
    c = dict(architecture="Bekulix", layers=layers, norm=dict(eps=eps), streams=streams, vocab=vocab, width=width)
    if loop is not None:
        c["loop"] = loop
    return c


SHAPES = {
    # every kind, a looped middle, a layer without a feed-forward
    "looped_middle": cfg_of([layer("attention_2", DIF, 20), layer("attention", ATT, 9), layer("latent_attention", LAT),
                             layer("attention", dict(ATT, heads=2, kv_heads=2, scale=1.1, q_temp=dict(coef=0.2, every=3)), 17)],
                            loop=dict(start=1, stop=3, times=2)),
    # no loop; one key/value head, one query head, a window of one and a block of one position, one stream
    "plain": cfg_of([layer("latent_attention", dict(LAT, mask=dict(size=1), heads=1), 8),
                     layer("attention", dict(ATT, heads=1, kv_heads=1, q_temp=dict(coef=1.5, every=1))),
                     layer("attention_2", dict(DIF, heads=3, kv_heads=1, mask=dict(size=1)), 11)], width=20, streams=1),
    # the whole model is the loop, three passes, many streams, windows and blocks wider than the sequence
    "all_looped": cfg_of([layer("latent_attention", dict(LAT, mask=dict(size=500), kv_rank=5)),
                          layer("attention_2", dict(DIF, heads=5, kv_heads=5, vdim=3, mask=dict(size=400), diff=0.0), 6)],
                         loop=dict(start=0, stop=2, times=3), width=18, streams=9, eps=1e-3),
    # the loop runs once and ends the model
    "loop_once": cfg_of([layer("attention", dict(ATT, dim=3, vdim=3, heads=4, kv_heads=1), 5), layer("attention_2", DIF, 16)],
                        loop=dict(start=1, stop=2, times=1), width=24, streams=2),
}


def close(got, want, tol=3e-4):
    got, want = got.detach().cpu().to(F64), want.to(F64)
    err = (got - want).abs().max().item()
    assert err <= tol * max(1.0, want.abs().max().item()), f"max abs error {err}"


class Pages:
    """A scattered page table over pools of garbage, and the batches of one sequence fed in portions."""

    def __init__(self, T, device, page):
        self.page, self.device = page, device
        self.num = (T + page - 1) // page + 3
        order = torch.randperm(self.num, generator=torch.Generator().manual_seed(T)).tolist()
        self.table = order

    def pool(self, heads, dim, dtype=torch.float32):
        return torch.full((self.num, self.page, heads, dim), float("nan"), device=self.device, dtype=dtype)

    def batches(self, cuts):
        at = 0
        for n in cuts:
            need = (at + n + self.page - 1) // self.page
            yield slice(at, at + n), RaggedBatch.build([n], [at], [0], self.device, [self.table[:need]], self.page)
            at += n


def rand(seed, *shape):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed))


def cuts_of(T, edge):
    """Whole; cut at the special place; just before and after it; in pairs; the tail decoded."""
    out = [[T], [edge, T - edge], [edge - 1, 2, T - edge - 1], [T - 9] + [1] * 9]
    if T <= 60:
        out.append([2] * (T // 2) + [1] * (T % 2))
    return [[n for n in c if n > 0] for c in out]


# ------------------------------------------------------------- shared keys and values
def framework_shared(q, k, wq, wk, c, eps, device, cuts, page):
    T, (G, D) = q.shape[0], k.shape[1:]
    pg = Pages(T, device, page)
    pool, fac = pg.pool(G, D), pg.pool(G, 1)[..., 0].contiguous()
    t = c.get("q_temp") or dict(coef=0.0, every=0)
    out = []
    for sl, batch in pg.batches(cuts):
        qn = normed_keys.query_norm_key_write(q[sl].to(device), k[sl].to(device), (wq * wk).to(device), eps, pool, fac, batch,
                                              t["coef"], t["every"])
        out.append(paged_attention(qn, pool, pool, batch, c["scale"], key_factors=fac))
    return torch.cat(out, 0)


def oracle_shared(q, k, wq, wk, c, eps):
    q, raw = q.to(F64), k.to(F64)
    T, H, G = q.shape[0], q.shape[1], raw.shape[1]
    qn, kn = O.unit_rms(q, eps) * wq.to(F64), O.unit_rms(raw, eps) * wk.to(F64)
    t = c.get("q_temp")
    if t:
        qn = qn * torch.tensor([O.query_temperature(p, t["coef"], t["every"]) for p in range(T)], dtype=F64).view(T, 1, 1)
    return torch.stack([O.attend(qn[:, h], kn[:, h // (H // G)], raw[:, h // (H // G)], c["scale"], O.sees_causal)
                        for h in range(H)], 1)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,temp", [(6, 3, 10, dict(coef=0.7, every=5)), (4, 1, 3, None), (2, 2, 16, dict(coef=2.0, every=1)),
                                        (5, 5, 8, dict(coef=-0.1, every=64)), (8, 1, 24, dict(coef=0.5, every=7))])
def test_values_are_the_keys_before_their_norm(device, H, G, D, temp):
    T, c = 45, dict(scale=0.5, q_temp=temp)
    q, k = rand(1, T, H, D) * 2, rand(2, T, G, D) * torch.linspace(0.2, 4, T)[:, None, None]
    wq, wk = 1 + 0.5 * rand(3, D), 1 + 0.5 * rand(4, D)
    want = oracle_shared(q, k, wq, wk, c, 1e-4)
    for cuts in cuts_of(T, 17):
        close(framework_shared(q, k, wq, wk, c, 1e-4, device, cuts, 4), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("far", [0, 1, 3, 4, 63, 64, 127, 128, 300, 388, 389])
@pytest.mark.parametrize("D", [24, 10])
def test_one_key_far_back_takes_the_weight(device, far, D):
    """Among several hundred keys the last query's score stands out at one place: the first tokens, both sides of
    a page border, the query itself. In a prompt portion and as a decoded token."""
    T, H, G = 390, 2, 1
    c = dict(scale=1.0, q_temp=None)
    q, k, one = rand(5, T, H, D), rand(6, T, G, D), torch.ones(D)
    k = k / k.pow(2).mean(-1, keepdim=True).sqrt() * (0.5 + torch.rand(T, G, 1, generator=torch.Generator().manual_seed(1)))
    q[T - 1] = k[far, 0]
    c["scale"] = 4.0 if D < 20 else 2.0
    qn, kn = O.unit_rms(q.to(F64), 1e-5), O.unit_rms(k.to(F64), 1e-5)
    want = torch.stack([O.attend(qn[T - 1 :, h], kn[:, 0], k[:, 0].to(F64), c["scale"], lambda i, j: True) for h in range(H)], 1)
    assert (want[0, 0] - k[far, 0].to(F64)).abs().max() < 0.05, "the test's spike does not stand out"
    for cuts in ([T], [T - 1, 1], [T - 19, 19]):
        close(framework_shared(q, k, one, one, c, 1e-5, device, cuts, 64)[T - 1 :], want)


@pytest.mark.parametrize("every", [1, 2, 7, 100, 2.5])
def test_growth_steps_at_the_right_position(every):
    pos = torch.arange(0, 300, dtype=torch.int32)
    got = normed_keys.position_growth(pos, 0.3, every)
    close(got, torch.tensor([O.query_temperature(p, 0.3, every) for p in range(300)]), 1e-6)
    if every == 7:
        assert float(got[5]) == 1.0 < float(got[6]) == float(got[12]) < float(got[13])


# --------------------------------------------------------------- windowed latent attention
def framework_latent(q, dkv, w_uk, w_uv, norm_w, c, device, cuts, page, eps=1e-5):
    T, H, D = q.shape
    rank = dkv.shape[1]
    pg = Pages(T, device, page)
    pool, out = pg.pool(1, rank), []
    uv = w_uv.view(H, -1, rank).to(device)
    for sl, batch in pg.batches(cuts):
        latent_attention.latent_kv_write(dkv[sl].to(device), norm_w.to(device), eps, None, pool, batch)
        out.append(latent_attention.latent_attention(q[sl].to(device), w_uk.view(H, D, rank).to(device), uv, pool, batch,
                                                     c["scale"], None, rank, window=c["mask"]["size"],
                                                     w_uv_t=uv.transpose(1, 2).contiguous() if sl.start % 2 else None))
    return torch.cat(out, 0)


def oracle_latent(q, dkv, w_uk, w_uv, norm_w, c, size=None, eps=1e-5):
    T, H, D = q.shape
    size = c["mask"]["size"] if size is None else size
    lat = O.unit_rms(dkv.to(F64), eps) * norm_w.to(F64)
    k, v = O.lin(lat, w_uk).view(T, H, D), O.lin(lat, w_uv).view(T, H, -1)
    return torch.cat([O.attend(q[:, h].to(F64), k[:, h], v[:, h], c["scale"], lambda i, j: O.sees_window(i, j, size))
                      for h in range(H)], -1)


def latent_inputs(T, H, D, Dv, rank, seed, spike=None):
    q, dkv = rand(seed, T, H, D), rand(seed + 1, T, rank)
    w_uk, w_uv = rand(seed + 2, H * D, rank) / rank ** 0.5, rand(seed + 3, H * Dv, rank) / rank ** 0.5
    norm_w = 1 + 0.2 * rand(seed + 4, rank)
    if spike is not None:
        i, j = spike
        lat = O.unit_rms(dkv[j : j + 1].to(F64), 1e-5) * norm_w.to(F64)
        q[i] = 10.0 * O.lin(lat, w_uk).view(H, D).float()
    return q, dkv, w_uk, w_uv, norm_w


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,Dv,rank,size", [(3, 7, 5, 12, 6), (1, 4, 8, 16, 1), (2, 8, 8, 3, 17), (4, 5, 9, 20, 200), (2, 3, 2, 9, 2)])
def test_windowed_latent_attention(device, H, D, Dv, rank, size):
    T, c = 43, dict(scale=0.8, mask=dict(size=size))
    args = latent_inputs(T, H, D, Dv, rank, 10)
    want = oracle_latent(*args, c)
    for cuts in cuts_of(T, 16):
        close(framework_latent(*args, c, device, cuts, 4), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,back", [(33, 32), (33, 33), (64, 63), (64, 64), (64, 65), (100, 99), (100, 100), (5, 0)])
def test_a_spike_at_the_windows_edge(device, size, back):
    """The last query's score stands out ``back`` places before it: inside the window it takes the weight, outside it
    is not seen at all."""
    T, c = 150, dict(scale=1.0, mask=dict(size=size))
    args = latent_inputs(T, 2, 16, 6, 24, 20, spike=(T - 1, T - 1 - back))
    want = oracle_latent(*args, c)
    if back in (size - 1, size):  # one token more or less in the window shows
        off = oracle_latent(*args, c, size=size - 1 if back < size else size + 1)
        assert (off[T - 1] - want[T - 1]).abs().max() > 0.3
    for cuts in ([T], [T - 1, 1], [T - 20, 20], [T - 3, 2, 1], [64, 64, T - 128]):
        close(framework_latent(*args, c, device, cuts, 16), want)


# ----------------------------------------------------------- chunked differential attention
def framework_differential(q, k, v, lam, c, eps, device, cuts, page):
    """q [T, H, 2, D], k [T, G, 2, D], v [T, G, Dv]."""
    T, H, _, D = q.shape
    G, Dv = v.shape[1:]
    qm = differential.map_major(q.reshape(T, -1).t().contiguous(), H, G, D).t().reshape(T, 2 * H, D)
    pg = Pages(T, device, page)
    kpool, vpool, out = pg.pool(2 * G, D), pg.pool(G, Dv), []
    for sl, batch in pg.batches(cuts):
        paged_kv_write(k[sl].reshape(-1, 2 * G, D).to(device), v[sl].to(device), kpool, vpool, batch)
        a = paged_attention(qm[sl].contiguous().to(device), kpool, vpool, batch, c["scale"], chunk=c["mask"]["size"],
                            out_dtype=torch.float32)
        out.append(differential.difference_norm(a, G, lam, 1.0 - c["diff"], eps, torch.float32))
    return torch.cat(out, 0)


def oracle_differential(q, k, v, lam, c, eps, size=None):
    T, H = q.shape[:2]
    G = k.shape[1]
    size = c["mask"]["size"] if size is None else size
    q, k, v = q.to(F64), k.to(F64), v.to(F64)
    heads = []
    for h in range(H):
        g = h // (H // G)
        a = [O.attend(q[:, h, m], k[:, g, m], v[:, g], c["scale"], lambda i, j: O.sees_chunk(i, j, size)) for m in (0, 1)]
        heads.append(O.combine_maps(a[0], a[1], lam, c["diff"], eps))
    return torch.cat(heads, -1)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv,size,diff", [(4, 2, 6, 9, 7, 0.45), (3, 1, 8, 16, 16, 0.0), (2, 2, 5, 3, 1, 0.9), (6, 3, 4, 8, 100, 0.2),
                                                (8, 2, 16, 8, 13, -0.3)])
def test_differential_attention_inside_blocks(device, H, G, D, Dv, size, diff):
    T, c, lam = 45, dict(scale=0.6, mask=dict(size=size), diff=diff), 0.35 + diff
    q, k, v = rand(30, T, H, 2, D), rand(31, T, G, 2, D), rand(32, T, G, Dv)
    want = oracle_differential(q, k, v, lam, c, 1e-4)
    edge = min(size * (T // 2 // size), 40) or 20
    for cuts in cuts_of(T, edge):
        close(framework_differential(q, k, v, lam, c, 1e-4, device, cuts, 4), want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,i,j", [(50, 100, 100), (50, 100, 99), (50, 149, 100), (50, 149, 99), (64, 127, 64), (64, 127, 63),
                                      (64, 128, 127), (33, 98, 66), (33, 98, 65), (33, 99, 98)])
def test_a_spike_at_a_blocks_border(device, size, i, j):
    """Query ``i``'s first map points at key ``j``: the first or last token of its block, or the one before the block,
    which is not seen. Prompt cut anywhere, and decoded."""
    T, H, G, D, Dv = i + 1, 2, 1, 12, 8
    c, lam = dict(scale=1.0, mask=dict(size=size), diff=0.3), 0.4
    q, k, v = rand(40, T, H, 2, D), rand(41, T, G, 2, D), rand(42, T, G, Dv)
    q[i, :, 0] = 3.0 * k[j, 0, 0]
    want = oracle_differential(q, k, v, lam, c, 1e-5)
    moved = v.clone()
    moved[j] += 5 * rand(43, G, Dv)  # the key's value enters the query's output if, and only if, the block shows it
    moved = (oracle_differential(q, k, moved, lam, c, 1e-5)[i] - want[i]).abs().max()
    assert moved > 0.3 if i // size == j // size else moved == 0
    for cuts in ([T], [T - 1, 1], [T - 3, 2, 1], [size - 1] + [T - size + 1], [40, T - 40]):
        close(framework_differential(q, k, v, lam, c, 1e-5, device, [n for n in cuts if n > 0], 16), want)


def test_difference_weight_and_row_order():
    lq1, lk1, lq2, lk2 = (rand(50 + i, 9) * 0.5 for i in range(4))
    assert abs(differential.difference_weight(lq1, lk1, lq2, lk2, 0.4) - O.difference_weight(lq1, lk1, lq2, lk2, 0.4)) < 1e-6
    H, G, D = 6, 2, 3
    rows = torch.arange(H * 2 * D)
    got = differential.map_major(rows, H, G, D).view(G, 2, H // G, D)
    for h in range(H):
        for m in (0, 1):
            assert torch.equal(got[h // (H // G), m, h % (H // G)], rows.view(H, 2, D)[h, m])


@pytest.mark.parametrize("device", DEVICES)
def test_nearly_equal_maps_keep_their_difference(device):
    """With lambda = 1 and maps that differ by 1e-3 the normed difference is of order one."""
    N, G, R, Dv = 5, 2, 3, 20
    a = rand(60, N, G, 1, R, Dv)
    o = torch.cat([a, a + 1e-3 * rand(61, N, G, 1, R, Dv)], 2).reshape(N, 2 * G * R, Dv)
    x = o.to(F64).view(N, G, 2, R, Dv)
    want = O.combine_maps(x[:, :, 0], x[:, :, 1], 1.0, 0.25, 1e-9).reshape(N, -1)
    close(differential.difference_norm(o.to(device), G, 1.0, 0.75, 1e-9), want, 2e-3)


# ----------------------------------------------------------------------- streams, feed-forward
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("S,W", [(1, 20), (2, 64), (3, 28), (4, 1030), (5, 12), (7, 24), (8, 2052), (9, 30), (16, 8)])
def test_streams(device, S, W):
    """Start, two updates in a row and the closing sum, against the equations; the mix is not symmetric."""
    N = 6
    table, toks = rand(70, 11, W), torch.tensor([3, 0, 10, 7, 7, 1])
    read = [rand(71 + i, S) for i in range(2)]
    mix, write = [rand(75 + i, S, S) for i in range(2)], [rand(79 + i, S) for i in range(2)]
    w = [1 + 0.3 * rand(83 + i, W) for i in range(3)]
    ys = [rand(90 + i, N, W) for i in range(2)]
    X = torch.stack([table[toks].to(F64)] * S)

    def normed(u, i):
        return O.one_plus_norm(u, w[i] - 1, 1e-4)

    d = device
    x, h = streams.streams_start(table.to(d), toks.to(d), S, read[0].to(d), w[0].to(d), 1e-4)
    close(x.transpose(0, 1), X)
    close(h, normed(O.read_streams(X, read[0]), 0), 1e-4)
    X = O.write_streams(X, mix[0], write[0], ys[0])
    h = streams.streams_update(x, ys[0].to(d), mix[0].to(d), write[0].to(d), read[1].to(d), w[1].to(d), 1e-4)
    close(x.transpose(0, 1), X, 1e-5)
    close(h, normed(O.read_streams(X, read[1]), 1), 1e-4)
    X = O.write_streams(X, mix[1], write[1], ys[1])
    h = streams.streams_update(x, ys[1].to(d), mix[1].to(d), write[1].to(d), None, w[2].to(d), 1e-4)
    close(x.transpose(0, 1), X, 1e-5)
    close(h, normed(X.sum(0), 2), 1e-4)
    assert streams.streams_update(x, ys[0].to(d), mix[0].to(d), write[0].to(d), None, None, 1e-4) is None
    close(x.transpose(0, 1), O.write_streams(X, mix[0], write[0], ys[0]), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("ff", [21, 64])
def test_dense_feed_forward_activation(device, ff):
    packed = rand(0, 9, 2 * ff) * 3
    close(relu_mul(packed.to(device)), torch.clamp(packed[:, :ff].to(F64), min=0) * packed[:, ff:].to(F64), 1e-6)


# -------------------------------------------------------------------- whole models
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("shape", sorted(SHAPES))
def test_whole_model_and_every_layer_run(device, shape):
    cfg = SHAPES[shape]
    P = {k: v.float() for k, v in O.random_checkpoint(cfg, seed=5).items()}
    toks = torch.randint(0, cfg["vocab"], (33,), generator=torch.Generator().manual_seed(7)).tolist()
    want_res = []
    want = O.forward(cfg, P, toks, want_res)
    assert model_class_for(cfg) is BekulixForCausalLM
    model = BekulixForCausalLM.from_checkpoint(cfg, P, dtype=torch.float32, device=device)
    assert len(model.runs) == len(want_res) == len(model.kv_layer_shapes()) == len(model.state_layer_buffers())
    assert model.config.from_dict(model.config.to_dict()) == model.config
    page = 8
    kv = KVCacheManager(len(model.runs), 0, 0, num_blocks=6, block_size=page, device=device, dtype=torch.float32,
                        layer_shapes=model.kv_layer_shapes(), layer_key_factors=model.kv_layer_key_factors())
    batch = RaggedBatch.build([33], [0], [0], device, [[5, 1, 0, 4, 2]], page)
    got_res = []
    with torch.no_grad():
        got = model.forward_ragged(torch.tensor(toks, device=device), batch, kv, None, None, got_res)
        rows = model.forward_ragged(torch.tensor(toks, device=device), batch, kv, None, torch.tensor([32, 0, 7], device=device))
    for a, b in zip(got_res, want_res):
        close(a, b, 2e-4)
    close(got, want)
    close(rows, want[[32, 0, 7]])
    with torch.no_grad():
        close(model(torch.tensor([toks, toks[::-1]], device=device))[1], O.forward(cfg, P, toks[::-1]))


def test_passes_of_a_looped_layer_keep_pages_of_their_own():
    model = BekulixForCausalLM.from_checkpoint(SHAPES["looped_middle"], O.random_checkpoint(SHAPES["looped_middle"], 1))
    assert model.runs == [0, 1, 2, 1, 2, 3]
    kv = KVCacheManager(6, 0, 0, num_blocks=2, block_size=4, device="cpu", layer_shapes=model.kv_layer_shapes(),
                        layer_key_factors=model.kv_layer_key_factors())
    assert kv.k_pools[1].data_ptr() != kv.k_pools[3].data_ptr() and kv.k_factors[1].shape == (2, 4, 3)
    assert kv.v_pools[1].numel() == 0  # keys serve as values
    assert kv.k_pools[0].shape == (2, 4, 4, 6) and kv.v_pools[0].shape == (2, 4, 2, 9)


def test_loader_refuses_stray_and_missing_tensors():
    cfg = SHAPES["looped_middle"]
    P = O.random_checkpoint(cfg, seed=1)
    with pytest.raises(ValueError):
        BekulixForCausalLM.from_checkpoint(cfg, dict(P, extra=torch.zeros(3)), dtype=torch.float32)
    Q = dict(P)
    del Q["l0.hc2.mix"]
    with pytest.raises(KeyError):
        BekulixForCausalLM.from_checkpoint(cfg, Q, dtype=torch.float32)
    bad = copy.deepcopy(cfg)
    bad["layers"][0]["type"] = "something_else"
    with pytest.raises(ValueError):
        BekulixForCausalLM.from_checkpoint(bad, P, dtype=torch.float32)
    bad = copy.deepcopy(cfg)
    bad["layers"][1]["mixer"]["vdim"] = 4
    with pytest.raises(ValueError):
        BekulixForCausalLM.from_checkpoint(bad, P, dtype=torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("shape", sorted(SHAPES) + ["tiled"])
def test_bfloat16_serving(shape):
    """bfloat16 matrices and activations, float32 streams, norms, scores and maps: sizes that are no multiples of 8,
    and sizes the matrix-core kernel tiles. A whole prompt and small steps agree with each other and with the oracle."""
    from colossalai_amd.inference import ContinuousBatchEngine, InferenceConfig

    tiled = cfg_of([layer("attention", dict(ATT, dim=32, vdim=32, heads=4, kv_heads=2, scale=0.1), 96),
                    layer("attention_2", dict(DIF, dim=16, vdim=40, heads=4, kv_heads=2, scale=0.12, diff=0.2, mask=dict(size=24)), 64),
                    layer("latent_attention", dict(LAT, dim=24, vdim=16, heads=4, kv_rank=48, mask=dict(size=20), scale=0.2), 64)],
                   loop=dict(start=0, stop=2, times=2), width=64, vocab=80, streams=4)
    cfg = dict(SHAPES, tiled=tiled)[shape]
    P = {k: v.float() for k, v in O.random_checkpoint(cfg, seed=6).items()}
    toks = torch.randint(0, cfg["vocab"], (70,), generator=torch.Generator().manual_seed(8)).tolist()
    want = O.forward(cfg, P, toks).float()

    def run(cuts):
        model = BekulixForCausalLM.from_checkpoint(cfg, P, dtype=torch.bfloat16, device="cuda")
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
        assert err.median().item() < 0.03 and (err < 0.15).float().mean().item() > 0.9
