"""Rotary positions on neighbouring pairs of a ragged serving batch.

Dimension ``2i`` is paired with ``2i + 1`` (the interleaved layout), ``i`` from
0 to ``dims / 2 - 1``; the pair ``(u, v)`` of a token at position ``p`` becomes
``(u cos a - v sin a, v cos a + u sin a)`` with ``a = p * f_i`` and
``f_i = base^(-2 i / dims)``. Only the first ``dims`` channels of a vector turn;
the rest pass unchanged. Positions, angles, sine and cosine are float32 (the
frequencies are formed in float64 and rounded once).

``pair_frequencies`` optionally stretches long wavelengths (``scaling``):
with ``l = 2 pi / f``, a frequency stays where ``l < original / high``, becomes
``f / factor`` where ``l > original / low``, and is mixed linearly in
``original / l`` between the two. ``rotate_qk_write`` turns a step's queries in
place and puts its turned keys and its values into the pages, in one launch.
``halves_to_pairs`` reorders the output rows of a projection whose rotated
channels are paired ``(i, i + dims / 2)`` so that the pairs become neighbours:
when queries and keys are both reordered the scores are the same, and a model
in that layout runs on the kernels of this one.
"""

import math
from typing import Optional

import torch

from ._kernels import serving_kernels, use_serving_hip as use_hip
from .ragged import RaggedBatch

__all__ = ["pair_frequencies", "rotate_pairs", "rotate_pairs_ref", "rotate_qk_write", "rotate_qk_write_ref",
           "halves_to_pairs"]


def pair_frequencies(base: float, dims: int, device=None, scaling: Optional[dict] = None) -> torch.Tensor:
    """f_i = base^(-2 i / dims), i = 0 .. dims / 2 - 1, float32. ``scaling`` = {"factor", "low", "high", "original"}."""
    assert dims % 2 == 0, "pairs need an even number of rotated channels"
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / dims)
    if scaling:
        factor, low, high, original = (float(scaling[n]) for n in ("factor", "low", "high", "original"))
        turns = original * f / (2.0 * math.pi)      # original / wavelength
        mix = (turns - low) / (high - low) if high != low else torch.zeros_like(f)
        f = torch.where(turns > high, f, torch.where(turns < low, f / factor, (1.0 - mix) * f / factor + mix * f))
    return f.to(torch.float32).to(device)


def halves_to_pairs(rows: torch.Tensor, heads: int, size: int, first: int, dims: int) -> torch.Tensor:
    """Reorder the rows [heads * size, ...] of a projection: of every head's ``size`` outputs, the ``dims`` from
    ``first`` on go from the order ``(i, i + dims / 2)`` per pair to neighbouring places."""
    assert dims % 2 == 0 and first + dims <= size and rows.shape[0] == heads * size
    place = torch.arange(size)
    place[first : first + dims] = first + torch.arange(dims).view(2, dims // 2).t().reshape(-1)
    return rows.view(heads, size, *rows.shape[1:])[:, place.to(rows.device)].reshape(rows.shape)


def rotate_pairs_ref(x, positions, freqs, out: Optional[torch.Tensor] = None):
    dims = 2 * freqs.numel()
    ang = positions.to(torch.float32)[:, None] * freqs.to(torch.float32)[None, :]     # [N, dims / 2]
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [dims // 2]
    c, s = torch.cos(ang).view(shape), torch.sin(ang).view(shape)
    xf = x.float()
    u, v = xf[..., 0:dims:2], xf[..., 1:dims:2]
    y = xf.clone()
    y[..., 0:dims:2] = u * c - v * s
    y[..., 1:dims:2] = v * c + u * s
    if out is None:
        return y.to(x.dtype)
    out.copy_(y.to(out.dtype))
    return out


def rotate_pairs(x, positions, freqs, out: Optional[torch.Tensor] = None):
    """x [N, H, R] (any row and head strides, unit channel stride), positions [N] int32, freqs [dims / 2] float32
    with ``dims <= R``. Writes to ``out`` (same shape, its own strides; may be ``x`` itself) or a new tensor."""
    assert x.dim() == 3 and 2 * freqs.numel() <= x.shape[-1]
    if use_hip(x):
        if out is None:
            out = torch.empty(x.shape, dtype=x.dtype, device=x.device)
        serving_kernels().rotate_pairs(x, positions, freqs, out)
        return out
    return rotate_pairs_ref(x, positions, freqs, out)


def rotate_qk_write_ref(q, k, v, freqs, kpool, vpool, batch: RaggedBatch):
    rotate_pairs_ref(q, batch.positions, freqs, out=q)
    rows = batch.kv_rows.long()
    kpool.view(-1, *kpool.shape[2:])[rows] = rotate_pairs_ref(k, batch.positions, freqs).to(kpool.dtype)
    vpool.view(-1, *vpool.shape[2:])[rows] = v.to(vpool.dtype)


def rotate_qk_write(q, k, v, freqs, kpool, vpool, batch: RaggedBatch) -> None:
    """q [N, H, D] (dense heads, any row stride) is turned in place; k [N, G, D], turned, and v [N, G, Dv] go to rows
    ``batch.kv_rows`` of the pools ([pages, page_size, G, D] / [.., Dv]). freqs [dims / 2] float32, ``dims <= D``."""
    assert q.shape[-1] == k.shape[-1] and 2 * freqs.numel() <= q.shape[-1]
    if use_hip(q):
        serving_kernels().rotate_qk_write(q, k, v, freqs, batch.positions, kpool, vpool, batch.kv_rows)
        return
    rotate_qk_write_ref(q, k, v, freqs, kpool, vpool, batch)
