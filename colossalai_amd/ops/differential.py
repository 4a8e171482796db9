"""Differential attention: two softmax maps per head over the same values.

Query head ``h`` has two queries and key head ``g`` two keys; with ``a1``, ``a2`` the
outputs of the two maps, the head's output is

    mult * unit(a1 - lambda * a2),   unit(d) = d / sqrt(mean(d^2) + eps).

For the attention op the maps are key heads of their own, ``[map 1, map 2]`` per
key/value head, that share a value head; its queries come in the order (key/value
head, map, query head of the group), which ``map_major`` brings the rows of a query
projection into once, at load time. The op hands back float32, so the difference
of two nearly equal outputs loses nothing to rounding; ``difference_norm`` forms
the heads' outputs in one pass.
"""

import torch

from ._kernels import serving_kernels, use_serving_hip as use_hip

__all__ = ["map_major", "difference_norm", "difference_norm_ref", "difference_weight"]


def map_major(rows: torch.Tensor, heads: int, kv_heads: int, dim: int) -> torch.Tensor:
    """Reorder the rows of a query projection (or its bias) from (head, map, channel) to (key/value head, map, query
    head of the group, channel)."""
    tail = rows.shape[1:]
    r = rows.view(kv_heads, heads // kv_heads, 2, dim, *tail)
    return r.transpose(1, 2).reshape(heads * 2 * dim, *tail).contiguous()


def difference_weight(lq1, lk1, lq2, lk2, base: float) -> float:
    """``exp(lq1 . lk1) - exp(lq2 . lk2) + base`` in float32."""
    a, b = (lq1.float() * lk1.float()).sum(), (lq2.float() * lk2.float()).sum()
    return float(torch.exp(a) - torch.exp(b)) + base


def difference_norm_ref(o, kv_heads: int, lam: float, mult: float, eps: float, out_dtype=None):
    N, H2, Dv = o.shape
    a = o.float().view(N, kv_heads, 2, H2 // 2 // kv_heads, Dv)
    d = a[:, :, 0] - lam * a[:, :, 1]
    d = d / torch.sqrt(d.pow(2).mean(-1, keepdim=True) + eps) * mult
    return d.reshape(N, H2 // 2 * Dv).to(out_dtype or o.dtype)


def difference_norm(o, kv_heads: int, lam: float, mult: float, eps: float, out_dtype=None):
    """o [N, 2H, Dv] float32 in the order (key/value head, map, query head of the group) -> [N, H * Dv], heads in
    their own order."""
    if use_hip(o):
        return serving_kernels().difference_norm(o, kv_heads, float(lam), float(mult), float(eps), out_dtype or o.dtype)
    return difference_norm_ref(o, kv_heads, lam, mult, eps, out_dtype)
