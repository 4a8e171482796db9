"""Attention whose keys are RMS-normed per head while its values are the same
projections before that norm: one cached row per token and key head.

The cache holds the key as projected, ``k``, and the float32 number
``f = 1 / sqrt(mean(k^2) + eps)`` next to it. A normed key is ``f * (w_k * k)``, so

    (w_q * q / rms(q)) . (f * w_k * k)  =  f * ((w_q * w_k * q / rms(q)) . k):

the query takes both norms' weights, the attention op multiplies a key's score
by its factor (``key_factors``) and reads keys and values from the same pool.
Half the cache and half the bytes of a decode step, and the key is not rounded a
second time after its norm.

``query_norm_key_write`` does a step's share in one launch: it norms the queries
(optionally grown with their position, ``1 + coef * ln(floor((p + 1) / every) + 1)``)
and writes keys and factors into the pool.
"""

import torch

from ._kernels import serving_kernels, use_serving_hip as use_hip
from .ragged import RaggedBatch

__all__ = ["query_norm_key_write", "query_norm_key_write_ref", "position_growth"]


def position_growth(positions, coef: float, every: float):
    """Factor of a query at position p (float32): ``1 + coef * ln(floor((p + 1) / every) + 1)``."""
    steps = torch.floor((positions.double() + 1.0) / every) + 1.0
    return 1.0 + coef * torch.log(steps.float())


def query_norm_key_write_ref(q, k, weight, eps: float, kpool, key_factors, batch: RaggedBatch, coef: float = 0.0,
                             every: float = 0.0):
    qf, kf = q.float(), k.float()
    y = qf / torch.sqrt(qf.pow(2).mean(-1, keepdim=True) + eps)
    if every > 0:
        y = y * position_growth(batch.positions, coef, every)[:, None, None]
    rows = batch.kv_rows.long()
    kpool.view(-1, *kpool.shape[2:])[rows] = k.to(kpool.dtype)
    key_factors.view(-1, key_factors.shape[2])[rows] = 1.0 / torch.sqrt(kf.pow(2).mean(-1) + eps)
    return (y * weight.float()).to(q.dtype)


def query_norm_key_write(q, k, weight, eps: float, kpool, key_factors, batch: RaggedBatch, coef: float = 0.0,
                         every: float = 0.0):
    """q [N, H, D], k [N, G, D] as projected (rows may be strided); ``weight`` [D] the product of both norms' weights.
    Writes k to rows ``batch.kv_rows`` of ``kpool`` [pages, page, G, D] and its factors to ``key_factors``
    [pages, page, G]; returns the normed queries [N, H, D] in q's dtype. ``every == 0``: no growth with position."""
    if use_hip(q):
        return serving_kernels().query_norm_key_write(q, k, weight, eps, float(coef), float(every), batch.positions, kpool,
                                                      key_factors, batch.kv_rows)
    return query_norm_key_write_ref(q, k, weight, eps, kpool, key_factors, batch, coef, every)
