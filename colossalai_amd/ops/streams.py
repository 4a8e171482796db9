"""Parallel residual streams ("hyper-connections").

A token carries ``S`` residual rows ``x_1 .. x_S`` (float32 ``[N, S, W]``) instead of
one. A sublayer reads ``u = sum_s read[s] x_s``; from its output ``y`` every stream is
formed anew, all at once from the old ones:

    x_t <- sum_s mix[s, t] x_s + write[t] * y        (mix indexed [from, to]).

``streams_start`` makes every stream the token's (scaled) embedding row and forms the first
sublayer's normed input. ``streams_update`` does one sublayer's write, in place,
together with the read and RMS norm of whatever comes next — the next sublayer,
or the output head, which reads the plain sum (``read=None``) — so each stream
element is read and written once per sublayer.
"""

from typing import Optional

import torch

from ._kernels import serving_kernels, use_serving_hip as use_hip
from .group_norm import grouped_rms_norm_ref

__all__ = ["streams_start", "streams_start_ref", "streams_update", "streams_update_ref"]


def _read_norm(x, read, weight, eps, out_dtype):
    u = x.sum(1) if read is None else torch.einsum("nsw,s->nw", x, read.float())
    return grouped_rms_norm_ref(u, weight, 1, eps, None, out_dtype)


def streams_start_ref(table, tokens, streams: int, read, weight, eps: float, scale: float = 1.0):
    x = (table[tokens].float() * scale)[:, None, :].repeat(1, streams, 1)
    return x, _read_norm(x, read, weight, eps, table.dtype)


def streams_start(table, tokens, streams: int, read, weight, eps: float, scale: float = 1.0):
    """table [vocab, W], tokens [N] int64 -> (streams [N, S, W] float32 = ``scale`` times the rows, ``rms_norm(u) *
    weight`` in the table's dtype). With one stream that is the start of an ordinary pre-norm model."""
    if use_hip(table):
        return tuple(serving_kernels().streams_start(table, tokens, streams, read, weight, eps, float(scale)))
    return streams_start_ref(table, tokens, streams, read, weight, eps, scale)


def streams_update_ref(x, y, mix, write, read, weight, eps: float, out_dtype=None):
    x.copy_(torch.einsum("nsw,st->ntw", x, mix.float()) + write.float()[None, :, None] * y.float()[:, None, :])
    return None if weight is None else _read_norm(x, read, weight, eps, out_dtype or y.dtype)


def streams_update(x, y, mix, write, read: Optional[torch.Tensor], weight: Optional[torch.Tensor], eps: float,
                   out_dtype=None):
    """x [N, S, W] float32, updated in place from the sublayer's output y [N, W]; ``mix`` [S, S], ``write`` [S]. Returns
    ``rms_norm(sum_s read[s] x_s) * weight`` of the new streams in ``out_dtype`` (``read=None``: the plain sum), or
    None when ``weight`` is None."""
    if use_hip(x):
        return serving_kernels().streams_update(x, y.contiguous(), mix, write, read, weight, eps, out_dtype or y.dtype)
    return streams_update_ref(x, y, mix, write, read, weight, eps, out_dtype)
