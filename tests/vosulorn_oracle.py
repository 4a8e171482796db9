"""A plain, slow float64 implementation of the Vosulorn design, one function per
mechanism, written from the design's equations. It shares no code with
``colossalai_amd``: the tests compare the framework against it.

Notation: ``h`` is a sublayer's input ``[T, W]`` (one sequence, T tokens from
position 0), weights are ``[out, in]`` and applied as ``h @ W.T``; ``P`` is a
dict of the checkpoint's tensors by name.
"""

import math

import torch

F64 = torch.float64
UNIT_EPS = 1e-6


def lin(h, w, b=None):
    y = h @ w.to(F64).T
    return y if b is None else y + b.to(F64)


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(F64)


def silu(z):
    return z / (1.0 + torch.exp(-z))


# ---------------------------------------------------------------------- positions
def frequencies(base, dims):
    return [base ** (-2.0 * i / dims) for i in range(dims // 2)]


def stretched(f, s):
    """One frequency under the wavelength-dependent scaling: short waves stay, long ones are divided by the factor, a
    linear mix between the two."""
    wave = 2.0 * math.pi / f
    if wave < s["original"] / s["high"]:
        return f
    if wave > s["original"] / s["low"]:
        return f / s["factor"]
    mix = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
    return (1.0 - mix) * f / s["factor"] + mix * f


def rotation_frequencies(rot):
    fs = frequencies(rot["base"], rot["dims"])
    return [stretched(f, rot["scaling"]) for f in fs] if rot.get("scaling") else fs


def turn(x, first, second, angle):
    """Channels ``first`` and ``second`` of x [T, ...] as the pair (u, v), turned by angle [T]."""
    out = x.clone()
    shape = [-1] + [1] * (x.dim() - 2)
    c, s = torch.cos(angle).view(shape), torch.sin(angle).view(shape)
    u, v = x[..., first], x[..., second]
    out[..., first] = u * c - v * s
    out[..., second] = v * c + u * s
    return out


def rotate_neighbours(x, freqs):
    """x [T, heads, D]: channel 2i with 2i + 1."""
    p = torch.arange(x.shape[0], dtype=F64)
    for i, f in enumerate(freqs):
        x = turn(x, 2 * i, 2 * i + 1, p * f)
    return x


def rotate_halves(x, freqs):
    """x [T, heads, D]: channel i with i + len(freqs)."""
    p = torch.arange(x.shape[0], dtype=F64)
    for i, f in enumerate(freqs):
        x = turn(x, i, i + len(freqs), p * f)
    return x


# --------------------------------------------------------------------- visibility
def sees_causal(i, j):
    return j <= i


def sees_chunk(i, j, size):
    """Positions up to the query inside the query's own block of ``size`` positions."""
    return (j <= i) & (i // size == j // size)


def attend(q, k, v, scale, sees, sink=None):
    """One head: q [T, D], k [S, D], v [S, Dv]; ``sees(i, j)`` says whether query i reads the keys j (a tensor of
    places). Query by query. ``sink``: a score without key and value that enters the denominator once."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F64)
    places = torch.arange(k.shape[0])
    for i in range(q.shape[0]):
        vis = places[sees(torch.tensor(i), places)]
        s = (k[vis] @ q[i]) * scale
        top = float(s.max()) if sink is None else max(float(s.max()), float(sink))
        w = torch.exp(s - top)
        den = w.sum() + (0.0 if sink is None else math.exp(float(sink) - top))
        out[i] = (w / den) @ v[vis]
    return out


# ------------------------------------------------------------------------- mixers
def short_conv(x, taps):
    """x [T, C], taps [C, K]: the last tap is the current token's, zeros ahead of the start, then silu."""
    T, K = x.shape[0], taps.shape[1]
    t = taps.to(F64)
    y = torch.zeros_like(x)
    for i in range(T):
        for d in range(K):
            if i - d >= 0:
                y[i] += t[:, K - 1 - d] * x[i - d]
    return silu(y)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def head_decay(a, A_log, dt_bias):
    """a [T, H] -> the factor a head's state is multiplied with."""
    z = a + dt_bias.to(F64)
    softplus = torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))
    return torch.exp(-torch.exp(A_log.to(F64)) * softplus)


def delta_scan(q, k, v, g, beta, S=None):
    """One head, token by token: q, k [T, D] (k a unit vector), v [T, Dv], g and beta [T]. Returns the outputs and
    the final state [D, Dv]."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=F64) if S is None else S
    out = []
    for t in range(q.shape[0]):
        S = g[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out.append(S.T @ q[t])
    return torch.stack(out), S


def delta_mixer(h, P, pre, c, eps):
    T, H, G, D, Dv = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (short_conv(lin(h, P[pre + n]), P[pre + n + ".conv"]) for n in ("q", "k", "v"))
    q, k, v = unit(q.view(T, G, D)) * D ** -0.5, unit(k.view(T, G, D)), v.view(T, H, Dv)
    beta = 1.0 / (1.0 + torch.exp(-lin(h, P[pre + "b"])))
    g = head_decay(lin(h, P[pre + "a"]), P[pre + "A_log"], P[pre + "dt_bias"])
    heads = [delta_scan(q[:, x // (H // G)], k[:, x // (H // G)], v[:, x], g[:, x], beta[:, x])[0] for x in range(H)]
    o = rms_norm(torch.stack(heads, 1), P[pre + "norm"], eps).reshape(T, H * Dv)
    return lin(o * silu(lin(h, P[pre + "g"])), P[pre + "o"])


def chunked_attention(h, P, pre, c, eps):
    T, H, G, D, Dv = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    f = rotation_frequencies(c["rot"])
    q = rotate_neighbours(lin(h, P[pre + "q"], P[pre + "q.b"]).view(T, H, D), f)
    k = rotate_neighbours(lin(h, P[pre + "k"], P[pre + "k.b"]).view(T, G, D), f)
    v = lin(h, P[pre + "v"], P[pre + "v.b"]).view(T, G, Dv)
    size = c["mask"]["size"]
    heads = [attend(q[:, x], k[:, x // (H // G)], v[:, x // (H // G)], c["scale"], lambda i, j: sees_chunk(i, j, size),
                    P[pre + "sink"][x]) for x in range(H)]
    return lin(torch.cat(heads, -1), P[pre + "o"], P[pre + "o.b"])


def latent_rows(h, P, pre, c, eps):
    """What a token keeps: the normed latent and the rotated key part that all heads share."""
    y = lin(h, P[pre + "dkv"])
    r = c["kv_rank"]
    lat = rms_norm(y[:, :r], P[pre + "dkv.norm"], eps)
    return lat, rotate_halves(y[:, None, r:], rotation_frequencies(c["rot"]))[:, 0]


def latent_attention(h, P, pre, c, rows):
    """``rows``: the (latent, rotated key part) pair, this layer's own or an earlier layer's."""
    T, H, D, R = h.shape[0], c["heads"], c["dim"], c["rot_dim"]
    lat, shared = rows
    q = lin(h, P[pre + "q"]).view(T, H, D + R)
    qr = rotate_halves(q[..., D:], rotation_frequencies(c["rot"]))
    k, v = lin(lat, P[pre + "uk"]).view(T, H, D), lin(lat, P[pre + "uv"]).view(T, H, c["vdim"])
    heads = [attend(torch.cat([q[:, x, :D], qr[:, x]], -1), torch.cat([k[:, x], shared], -1), v[:, x], c["scale"],
                    sees_causal) for x in range(H)]
    return lin(torch.cat(heads, -1), P[pre + "o"])


# ------------------------------------------------------------------------ experts
def route(h, router, bias, top):
    """ids [T, top] and weights: the largest logits, softmax over those alone."""
    z = lin(h, router, bias)
    ids = torch.sort(z, dim=-1, descending=True, stable=True).indices[:, :top]
    picked = z.gather(1, ids)
    w = torch.exp(picked - picked.max(-1, keepdim=True).values)
    return ids, w / w.sum(-1, keepdim=True)


def expert(h, P, pre):
    return lin(silu(lin(h, P[pre + "gate"])) * lin(h, P[pre + "up"]), P[pre + "down"])


def moe(h, P, pre, c):
    ids, w = route(h, P[pre + "router"], P[pre + "router.b"], c["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, x in zip(ids[t].tolist(), w[t]):
            out[t] += x * expert(h[t : t + 1], P, pre + "e%d." % e)[0]
    return out


# ------------------------------------------------------------------------- model
def forward(cfg, P, tokens, residuals=None):
    """tokens: list of ids of one sequence -> float64 logits [T, vocab]; ``residuals`` receives the stream after
    every layer."""
    eps = cfg["norm"]["eps"]
    x = P["embed"].to(F64)[torch.tensor(tokens)] * cfg["embedding"]["scale"]
    rows = {}
    for i, spec in enumerate(cfg["layers"]):
        pre, c = "l%d." % i, spec["mixer"]
        h = rms_norm(x, P[pre + "norm1"], eps)
        if spec["type"] == "delta":
            y = delta_mixer(h, P, pre + "mix.", c, eps)
        elif spec["type"] == "attention":
            y = chunked_attention(h, P, pre + "mix.", c, eps)
        else:
            src = c.get("kv_from")
            rows[i] = rows[src] if src is not None else latent_rows(h, P, pre + "mix.", c, eps)
            y = latent_attention(h, P, pre + "mix.", c, rows[i])
        x = x + y
        if spec.get("mlp") is not None:
            x = x + moe(rms_norm(x, P[pre + "norm2"], eps), P, pre + "mlp.", spec["mlp"])
        if residuals is not None:
            residuals.append(x.clone())
    return lin(rms_norm(x, P["final.norm"], eps), P["head"])


# ------------------------------------------------------------------ random models
def random_checkpoint(cfg, seed=0, dtype=torch.bfloat16):
    """Random tensors of a config's shapes, rounded to ``dtype`` (what a checkpoint would hold)."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    P = {}

    def mat(name, o, i, gain=1.0):
        P[name] = (torch.randn(o, i, generator=g) * gain / math.sqrt(i)).to(dtype)

    def vec(name, size, mean=0.0, std=0.1):
        P[name] = (mean + std * torch.randn(size, generator=g)).to(dtype)

    mat("embed", cfg["vocab"], W)
    mat("head", cfg["vocab"], W)
    vec("final.norm", W, 1.0)
    for i, spec in enumerate(cfg["layers"]):
        p, c = "l%d.mix." % i, spec["mixer"]
        H, D, Dv = c["heads"], c["dim"], c["vdim"]
        vec("l%d.norm1" % i, W, 1.0)
        mat(p + "o", W, H * Dv)
        if spec["type"] == "delta":
            G = c["kv_heads"]
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                mat(p + n, rows, W, 1.5)
                vec(p + n + ".conv", rows * c["conv"], 0.0, 0.6)
                P[p + n + ".conv"] = P[p + n + ".conv"].view(rows, c["conv"])
            mat(p + "g", H * Dv, W)
            mat(p + "b", H, W)
            mat(p + "a", H, W)
            vec(p + "A_log", H, 0.0, 0.7)
            vec(p + "dt_bias", H, -2.0, 1.0)
            vec(p + "norm", Dv, 1.0)
        elif spec["type"] == "attention":
            G = c["kv_heads"]
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                mat(p + n, rows, W, 1.5)
                vec(p + n + ".b", rows, 0.0, 0.3)
            vec(p + "o.b", W, 0.0, 0.3)
            vec(p + "sink", H, 0.5, 1.0)
        else:
            mat(p + "q", H * (D + c["rot_dim"]), W, 1.5)
            if c.get("kv_from") is None:
                mat(p + "dkv", c["kv_rank"] + c["rot_dim"], W, 1.5)
                vec(p + "dkv.norm", c["kv_rank"], 1.0)
            mat(p + "uk", H * D, c["kv_rank"], 1.5)
            mat(p + "uv", H * Dv, c["kv_rank"])
        f = spec.get("mlp")
        if f is None:
            continue
        b = "l%d.mlp." % i
        vec("l%d.norm2" % i, W, 1.0)
        mat(b + "router", f["router"]["experts"], W, 2.0)
        vec(b + "router.b", f["router"]["experts"], 0.0, 0.5)
        for e in range(f["router"]["experts"]):
            mat(b + "e%d.gate" % e, f["expert"]["ff"], W)
            mat(b + "e%d.up" % e, f["expert"]["ff"], W)
            mat(b + "e%d.down" % e, W, f["expert"]["ff"])
    return P
