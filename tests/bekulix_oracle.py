"""A plain, slow float64 implementation of the Bekulix design, one function per
mechanism, written from the design's equations. It shares no code with
``colossalai_amd``: the tests compare the framework against it.

Notation: ``h`` is a sublayer's input ``[T, W]`` (one sequence, T tokens from
position 0), weights are ``[out, in]`` and applied as ``h @ W.T``; ``P`` is a
dict of the checkpoint's tensors by name.
"""

import math

import torch

F64 = torch.float64


def lin(h, w, b=None):
    y = h @ w.to(F64).T
    return y if b is None else y + b.to(F64)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def one_plus_norm(x, w, eps):
    return unit_rms(x, eps) * (1.0 + w.to(F64))


# --------------------------------------------------------------------- visibility
def sees_causal(i, j):
    return j <= i


def sees_window(i, j, size):
    """The query itself and the size - 1 positions before it."""
    return 0 <= i - j < size


def sees_chunk(i, j, size):
    """Positions up to the query inside the query's own block of ``size`` positions."""
    return j <= i and i // size == j // size


def attend(q, k, v, scale, sees):
    """One head: q [T, D], k [S, D], v [S, Dv]; ``sees(i, j)`` says whether query i reads key j. Query by query."""
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F64)
    for i in range(q.shape[0]):
        vis = [j for j in range(k.shape[0]) if sees(i, j)]
        s = (k[vis] @ q[i]) * scale
        w = torch.exp(s - s.max())
        out[i] = (w / w.sum()) @ v[vis]
    return out


# ------------------------------------------------------------------------- mixers
def query_temperature(p, coef, every):
    return 1.0 + coef * math.log(math.floor((p + 1) / every) + 1)


def shared_key_value_attention(h, P, pre, c, eps):
    """Grouped queries; the values are the key projections before their norm; queries grow with position."""
    T, H, G, D = h.shape[0], c["heads"], c["kv_heads"], c["dim"]
    q = unit_rms(lin(h, P[pre + "q"]).view(T, H, D), eps) * P[pre + "q.norm"].to(F64)
    raw = lin(h, P[pre + "k"]).view(T, G, D)
    k = unit_rms(raw, eps) * P[pre + "k.norm"].to(F64)
    t = c.get("q_temp")
    if t:
        q = q * torch.tensor([query_temperature(p, t["coef"], t["every"]) for p in range(T)], dtype=F64).view(T, 1, 1)
    heads = [attend(q[:, x], k[:, x // (H // G)], raw[:, x // (H // G)], c["scale"], sees_causal) for x in range(H)]
    return lin(torch.cat(heads, -1), P[pre + "o"])


def windowed_latent_attention(h, P, pre, c, eps):
    """Keys and values of every head are up-projections of one normed latent per token; sliding window."""
    T, H, D, Dv = h.shape[0], c["heads"], c["dim"], c["vdim"]
    q = lin(h, P[pre + "q"]).view(T, H, D)
    lat = unit_rms(lin(h, P[pre + "dkv"]), eps) * P[pre + "dkv.norm"].to(F64)
    k, v = lin(lat, P[pre + "uk"]).view(T, H, D), lin(lat, P[pre + "uv"]).view(T, H, Dv)
    size = c["mask"]["size"]
    heads = [attend(q[:, x], k[:, x], v[:, x], c["scale"], lambda i, j: sees_window(i, j, size)) for x in range(H)]
    return lin(torch.cat(heads, -1), P[pre + "o"])


def difference_weight(lq1, lk1, lq2, lk2, diff):
    lq1, lk1, lq2, lk2 = (t.to(F64) for t in (lq1, lk1, lq2, lk2))
    return float(torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum())) + diff


def combine_maps(a1, a2, lam, diff, eps):
    """Two maps' outputs of a head [T, Dv] -> normed difference, scaled."""
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def chunked_differential_attention(h, P, pre, c, eps):
    """Two softmax maps per head over the same values, inside fixed blocks of positions."""
    T, H, G, D, Dv = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = lin(h, P[pre + "q"], P[pre + "q.b"]).view(T, H, 2, D)
    k = lin(h, P[pre + "k"], P[pre + "k.b"]).view(T, G, 2, D)
    v = lin(h, P[pre + "v"], P[pre + "v.b"]).view(T, G, Dv)
    lam = difference_weight(P[pre + "lq1"], P[pre + "lk1"], P[pre + "lq2"], P[pre + "lk2"], c["diff"])
    size = c["mask"]["size"]
    heads = []
    for x in range(H):
        g = x // (H // G)
        a = [attend(q[:, x, m], k[:, g, m], v[:, g], c["scale"], lambda i, j: sees_chunk(i, j, size)) for m in (0, 1)]
        heads.append(combine_maps(a[0], a[1], lam, c["diff"], eps))
    return lin(torch.cat(heads, -1), P[pre + "o"])


MIX = {"attention": shared_key_value_attention, "latent_attention": windowed_latent_attention,
       "attention_2": chunked_differential_attention}


def relu_feed_forward(h, P, pre):
    return lin(torch.clamp(lin(h, P[pre + "gate"]), min=0.0) * lin(h, P[pre + "up"]), P[pre + "down"])


# ------------------------------------------------------------------------ streams
def read_streams(X, w_in):
    """X [s, T, W] -> the sublayer's input before its norm."""
    return sum(w_in.to(F64)[s] * X[s] for s in range(X.shape[0]))


def write_streams(X, mix, w_out, y):
    """Every new stream from the old ones (mix indexed [from, to]) plus its share of the sublayer's output."""
    n = X.shape[0]
    return torch.stack([sum(mix.to(F64)[s, t] * X[s] for s in range(n)) + w_out.to(F64)[t] * y for t in range(n)])


def layer_order(cfg):
    n, lp = len(cfg["layers"]), cfg.get("loop")
    order = []
    if not lp:
        return list(range(n))
    order += range(0, lp["start"])
    for _ in range(lp["times"]):
        order += range(lp["start"], lp["stop"])
    order += range(lp["stop"], n)
    return order


def forward(cfg, P, tokens, residuals=None):
    """tokens: list of ids of one sequence -> float64 logits [T, vocab]. ``residuals`` receives the sum of the
    streams after every layer run."""
    eps = cfg["norm"]["eps"]
    e = P["embed"].to(F64)[torch.tensor(tokens)]
    X = torch.stack([e] * cfg["streams"])
    for i in layer_order(cfg):
        spec, pre = cfg["layers"][i], "l%d." % i
        u = read_streams(X, P[pre + "hc1.in"])
        y = MIX[spec["type"]](one_plus_norm(u, P[pre + "norm1"], eps), P, pre + "mix.", spec["mixer"], eps)
        X = write_streams(X, P[pre + "hc1.mix"], P[pre + "hc1.out"], y)
        if spec.get("mlp") is not None:
            u = read_streams(X, P[pre + "hc2.in"])
            y = relu_feed_forward(one_plus_norm(u, P[pre + "norm2"], eps), P, pre + "mlp.")
            X = write_streams(X, P[pre + "hc2.mix"], P[pre + "hc2.out"], y)
        if residuals is not None:
            residuals.append(X.sum(0))
    return lin(one_plus_norm(X.sum(0), P["final.norm"], eps), P["head"])


# ------------------------------------------------------------------ random models
def random_checkpoint(cfg, seed=0, dtype=torch.bfloat16):
    """Random tensors of a config's shapes, rounded to ``dtype`` (what a checkpoint would hold)."""
    g = torch.Generator().manual_seed(seed)
    W, n = cfg["width"], cfg["streams"]
    P = {}

    def mat(name, o, i, gain=1.0):
        P[name] = (torch.randn(o, i, generator=g) * gain / math.sqrt(i)).to(dtype)

    def vec(name, size, mean=0.0, std=0.1):
        P[name] = (mean + std * torch.randn(size, generator=g)).to(dtype)

    def streams(name):
        vec(name + ".in", n, 1.0 / n, 0.3 / n)
        vec(name + ".out", n, 0.8, 0.3)
        P[name + ".mix"] = (0.8 * torch.eye(n) + 0.2 / n * torch.randn(n, n, generator=g)).to(dtype)

    mat("embed", cfg["vocab"], W, math.sqrt(W))
    mat("head", cfg["vocab"], W)
    vec("final.norm", W)
    for i, spec in enumerate(cfg["layers"]):
        p, c = "l%d." % i, spec["mixer"]
        H, D = c["heads"], c["dim"]
        vec(p + "norm1", W)
        streams(p + "hc1")
        if spec["type"] == "attention":
            mat(p + "mix.q", H * D, W)
            mat(p + "mix.k", c["kv_heads"] * D, W, 1.5)
            vec(p + "mix.q.norm", D, 1.3)
            vec(p + "mix.k.norm", D, 0.9)
            mat(p + "mix.o", W, H * D)
        elif spec["type"] == "latent_attention":
            mat(p + "mix.q", H * D, W, 2.0)
            mat(p + "mix.dkv", c["kv_rank"], W, 2.0)
            vec(p + "mix.dkv.norm", c["kv_rank"], 1.0)
            mat(p + "mix.uk", H * D, c["kv_rank"], 2.0)
            mat(p + "mix.uv", H * c["vdim"], c["kv_rank"])
            mat(p + "mix.o", W, H * c["vdim"])
        else:
            G, Dv = c["kv_heads"], c["vdim"]
            for name, rows in (("q", 2 * H * D), ("k", 2 * G * D), ("v", G * Dv)):
                mat(p + "mix." + name, rows, W, 1.5)
                vec(p + "mix." + name + ".b", rows, 0.0, 0.3)
            for name in ("lq1", "lk1", "lq2", "lk2"):
                vec(p + "mix." + name, D, 0.0, 0.3)
            mat(p + "mix.o", W, H * Dv)
        f = spec.get("mlp")
        if f is None:
            continue
        vec(p + "norm2", W)
        streams(p + "hc2")
        mat(p + "mlp.gate", f["ff"], W)
        mat(p + "mlp.up", f["ff"], W)
        mat(p + "mlp.down", W, f["ff"])
    return P
