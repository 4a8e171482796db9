"""Vosulorn: a decoder-only language model of latent attention with shared latents,
chunked rotary attention with a learned sink, and a gated delta rule, every layer
with softmax-routed gated experts; served from paged keys and latents plus
fixed-size state.

Every layer is pre-norm, ``x <- x + mixer(norm1(x))``, ``x <- x + ff(norm2(x))``
(RMS norms with a weight, float32 residual). The embedding is scaled by a
constant on the way in. A checkpoint's ``layers`` list picks per layer

* mixer ``latent_attention`` — keys and values are up-projections of one RMS-normed
  latent per token plus one rotated key part that all heads share; causal softmax.
  Only the latent and the rotated part are paged (``ops/latent_attention.py``). A
  layer with ``kv_from: j`` has no such projection of its own: it attends over layer
  ``j``'s cached rows with its own queries and up-projections. The checkpoint pairs
  rotated channels ``(i, i + dims / 2)``; queries and shared key parts are brought to
  neighbouring pairs when they are loaded (``ops/pair_rotary.halves_to_pairs``), which
  leaves every score as it is.
* mixer ``attention`` — grouped queries, biased projections, rotary positions on
  neighbouring pairs with wavelength-dependent frequency scaling, a query sees the
  keys of its own fixed block of positions, and the softmax denominator holds one
  more learned term per head.
* mixer ``delta`` — short causal convolutions with SiLU on q/k/v, unit-length q/k, a
  delta rule with one decay per head and token (``ops/linear_recurrence.py``), a
  per-head RMS norm and a SiLU gate on its output.
* feed-forward ``moe`` — experts ``down(silu(gate h) * up h)``; the router has a bias,
  chooses by its float32 logits and weights by the softmax over the chosen ones — or
  none.

The module holds the packed layout the kernels want (all input projections of a
mixer are one matrix, gate/up of an expert are stacked, the experts are stacked
``[E, out, in]``). Serving goes through ``forward_ragged`` (a ragged step over the
engine's pages and state slots); ``forward`` runs whole sequences through the same
path with throw-away caches.
"""

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..ops.group_norm import add_rms_norm, head_rms_norm_gate
from ..ops.latent_attention import latent_attention, latent_kv_write
from ..ops.linear_recurrence import conv_gated_delta_rule
from ..ops.paged_attention import paged_attention
from ..ops.pair_rotary import halves_to_pairs, pair_frequencies, rotate_qk_write
from ..ops.ragged import RaggedBatch
from ..ops.routed_experts import grouped_topk_route, routed_expert_ffn
from ..ops.streams import streams_start
from .packed import PackedLinear
from .registry import register_model

__all__ = ["VosulornConfig", "VosulornForCausalLM"]

UNIT_EPS = 1e-6  # inside the root of the delta rule's q/k unit-length scaling


@dataclass
class VosulornConfig:
    vocab: int
    width: int
    layers: List[dict]
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0

    @classmethod
    def from_dict(cls, d: dict) -> "VosulornConfig":
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=list(d["layers"]),
                   norm_eps=float(d["norm"]["eps"]),
                   embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)))

    def to_dict(self) -> dict:
        return {"architecture": "Vosulorn", "embedding": {"scale": self.embedding_scale}, "layers": self.layers,
                "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}


def _vec(n, value=1.0):
    return nn.Parameter(torch.full((n,), value, dtype=torch.float32))


def _grouped_heads(c: dict):
    H, G = int(c["heads"]), int(c["kv_heads"])
    if H % G:
        raise ValueError(f"{H} query heads do not split over {G} key/value heads")
    return H, G


def _rotation(c: dict, size: int):
    """(dims, frequencies) of a mixer's ``rot``, which turns the first ``dims`` of ``size`` channels."""
    rot = c.get("rot") or {}
    dims = int(rot.get("dims", 0))
    if dims % 2 or dims > size:
        raise ValueError(f"cannot rotate {dims} of {size} channels in pairs")
    return dims, pair_frequencies(float(rot.get("base", 10000.0)), dims, scaling=rot.get("scaling"))


class VosulornLatentAttention(nn.Module):
    def __init__(self, width: int, c: dict, eps: float):
        super().__init__()
        self.eps, self.scale = eps, float(c["scale"])
        self.H, self.D, self.R, self.Dv = int(c["heads"]), int(c["dim"]), int(c["rot_dim"]), int(c["vdim"])
        self.rank = int(c["kv_rank"])
        self.kv_from = None if c.get("kv_from") is None else int(c["kv_from"])
        parts = {"q": self.H * (self.D + self.R)}
        if self.kv_from is None:
            parts["dkv"] = self.rank + self.R
            self.dkv_norm = _vec(self.rank)
        self.in_proj = PackedLinear(width, parts)
        self.uk = nn.Parameter(torch.randn(self.H, self.D, self.rank) * self.rank ** -0.5)
        self.uv = nn.Parameter(torch.randn(self.H, self.Dv, self.rank) * self.rank ** -0.5)
        self.o = nn.Linear(self.H * self.Dv, width, bias=False)
        self.rot_dims, freqs = _rotation(c, self.R)
        self.register_buffer("freqs", freqs if self.R else None, persistent=False)
        self.register_buffer("uv_t", None, persistent=False)  # uv with its last two axes swapped, for decode steps

    def kv_shape(self):
        """One key head holding the latent and the shared rotated part; the values are a view of it. None for a layer
        that reads another's."""
        return (1, self.rank + self.R, 0) if self.kv_from is None else None

    def state_buffers(self):
        return None

    def prepare(self):
        self.uv_t = self.uv.detach().transpose(1, 2).contiguous()

    def pair_rows(self, name: str, rows: torch.Tensor) -> torch.Tensor:
        """A checkpoint's projection rows with the rotated channels as neighbouring pairs."""
        if name == "q":
            return halves_to_pairs(rows, self.H, self.D + self.R, self.D, self.rot_dims)
        return halves_to_pairs(rows, 1, self.rank + self.R, self.rank, self.rot_dims)

    def forward(self, h, batch: RaggedBatch, kv, layer: int, state):
        N = h.shape[0]
        p, _ = self.in_proj(h)
        pool = kv.k_pools[layer]
        if self.kv_from is None:
            latent_kv_write(p["dkv"], self.dkv_norm, self.eps, self.freqs, pool, batch)
        o = latent_attention(p["q"].view(N, self.H, self.D + self.R), self.uk, self.uv, pool, batch, self.scale, self.freqs,
                             self.rank, w_uv_t=self.uv_t)
        return self.o(o)


class VosulornAttention(nn.Module):
    """Rotary grouped-query attention inside fixed blocks of positions, with a learned sink."""

    kv_from = None

    def __init__(self, width: int, c: dict, eps: float):
        super().__init__()
        self.scale = float(c["scale"])
        self.H, self.G = _grouped_heads(c)
        self.D, self.Dv = int(c["dim"]), int(c["vdim"])
        self.chunk = int((c.get("mask") or {}).get("size") or 0)  # 0: causal only
        self.in_proj = PackedLinear(width, {"q": self.H * self.D, "k": self.G * self.D, "v": self.G * self.Dv}, bias=True)
        self.o = nn.Linear(self.H * self.Dv, width, bias=True)
        self.sink = _vec(self.H, 0.0)
        _, freqs = _rotation(c, self.D)
        self.register_buffer("freqs", freqs, persistent=False)

    def kv_shape(self):
        return (self.G, self.D, self.Dv)

    def state_buffers(self):
        return None

    def forward(self, h, batch: RaggedBatch, kv, layer: int, state):
        N = h.shape[0]
        p, _ = self.in_proj(h)
        kpool, vpool = kv.k_pools[layer], kv.v_pools[layer]
        q = p["q"].view(N, self.H, self.D)
        rotate_qk_write(q, p["k"].view(N, self.G, self.D), p["v"].view(N, self.G, self.Dv), self.freqs, kpool, vpool, batch)
        o = paged_attention(q, kpool, vpool, batch, self.scale, chunk=self.chunk, sink_logits=self.sink)
        return self.o(o.view(N, self.H * self.Dv))


class VosulornDelta(nn.Module):
    """Gated delta rule with one decay per head."""

    kv_from = None

    def __init__(self, width: int, c: dict, eps: float):
        super().__init__()
        self.eps = eps
        self.H, self.G = _grouped_heads(c)
        self.D, self.Dv, self.K = int(c["dim"]), int(c["vdim"]), int(c["conv"])
        self.Cq, self.Cv = self.G * self.D, self.H * self.Dv
        self.C = 2 * self.Cq + self.Cv
        self.in_proj = PackedLinear(width, {"q": self.Cq, "k": self.Cq, "v": self.Cv, "g": self.Cv, "b": self.H, "a": self.H})
        self.conv = nn.Parameter(torch.randn(self.C, self.K, dtype=torch.float32) * 0.5)
        self.A_log, self.dt_bias = _vec(self.H, 0.0), _vec(self.H, 0.0)
        self.norm = _vec(self.Dv)
        self.o = nn.Linear(self.Cv, width, bias=False)

    def kv_shape(self):
        return None

    def state_buffers(self):
        buf = {"S": (self.H, self.D, self.Dv)}
        if self.K > 1:
            buf["tail"] = (self.K - 1, self.C)
        return buf

    def forward(self, h, batch: RaggedBatch, kv, layer: int, state):
        p, y = self.in_proj(h)
        o = conv_gated_delta_rule(y[:, : self.C], self.conv, state.get("tail"), self.G, self.D, p["b"], p["a"], self.A_log,
                                  self.dt_bias, state["S"], batch, UNIT_EPS, self.D ** -0.5)
        o = head_rms_norm_gate(o, self.norm, self.eps, p["g"], h.dtype, act="silu")
        return self.o(o.view(-1, self.Cv))


class VosulornMoE(nn.Module):
    def __init__(self, width: int, c: dict):
        super().__init__()
        r = c["router"]
        self.E, self.top = int(r["experts"]), int(r["top"])
        if not 0 < self.top <= self.E:
            raise ValueError(f"cannot choose {self.top} of {self.E} experts")
        ff = int(c["expert"]["ff"])
        self.router = nn.Parameter(torch.randn(self.E, width, dtype=torch.float32) * width ** -0.5)  # float32 always
        self.router_b = _vec(self.E, 0.0)
        self.w_up = nn.Parameter(torch.randn(self.E, 2 * ff, width) * width ** -0.5)     # [gate; up] per expert
        self.w_down = nn.Parameter(torch.randn(self.E, width, ff) * ff ** -0.5)

    def forward(self, h):
        logits = F.linear(h.float(), self.router, self.router_b)
        ids, weights = grouped_topk_route(logits, None, self.top, score="logits")
        return routed_expert_ffn(h, self.w_up, self.w_down, ids, weights, None, "silu_gated")


MIXERS = {"latent_attention": VosulornLatentAttention, "attention": VosulornAttention, "delta": VosulornDelta}
MLPS = {"moe": VosulornMoE}


class VosulornLayer(nn.Module):
    def __init__(self, cfg: VosulornConfig, spec: dict):
        super().__init__()
        if spec["type"] not in MIXERS:
            raise ValueError(f"unknown mixer type {spec['type']!r}")
        self.kind = spec["type"]
        self.norm1 = _vec(cfg.width)
        self.mix = MIXERS[spec["type"]](cfg.width, spec["mixer"], cfg.norm_eps)
        m = spec.get("mlp")
        if m is not None and m.get("kind", "moe") not in MLPS:
            raise ValueError(f"unknown feed-forward kind {m.get('kind')!r}")
        self.mlp = MLPS[m.get("kind", "moe")](cfg.width, m) if m is not None else None
        self.norm2 = _vec(cfg.width) if m is not None else None


@register_model("Vosulorn")
class VosulornForCausalLM(nn.Module):
    config_class = VosulornConfig
    serves_ragged = True  # the serving engines drive forward_ragged

    def __init__(self, cfg: VosulornConfig):
        super().__init__()
        if not cfg.layers:
            raise ValueError("a model needs at least one layer")
        self.config = cfg
        self.embed = nn.Embedding(cfg.vocab, cfg.width)
        self.layers = nn.ModuleList([VosulornLayer(cfg, s) for s in cfg.layers])
        self.final_norm = _vec(cfg.width)
        self.head = nn.Linear(cfg.width, cfg.vocab, bias=False)
        self.register_buffer("one", torch.ones(1), persistent=False)  # the residual as a single stream, read as it is
        for i, layer in enumerate(self.layers):
            a, j = layer.mix, layer.mix.kv_from
            if j is None:
                continue
            if not 0 <= j < i or self.layers[j].kind != "latent_attention" or self.layers[j].mix.kv_from is not None:
                raise ValueError(f"layer {i} reads latents of layer {j}, which must come earlier and have its own")
            b = self.layers[j].mix
            same_turn = a.R == 0 or torch.equal(a.freqs.cpu(), b.freqs.cpu())
            if (a.rank, a.R, a.rot_dims) != (b.rank, b.R, b.rot_dims) or not same_turn:
                raise ValueError(f"layer {i} and the layer {j} whose latents it reads differ in their sizes or rotation")

    # ------------------------------------------------------------ cache plan
    def kv_layer_shapes(self):
        """Per layer ``(kv_heads, key_dim, value_dim)``, None for a layer without keys of its own."""
        return [l.mix.kv_shape() for l in self.layers]

    def kv_layer_sources(self):
        """Per layer the layer whose pools it reads, None for its own."""
        return [l.mix.kv_from for l in self.layers]

    def state_layer_buffers(self):
        """Per layer ``{name: shape}`` of float32 state kept per sequence, or None."""
        return [l.mix.state_buffers() for l in self.layers]

    @property
    def act_dtype(self):
        return self.head.weight.dtype

    # ---------------------------------------------------------------- serve
    def forward_ragged(self, tokens: torch.Tensor, batch: RaggedBatch, kv, state,
                       want: Optional[torch.Tensor] = None, residuals: Optional[list] = None) -> torch.Tensor:
        """tokens [N] (flat, sequence after sequence as ``batch`` says); ``kv`` a KVCacheManager and ``state`` a
        StateCacheManager laid out by ``kv_layer_shapes`` / ``kv_layer_sources`` / ``state_layer_buffers``. Returns
        float32 logits of the rows ``want`` (indices into the flat token axis; all rows if None). ``residuals``, when a
        list, receives a copy of the float32 residual stream after every layer."""
        cfg, act, n = self.config, self.act_dtype, len(self.layers)
        eps = cfg.norm_eps
        x, h = streams_start(self.embed.weight, tokens, 1, self.one, self.layers[0].norm1, eps, cfg.embedding_scale)
        x = x.view(-1, cfg.width)
        for i, layer in enumerate(self.layers):
            y = layer.mix(h, batch, kv, i, state.layers[i])
            if layer.mlp is not None:
                h = add_rms_norm(x, y, None, layer.norm2, eps, act)
                y = layer.mlp(h)
            last = i + 1 == n
            if last and want is not None and residuals is None:  # the last sum is per row: the wanted rows only
                x, y = x.index_select(0, want), y.index_select(0, want)
            h = add_rms_norm(x, y, None, self.final_norm if last else self.layers[i + 1].norm1, eps, act)
            if residuals is not None:
                residuals.append(x.clone())
        if want is not None and residuals is not None:
            h = h.index_select(0, want)
        return self.head(h).float()

    def forward(self, input_ids: torch.Tensor) -> torch.Tensor:
        """input_ids [B, S] -> logits [B, S, vocab] (float32), every sequence from position 0 with caches that
        live for this call only."""
        from ..inference.kv_cache import KVCacheManager
        from ..inference.state_cache import StateCacheManager

        B, S = input_ids.shape
        dev = input_ids.device
        page = 16
        pages = (S + page - 1) // page
        kv = KVCacheManager(len(self.layers), 0, 0, num_blocks=B * pages, block_size=page, device=dev,
                            dtype=self.act_dtype, layer_shapes=self.kv_layer_shapes(),
                            layer_sources=self.kv_layer_sources())
        state = StateCacheManager(self.state_layer_buffers(), B, device=dev)
        tables = [list(range(b * pages, (b + 1) * pages)) for b in range(B)]
        batch = RaggedBatch.build([S] * B, [0] * B, list(range(B)), dev, tables, page)
        with torch.no_grad():
            return self.forward_ragged(input_ids.reshape(-1), batch, kv, state).view(B, S, -1)

    # -------------------------------------------------------------- weights
    def prepare(self) -> None:
        """Refresh what is derived from the weights (after loading or changing them)."""
        for layer in self.layers:
            if hasattr(layer.mix, "prepare"):
                layer.mix.prepare()

    def load_checkpoint_tensors(self, tensors: Dict[str, torch.Tensor]) -> None:
        """Pack a checkpoint's tensors (``embed``, ``head``, ``final.norm``, ``l<i>.norm{1,2}``, ``l<i>.mix.*``,
        ``l<i>.mlp.*``) into this module's parameters. Every tensor must be used and every parameter filled."""
        used = set()

        def get(name):
            used.add(name)
            return tensors[name]

        def put(param, value):
            assert tuple(param.shape) == tuple(value.shape), (tuple(param.shape), tuple(value.shape))
            param.data.copy_(value.to(param.dtype))

        put(self.embed.weight, get("embed"))
        put(self.head.weight, get("head"))
        put(self.final_norm, get("final.norm"))
        for i, layer in enumerate(self.layers):
            p, m = f"l{i}.", layer.mix
            a = p + "mix."
            put(layer.norm1, get(p + "norm1"))
            put(m.o.weight, get(a + "o"))
            if layer.kind == "latent_attention":
                put(m.in_proj.weight, torch.cat([m.pair_rows(n, get(a + n)) for n in m.in_proj.parts], 0))
                if m.kv_from is None:
                    put(m.dkv_norm, get(a + "dkv.norm"))
                put(m.uk, get(a + "uk").view(m.H, m.D, m.rank))
                put(m.uv, get(a + "uv").view(m.H, m.Dv, m.rank))
            elif layer.kind == "attention":
                put(m.in_proj.weight, torch.cat([get(a + n) for n in m.in_proj.parts], 0))
                put(m.in_proj.bias, torch.cat([get(a + n + ".b") for n in m.in_proj.parts], 0))
                put(m.o.bias, get(a + "o.b"))
                put(m.sink, get(a + "sink"))
            else:
                put(m.in_proj.weight, torch.cat([get(a + n) for n in m.in_proj.parts], 0))
                put(m.conv, torch.cat([get(a + n + ".conv") for n in ("q", "k", "v")], 0))
                put(m.A_log, get(a + "A_log"))
                put(m.dt_bias, get(a + "dt_bias"))
                put(m.norm, get(a + "norm"))
            f, b = layer.mlp, p + "mlp."
            if f is None:
                used.update(n for n in (p + "norm2",) if n in tensors)  # carried, but unused without a feed-forward
                continue
            put(layer.norm2, get(p + "norm2"))
            put(f.router, get(b + "router"))
            put(f.router_b, get(b + "router.b"))
            put(f.w_up, torch.stack([torch.cat([get(b + f"e{e}.gate"), get(b + f"e{e}.up")], 0) for e in range(f.E)], 0))
            put(f.w_down, torch.stack([get(b + f"e{e}.down") for e in range(f.E)], 0))
        missing = set(tensors) - used
        if missing:
            raise ValueError(f"checkpoint tensors without a place in the model: {sorted(missing)[:8]}")
        self.prepare()

    def serving_dtype(self, dtype) -> "VosulornForCausalLM":
        """Give matrices and projection biases ``dtype``; norm weights, the convolution, decays, sinks and the router
        stay float32."""
        keep32 = {id(l.mlp.router) for l in self.layers if l.mlp is not None}
        keep32 |= {id(l.mix.conv) for l in self.layers if l.kind == "delta"}
        for p in self.parameters():
            if p.dim() >= 2 and id(p) not in keep32:
                p.data = p.data.to(dtype)
        for layer in self.layers:
            if layer.kind == "attention":
                layer.mix.in_proj.bias.data = layer.mix.in_proj.bias.data.to(dtype)
                layer.mix.o.bias.data = layer.mix.o.bias.data.to(dtype)
        self.prepare()
        return self

    @classmethod
    def from_checkpoint(cls, config: dict, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16, device="cpu"):
        """Build from a parsed config.json and a name -> tensor mapping."""
        model = cls(VosulornConfig.from_dict(config)).serving_dtype(dtype)
        model.load_checkpoint_tensors(tensors)
        return model.to(device).eval()
