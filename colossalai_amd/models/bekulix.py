"""Bekulix: a decoder-only language model with parallel residual streams, three kinds
of attention without rotary positions and a looped block, served from paged keys
and latents.

A token carries ``streams`` float32 residual rows (hyper-connections,
``ops/streams.py``), all equal to its embedding at the start; a sublayer reads a
weighted sum of them, RMS-normed with a weight stored around zero, and writes back
through a ``[from, to]`` mixing matrix and one output weight per stream. The logits are
``head(norm(sum of the streams))``. A checkpoint's ``layers`` list picks per layer

* mixer ``attention`` — grouped queries, RMS norm per head on queries and keys (plain
  weights), the values are the key projections *before* that norm, queries grow with
  position by ``1 + coef * ln(floor((p + 1) / every) + 1)``; causal. One cached row per
  token and key head serves as key and value (``ops/normed_keys.py``).
* mixer ``latent_attention`` — keys and values are up-projections of one RMS-normed
  latent per token, no rotated part; sliding window. Only the latent is paged
  (``ops/latent_attention.py``).
* mixer ``attention_2`` — differential attention (``ops/differential.py``): two softmax
  maps per head over the same values, biased projections; a query sees the keys of its
  own fixed block of positions.
* feed-forward ``dense`` — ``down(relu(gate h) * up h)`` — or none.

``loop = {start, stop, times}`` runs layers ``start .. stop - 1`` ``times`` times in a row
with the same weights; each pass keeps its own pages (the cache plan below is per
layer *run*).

Serving goes through ``forward_ragged`` (a ragged step over the engine's pages);
``forward`` runs whole sequences through the same path with throw-away caches.
"""

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from ..ops.activation import relu_mul
from ..ops.differential import difference_norm, difference_weight, map_major
from ..ops.latent_attention import latent_attention, latent_kv_write
from ..ops.normed_keys import query_norm_key_write
from ..ops.paged_attention import paged_attention, paged_kv_write
from ..ops.ragged import RaggedBatch
from ..ops.streams import streams_start, streams_update
from .looped import layer_runs, parse_loop
from .packed import PackedLinear
from .registry import register_model

__all__ = ["BekulixConfig", "BekulixForCausalLM"]


@dataclass
class BekulixConfig:
    vocab: int
    width: int
    layers: List[dict]
    norm_eps: float = 1e-6
    streams: int = 2
    loop: Optional[dict] = None  # {"start", "stop", "times"}

    @classmethod
    def from_dict(cls, d: dict) -> "BekulixConfig":
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=list(d["layers"]),
                   norm_eps=float(d["norm"]["eps"]), streams=int(d["streams"]), loop=parse_loop(d))

    def to_dict(self) -> dict:
        d = {"architecture": "Bekulix", "layers": self.layers, "norm": {"eps": self.norm_eps}, "streams": self.streams,
             "vocab": self.vocab, "width": self.width}
        if self.loop is not None:
            d["loop"] = dict(self.loop)
        return d

    def layer_runs(self):
        """The order in which layers run: ``(layer, pass number or None, first of its pass)``."""
        return layer_runs(len(self.layers), self.loop)


def _vec(n, value=1.0):
    return nn.Parameter(torch.full((n,), value, dtype=torch.float32))


def _mask_size(c: dict) -> int:
    return int((c.get("mask") or {}).get("size") or 0)  # 0: causal only


def _grouped_heads(c: dict):
    H, G = int(c["heads"]), int(c["kv_heads"])
    if H % G:
        raise ValueError(f"{H} query heads do not split over {G} key/value heads")
    return H, G


class BekulixAttention(nn.Module):
    """Normed queries and keys, values = keys before their norm, queries grow with position."""

    key_factors = True

    def __init__(self, width: int, c: dict, eps: float):
        super().__init__()
        self.eps, self.scale = eps, float(c["scale"])
        self.H, self.G = _grouped_heads(c)
        self.D = int(c["dim"])
        if int(c.get("vdim", self.D)) != self.D:
            raise ValueError("the values are the keys: their sizes must agree")
        t = c.get("q_temp")
        self.coef, self.every = (float(t["coef"]), float(t["every"])) if t else (0.0, 0.0)
        self.in_proj = PackedLinear(width, {"q": self.H * self.D, "k": self.G * self.D})
        self.qk_norm = _vec(self.D)  # the product of both norms' weights: only it enters a score
        self.o = nn.Linear(self.H * self.D, width, bias=False)

    def kv_shape(self):
        return (self.G, self.D, 0)

    def forward(self, h, batch: RaggedBatch, kv, run: int):
        N = h.shape[0]
        p, _ = self.in_proj(h)
        pool, factors = kv.k_pools[run], kv.k_factors[run]
        q = query_norm_key_write(p["q"].view(N, self.H, self.D), p["k"].view(N, self.G, self.D), self.qk_norm, self.eps,
                                 pool, factors, batch, self.coef, self.every)
        o = paged_attention(q, pool, pool, batch, self.scale, key_factors=factors)
        return self.o(o.view(N, self.H * self.D))


class BekulixLatentAttention(nn.Module):
    """Keys and values from one normed latent per token; sliding window; no positions in the scores."""

    key_factors = False

    def __init__(self, width: int, c: dict, eps: float):
        super().__init__()
        self.eps, self.scale, self.window = eps, float(c["scale"]), _mask_size(c)
        self.H, self.D, self.Dv, self.rank = int(c["heads"]), int(c["dim"]), int(c["vdim"]), int(c["kv_rank"])
        self.in_proj = PackedLinear(width, {"q": self.H * self.D, "dkv": self.rank})
        self.dkv_norm = _vec(self.rank)
        self.uk = nn.Parameter(torch.randn(self.H, self.D, self.rank) * self.rank ** -0.5)
        self.uv = nn.Parameter(torch.randn(self.H, self.Dv, self.rank) * self.rank ** -0.5)
        self.o = nn.Linear(self.H * self.Dv, width, bias=False)
        self.register_buffer("uv_t", None, persistent=False)  # uv with its last two axes swapped, for decode steps

    def kv_shape(self):
        """One key head holding the latent; the values are a view of it."""
        return (1, self.rank, 0)

    def prepare(self):
        self.uv_t = self.uv.detach().transpose(1, 2).contiguous()

    def forward(self, h, batch: RaggedBatch, kv, run: int):
        N = h.shape[0]
        p, _ = self.in_proj(h)
        pool = kv.k_pools[run]
        latent_kv_write(p["dkv"], self.dkv_norm, self.eps, None, pool, batch)
        o = latent_attention(p["q"].view(N, self.H, self.D), self.uk, self.uv, pool, batch, self.scale, None, self.rank,
                             window=self.window, w_uv_t=self.uv_t)
        return self.o(o)


class BekulixDifferentialAttention(nn.Module):
    """Two softmax maps per head over the same values, inside fixed blocks of positions."""

    key_factors = False

    def __init__(self, width: int, c: dict, eps: float):
        super().__init__()
        self.eps, self.scale, self.chunk = eps, float(c["scale"]), _mask_size(c)
        self.H, self.G = _grouped_heads(c)
        self.D, self.Dv, self.diff = int(c["dim"]), int(c["vdim"]), float(c["diff"])
        # query rows in the order (key/value head, map, query head of the group)
        self.in_proj = PackedLinear(width, {"q": 2 * self.H * self.D, "k": 2 * self.G * self.D, "v": self.G * self.Dv},
                                    bias=True)
        self.lq1, self.lk1, self.lq2, self.lk2 = (_vec(self.D, 0.0) for _ in range(4))
        self.o = nn.Linear(self.H * self.Dv, width, bias=False)
        self._lam = None

    def kv_shape(self):
        return (2 * self.G, self.D, self.Dv, self.G)

    def prepare(self):
        self._lam = difference_weight(*(t.detach().cpu() for t in (self.lq1, self.lk1, self.lq2, self.lk2)), self.diff)

    def forward(self, h, batch: RaggedBatch, kv, run: int):
        N = h.shape[0]
        if self._lam is None:
            self.prepare()
        p, _ = self.in_proj(h)
        kpool, vpool = kv.k_pools[run], kv.v_pools[run]
        paged_kv_write(p["k"].view(N, 2 * self.G, self.D), p["v"].view(N, self.G, self.Dv), kpool, vpool, batch)
        a = paged_attention(p["q"].view(N, 2 * self.H, self.D), kpool, vpool, batch, self.scale, chunk=self.chunk,
                            out_dtype=torch.float32)
        return self.o(difference_norm(a, self.G, self._lam, 1.0 - self.diff, self.eps, h.dtype))


class BekulixDenseMLP(nn.Module):
    def __init__(self, width: int, c: dict):
        super().__init__()
        ff = int(c["ff"])
        self.in_proj = PackedLinear(width, {"gate": ff, "up": ff})
        self.down = nn.Linear(ff, width, bias=False)

    def forward(self, h):
        _, y = self.in_proj(h)
        return self.down(relu_mul(y))


class BekulixStreams(nn.Module):
    """One sublayer's weights on the residual streams (float32)."""

    def __init__(self, streams: int):
        super().__init__()
        self.read = _vec(streams, 1.0 / streams)
        self.write = _vec(streams)
        self.mix = nn.Parameter(torch.eye(streams, dtype=torch.float32))  # [from, to]


MIXERS = {"attention": BekulixAttention, "latent_attention": BekulixLatentAttention,
          "attention_2": BekulixDifferentialAttention}
MLPS = {"dense": BekulixDenseMLP}


class BekulixLayer(nn.Module):
    def __init__(self, cfg: BekulixConfig, spec: dict):
        super().__init__()
        if spec["type"] not in MIXERS:
            raise ValueError(f"unknown mixer type {spec['type']!r}")
        self.kind = spec["type"]
        self.norm1 = _vec(cfg.width)  # 1 + the stored weight
        self.hc1 = BekulixStreams(cfg.streams)
        self.mix = MIXERS[spec["type"]](cfg.width, spec["mixer"], cfg.norm_eps)
        m = spec.get("mlp")
        if m is not None and m.get("kind") not in MLPS:
            raise ValueError(f"unknown feed-forward kind {m.get('kind')!r}")
        self.mlp = MLPS[m["kind"]](cfg.width, m) if m is not None else None
        if self.mlp is not None:
            self.norm2 = _vec(cfg.width)
            self.hc2 = BekulixStreams(cfg.streams)


@register_model("Bekulix")
class BekulixForCausalLM(nn.Module):
    config_class = BekulixConfig
    serves_ragged = True  # the serving engines drive forward_ragged

    def __init__(self, cfg: BekulixConfig):
        super().__init__()
        self.config = cfg
        self.embed = nn.Embedding(cfg.vocab, cfg.width)
        self.layers = nn.ModuleList([BekulixLayer(cfg, s) for s in cfg.layers])
        self.final_norm = _vec(cfg.width)
        self.head = nn.Linear(cfg.width, cfg.vocab, bias=False)
        self.runs = [i for i, _, _ in cfg.layer_runs()]

    # ------------------------------------------------------------ cache plan
    def kv_layer_shapes(self):
        """Per layer *run* ``(key heads, key_dim, value_dim[, value heads])``: a looped layer has one entry per pass."""
        return [self.layers[i].mix.kv_shape() for i in self.runs]

    def kv_layer_key_factors(self):
        """Per layer run whether it keeps a float32 factor beside each key."""
        return [self.layers[i].mix.key_factors for i in self.runs]

    def state_layer_buffers(self):
        """No layer keeps state outside the pages."""
        return [None] * len(self.runs)

    @property
    def act_dtype(self):
        return self.head.weight.dtype

    # ---------------------------------------------------------------- serve
    def forward_ragged(self, tokens: torch.Tensor, batch: RaggedBatch, kv, state,
                       want: Optional[torch.Tensor] = None, residuals: Optional[list] = None) -> torch.Tensor:
        """tokens [N] (flat, sequence after sequence as ``batch`` says); ``kv`` a KVCacheManager laid out by
        ``kv_layer_shapes`` / ``kv_layer_key_factors``. Returns float32 logits of the rows ``want`` (indices into the
        flat token axis; all rows if None). ``residuals``, when a list, receives the float32 sum of the streams after
        every layer run."""
        eps, act = self.config.norm_eps, self.act_dtype
        layers = [self.layers[i] for i in self.runs]
        x, h = streams_start(self.embed.weight, tokens, self.config.streams, layers[0].hc1.read, layers[0].norm1, eps)
        for r, layer in enumerate(layers):
            last = r + 1 == len(layers)
            after = (None, self.final_norm) if last else (layers[r + 1].hc1.read, layers[r + 1].norm1)
            y, hc = layer.mix(h, batch, kv, r), layer.hc1
            if layer.mlp is not None:
                h = streams_update(x, y, hc.mix, hc.write, layer.hc2.read, layer.norm2, eps, act)
                y, hc = layer.mlp(h), layer.hc2
            if last and want is not None and residuals is None:  # the last write is per row: the wanted rows only
                x, y = x.index_select(0, want), y.index_select(0, want)
            h = streams_update(x, y, hc.mix, hc.write, *after, eps, act)
            if residuals is not None:
                residuals.append(x.sum(1))
        if want is not None and residuals is not None:
            h = h.index_select(0, want)
        return self.head(h).float()

    def forward(self, input_ids: torch.Tensor) -> torch.Tensor:
        """input_ids [B, S] -> logits [B, S, vocab] (float32), every sequence from position 0 with caches that
        live for this call only."""
        from ..inference.kv_cache import KVCacheManager

        B, S = input_ids.shape
        dev = input_ids.device
        page = 16
        pages = (S + page - 1) // page
        kv = KVCacheManager(len(self.runs), 0, 0, num_blocks=B * pages, block_size=page, device=dev,
                            dtype=self.act_dtype, layer_shapes=self.kv_layer_shapes(),
                            layer_key_factors=self.kv_layer_key_factors())
        tables = [list(range(b * pages, (b + 1) * pages)) for b in range(B)]
        batch = RaggedBatch.build([S] * B, [0] * B, list(range(B)), dev, tables, page)
        with torch.no_grad():
            return self.forward_ragged(input_ids.reshape(-1), batch, kv, None).view(B, S, -1)

    # -------------------------------------------------------------- weights
    def prepare(self) -> None:
        """Refresh what is derived from the weights (after loading or changing them)."""
        for layer in self.layers:
            if hasattr(layer.mix, "prepare"):
                layer.mix.prepare()

    def load_checkpoint_tensors(self, tensors: Dict[str, torch.Tensor]) -> None:
        """Pack a checkpoint's tensors (``embed``, ``head``, ``final.norm``, ``l<i>.norm{1,2}``,
        ``l<i>.hc{1,2}.{in,out,mix}``, ``l<i>.mix.*``, ``l<i>.mlp.*``) into this module's parameters. Every tensor must
        be used and every parameter filled."""
        used = set()

        def get(name):
            used.add(name)
            return tensors[name]

        def put(param, value):
            assert tuple(param.shape) == tuple(value.shape), (tuple(param.shape), tuple(value.shape))
            param.data.copy_(value.to(param.dtype))

        def put_streams(hc, p):
            put(hc.read, get(p + "in"))
            put(hc.write, get(p + "out"))
            put(hc.mix, get(p + "mix"))

        put(self.embed.weight, get("embed"))
        put(self.head.weight, get("head"))
        put(self.final_norm, 1.0 + get("final.norm").float())
        for i, layer in enumerate(self.layers):
            p, m = f"l{i}.", layer.mix
            a = p + "mix."
            put(layer.norm1, 1.0 + get(p + "norm1").float())
            put_streams(layer.hc1, p + "hc1.")
            put(m.o.weight, get(a + "o"))
            if layer.kind == "attention":
                put(m.in_proj.weight, torch.cat([get(a + "q"), get(a + "k")], 0))
                put(m.qk_norm, get(a + "q.norm").float() * get(a + "k.norm").float())
            elif layer.kind == "latent_attention":
                put(m.in_proj.weight, torch.cat([get(a + "q"), get(a + "dkv")], 0))
                put(m.dkv_norm, get(a + "dkv.norm"))
                put(m.uk, get(a + "uk").view(m.H, m.D, m.rank))
                put(m.uv, get(a + "uv").view(m.H, m.Dv, m.rank))
            else:
                q, qb = (map_major(get(a + n), m.H, m.G, m.D) for n in ("q", "q.b"))
                put(m.in_proj.weight, torch.cat([q, get(a + "k"), get(a + "v")], 0))
                put(m.in_proj.bias, torch.cat([qb, get(a + "k.b"), get(a + "v.b")], 0))
                for n in ("lq1", "lk1", "lq2", "lk2"):
                    put(getattr(m, n), get(a + n))
            if layer.mlp is None:
                used.update(n for n in tensors if n == p + "norm2" or n.startswith(p + "hc2."))
                continue
            put(layer.norm2, 1.0 + get(p + "norm2").float())
            put_streams(layer.hc2, p + "hc2.")
            put(layer.mlp.in_proj.weight, torch.cat([get(p + "mlp.gate"), get(p + "mlp.up")], 0))
            put(layer.mlp.down.weight, get(p + "mlp.down"))
        missing = set(tensors) - used
        if missing:
            raise ValueError(f"checkpoint tensors without a place in the model: {sorted(missing)[:8]}")
        self.prepare()

    def serving_dtype(self, dtype) -> "BekulixForCausalLM":
        """Give matrices and projection biases ``dtype``; norm weights, the weights on the streams and the difference
        weight's vectors stay float32."""
        keep32 = {id(hc.mix) for hc in self.modules() if isinstance(hc, BekulixStreams)}
        for p in self.parameters():
            if p.dim() >= 2 and id(p) not in keep32:
                p.data = p.data.to(dtype)
        for layer in self.layers:
            if layer.kind == "attention_2":
                layer.mix.in_proj.bias.data = layer.mix.in_proj.bias.data.to(dtype)
        self.prepare()
        return self

    @classmethod
    def from_checkpoint(cls, config: dict, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16, device="cpu"):
        """Build from a parsed config.json and a name -> tensor mapping."""
        model = cls(BekulixConfig.from_dict(config)).serving_dtype(dtype)
        model.load_checkpoint_tensors(tensors)
        return model.to(device).eval()
