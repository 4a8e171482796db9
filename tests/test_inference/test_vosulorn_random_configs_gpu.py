"""Vosulorn models of random shapes (layer order, shared latents, head counts and sizes that are no multiple of eight,
rotations, block lengths, latent sizes, taps, experts or no feed-forward) through the engine on the GPU, in float32 and bfloat16, a whole prompt per step and a mixed schedule of portions
and decode tokens of two requests, against the float64 oracle."""

import os
import random
import sys

import pytest
import torch

ROOT = os.path.dirname(os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
sys.path.insert(0, os.path.join(ROOT, "tests"))
import vosulorn_oracle as O  # noqa: E402

from colossalai_amd.inference import ContinuousBatchEngine, InferenceConfig  # noqa: E402
from colossalai_amd.models import VosulornForCausalLM  # noqa: E402

pytestmark = pytest.mark.gpu


def random_config(rng):
    def attention(i):
        G, D = rng.choice([1, 2, 3, 4]), rng.choice([8, 20, 32, 40, 64, 96, 128])
        a = dict(dim=D, vdim=rng.choice([8, 20, 64, 128]), heads=G * rng.choice([1, 2, 3, 4]), kv_heads=G,
                 scale=rng.choice([0.7, 1.0, 1.5]) * D ** -0.5, mask=dict(size=rng.choice([1, 5, 17, 33, 64, 100, 500])),
                 rot=dict(base=rng.choice([100.0, 1e4, 5e5]), dims=rng.choice([2, D // 2 // 2 * 2, D])))
        if rng.random() < 0.7:
            a["rot"]["scaling"] = dict(factor=rng.choice([2.0, 8.0]), low=1.0, high=rng.choice([2.0, 4.0]),
                                       original=rng.choice([20, 64, 500]))
        return dict(type="attention", mixer=a)

    def latent(i):
        own = [j for j in range(i) if layers[j]["type"] == "latent_attention" and "kv_from" not in layers[j]["mixer"]]
        c = dict(dim=rng.choice([8, 15, 32, 48, 64]), vdim=rng.choice([8, 30, 64, 128]), heads=rng.choice([1, 3, 4, 8]))
        if own and rng.random() < 0.7:
            j = rng.choice(own)
            c.update({n: layers[j]["mixer"][n] for n in ("rot_dim", "kv_rank", "rot")}, kv_from=j)
        else:
            R = rng.choice([2, 8, 16, 64])
            c.update(rot_dim=R, kv_rank=rng.choice([16, 40, 64, 100, 256]), rot=dict(base=rng.choice([50.0, 1e4, 1e6]), dims=R))
        c["scale"] = rng.choice([0.5, 1.0]) * (c["dim"] + c["rot_dim"]) ** -0.5
        return dict(type="latent_attention", mixer=c)

    def delta(i):
        G = rng.choice([1, 2, 3])
        return dict(type="delta", mixer=dict(heads=G * rng.choice([1, 2, 4]), kv_heads=G, dim=rng.choice([8, 20, 32, 64, 100, 128]),
                                             vdim=rng.choice([8, 17, 32, 64, 128, 160]), conv=rng.choice([1, 2, 3, 4, 6])))

    layers = []
    for i in range(rng.randint(3, 6)):
        spec = rng.choice([attention, delta, latent])(i)
        E = rng.choice([1, 3, 8, 13])
        spec["mlp"] = None if rng.random() < 0.2 else dict(
            kind="moe", expert=dict(ff=rng.choice([24, 32, 50, 96])), router=dict(experts=E, top=rng.randint(1, E)))
        layers.append(spec)
    return dict(architecture="Vosulorn", vocab=rng.choice([50, 333]), width=rng.choice([64, 90, 160, 256]),
                norm=dict(eps=rng.choice([1e-6, 1e-5])), embedding=dict(scale=rng.choice([1.0, 7.5, 16.0])), layers=layers)


def run(cfg, P, toks, dtype, plan):
    model = VosulornForCausalLM.from_checkpoint(cfg, P, dtype=dtype, device="cuda")
    eng = ContinuousBatchEngine(model, InferenceConfig(max_batch_size=4, dtype=dtype), num_blocks=64, block_size=16)
    outs, at = {k: [] for k in toks}, {k: 0 for k in toks}
    for step in plan:
        items = []
        for k, n in step:
            n = min(n, len(toks[k]) - at[k])
            if n > 0:
                items.append((k, toks[k][at[k] : at[k] + n], list(range(n))))
                at[k] += n
        if items:
            logits, o = eng.run_ragged(items), 0
            for k, t, _ in items:
                outs[k].append(logits[o : o + len(t)].float().cpu())
                o += len(t)
    assert all(at[k] == len(toks[k]) for k in toks)
    return {k: torch.cat(v) for k, v in outs.items()}


@pytest.mark.parametrize("seed", range(10))
def test_random_configuration(seed):
    rng = random.Random(seed)
    cfg = random_config(rng)
    P = {k: v.float() for k, v in O.random_checkpoint(cfg, seed).items()}
    g = torch.Generator().manual_seed(seed)
    toks = {"a": torch.randint(0, cfg["vocab"], (rng.choice([110, 150]),), generator=g).tolist(),
            "b": torch.randint(0, cfg["vocab"], (rng.choice([3, 40, 70]),), generator=g).tolist()}
    whole = [[("a", 10 ** 6), ("b", 10 ** 6)]]
    mixed = ([[("a", 37)], [("a", 2), ("b", 5)], [("a", 64), ("b", 1)], [("a", 1), ("b", 30)], [("a", 130), ("b", 1)]]
             + [[("a", 1), ("b", 1)]] * 30 + [[("a", 10 ** 6), ("b", 2)], [("b", 10 ** 6)]])
    for dtype in (torch.float32, torch.bfloat16):
        if dtype == torch.bfloat16:  # choices that no bfloat16 rounding turns: biases well apart, small products
            for name in P:
                if name.endswith("mlp.router"):
                    P[name] *= 0.1
                elif name.endswith("mlp.router.b"):
                    P[name] = torch.linspace(-6, 6, P[name].numel())[torch.randperm(P[name].numel(), generator=g)]
        want = {k: O.forward(cfg, P, v).float() for k, v in toks.items()}
        for plan in (whole, mixed):
            got = run(cfg, P, toks, dtype, plan)
            err = torch.cat([(got[k] - want[k]).pow(2).mean(-1).sqrt() / want[k].pow(2).mean().sqrt() for k in toks])
            if dtype == torch.float32:
                assert err.max().item() < 3e-4, (cfg, err.max().item())
            else:
                assert err.median().item() < 0.03 and (err > 0.1).float().mean().item() < 0.05, (cfg, err.median().item())
