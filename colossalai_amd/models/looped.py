"""Models whose checkpoint runs a block of layers several times with the same weights."""

from typing import List, Optional, Tuple

__all__ = ["parse_loop", "layer_runs"]


def parse_loop(d: dict) -> Optional[dict]:
    """The ``loop`` entry of a config (``start``, ``stop``, ``times``) as ints, or None."""
    loop = d.get("loop")
    return None if loop is None else {k: int(loop[k]) for k in ("start", "stop", "times")}


def layer_runs(num_layers: int, loop: Optional[dict]) -> List[Tuple[int, Optional[int], bool]]:
    """The order in which layers run: ``(layer, pass number or None, first of its pass)``. Layers ``start .. stop - 1``
    run ``times`` times in a row; every run of a layer has caches of its own."""
    if loop is None or loop["stop"] <= loop["start"] or loop["times"] < 1:
        return [(i, None, False) for i in range(num_layers)]
    if not 0 <= loop["start"] < loop["stop"] <= num_layers:
        raise ValueError(f"loop {loop} does not fit {num_layers} layers")
    runs = [(i, None, False) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None, False) for i in range(loop["stop"], num_layers)]
