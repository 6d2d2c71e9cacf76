"""What decoders share whose config.json lists their layers one by one and may run a block of them several times."""
from typing import List, Tuple


def layer_runs(cfg: dict) -> List[Tuple[int, bool]]:
    """[(layer, does a pass of the loop begin here?)] in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    if not (0 <= start < stop <= n) or times < 1:
        raise ValueError(f"loop over layers {start} .. {stop - 1}, {times} times, of a model of {n} layers")
    runs = [(i, False) for i in range(start)]
    for _ in range(times):
        runs += [(i, i == start) for i in range(start, stop)]
    return runs + [(i, False) for i in range(stop, n)]
