"""What configurations of layer-by-layer designs share: a list of layers, each with its own mixer and feed-forward sizes, and a span
of them that runs several times in a row with the same weights."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional


@dataclass
class LayeredConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: List[Dict[str, Any]]
    eps: float
    loop: Optional[Dict[str, int]] = None
    num_local_experts: int = field(default=0, init=False)

    def check(self, mixers, feed_forwards) -> None:
        for i, lay in enumerate(self.layers):
            if lay["type"] not in mixers:
                raise ValueError(f"layer {i}: unknown mixer {lay['type']!r} (have {sorted(mixers)})")
            if lay.get("mlp") is not None and lay["mlp"]["kind"] not in feed_forwards:
                raise ValueError(f"layer {i}: unknown feed-forward {lay['mlp']['kind']!r}")
        lp = self.loop
        if lp is not None and not (0 <= lp["start"] < lp["stop"] <= len(self.layers) and lp["times"] >= 1):
            raise ValueError(f"loop {lp} does not fit {len(self.layers)} layers")

    def runs(self):
        """(layer, number of the pass that begins right before it, or None) in execution order."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        a, b, times = self.loop["start"], self.loop["stop"], self.loop["times"]
        body = [(i, t if i == a else None) for t in range(times) for i in range(a, b)]
        return [(i, None) for i in range(a)] + body + [(i, None) for i in range(b, n)]

    @property
    def num_hidden_layers(self) -> int:
        return len(self.runs())
