"""Execution order of a stack that runs a stretch of its layers several times with the same weights: layers [0, start), then
`times` passes over [start, stop), then [stop, n).  Every pass has caches and states of its own; a pass's number is the
layer's "lane" (0 outside the loop)."""
from __future__ import annotations


class LoopedLayers:
    """Mixin of configuration objects: read_loop(config.json's "loop" or None, number of layers)."""

    def read_loop(self, loop: dict | None, n: int) -> None:
        self.loop_start, self.loop_stop, self.loop_times = (int(loop["start"]), int(loop["stop"]), int(loop["times"])) \
            if loop else (0, 0, 0)
        assert 0 <= self.loop_start <= self.loop_stop <= n and (not loop or self.loop_times >= 1), loop
        self._n_layers = n

    @property
    def layer_runs(self):
        """[(layer, lane, pass number on a pass's first layer or None)] in execution order"""
        a, b, n = self.loop_start, self.loop_stop, self._n_layers
        if not self.loop_times or a == b:
            return [(i, 0, None) for i in range(n)]
        runs = [(i, 0, None) for i in range(a)]
        for t in range(self.loop_times):
            runs += [(i, t, t if i == a else None) for i in range(a, b)]
        return runs + [(i, 0, None) for i in range(b, n)]

    def lanes_of(self, i: int) -> int:
        return self.loop_times if self.loop_times and self.loop_start <= i < self.loop_stop else 1
