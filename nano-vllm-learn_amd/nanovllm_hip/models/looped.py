"""Order of layers where a run of them, loop = dict(start, stop, times), is passed through several times with the same weights."""


class LoopedLayers:
    """Mixin of a configuration with `layers` and `loop` (or None)."""

    @property
    def num_hidden_layers(self):
        return len(self.layers)

    def check_loop(self):
        loop, n = self.loop, len(self.layers)
        if loop is not None and not (0 <= loop["start"] <= loop["stop"] <= n and loop["times"] >= 1):
            raise ValueError(f"loop {loop} over {n} layers")

    def passes(self, index):
        """How often layer `index` runs."""
        return self.loop["times"] if self.loop is not None and self.loop["start"] <= index < self.loop["stop"] else 1

    def runs(self):
        """(layer, pass) in the order they run."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, 0) for i in range(n)]
        a, b = self.loop["start"], self.loop["stop"]
        return [(i, 0) for i in range(a)] + [(i, t) for t in range(self.loop["times"]) for i in range(a, b)] + [(i, 0) for i in range(b, n)]
