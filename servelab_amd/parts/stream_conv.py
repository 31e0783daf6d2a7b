"""A short causal convolution over the residual stream, in front of a mixer: the mixer reads
h_t = x_t + sum_j taps[:, j] x_(t - n + 1 + j), channel by channel, zeros before the sequence's start.

The stream and the last n - 1 rows of it that a sequence keeps are float32 in both activation types;
h is rounded once, to the rows the mixer's products read.  What still has to join the stream (the
normed output of the sublayer before, ``NormedDelta``) is added in the same kernel call.
"""
from .base import Part, ParamSpec, StateSpec
from .norm import NormedDelta


class StreamConvolution(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, taps: int, name: str = "conv"):
        self.hidden_size, self.taps, self.name = int(hidden_size), int(taps), name
        if self.taps < 1:
            raise ValueError("the convolution has at least one tap")

    def param_specs(self):
        return {self.name: ParamSpec((self.hidden_size, self.taps))}

    def cache_specs(self):
        return [StateSpec(((self.taps - 1) * self.hidden_size,), "float32")] if self.taps > 1 else []

    def load(self, tensors, rt):
        self.rt = rt
        self.weight = rt.vector(tensors(self.name).t())            # [taps, width]
        self.no_state = None
        if self.taps == 1:                                         # a factor per channel, nothing carried
            self.no_state = rt.vector(tensors(self.name).new_zeros((1, 1)))

    def forward(self, resid, delta, batch, cache):
        """``delta``: None or a ``NormedDelta``; ``cache``: the binding of the kept rows (None with one
        tap).  Returns the mixer's rows in the activation dtype."""
        state, write = (cache.state, cache.write) if cache is not None else (self.no_state, False)
        y = {}
        if isinstance(delta, NormedDelta):
            y = {"y": delta.y, "y_weight": delta.weight, "y_eps": delta.eps}
        return self.rt.ops.stream_conv(resid, self.weight, state, 0, batch, write, **y)
