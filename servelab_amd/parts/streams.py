"""A residual stream kept in several copies.

Every copy starts as the embedding output.  A sublayer reads one weighted sum of the copies,
u = sum_s in_s x_s, through its norm; its output y is then written to all of them at once from the
old ones, x_t <- sum_s mix[s, t] x_s + out_t y (mix is indexed [from, to]).  The final norm reads the
plain sum of the copies.  The copies lie side by side, float32 [T, streams, H], and the write of one
sublayer's output, the read of the next and its norm are one kernel call.
"""
from .base import Part, ParamSpec


class StreamLink(Part):
    """How one sublayer is tied to the copies: ``in`` [streams], ``out`` [streams] and ``mix``
    [streams, streams], all float32."""
    graph_safe = True

    def __init__(self, streams: int, names=("in", "out", "mix")):
        self.streams, self.names = int(streams), tuple(names)
        if self.streams < 1:
            raise ValueError("there is at least one stream")

    def param_specs(self):
        s = self.streams
        return {self.names[0]: ParamSpec((s,), init="gain"), self.names[1]: ParamSpec((s,), init="gain"),
                self.names[2]: ParamSpec((s, s))}

    def load(self, tensors, rt):
        self.rt = rt
        self.weights = rt.vector(tensors(self.names[0]))
        self.out = rt.vector(tensors(self.names[1]))
        self.mix = rt.vector(tensors(self.names[2]))

    def read(self, ops, resid, delta, weight, bias, eps, center):
        """The normed rows of this sublayer, after what is pending (``delta``: a ``StreamsDelta`` or None)
        has been written to the copies."""
        if delta is None:
            return ops.streams_norm(resid, [], None, None, self.weights, weight, bias, eps, center=center)
        return ops.streams_norm(resid, delta.outputs(ops), delta.link.mix, delta.link.out, self.weights, weight,
                                bias, eps, center=center)
