"""RMSNorm: y = x * rsqrt(mean(x^2) + eps) * w in float32; LayerNorm with a gain and,
if named, a bias: y = (x - mean) / sqrt(var + eps) * w + b, var the mean of the squared deviations.

Reference: servelab/attention/triton/paged_attention.py:76-91 and the vector
in tests/test_triton_kernels.py:57-59.  Here the residual add that precedes
every use (servelab/parallel/tp_model.py:131-133) is fused in.
"""
from .base import Norm, ParamSpec


class StreamsDelta:
    """A sublayer's output that joins a stream kept in several copies: every copy becomes a weighted
    sum of all of them plus its own multiple of the output (``link``: a ``StreamLink``).  ``y``: a
    plain value, a ``NormedDelta``, or a tuple of them (their sum joins)."""
    __slots__ = ("y", "link")

    def __init__(self, y, link):
        self.y, self.link = y, link

    def outputs(self, ops):
        """[(rows, gain of their own norm or None, its eps)]"""
        ys = self.y if isinstance(self.y, (tuple, list)) else (self.y,)
        return [(d.y, d.weight, d.eps) if isinstance(d, NormedDelta) else (ops.materialize(d), None, 0.0) for d in ys]

    def norm_rows(self, ops, resid, weight, bias, eps, center, rows):
        """Rows ``rows`` of the sum of all copies, normed; the copies stay as they are."""
        return ops.streams_norm(resid, self.outputs(ops), self.link.mix, self.link.out, None, weight, bias, eps,
                                center=center, rows=rows)


class NormedDelta:
    """A sublayer's output that joins the stream through an RMS norm of its own:
    stream += y / sqrt(mean(y^2) + eps) * weight.  A block hands it on as its pending delta, and
    the RMS norm that reads the stream next does the add and its own norm in one kernel call."""
    __slots__ = ("y", "weight", "eps")

    def __init__(self, y, weight, eps):
        self.y, self.weight, self.eps = y, weight, float(eps)


def _settle(ops, resid, delta):
    """Of several deltas (sublayers that ran side by side), those with a norm of their own join the
    stream here; what is left for the reading norm's own add."""
    if not isinstance(delta, (tuple, list)) or not any(isinstance(d, NormedDelta) for d in delta):
        return delta
    for d in delta:
        if isinstance(d, NormedDelta):
            ops.add_postnorm(resid, d.y, d.weight, d.eps, 1.0, want_rows=False)
    return tuple(d for d in delta if not isinstance(d, NormedDelta)) or None


class RMSNorm(Norm):
    """``offset``: the stored weight w acts as the gain offset + w (1 for weights kept around
    zero); the sum is taken once at load, in float32."""
    graph_safe = True

    def __init__(self, size: int, eps: float, name: str = "weight", offset: float = 0.0):
        self.size = int(size)
        self.eps = float(eps)
        self.name = name
        self.offset = float(offset)

    def param_specs(self):
        return {self.name: ParamSpec((self.size,), init="gain" if not self.offset else "normal")}

    def load(self, tensors, rt):
        self.rt = rt
        self.weight = rt.vector(tensors(self.name))
        if self.offset:
            self.weight = (self.weight + self.offset).contiguous()

    def forward(self, resid, delta, fuse=False):
        if isinstance(delta, NormedDelta):
            return self.rt.ops.add_normed_rmsnorm(resid, delta.y, delta.weight, delta.eps, self.weight, self.eps)
        delta = _settle(self.rt.ops, resid, delta)
        return self.rt.ops.add_rmsnorm(resid, delta, self.weight, self.eps, fuse=fuse)

    def forward_rows(self, resid, delta, rows, fuse=False):
        if isinstance(delta, NormedDelta):
            return self.rt.ops.add_normed_rmsnorm(resid, delta.y, delta.weight, delta.eps, self.weight, self.eps,
                                                  rows=rows)
        if isinstance(delta, StreamsDelta):
            return delta.norm_rows(self.rt.ops, resid, self.weight, None, self.eps, False, rows)
        delta = _settle(self.rt.ops, resid, delta)
        return self.rt.ops.rows_add_rmsnorm(resid, delta, rows, self.weight, self.eps, fuse=fuse)

    def forward_streams(self, resid, delta, link):
        return link.read(self.rt.ops, resid, delta, self.weight, None, self.eps, False)

    def normed(self, y):
        """``y`` as a delta that joins the stream through this norm."""
        return NormedDelta(self.rt.ops.materialize(y), self.weight, self.eps)


class LayerNorm(Norm):
    """Layer norm with a gain and (``bias_name`` given) a bias, in float32, fused with the residual
    add before it.  ``delta`` may be a tuple of values that are all added (the
    outputs of sublayers that ran side by side).  Its rows are plain normed rows
    (``fuse`` is not taken up)."""
    graph_safe = True

    def __init__(self, size: int, eps: float, name: str = "weight", bias_name=None):
        self.size = int(size)
        self.eps = float(eps)
        self.name, self.bias_name = name, bias_name

    def param_specs(self):
        specs = {self.name: ParamSpec((self.size,), init="gain")}
        if self.bias_name is not None:
            specs[self.bias_name] = ParamSpec((self.size,))
        return specs

    def load(self, tensors, rt):
        self.rt = rt
        self.weight = rt.vector(tensors(self.name))
        self.bias = rt.vector(tensors(self.bias_name)) if self.bias_name is not None else None

    def _more(self):
        return {} if self.bias is None else {"bias": self.bias}

    def forward(self, resid, delta, fuse=False):
        delta = _settle(self.rt.ops, resid, (delta,) if isinstance(delta, NormedDelta) else delta)
        return self.rt.ops.add_layernorm(resid, delta, self.weight, self.eps, **self._more())

    def forward_rows(self, resid, delta, rows, fuse=False):
        if isinstance(delta, StreamsDelta):
            return delta.norm_rows(self.rt.ops, resid, self.weight, self.bias, self.eps, True, rows)
        delta = _settle(self.rt.ops, resid, (delta,) if isinstance(delta, NormedDelta) else delta)
        return self.rt.ops.add_layernorm(resid, delta, self.weight, self.eps, rows=rows, **self._more())

    def forward_streams(self, resid, delta, link):
        return link.read(self.rt.ops, resid, delta, self.weight, self.bias, self.eps, True)


class PostRMSNorm(RMSNorm):
    """An RMS norm on a sublayer's output instead of its input: the stream takes
    ``mult`` times the normed output, and the sublayers read the stream itself.
    ``forward_post(resid, y)`` adds mult * norm(y) into the float32 stream in
    place and returns the stream's rows in the activation dtype, which is what
    the next sublayer reads (``y`` None: only those rows)."""

    def __init__(self, size: int, eps: float, mult: float = 1.0, name: str = "weight"):
        super().__init__(size, eps, name)
        self.mult = float(mult)

    def load(self, tensors, rt):
        super().load(tensors, rt)
        self.delta_weight = self.weight if self.mult == 1.0 else (self.weight * self.mult).contiguous()

    def normed(self, y):
        return NormedDelta(self.rt.ops.materialize(y), self.delta_weight, self.eps)

    def forward_post(self, resid, y):
        return self.rt.ops.add_postnorm(resid, y, self.weight, self.eps, self.mult)
