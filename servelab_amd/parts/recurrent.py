"""Mixers whose memory is a matrix per head, carried from token to token in a state slot.

All of them keep, per head, S [dim, vdim] in float32 and read a token's output as S^T q:

``MatrixLSTM``: scalar gates per head with a running maximum m (m_0 = 0):
    i = cap tanh(i~ / cap), f = logsigmoid(cap tanh(f~ / cap)), m' = max(f + m, i),
    S' = e^(f + m - m') S + e^(i - m') k v^T, n' likewise with k alone,
    o = S'^T q / (max(|n' . q|, e^(-m')) + 1e-6);
each head's o divided by its root mean square, a gain over all heads, a sigmoid output gate.

``GatedLinearAttention``: a decay per key channel, alpha = sigmoid(z)^(1/tau) with z from a
low-rank projection plus bias: S' = diag(alpha) S + k v^T; o RMS-normed per head with a gain
shared by the heads, times silu of a full-rank gate.

``GatedDeltaRule``: q, k, v pass a short causal convolution over time and silu; q and k become
unit vectors per head; S' = diag(g) S, u = beta (v - S'^T k), S' += k u^T, o = S'^T q (the
read-out sees the token's own write); g = exp(-exp(A_log_h) softplus(a + dt_bias)) per head and
key channel, a from a low-rank projection; the gain is shared by the heads and the sigmoid
output gate comes from a low-rank projection.  The convolution's last taps - 1 inputs are part
of the state.  ``decay`` "head": one g per head, a straight from the input; ``gate`` "silu": silu of a
full projection in place of the sigmoid of a low-rank one.

``SelectiveStateMixer`` (Mamba): a state per channel c and place n; the projection gives x and a gate z,
x passes a short causal convolution with a bias and silu; a second projection of x gives a low-rank
step, B and C; dt = softplus(W_dt step + b) per channel; S'[c, n] = exp(-exp(A_log[c, n]) dt_c) S[c, n]
+ dt_c x_c B_n, y_c = sum_n S'[c, n] C_n + D_c x_c, times silu(z).  The convolution's last taps - 1
inputs are part of the state.

``StateSpaceMixer``: one projection gives a gate z, the inputs x, B and C (B and C shared by the
heads of a group) and a step size per head; x, B and C pass a short causal convolution with a bias
and silu; dt = softplus(dt~ + dt_bias_h); S' = exp(-exp(A_log_h) dt) S + dt B x^T (one decay for
the whole head), y = S'^T C + D_h x; y times silu(z), then RMS-normed in equal parts with a gain
over the whole row.  The convolution's last taps - 1 inputs are part of the state.

``BoundedForgetAttention`` (HGRN2): a forget gate per key channel that also says how much is written,
f = l + (1 - l) sigmoid(z) with a stored lower bound l: S' = diag(f) S + (1 - f) v^T, read by silu(q);
o RMS-normed per head with a gain shared by the heads, no output gate.

Gates, decays, unit norms, state and read-out are float32 in both activation types; the input
projection (one product for everything a mixer projects from its input) returns float32 sums.
A state starts from zero at a sequence's first token, whatever the slot held.  Every size and
constant is a constructor parameter, checkpoint names too (``names``).
"""
import torch

from .base import Mixer, ParamSpec, StateSpec
from .norm import PostRMSNorm


def _rows(blocks):
    """Row-concatenated matrices and where each starts: ({name: first row}, matrix)."""
    at, n = {}, 0
    for name, t in blocks:
        at[name] = n
        n += t.shape[0]
    return at, torch.cat([t for _, t in blocks], 0)


class _MatrixMemoryMixer(Mixer):
    graph_safe = True

    def _project(self, x):
        return self.rt.ops.linear(x, self.w_in, self.b_in, out_f32=True)

    def _load_in(self, blocks, rt, biases=None):
        """One input matrix out of ``blocks`` [(name, tensor)], padded to a multiple of 8 rows;
        ``biases`` {name: tensor} are the rows' biases (others zero)."""
        self.at, w = _rows(blocks)
        extra = -w.shape[0] % 8
        if extra:
            w = torch.cat([w, w.new_zeros(extra, w.shape[1])], 0)
        self.w_in = rt.linear_weight(w)
        self.b_in = None
        if biases:
            b = torch.zeros(w.shape[0], dtype=torch.float32, device=w.device)
            for name, t in biases.items():
                b[self.at[name]:self.at[name] + t.shape[0]] = t.float()
            self.b_in = rt.vector(b)


class MatrixLSTM(_MatrixMemoryMixer):
    NAMES = {"q": "q", "k": "k", "v": "v", "gate": "g", "out": "o", "norm": "norm",
             "i": "i", "i_bias": "i.b", "f": "f", "f_bias": "f.b"}

    def __init__(self, hidden_size, heads, dim, vdim, gate_cap, norm_eps, names=None):
        self.hidden_size, self.heads, self.dim, self.vdim = int(hidden_size), int(heads), int(dim), int(vdim)
        self.gate_cap, self.norm_eps = float(gate_cap), float(norm_eps)
        self.names = dict(self.NAMES, **(names or {}))

    def param_specs(self):
        n, h, H, D, Dv = self.names, self.hidden_size, self.heads, self.dim, self.vdim
        return {n["q"]: ParamSpec((H * D, h)), n["k"]: ParamSpec((H * D, h)), n["v"]: ParamSpec((H * Dv, h)),
                n["gate"]: ParamSpec((H * Dv, h)), n["out"]: ParamSpec((h, H * Dv)),
                n["norm"]: ParamSpec((H * Dv,), init="gain"),
                n["i"]: ParamSpec((H, h)), n["i_bias"]: ParamSpec((H,)),
                n["f"]: ParamSpec((H, h)), n["f_bias"]: ParamSpec((H,))}

    def cache_spec(self):
        H, D, Dv = self.heads, self.dim, self.vdim
        return StateSpec((H * D * Dv + H * D + H,), "float32")        # S, n, m

    def load(self, tensors, rt):
        self.rt = rt
        n = self.names
        self._load_in([(x, tensors(n[x])) for x in ("q", "k", "v", "gate", "i", "f")], rt,
                      {"i": tensors(n["i_bias"]), "f": tensors(n["f_bias"])})
        self.gain = rt.vector(tensors(n["norm"]))
        self.w_o = rt.linear_weight(tensors(n["out"]), delta=True)

    def forward(self, x, batch, cache, shared):
        ops, at = self.rt.ops, self.at
        H, D, Dv = self.heads, self.dim, self.vdim
        buf = self._project(x)
        o = ops.mlstm_scan(buf, at["q"], at["k"], at["v"], at["i"], at["f"], H, D, Dv, self.gate_cap,
                           D ** -0.5, cache.state, batch, cache.write)
        y = ops.head_norm_gate(o, H, Dv, self.gain, True, self.norm_eps, buf, at["gate"], "sigmoid")
        return ops.linear(y, self.w_o, None)


class GatedLinearAttention(_MatrixMemoryMixer):
    NAMES = {"q": "q", "k": "k", "v": "v", "gate": "g", "out": "o", "norm": "norm",
             "decay_in": "a1", "decay_out": "a2", "decay_bias": "a2.b"}

    def __init__(self, hidden_size, heads, dim, vdim, tau, decay_rank, norm_eps, names=None):
        self.hidden_size, self.heads, self.dim, self.vdim = int(hidden_size), int(heads), int(dim), int(vdim)
        self.tau, self.decay_rank, self.norm_eps = float(tau), int(decay_rank), float(norm_eps)
        self.names = dict(self.NAMES, **(names or {}))

    def param_specs(self):
        n, h, H, D, Dv, r = self.names, self.hidden_size, self.heads, self.dim, self.vdim, self.decay_rank
        return {n["q"]: ParamSpec((H * D, h)), n["k"]: ParamSpec((H * D, h)), n["v"]: ParamSpec((H * Dv, h)),
                n["gate"]: ParamSpec((H * Dv, h)), n["out"]: ParamSpec((h, H * Dv)),
                n["norm"]: ParamSpec((Dv,), init="gain"),
                n["decay_in"]: ParamSpec((r, h)), n["decay_out"]: ParamSpec((H * D, r)),
                n["decay_bias"]: ParamSpec((H * D,))}

    def cache_spec(self):
        return StateSpec((self.heads * self.dim * self.vdim,), "float32")

    def load(self, tensors, rt):
        self.rt = rt
        n = self.names
        self._load_in([(x, tensors(n[x])) for x in ("q", "k", "v", "gate", "decay_in")], rt)
        self.decay_out = rt.vector(tensors(n["decay_out"]))
        self.decay_bias = rt.vector(tensors(n["decay_bias"]))
        self.gain = rt.vector(tensors(n["norm"]))
        self.w_o = rt.linear_weight(tensors(n["out"]), delta=True)

    def forward(self, x, batch, cache, shared):
        ops, at = self.rt.ops, self.at
        H, D, Dv = self.heads, self.dim, self.vdim
        buf = self._project(x)
        log_decay = ops.lowrank_expand(buf, at["decay_in"], self.decay_out, self.decay_bias,
                                       "log_sigmoid", heads=H, divisor=self.tau)
        o = ops.decay_scan(buf, at["q"], at["k"], at["v"], H, H, D, Dv, log_decay, D ** -0.5,
                           None, 0, cache.state, batch, cache.write)
        y = ops.head_norm_gate(o, H, Dv, self.gain, False, self.norm_eps, buf, at["gate"], "silu")
        return ops.linear(y, self.w_o, None)


class GatedDeltaRule(_MatrixMemoryMixer):
    NAMES = {"q": "q", "k": "k", "v": "v", "q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv",
             "beta": "b", "rate": "A_log", "norm": "norm", "decay_in": "a1", "decay_out": "a2",
             "decay_bias": "dt_bias", "gate_in": "g1", "gate_out": "g2", "out": "o", "decay": "a", "gate": "g"}

    def __init__(self, hidden_size, heads, kv_heads, dim, vdim, conv, decay_rank, gate_rank, norm_eps,
                 unit_eps=1e-6, names=None, decay="channel", gate="sigmoid"):
        if heads % kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if decay not in ("channel", "head") or gate not in ("sigmoid", "silu"):
            raise ValueError("the decay is per 'channel' (low-rank) or per 'head', the gate 'sigmoid' (low-rank) or 'silu'")
        self.decay, self.gate = decay, gate
        self.hidden_size, self.heads, self.kv_heads = int(hidden_size), int(heads), int(kv_heads)
        self.dim, self.vdim, self.conv = int(dim), int(vdim), int(conv)
        self.decay_rank, self.gate_rank = int(decay_rank), int(gate_rank)
        self.norm_eps, self.unit_eps = float(norm_eps), float(unit_eps)
        self.names = dict(self.NAMES, **(names or {}))

    @property
    def channels(self):
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    def param_specs(self):
        n, h = self.names, self.hidden_size
        H, G, D, Dv, taps = self.heads, self.kv_heads, self.dim, self.vdim, self.conv
        return {n["q"]: ParamSpec((G * D, h)), n["q_conv"]: ParamSpec((G * D, taps)),
                n["k"]: ParamSpec((G * D, h)), n["k_conv"]: ParamSpec((G * D, taps)),
                n["v"]: ParamSpec((H * Dv, h)), n["v_conv"]: ParamSpec((H * Dv, taps)),
                n["beta"]: ParamSpec((H, h)), n["rate"]: ParamSpec((H,)),
                n["norm"]: ParamSpec((Dv,), init="gain"),
                **self._decay_and_gate(n, h, H, D, Dv), n["out"]: ParamSpec((h, H * Dv))}

    def _decay_and_gate(self, n, h, H, D, Dv):
        if self.decay == "head":
            specs = {n["decay"]: ParamSpec((H, h)), n["decay_bias"]: ParamSpec((H,))}
        else:
            specs = {n["decay_in"]: ParamSpec((self.decay_rank, h)), n["decay_out"]: ParamSpec((H * D, self.decay_rank)),
                     n["decay_bias"]: ParamSpec((H * D,))}
        if self.gate == "silu":
            return dict(specs, **{n["gate"]: ParamSpec((H * Dv, h))})
        return dict(specs, **{n["gate_in"]: ParamSpec((self.gate_rank, h)),
                              n["gate_out"]: ParamSpec((H * Dv, self.gate_rank))})

    def cache_spec(self):
        H, D, Dv = self.heads, self.dim, self.vdim
        return StateSpec((H * D * Dv + (self.conv - 1) * self.channels,), "float32")   # S, last inputs

    def load(self, tensors, rt):
        self.rt = rt
        n = self.names
        self._load_in([(x, tensors(n[x])) for x in
                       ("q", "k", "v", "beta", "decay" if self.decay == "head" else "decay_in",
                        "gate" if self.gate == "silu" else "gate_in")], rt)
        self.taps = rt.vector(torch.cat([tensors(n[x]) for x in ("q_conv", "k_conv", "v_conv")], 0))
        self.rate = rt.vector(tensors(n["rate"]))
        if self.decay == "channel":
            self.decay_out = rt.vector(tensors(n["decay_out"]))
        self.decay_bias = rt.vector(tensors(n["decay_bias"]))
        if self.gate == "sigmoid":
            self.gate_out = rt.vector(tensors(n["gate_out"]))
        self.gain = rt.vector(tensors(n["norm"]))
        self.w_o = rt.linear_weight(tensors(n["out"]), delta=True)

    def forward(self, x, batch, cache, shared):
        ops, at = self.rt.ops, self.at
        H, G, D, Dv = self.heads, self.kv_heads, self.dim, self.vdim
        buf = self._project(x)
        # q, k and v lie side by side in the projection: one convolution over all their channels,
        # then q and k heads made unit vectors (q also times dim^-1/2)
        qkv = ops.short_conv(buf, at["q"], self.taps, cache.state, H * D * Dv, batch, cache.write,
                             unit_heads=2 * G, unit_dim=D, unit_eps=self.unit_eps,
                             scaled_heads=G, scale=D ** -0.5)
        if self.decay == "head":
            o = ops.head_delta_scan(qkv, 0, G * D, 2 * G * D, H, G, D, Dv, buf, at["beta"], at["decay"], self.rate,
                                    self.decay_bias, cache.state, batch, cache.write)
        else:
            log_decay = ops.lowrank_expand(buf, at["decay_in"], self.decay_out, self.decay_bias,
                                           "rate_softplus", heads=H, rates=self.rate)
            o = ops.decay_scan(qkv, 0, G * D, 2 * G * D, H, G, D, Dv, log_decay, 1.0,
                               buf, at["beta"], cache.state, batch, cache.write)
        if self.gate == "silu":
            y = ops.head_norm_gate(o, H, Dv, self.gain, False, self.norm_eps, buf, at["gate"], "silu")
            return ops.linear(y, self.w_o, None)
        gate = ops.lowrank_expand(buf, at["gate_in"], self.gate_out, None, "plain", heads=H)
        y = ops.head_norm_gate(o, H, Dv, self.gain, False, self.norm_eps, gate, 0, "sigmoid")
        return ops.linear(y, self.w_o, None)


class StateSpaceMixer(_MatrixMemoryMixer):
    NAMES = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "step_bias": "dt_bias", "rate": "A_log",
             "skip": "D", "norm": "norm", "out": "o"}

    def __init__(self, hidden_size, heads, vdim, state, groups, conv, norm_groups, norm_eps, names=None):
        if heads % groups or (heads * vdim) % norm_groups:
            raise ValueError("heads must be a multiple of groups, heads * vdim of norm_groups")
        self.hidden_size, self.heads, self.vdim, self.state = int(hidden_size), int(heads), int(vdim), int(state)
        self.groups, self.conv, self.norm_groups = int(groups), int(conv), int(norm_groups)
        self.norm_eps = float(norm_eps)
        self.names = dict(self.NAMES, **(names or {}))

    @property
    def inner(self):
        return self.heads * self.vdim

    @property
    def channels(self):
        """What passes the convolution: x, B and C."""
        return self.inner + 2 * self.groups * self.state

    def param_specs(self):
        n, h, H = self.names, self.hidden_size, self.heads
        return {n["in"]: ParamSpec((2 * self.inner + 2 * self.groups * self.state + H, h)),
                n["conv"]: ParamSpec((self.channels, self.conv)), n["conv_bias"]: ParamSpec((self.channels,)),
                n["step_bias"]: ParamSpec((H,)), n["rate"]: ParamSpec((H,)), n["skip"]: ParamSpec((H,)),
                n["norm"]: ParamSpec((self.inner,), init="gain"), n["out"]: ParamSpec((h, self.inner))}

    def cache_spec(self):
        return StateSpec((self.inner * self.state + (self.conv - 1) * self.channels,), "float32")   # S, last inputs

    def load(self, tensors, rt):
        self.rt = rt
        n = self.names
        w = tensors(n["in"])
        # the projection's rows are [z | x | B | C | dt]
        self._load_in([("z", w[:self.inner]), ("xbc", w[self.inner:self.inner + self.channels]),
                       ("dt", w[self.inner + self.channels:])], rt)
        self.taps = rt.vector(tensors(n["conv"]))
        self.conv_bias = rt.vector(tensors(n["conv_bias"]))
        self.step_bias = rt.vector(tensors(n["step_bias"]))
        self.rate = rt.vector(tensors(n["rate"]))
        self.skip = rt.vector(tensors(n["skip"]))
        self.gain = rt.vector(tensors(n["norm"]))
        self.w_o = rt.linear_weight(tensors(n["out"]), delta=True)

    def forward(self, x, batch, cache, shared):
        ops, at = self.rt.ops, self.at
        H, P, N, G = self.heads, self.vdim, self.state, self.groups
        buf = self._project(x)
        xbc = ops.short_conv(buf, at["xbc"], self.taps, cache.state, self.inner * N, batch, cache.write,
                             bias=self.conv_bias)
        y = ops.ssd_scan(xbc, 0, self.inner, self.inner + G * N, H, G, N, P, buf, at["dt"], self.rate,
                         self.step_bias, self.skip, cache.state, batch, cache.write)
        # the gate comes before the norm, which takes the row in `norm_groups` equal parts
        y = ops.head_norm_gate(y, self.norm_groups, self.inner // self.norm_groups, self.gain, True,
                               self.norm_eps, buf, at["z"], "silu", gate_first=True)
        return ops.linear(y, self.w_o, None)


class BoundedForgetAttention(_MatrixMemoryMixer):
    NAMES = {"q": "q", "f": "f", "f_bias": "f.b", "lower": "lower", "v": "v", "norm": "norm", "out": "o"}

    def __init__(self, hidden_size, heads, dim, vdim, norm_eps, names=None):
        self.hidden_size, self.heads, self.dim, self.vdim = int(hidden_size), int(heads), int(dim), int(vdim)
        self.norm_eps = float(norm_eps)
        self.names = dict(self.NAMES, **(names or {}))

    def param_specs(self):
        n, h, H, D, Dv = self.names, self.hidden_size, self.heads, self.dim, self.vdim
        return {n["q"]: ParamSpec((H * D, h)), n["f"]: ParamSpec((H * D, h)), n["f_bias"]: ParamSpec((H * D,)),
                n["lower"]: ParamSpec((H * D,), init="normal"), n["v"]: ParamSpec((H * Dv, h)),
                n["norm"]: ParamSpec((Dv,), init="gain"), n["out"]: ParamSpec((h, H * Dv))}

    def cache_spec(self):
        return StateSpec((self.heads * self.dim * self.vdim,), "float32")

    def load(self, tensors, rt):
        self.rt = rt
        n = self.names
        self._load_in([(x, tensors(n[x])) for x in ("q", "f", "v")], rt, {"f": tensors(n["f_bias"])})
        self.lower = rt.vector(tensors(n["lower"]))
        self.gain = rt.vector(tensors(n["norm"]))
        self.w_o = rt.linear_weight(tensors(n["out"]), delta=True)

    def forward(self, x, batch, cache, shared):
        ops, at = self.rt.ops, self.at
        H, D, Dv = self.heads, self.dim, self.vdim
        buf = self._project(x)
        o = ops.forget_scan(buf, at["q"], at["f"], at["v"], H, D, Dv, self.lower, cache.state, batch, cache.write)
        return ops.linear(ops.head_norm_gate(o, H, Dv, self.gain, False, self.norm_eps), self.w_o, None)


class SelectiveStateMixer(_MatrixMemoryMixer):
    NAMES = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "proj": "x", "step": "dt", "step_bias": "dt.b",
             "rate": "A_log", "skip": "D", "out": "o"}

    def __init__(self, hidden_size, inner, state, step_rank, conv, names=None):
        self.hidden_size, self.inner, self.state = int(hidden_size), int(inner), int(state)
        self.step_rank, self.conv = int(step_rank), int(conv)
        if min(self.inner, self.state, self.step_rank, self.conv) < 1:
            raise ValueError("inner, state, step_rank and conv must be positive")
        self.names = dict(self.NAMES, **(names or {}))

    def param_specs(self):
        n, h, C, N, R = self.names, self.hidden_size, self.inner, self.state, self.step_rank
        return {n["in"]: ParamSpec((2 * C, h)), n["conv"]: ParamSpec((C, self.conv)), n["conv_bias"]: ParamSpec((C,)),
                n["proj"]: ParamSpec((R + 2 * N, C)), n["step"]: ParamSpec((C, R)), n["step_bias"]: ParamSpec((C,)),
                n["rate"]: ParamSpec((C, N)), n["skip"]: ParamSpec((C,)), n["out"]: ParamSpec((h, C))}

    def cache_spec(self):
        return StateSpec((self.inner * self.state + (self.conv - 1) * self.inner,), "float32")   # S [state, inner], last inputs

    def load(self, tensors, rt):
        self.rt = rt
        n, C = self.names, self.inner
        w = tensors(n["in"])
        self._load_in([("x", w[:C]), ("z", w[C:])], rt)
        self.taps = rt.vector(tensors(n["conv"]))
        self.conv_bias = rt.vector(tensors(n["conv_bias"]))
        proj = tensors(n["proj"])
        extra = -proj.shape[0] % 8
        if extra:
            proj = torch.cat([proj, proj.new_zeros(extra, proj.shape[1])], 0)
        self.w_proj = rt.linear_weight(proj)
        self.step = rt.vector(tensors(n["step"]))
        self.step_t = rt.vector(tensors(n["step"]).float().t())
        self.step_bias = rt.vector(tensors(n["step_bias"]))
        self.rate = rt.vector(-torch.exp(tensors(n["rate"]).float()).t())          # [state, inner]
        self.skip = rt.vector(tensors(n["skip"]))
        self.w_o = rt.linear_weight(tensors(n["out"]), delta=True)

    def forward(self, x, batch, cache, shared):
        ops, at, R, N = self.rt.ops, self.at, self.step_rank, self.state
        buf = self._project(x)
        u, rows = ops.short_conv(buf, at["x"], self.taps, cache.state, self.inner * N, batch, cache.write,
                                 bias=self.conv_bias, want_rows=True)
        proj = ops.linear(rows, self.w_proj, None, out_f32=True)                   # [step | B | C]
        y = ops.selective_scan(u, proj, R, N, self.step, self.step_t, self.step_bias, self.rate, self.skip,
                               buf, at["z"], cache.state, batch, cache.write)
        return ops.linear(y, self.w_o, None)


def _needs(part):
    """What a mixer needs cached, as a list (most have one need or none)."""
    several = getattr(part, "cache_specs", None)
    if several is not None:
        return list(several())
    spec = part.cache_spec()
    return [] if spec is None else [spec]


class SideBySide(Mixer):
    """Two mixers that read the same rows; the result is left_scale * left + right_scale *
    right.  Each keeps a cache of its own kind: the block hands over their bindings
    (``cache_specs``).  ``out_norms`` (the names of two gains): each output is first RMS-normed over
    ``hidden_size`` with its gain; the result is then a pair of ``NormedDelta``, which the norm that
    reads the stream next adds."""

    def __init__(self, left, right, left_scale, right_scale, names=("left.", "right."), out_norms=None,
                 hidden_size=0, norm_eps=0.0):
        self.left, self.right = left, right
        self.left_scale, self.right_scale = float(left_scale), float(right_scale)
        self.names = tuple(names)
        self.norms = None
        if out_norms is not None:
            self.norms = tuple(PostRMSNorm(hidden_size, norm_eps, mult, name=name)
                               for name, mult in zip(out_norms, (self.left_scale, self.right_scale)))

    @property
    def graph_safe(self):
        return self.left.graph_safe and self.right.graph_safe

    def _sides(self):
        return list(zip(self.names, (self.left, self.right)))

    def param_specs(self):
        specs = {}
        for prefix, part in self._sides():
            for name, spec in part.param_specs().items():
                specs[prefix + name] = spec
        for norm in self.norms or ():
            specs.update(norm.param_specs())
        return specs

    def cache_specs(self):
        return _needs(self.left) + _needs(self.right)

    def load(self, tensors, rt):
        from .base import prefixed
        self.rt = rt
        for prefix, part in self._sides():
            part.load(prefixed(prefix, tensors), rt)
        for norm in self.norms or ():
            norm.load(tensors, rt)

    def forward(self, x, batch, caches, shared):
        ops = self.rt.ops
        caches = list(caches)
        outs = []
        for _, part in self._sides():
            n = len(_needs(part))
            own, caches = caches[:n], caches[n:]
            several = hasattr(part, "cache_specs")
            outs.append(part.forward(x, batch, own if several else (own[0] if own else None), shared))
        a, b = outs
        if self.norms is not None:
            return (self.norms[0].normed(a), self.norms[1].normed(b))
        return ops.scaled_sum(ops.materialize(a), self.left_scale, ops.materialize(b), self.right_scale)
