"""A slow, whole-sequence implementation of the Kelutar design in float64, one function per
mechanism, written from the design's equations.  It shares no code with servelab_amd: the tests
hold the engine to it.

config: the dict of config.json.  weights: {tensor name: torch tensor}.  Everything runs on the
CPU over one whole sequence, token by token where the design is a recurrence.

The design in short.  The stream starts as a multiple of the token's embedding plus a learned vector
of the position.  A layer is x += N1(Mixer(h)), x += N2(FF(x)), N an RMS norm with a plain gain and
h = x + Conv(x), a causal convolution over time on each channel of the stream.  Mixers: softmax
attention over a window whose values are the keys as projected, with biases, a norm per head, a
factor per head on the scores and a sigmoid gate on every channel of its output; and a linear
attention (HGRN2) whose forget gate, bounded from below, also says how much is written.  The
feed-forward is down(relu(up)^2) or absent.  Layers may run another layer's tensors."""
import math

import torch

F = torch.float64


def rms_norm(x, gain, eps):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if gain is None else y * gain


def linear(x, w, b=None):
    y = x @ w.T
    return y if b is None else y + b


def embed(cfg, w, tokens):
    """scale * table row + the position's vector (which is not scaled)."""
    ids = torch.as_tensor(tokens, dtype=torch.long)
    return w["embed"][ids] * float(cfg["embedding"]["scale"]) + w["pos"][torch.arange(len(ids))]


def stream_convolution(x, taps):
    """x [T, C], taps [C, n]: h_t = x_t + sum_j taps[:, j] x_(t - n + 1 + j), zeros before the start."""
    T, C = x.shape
    n = taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, C, dtype=x.dtype), x], 0)
    h = x.clone()
    for j in range(n):
        h = h + taps[:, j][None, :] * padded[j:j + T]
    return h


def visible(T, size):
    """[T, T] bool: query i sees key j when 0 <= i - j (< size, if there is a window)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if size:
        seen &= (i - j) < size
    return seen


def attention(h, m, w, p, eps):
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q = linear(h, w[p + "q"], w[p + "q.b"]).view(T, H, D)
    k = linear(h, w[p + "k"], w[p + "k.b"]).view(T, G, D)
    v = k                                                    # (before the norm)
    q = rms_norm(q, w[p + "q.norm"], eps)
    k = rms_norm(k, w[p + "k.norm"], eps)
    k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    scores = torch.einsum("ihd,jhd->hij", q, k) * float(m["scale"]) * w[p + "temp"][:, None, None]
    seen = visible(T, (m.get("mask") or {}).get("size"))
    weights = torch.softmax(scores.masked_fill(~seen, -math.inf), -1)
    o = torch.einsum("hij,jhd->ihd", weights, v).reshape(T, H * D)
    return linear(o * torch.sigmoid(linear(h, w[p + "g"])), w[p + "o"])


def forget_gate(z, lower):
    return lower + (1.0 - lower) * torch.sigmoid(z)


def hgrn2(h, m, w, p, eps):
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    q = linear(h, w[p + "q"])
    q = (q * torch.sigmoid(q)).view(T, H, D)
    v = linear(h, w[p + "v"]).view(T, H, Dv)
    f = forget_gate(linear(h, w[p + "f"], w[p + "f.b"]), w[p + "lower"]).view(T, H, D)
    S = torch.zeros(H, D, Dv, dtype=h.dtype)
    out = torch.zeros(T, H, Dv, dtype=h.dtype)
    for t in range(T):
        S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return linear(rms_norm(out, w[p + "norm"], eps).reshape(T, H * Dv), w[p + "o"])


def feed_forward(x, w, p):
    return linear(torch.relu(linear(x, w[p + "up"])) ** 2, w[p + "down"])


MIXERS = {"attention": attention, "hgrn2": hgrn2}


def layer(x, entry, i, w, eps):
    p = f"l{i}."
    h = stream_convolution(x, w[p + "canon1"])
    x = x + rms_norm(MIXERS[entry["type"]](h, entry["mixer"], w, p + "mix.", eps), w[p + "norm1"], eps)
    if entry.get("mlp") is not None:
        x = x + rms_norm(feed_forward(x, w, p + "mlp."), w[p + "norm2"], eps)
    return x


def owner(cfg, i):
    """The layer whose tensors layer i runs."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg, weights, tokens, streams=None):
    """Logits [T, vocab]; ``streams``: a list that takes the stream after every layer."""
    w = {n: t.to(F) for n, t in weights.items()}
    eps = float(cfg["norm"]["eps"])
    x = embed(cfg, w, tokens)
    for i, entry in enumerate(cfg["layers"]):
        x = layer(x, entry, owner(cfg, i), w, eps)
        if streams is not None:
            streams.append(x)
    return linear(rms_norm(x, w["final.norm"], eps), w["head"])
