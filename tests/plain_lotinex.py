"""A slow, whole-sequence implementation of the Lotinex design in float64, one function per
mechanism, written from the design's equations.  It shares no code with servelab_amd: the tests
hold the engine to it.

config: the dict of config.json.  weights: {tensor name: torch tensor}.  Everything runs on the
CPU over one whole sequence, token by token where the design is a recurrence.

The design in short.  The stream has several copies, all equal to the scaled embedding at first.
Each sublayer reads one weighted sum of the copies through a layer norm with gain and bias; then
every copy becomes a weighted sum of all of them plus its own multiple of the sublayer's output.
At the end the copies are added up.  Mixers: softmax attention within chunks of positions, with a
norm per head, whose keys and values may be those of an earlier layer; the gated delta rule with one
decay a head; and two mixers side by side (softmax attention over a window behind a short
convolution, with a norm over the projection, blended frequencies, capped scores and a one in the
denominator; a selective scan with a decay per channel and state), each with a norm on its output.
Feed-forwards: gated by silu, dense or experts chosen by the sigmoid of their logits, whose weight
multiplies their input.  The head is the embedding table."""
import math

import torch

F = torch.float64


def linear(x, w, b=None):
    y = x @ w.T
    return y if b is None else y + b


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def layer_norm(x, gain, bias, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * gain + bias


def rms_norm(x, gain, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * gain


def unit_vectors(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def short_convolution(u, taps, bias=None):
    """u [T, C], taps [C, n]: y_t = sum_j taps[:, j] u_(t - n + 1 + j), zeros before the start."""
    T, n = u.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, u.shape[1], dtype=u.dtype), u], 0)
    y = sum(taps[:, j][None, :] * padded[j:j + T] for j in range(n))
    return y if bias is None else y + bias


# --------------------------------------------------------------------------- rotation
def frequencies(rot):
    """([f of every pair], what cos and sin are multiplied by) of a mixer's ``rot`` section."""
    dims, base, sc = rot["dims"], float(rot["base"]), rot.get("scaling")
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return plain, 1.0
    factor, original = float(sc["factor"]), float(sc["original"])

    def pair_with(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(pair_with(sc["fast"])), 0)
    hi = min(math.ceil(pair_with(sc["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        r = min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001)))
        out.append(f / factor * r + f * (1.0 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_halves(x, rot):
    """x [T, heads, D]: channel i turns with channel i + dims / 2, i < dims / 2; the rest pass."""
    if not rot or not rot.get("dims"):
        return x
    freqs, mag = frequencies(rot)
    half = rot["dims"] // 2
    ang = torch.arange(x.shape[0], dtype=x.dtype)[:, None] * torch.tensor(freqs, dtype=x.dtype)[None, :]
    c, s = (torch.cos(ang) * mag)[:, None, :], (torch.sin(ang) * mag)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


# --------------------------------------------------------------------------- what a position sees
def sees_window(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    return seen & (i - j < size) if size else seen


def sees_chunk(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    return seen & (i // size == j // size) if size else seen


def softmax_over(scores, seen):
    return torch.softmax(scores.masked_fill(~seen, -math.inf), -1)


def softmax_plus_one(scores, seen):
    """exp(s_j) / (1 + sum exp(s_j)) over what is seen."""
    s = scores.masked_fill(~seen, -math.inf)
    top = torch.clamp(s.amax(-1, keepdim=True), min=0.0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attend(q, k, v, scale, seen, weights, softcap=None):
    """q [T, H, D], k [T, G, D], v [T, G, Dv] -> [T, H * Dv]; query head h reads kv head h // (H / G)."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // rep].T) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        out.append(weights(s, seen) @ v[:, h // rep])
    return torch.stack(out, 1).reshape(T, -1)


def _size(m):
    mask = m.get("mask")
    return int(mask["size"]) if mask and mask.get("size") else 0


# --------------------------------------------------------------------------- mixers
def chunk_attention(h, m, w, p, eps, kept):
    """``kept``: {layer: (keys, values)} of the layers before; the own pair is returned beside the output."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_halves(rms_norm(linear(h, w[p + "q"]).view(T, H, D), w[p + "q.norm"], eps), m.get("rot"))
    if m.get("kv_from") is not None:
        pair = kept[m["kv_from"]]
    else:
        k = rotate_halves(rms_norm(linear(h, w[p + "k"]).view(T, G, D), w[p + "k.norm"], eps), m.get("rot"))
        pair = (k, linear(h, w[p + "v"]).view(T, G, Dv))
    o = attend(q, pair[0], pair[1], m["scale"], sees_chunk(T, _size(m)), softmax_over)
    return linear(o, w[p + "o"]), pair


def gated_delta(h, m, w, p, eps):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(short_convolution(linear(h, w[p + "q"]), w[p + "q.conv"])).view(T, G, D)
    k = silu(short_convolution(linear(h, w[p + "k"]), w[p + "k.conv"])).view(T, G, D)
    v = silu(short_convolution(linear(h, w[p + "v"]), w[p + "v.conv"])).view(T, H, Dv)
    q = (unit_vectors(q) * D ** -0.5).repeat_interleave(H // G, 1)
    k = unit_vectors(k).repeat_interleave(H // G, 1)
    beta = torch.sigmoid(linear(h, w[p + "b"]))                                              # [T, H]
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(linear(h, w[p + "a"]) + w[p + "dt_bias"]))
    S = torch.zeros(H, D, Dv, dtype=h.dtype)
    out = torch.zeros(T, H, Dv, dtype=h.dtype)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    y = rms_norm(out, w[p + "norm"], eps).reshape(T, H * Dv) * silu(linear(h, w[p + "g"]))
    return linear(y, w[p + "o"])


def sink_attention(h, m, w, p, eps):
    """Over a window, behind a short convolution, a norm over the whole projection, a one in the denominator."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = linear(h, w[p + "q"]), linear(h, w[p + "k"]), linear(h, w[p + "v"])
    if m.get("conv"):
        q, k, v = (short_convolution(u, w[p + n + ".conv"]) for u, n in ((q, "q"), (k, "k"), (v, "v")))
    q = rotate_halves(rms_norm(q, w[p + "q.norm"], eps).view(T, H, D), m.get("rot"))
    k = rotate_halves(rms_norm(k, w[p + "k.norm"], eps).view(T, G, D), m.get("rot"))
    o = attend(q, k, v.view(T, G, Dv), m["scale"], sees_window(T, _size(m)), softmax_plus_one, m.get("softcap"))
    return linear(o, w[p + "o"])


def selective_scan(h, m, w, p):
    T = h.shape[0]
    C, N, R = m["inner"], m["state"], m["dt_rank"]
    x, z = linear(h, w[p + "in"]).split([C, C], -1)
    x = silu(short_convolution(x, w[p + "conv"], w[p + "conv.b"]))
    low, B, Cc = linear(x, w[p + "x"]).split([R, N, N], -1)
    dt = softplus(linear(low, w[p + "dt"], w[p + "dt.b"]))
    A = -torch.exp(w[p + "A_log"])
    S = torch.zeros(C, N, dtype=h.dtype)
    y = torch.zeros(T, C, dtype=h.dtype)
    for t in range(T):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ Cc[t] + w[p + "D"] * x[t]
    return linear(y * silu(z), w[p + "o"])


def side_by_side(h, m, w, p, eps):
    left = sink_attention(h, m["left"], w, p + "left.", eps)
    right = selective_scan(h, m["right"], w, p + "right.")
    return 0.5 * (rms_norm(left, w[p + "left.out"], eps) + rms_norm(right, w[p + "right.out"], eps))


# --------------------------------------------------------------------------- feed-forwards
def gated_ff(h, w, p):
    return linear(silu(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


def route(h, w, p, top):
    """([T, top] chosen experts, [T, top] their scores)."""
    s = torch.sigmoid(linear(h, w[p + "router"]))
    best = torch.topk(s, top, dim=-1)
    return best.indices, best.values


def routed_ff(h, c, w, p):
    chosen, scores = route(h, w, p, c["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(chosen[t].tolist(), scores[t]):
            out[t] += gated_ff(s * h[t:t + 1], w, f"{p}e{e}.")[0]
    return out


# --------------------------------------------------------------------------- the model
def read_streams(xs, w, p):
    """xs [streams, T, width] -> the rows a sublayer's norm reads."""
    return torch.einsum("s,stw->tw", w[p + "in"], xs)


def write_streams(xs, y, w, p):
    """Every stream from all the old ones (mix is indexed [from, to]) and from the output."""
    return torch.einsum("st,snw->tnw", w[p + "mix"], xs) + w[p + "out"][:, None, None] * y[None]


def layer(xs, i, entry, w, eps, kept):
    p = f"l{i}."
    h = layer_norm(read_streams(xs, w, p + "hc1."), w[p + "norm1"], w[p + "norm1.b"], eps)
    m = entry["mixer"]
    if entry["type"] == "attention":
        y, kept[i] = chunk_attention(h, m, w, p + "mix.", eps, kept)
    elif entry["type"] == "delta":
        y = gated_delta(h, m, w, p + "mix.", eps)
    else:
        y = side_by_side(h, m, w, p + "mix.", eps)
    xs = write_streams(xs, y, w, p + "hc1.")
    c = entry.get("mlp")
    if c is None:
        return xs
    h = layer_norm(read_streams(xs, w, p + "hc2."), w[p + "norm2"], w[p + "norm2.b"], eps)
    y = gated_ff(h, w, p + "mlp.") if c["kind"] == "dense" else routed_ff(h, c, w, p + "mlp.")
    return write_streams(xs, y, w, p + "hc2.")


def forward(config, weights, tokens, trace=None):
    """tokens: list of ids of one sequence -> logits [T, vocab].  ``trace`` (a list) receives the sum
    of the streams after every layer."""
    w = {n: t.to(F) for n, t in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)] * config["embedding"]["scale"]
    xs = torch.stack([x] * config["streams"])
    kept = {}
    for i, entry in enumerate(config["layers"]):
        xs = layer(xs, i, entry, w, eps, kept)
        if trace is not None:
            trace.append(xs.sum(0))
    return linear(layer_norm(xs.sum(0), w["final.norm"], w["final.norm.b"], eps), w["embed"])
