"""Small Lotinex configurations and weights for the tests, and what the tests hold them to.  The
configurations differ from each other in every size, in the order of their layers and in which
options they use; the weights are drawn so that every mechanism matters (links that mix the copies of
the stream unevenly, decays over a wide range, scores large enough to be capped, sinks that take a
share, experts whose scores differ)."""
import json
import os
import random

import numpy as np
import torch

import plain_lotinex as plain
from servelab_amd.weights.safetensors_io import write_safetensors

YARN = {"factor": 6.0, "original": 64, "fast": 8.0, "slow": 1.0}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def softmax(heads, kv_heads, dim, vdim, scale, size=None, rot=0, base=1000.0, scaling=None, **more):
    m = dict({"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}, **more)
    if rot:
        m["rot"] = {"base": base, "dims": rot}
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    if size:
        m["mask"] = {"size": size}
    return m


def attention(*args, mlp=None, **kwargs):
    return {"type": "attention", "mixer": softmax(*args, **kwargs), "mlp": mlp}


def delta(heads, kv_heads, dim, vdim, conv, mlp=None):
    return {"type": "delta", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def sides(left, inner, state, dt_rank, conv, mlp=None):
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": left, "right": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}}}


def config(width, vocab, streams, eps, scale, layers):
    return {"architecture": "Lotinex", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": layers}


MODELS = {
    # every mixer; a layer that reads another's keys over chunks twice and a half as long; no feed-forward once
    "A": config(72, 151, 3, 1e-5, 3.0, [
        attention(4, 2, 16, 24, 0.4, size=12, rot=8, mlp=dense(40)),
        sides(softmax(6, 3, 10, 14, 0.5, size=9, rot=10, scaling=YARN, softcap=3.0, conv=3), 56, 6, 5, 4, mlp=moe(5, 2, 24)),
        attention(8, 2, 16, 24, 0.3, size=30, rot=8, kv_from=0, mlp=moe(7, 1, 16)),
        delta(4, 2, 12, 18, 3)]),
    # one copy of the stream; no windows, no chunks, no cap, no rotation; one tap; chunks of one token
    "B": config(64, 97, 1, 1e-6, 0.5, [
        sides(softmax(3, 1, 8, 8, 0.6), 24, 16, 1, 1, mlp=dense(33)),
        attention(2, 2, 24, 10, 0.7), delta(1, 1, 32, 6, 1, mlp=moe(3, 3, 20)),
        attention(4, 2, 24, 10, 0.2, kv_from=1), attention(2, 1, 8, 8, 0.5, size=1, rot=2)]),
    # four copies; two layers that read the same keys, one nearer and one farther than their owner; wide scan
    "C": config(96, 200, 4, 1e-4, 8.0, [
        delta(6, 3, 9, 20, 4, mlp=dense(64)), attention(3, 3, 32, 16, 0.2, size=20, rot=32, mlp=dense(24)),
        attention(6, 3, 32, 16, 0.25, size=10, rot=32, kv_from=1), sides(
            softmax(2, 1, 32, 32, 0.3, size=40, rot=6, softcap=20.0, conv=5), 80, 24, 7, 2, mlp=moe(9, 4, 40)),
        attention(9, 3, 32, 16, 0.2, rot=32, kv_from=1, mlp=moe(4, 1, 8))]),
    # five copies; a state of seventy places a channel; no pages but the window's of two tokens
    "D": config(40, 61, 5, 1e-5, 1.0, [
        sides(softmax(1, 1, 6, 4, 1.0, size=2, rot=4, conv=2), 10, 70, 3, 3), delta(2, 1, 1, 1, 2, mlp=dense(24))]),
    # no attention at all: states and not one page; ten copies; wide key channels
    "E": config(136, 83, 10, 1e-5, 11.0, [
        delta(2, 2, 72, 5, 4, mlp=dense(16)), delta(5, 5, 16, 16, 2, mlp=moe(6, 2, 12)), delta(2, 1, 72, 5, 4)]),
    # the widest: heads as the matrix-core attention takes them, enough rows for every product kernel
    "F": config(256, 300, 2, 1e-5, 16.0, [
        delta(8, 4, 64, 48, 4, mlp=dense(512)),
        sides(softmax(8, 2, 64, 32, 0.125, size=100, rot=32, scaling=YARN, softcap=30.0, conv=4), 512, 40, 40, 4,
              mlp=moe(12, 2, 96)),
        attention(8, 4, 32, 32, 0.3, size=150, rot=32, mlp=dense(288)),
        attention(4, 4, 32, 32, 0.3, size=170, rot=32, kv_from=2, mlp=moe(8, 1, 160))]),
}


def tensor_shapes(cfg):
    """{name: shape} of every tensor a checkpoint of ``cfg`` holds (written from the design)."""
    w, s = cfg["width"], cfg["streams"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "final.norm.b": (w,)}

    def link(p, n):
        out.update({f"{p}norm{n}": (w,), f"{p}norm{n}.b": (w,), f"{p}hc{n}.in": (s,), f"{p}hc{n}.out": (s,),
                    f"{p}hc{n}.mix": (s, s)})

    def heads(x, m, norm):
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.update({x + "q": (H * D, w), x + "o": (w, H * Dv), x + "q.norm": (D if norm == "head" else H * D,)})
        if m.get("kv_from") is None:
            out.update({x + "k": (G * D, w), x + "v": (G * Dv, w), x + "k.norm": (D if norm == "head" else G * D,)})
        if m.get("conv"):
            out.update({x + "q.conv": (H * D, m["conv"]), x + "k.conv": (G * D, m["conv"]), x + "v.conv": (G * Dv, m["conv"])})
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        x = p + "mix."
        link(p, 1)
        if layer["type"] == "attention":
            heads(x, m, "head")
        elif layer["type"] == "delta":
            H, G, D, Dv, n = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            out.update({x + "q": (G * D, w), x + "q.conv": (G * D, n), x + "k": (G * D, w), x + "k.conv": (G * D, n),
                        x + "v": (H * Dv, w), x + "v.conv": (H * Dv, n), x + "b": (H, w), x + "a": (H, w),
                        x + "A_log": (H,), x + "dt_bias": (H,), x + "norm": (Dv,), x + "g": (H * Dv, w), x + "o": (w, H * Dv)})
        else:
            heads(x + "left.", m["left"], "all")
            r = m["right"]
            C, N, R = r["inner"], r["state"], r["dt_rank"]
            y = x + "right."
            out.update({y + "in": (2 * C, w), y + "conv": (C, r["conv"]), y + "conv.b": (C,), y + "x": (R + 2 * N, C),
                        y + "dt": (C, R), y + "dt.b": (C,), y + "A_log": (C, N), y + "D": (C,), y + "o": (w, C),
                        x + "left.out": (w,), x + "right.out": (w,)})
        c = layer["mlp"]
        if c is None:
            continue
        link(p, 2)
        if c["kind"] == "dense":
            out.update({p + "mlp.gate": (c["ff"], w), p + "mlp.up": (c["ff"], w), p + "mlp.down": (w, c["ff"])})
        else:
            f = c["expert"]["ff"]
            out[p + "mlp.router"] = (c["router"]["experts"], w)
            for e in range(c["router"]["experts"]):
                q = f"{p}mlp.e{e}."
                out.update({q + "gate": (f, w), q + "up": (f, w), q + "down": (w, f)})
    return out


def make_weights(cfg, seed):
    """Values that are exact in bfloat16, as float32 tensors."""
    g = torch.Generator().manual_seed(seed)
    s = cfg["streams"]

    def normal(shape, std=1.0, mean=0.0):
        return mean + std * torch.randn(shape, generator=g)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if name.endswith((".norm1.b", ".norm2.b", "final.norm.b")):
            t = normal(shape, 0.3)
        elif name == "embed":
            t = normal(shape)
        elif name.endswith((".in", ".out", ".mix")) and ".hc" in name:
            if last == "mix":
                t = 0.8 * torch.eye(s) + normal(shape, 0.3 / s)
            else:
                t = normal(shape, 0.4, 1.0) / (s if last == "in" else 1)
        elif last in ("norm", "norm1", "norm2", "out"):
            t = normal(shape, 0.25, 1.0)
        elif last == "A_log":
            t = normal(shape, 0.8, -0.5)
        elif last == "dt_bias" or name.endswith("dt.b"):
            t = normal(shape, 1.0, -1.0)
        elif last == "conv":
            t = normal(shape, 0.6)
        elif last in ("D", "b"):
            t = normal(shape, shape[-1] ** -0.5 if len(shape) == 2 else 1.0)
        else:
            t = normal(shape, (1.5 if last in ("q", "k", "dt") else 1.0) * shape[-1] ** -0.5)
        out[name] = t.to(torch.bfloat16).float()
    return out


def write_folder(tmp_path, cfg, seed, tag, weights=None):
    """(folder, weights): config.json and model.safetensors in bfloat16."""
    folder = os.path.join(str(tmp_path), f"lotinex_{tag}")
    os.makedirs(folder, exist_ok=True)
    weights = weights if weights is not None else make_weights(cfg, seed)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(folder, "model.safetensors"),
                      {n: t.to(torch.bfloat16) for n, t in weights.items()})
    return folder, weights


def make_requests(vocab, lengths, seed, avoid=()):
    rng = random.Random(seed)
    ids = [t for t in range(vocab) if t not in avoid]
    return {f"r{i}": [rng.choice(ids) for _ in range(n)] for i, n in enumerate(lengths)}


def reference(cfg, weights, requests):
    return {rid: plain.forward(cfg, weights, toks).float().numpy() for rid, toks in requests.items()}


def float32_bar(cfg, weights, requests, ref):
    """The bar for float32 logits: 1e-4 of the logits' range, or three times what the plain
    implementation itself loses when it runs in float32 where that is more."""
    plain.F = torch.float32
    try:
        lost = max(float(np.abs(plain.forward(cfg, weights, toks).double().numpy() - ref[rid]).max())
                   for rid, toks in requests.items())
    finally:
        plain.F = torch.float64
    return max(1e-4 * max(1.0, max(float(np.abs(r).max()) for r in ref.values())), 3.0 * lost)


MARK, WINDOW, CHUNK = 7, 48, 40
MARKED_KINDS = ("chunk", "shared", "window", "delta", "scan")


def marked_token_model(kind):
    """(config, weights) of a model in which one marked token decides every logit of a token that sees it.
    chunk, shared, window: every query points at the key that only the token MARK makes (shared: the keys are
    those of a layer with chunks a third as long, whose own output is nothing); delta, scan: every token
    keeps all the state has and only MARK writes."""
    if kind == "delta":
        layers = [delta(2, 1, 12, 20, 2)]
    elif kind == "chunk":
        layers = [attention(2, 1, 16, 16, 6.0, size=CHUNK)]
    elif kind == "shared":
        layers = [attention(2, 1, 16, 16, 6.0, size=CHUNK), attention(4, 1, 16, 16, 6.0, size=3 * CHUNK, kv_from=0)]
    else:
        layers = [sides(softmax(2, 1, 16, 16, 6.0, size=WINDOW, conv=2), 32, 12, 4, 2)]
    cfg = config(56, 120, 2, 1e-5, 2.0, layers)
    w = make_weights(cfg, 21)
    w["embed"][:, 0] = 0.0
    w["embed"][MARK, 0] = 8.0                        # only the marked token has anything in channel 0
    w["embed"][:, 1] = 2.0                           # channel 1 is the same for all tokens
    for n in w:
        if n.endswith((".norm1", ".norm2")):
            w[n][:2] = 1.0
        if n.endswith((".norm1.b", ".norm2.b")):
            w[n][:2] = 0.0
        if n.endswith("hc1.in") or n.endswith("hc1.out"):
            w[n][:] = 0.5
    if kind in ("chunk", "shared", "window"):
        p = "l0.mix.left." if kind == "window" else "l0.mix."
        w[p + "k"][15] = 0.0
        w[p + "k"][15, 0] = 4.0                      # channel 15 of the one kv head
        w[p + "k"][:15, 0] = 0.5
        for x in [p] + (["l1.mix."] if kind == "shared" else []):
            w[x + "q"][:, :] *= 0.1
            w[x + "q"][15::16] = 0.0
            w[x + "q"][15::16, 1] = 3.0              # every query head asks for channel 15
            w[x + "q.norm"][:] = 1.0
        w[p + "k.norm"][:] = 1.0
        w[p + "v"][:, 0] += 1.0
        if kind == "shared":
            w["l0.mix.o"][:] = 0.0
        if kind == "window":
            for x in ("q", "k", "v"):
                w[p + x + ".conv"][:] = torch.tensor([0.0, 1.0])         # (the mark stays with its own token)
            w["l0.mix.right.out"][:] = 0.0
    elif kind == "delta":
        p = "l0.mix."
        w[p + "A_log"][:] = -12.0                    # nothing fades
        w[p + "b"][:] = 0.0
        w[p + "b"][:, 1] = -12.0                     # hardly anything is written
        w[p + "b"][:, 0] = 8.0                       # but by the marked token
        for x in ("q", "k", "v"):
            w[p + x + ".conv"][:] = torch.tensor([0.0, 1.0])
        w[p + "q"][:, 1] = 2.0
        w[p + "k"][:, 0] = 2.0
        w[p + "v"][:, 0] = 1.0
    else:
        p = "l0.mix.right."
        w["l0.mix.left.out"][:] = 0.0
        w[p + "A_log"][:] = -9.0
        w[p + "D"][:] = 0.0
        w[p + "conv"][:] = torch.tensor([0.0, 1.0])
        w[p + "dt.b"][:] = -14.0
        w[p + "in"][:32, 0] = 1.0                    # the mark's x is large in every channel
        w[p + "in"][0] = 0.0
        w[p + "in"][0, 0] = 3.0                      # channel 0 is the mark alone
        w[p + "conv.b"][0] = 0.0
        w[p + "x"][:4] = 0.0
        w[p + "x"][:4, 0] = 1.0                      # and opens every channel's step
        w[p + "dt"][:] = w[p + "dt"].abs() + 0.5
        w[p + "x"][16:] *= 0.1
        w[p + "conv.b"][1] = 4.0                     # channel 1 is the same for all: what C reads
        w[p + "x"][16:, 1] = 1.0
    return cfg, {n: t.to(torch.bfloat16).float() for n, t in w.items()}


def marked_reach(kind, place):
    """The last token that sees the mark (None: all do)."""
    return {"chunk": place // CHUNK * CHUNK + CHUNK - 1, "shared": place // (3 * CHUNK) * 3 * CHUNK + 3 * CHUNK - 1,
            "window": place + WINDOW - 1, "delta": None, "scan": None}[kind]
