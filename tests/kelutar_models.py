"""Small Kelutar configurations and weights for the tests, and what the tests hold them to.  The
configurations differ from each other in every size, in the order of their layers and in which
options they use; the weights are drawn so that every mechanism matters (lower bounds over their
whole range, gates that open and close, factors per head that differ and change sign, convolutions
as large as the stream they read)."""
import json
import os
import random

import numpy as np
import torch

import plain_kelutar as plain
from servelab_amd.weights.safetensors_io import write_safetensors


def attention(heads, kv_heads, dim, scale, ff=None, window=None, borrows=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    return entry("attention", m, ff, borrows)


def hgrn2(heads, dim, vdim, ff=None, borrows=None):
    return entry("hgrn2", {"heads": heads, "dim": dim, "vdim": vdim}, ff, borrows)


def entry(kind, mixer, ff, borrows):
    out = {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}
    if borrows is not None:
        out["weights_of"] = borrows
    return out


def config(width, vocab, positions, eps, scale, taps, layers):
    return {"architecture": "Kelutar", "width": width, "vocab": vocab, "max_positions": positions,
            "norm": {"eps": eps}, "embedding": {"scale": scale}, "canon": {"taps": taps}, "layers": layers}


MODELS = {
    # both mixers with and without a feed-forward, layers that run others' tensors, three taps
    "A": config(72, 151, 260, 1e-5, 3.0, 3, [
        hgrn2(3, 10, 14), attention(4, 2, 16, 0.4, ff=40, window=9), hgrn2(2, 24, 8, ff=56),
        attention(4, 2, 16, 0.4, ff=40, window=9, borrows=1), hgrn2(3, 10, 14, borrows=0)]),
    # an attention over every earlier key ahead of everything, one kv head, five taps
    "B": config(64, 97, 130, 1e-6, 0.5, 5, [
        attention(6, 1, 10, 0.25), hgrn2(1, 32, 6, ff=33), attention(2, 2, 24, 0.7, window=30)]),
    # two taps; a chain of borrowed layers; key channels that are no multiple of anything
    "C": config(96, 200, 400, 1e-4, 8.0, 2, [
        hgrn2(4, 9, 20, ff=64), attention(3, 3, 32, 0.2, window=33), hgrn2(4, 9, 20, ff=64, borrows=0),
        hgrn2(4, 9, 20, ff=64, borrows=2)]),
    # one tap (a factor per channel, nothing kept), windows of two tokens and of one, a scale of 1
    "D": config(40, 61, 128, 1e-5, 1.0, 1, [
        attention(1, 1, 6, 1.0, ff=24, window=2), hgrn2(1, 1, 1), attention(2, 1, 8, 0.5, window=1)]),
    # no attention at all: states and not one page; wide key channels; four taps
    "E": config(136, 83, 140, 1e-5, 11.0, 4, [
        hgrn2(2, 72, 5, ff=16), hgrn2(5, 16, 16), hgrn2(2, 72, 5, ff=16, borrows=0)]),
    # the widest: heads as the matrix-core attention takes them, enough rows for every product kernel
    "F": config(256, 300, 700, 1e-5, 16.0, 4, [
        attention(8, 2, 64, 0.125, ff=512, window=100), hgrn2(4, 64, 96), hgrn2(8, 40, 32, ff=288),
        attention(4, 4, 32, 0.3, ff=160)]),
}


def tensor_shapes(cfg):
    """{name: shape} of every tensor a checkpoint of ``cfg`` holds (written from the design)."""
    w, taps = cfg["width"], cfg["canon"]["taps"]
    out = {"embed": (cfg["vocab"], w), "pos": (cfg["max_positions"], w), "final.norm": (w,), "head": (cfg["vocab"], w)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", layer["mixer"]
        x, H, D = p + "mix.", m["heads"], m["dim"]
        out.update({p + "norm1": (w,), p + "canon1": (w, taps)})
        if layer["type"] == "attention":
            G = m["kv_heads"]
            out.update({x + "q": (H * D, w), x + "q.b": (H * D,), x + "k": (G * D, w), x + "k.b": (G * D,),
                        x + "q.norm": (D,), x + "k.norm": (D,), x + "temp": (H,), x + "g": (H * D, w), x + "o": (w, H * D)})
        else:
            Dv = m["vdim"]
            out.update({x + "q": (H * D, w), x + "f": (H * D, w), x + "f.b": (H * D,), x + "lower": (H * D,),
                        x + "v": (H * Dv, w), x + "norm": (Dv,), x + "o": (w, H * Dv)})
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out.update({p + "norm2": (w,), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    return out


def make_weights(cfg, seed):
    """Values that are exact in bfloat16, as float32 tensors."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.25 * torch.randn(shape, generator=g)
        elif last == "temp":
            t = torch.randn(shape, generator=g) + 1.0
        elif last == "lower":
            t = 0.95 * torch.rand(shape, generator=g)
        elif last == "b":
            t = torch.randn(shape, generator=g) + (1.5 if name.endswith("f.b") else 0.0)
        elif last == "canon1":
            t = 0.5 * torch.randn(shape, generator=g)
        elif last in ("embed", "pos"):
            t = torch.randn(shape, generator=g)
        else:
            t = torch.randn(shape, generator=g) * (1.5 if last in ("q", "k", "f") else 1.0) * shape[-1] ** -0.5
            if last in ("q", "k", "v", "f", "g", "up"):
                # (the rows they read grow with the embedding's scale and the layers' outputs)
                t = t / max(1.0, cfg["embedding"]["scale"]) ** 0.5
        out[name] = t.to(torch.bfloat16).float()
    return out


def write_folder(tmp_path, cfg, seed, tag, weights=None):
    """(folder, weights): config.json and model.safetensors in bfloat16."""
    folder = os.path.join(str(tmp_path), f"kelutar_{tag}")
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


MARK, WINDOW = 7, 48
MARKED_KINDS = ("attention", "attention_w", "hgrn2", "conv")


def marked_token_model(kind):
    """(config, weights) of one layer in which one marked token decides every logit of a token that sees
    it: (attention, attention_w) every query points at the key that only the token MARK makes; (hgrn2)
    every gate keeps all it has, only MARK's writes; (conv) a token sees MARK through the convolution's
    three earlier taps alone."""
    taps = 4
    if kind == "hgrn2":
        layer = hgrn2(2, 12, 20)
    else:
        layer = attention(2, 1, 16, 6.0, window={"attention": None, "attention_w": WINDOW, "conv": 1}[kind])
    cfg = config(56, 120, 320, 1e-5, 2.0, taps, [layer])
    w = make_weights(cfg, 21)
    p = "l0.mix."
    w["l0.norm1"][:] = 1.0
    w["embed"][:, 0] = 0.0
    w["embed"][MARK, 0] = 8.0                        # only the marked token has anything in channel 0
    w["embed"][:, 1] = 2.0                           # channel 1 is the same for all tokens
    w["pos"][:, :2] = 0.0
    if kind == "conv":
        w[p + "k"][:, 0] = 4.0                       # the values read channel 0
        w["l0.canon1"][0] = 1.0
    else:
        w["l0.canon1"][:2] = 0.0                     # (the mark stays with its own token)
    if kind == "attention_w":
        w["l0.canon1"][:] = 0.0                      # (and so does everything else of it: a sharp edge)
    if kind == "hgrn2":
        w[p + "f"][:] = 0.0
        w[p + "f.b"][:] = 12.0                       # open: kept as it is, hardly anything written
        w[p + "f"][5::12, 0] = -2.0                  # the marked token closes channel 5 of every head
        w[p + "lower"][:] = 0.0
        w[p + "q"][5::12] = 0.0
        w[p + "q"][5::12, 1] = 1.0                   # and every token reads it
        w[p + "v"][:, 0] = 1.0
    elif kind != "conv":
        w[p + "q.b"][:] = 0.0
        w[p + "k.b"][15] = 0.0
        w[p + "k"][15] = 0.0
        w[p + "k"][15, 0] = 4.0                      # channel 15 of the one kv head
        w[p + "k"][:15, 0] = 0.5
        w[p + "q"][:, :] *= 0.1
        w[p + "q"][15::16] = 0.0
        w[p + "q"][15::16, 1] = 3.0                  # every query head asks for channel 15
        w[p + "q.norm"][:] = 1.0
        w[p + "k.norm"][:] = 1.0
        w[p + "temp"][:] = 1.0
    return cfg, {n: t.to(torch.bfloat16).float() for n, t in w.items()}


def marked_reach(kind, place):
    """The last token that sees the mark (None: all do)."""
    return {"attention": None, "attention_w": place + WINDOW - 1, "hgrn2": None, "conv": place + 3}[kind]
