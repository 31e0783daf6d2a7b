"""Kelutar without a GPU: configuration and registry, declared tensors against a written checkpoint,
cache needs and the run list of borrowed layers, the plain implementation's own mechanisms against
second closed forms, and the engine's host side (pages, state slots, run list, batching, replay)
over the kernel calls emulated in torch."""
import copy
import json
import math

import numpy as np
import pytest
import torch

import plain_kelutar as plain
import replay_schedules as rs
from emulated_ops import EmulatedOps
from kelutar_models import (MARK, MARKED_KINDS, MODELS, float32_bar, make_requests, make_weights, marked_reach,
                            marked_token_model, reference, tensor_shapes, write_folder)
from replay_harness import compare, replay_in_process
from servelab_amd import ConfigError, load_config
from servelab_amd.config import KelutarConfig, resolve_architecture
from servelab_amd.parts import PagedKVSpec, StateSpec
from servelab_amd.parts.model import build_model_spec
from servelab_amd.weights.loader import Checkpoint, check_tensors

F = torch.float64


# ------------------------------------------------------------------ configuration
@pytest.mark.parametrize("which", sorted(MODELS))
def test_config_round_trip_and_declared_tensors(tmp_path, which):
    cfg = MODELS[which]
    folder, _ = write_folder(tmp_path, cfg, seed=1, tag=which)
    assert resolve_architecture(json.load(open(folder + "/config.json"))).name == "Kelutar"
    config = load_config(folder)
    assert isinstance(config, KelutarConfig)
    again = KelutarConfig.from_hf(config.to_hf())
    assert again.layers == config.layers and again.to_hf() == config.to_hf()
    assert (again.embedding_scale, again.taps, again.max_positions) == \
        (cfg["embedding"]["scale"], cfg["canon"]["taps"], cfg["max_positions"])
    spec = build_model_spec(config)
    check_tensors({n: s.shape for n, s in spec.param_specs().items()}, Checkpoint(folder).shapes())
    assert {n: tuple(s.shape) for n, s in spec.param_specs().items()} == tensor_shapes(cfg)
    assert spec.max_position_embeddings == cfg["max_positions"] and spec.graph_safe


def test_missing_and_impossible_keys_name_themselves():
    base = MODELS["A"]
    for path, text in ((("width",), "width"), (("norm",), "norm"), (("embedding",), "embedding"),
                       (("max_positions",), "max_positions"), (("canon", "taps"), "taps"),
                       (("layers", 1, "mixer", "kv_heads"), "kv_heads"), (("layers", 1, "mixer", "scale"), "scale"),
                       (("layers", 0, "mixer", "vdim"), "vdim"), (("layers", 1, "mlp", "ff"), "ff"),
                       (("layers", 0, "type"), "type")):
        cfg = copy.deepcopy(base)
        node = cfg
        for k in path[:-1]:
            node = node[k]
        del node[path[-1]]
        with pytest.raises(ConfigError, match=text):
            KelutarConfig.from_hf(cfg)
    for change, text in ((lambda c: c["layers"][0].update(type="rnn"), "attention, hgrn2"),
                         (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "kv_heads"),
                         (lambda c: c["layers"][1]["mixer"].update(vdim=8), "vdim"),
                         (lambda c: c["layers"][1]["mlp"].update(kind="moe"), "dense"),
                         (lambda c: c["layers"][3].update(weights_of=3), "weights_of"),
                         (lambda c: c["layers"][3]["mixer"].update(scale=0.5), "describes another layer"),
                         (lambda c: c["canon"].update(taps=99), "taps")):
        cfg = copy.deepcopy(base)
        change(cfg)
        with pytest.raises(ConfigError, match=text):
            KelutarConfig.from_hf(cfg)


def test_keys_that_may_be_absent():
    """No mask: every earlier key; no convolution: blocks that read the stream itself; a borrowing entry
    takes what it leaves out from the layer it borrows from."""
    cfg = copy.deepcopy(MODELS["A"])
    cfg["layers"][1]["mixer"].pop("mask")
    cfg["layers"][3] = {"weights_of": 1}
    cfg.pop("canon")
    config = KelutarConfig.from_hf(cfg)
    assert config.layers[1].mixer.window == 0 and config.layers[3].mixer == config.layers[1].mixer and config.taps == 0
    spec = build_model_spec(config)
    assert not any("canon" in n for n in spec.param_specs())
    assert len(spec.stream_specs()) == 5


def test_cache_needs_and_the_run_list_of_borrowed_layers():
    spec = build_model_spec(KelutarConfig.from_hf(MODELS["A"]))
    assert [c.layer for c in spec.run] == [0, 1, 2, 1, 0] and len(spec.layers) == 3
    streams = spec.stream_specs()
    assert len(streams) == 10                            # every call keeps the convolution's inputs and its mixer's
    assert all(streams[2 * i] == StateSpec((2 * 72,), "float32") for i in range(5))
    assert streams[1] == streams[9] == StateSpec((3 * 10 * 14,), "float32")
    assert streams[3] == streams[7] == PagedKVSpec(2, 16, 9, value_dim=16)
    # one tap keeps nothing; a chain of borrowed layers ends at the one that owns its tensors
    one = build_model_spec(KelutarConfig.from_hf(MODELS["D"]))
    assert [type(s) for s in one.stream_specs().values()] == [PagedKVSpec, StateSpec, PagedKVSpec]
    assert [c.layer for c in build_model_spec(KelutarConfig.from_hf(MODELS["C"])).run] == [0, 1, 0, 0]


def test_without_a_convolution_the_blocks_read_the_stream(tmp_path):
    """Taps of zero and no taps are the same function; the second runs the blocks without a convolution."""
    cfg = copy.deepcopy(MODELS["A"])
    weights = make_weights(cfg, 3)
    for n in list(weights):
        if n.endswith("canon1"):
            weights[n] = torch.zeros_like(weights[n])
    requests = make_requests(cfg["vocab"], [19, 2], seed=1)
    ref = reference(cfg, weights, requests)
    bar = float32_bar(cfg, weights, requests, ref)
    cfg.pop("canon")
    folder, _ = write_folder(tmp_path, cfg, 3, "plain", {n: t for n, t in weights.items() if not n.endswith("canon1")})
    steps = rs.portions(requests, sizes=(5, 2, 1))
    out = str(tmp_path / "out")
    replay_in_process(folder, steps, out, "float32", rs.max_tokens_needed(steps), ops=EmulatedOps(torch.float32),
                      device="cpu", max_live=2)
    assert compare(out, steps, ref, cfg["vocab"])[0] < bar


# ------------------------------------------------------------------ the plain mechanisms
def test_plain_stream_convolution_is_a_sum_over_taps():
    g = torch.Generator().manual_seed(1)
    x, taps = torch.randn(7, 3, generator=g, dtype=F), torch.randn(3, 4, generator=g, dtype=F)
    got = plain.stream_convolution(x, taps)
    for t in range(7):
        want = x[t] + sum(taps[:, j] * x[t - 3 + j] for j in range(4) if t - 3 + j >= 0)
        assert torch.allclose(got[t], want, atol=1e-12)
    assert torch.allclose(plain.stream_convolution(x, taps[:, :1]), x * (1 + taps[:, 0]), atol=1e-12)


def test_plain_window_sees_itself_and_size_minus_one_before():
    seen = plain.visible(6, 3)
    assert seen[5].tolist() == [False, False, False, True, True, True]
    assert seen[1].tolist() == [True, True, False, False, False, False]
    assert plain.visible(4, None)[3].tolist() == [True] * 4 and plain.visible(4, 1)[3].tolist() == [False] * 3 + [True]


def test_plain_embedding_scales_the_token_and_not_the_position():
    w = {"embed": torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=F), "pos": torch.tensor([[0.5, 0], [0, 0.5]], dtype=F)}
    got = plain.embed({"embedding": {"scale": 10.0}}, w, [1, 0])
    assert got.tolist() == [[30.5, 40.0], [10.0, 20.5]]


def attention_weights(g, H, G, D, width):
    shapes = {"q": (H * D, width), "q.b": (H * D,), "k": (G * D, width), "k.b": (G * D,), "q.norm": (D,), "k.norm": (D,),
              "temp": (H,), "g": (H * D, width), "o": (width, H * D)}
    return {n: torch.randn(s, generator=g, dtype=F) for n, s in shapes.items()}


def test_plain_attention_with_one_token_returns_its_gated_key():
    g = torch.Generator().manual_seed(2)
    w = attention_weights(g, 2, 1, 4, 6)
    m = {"heads": 2, "kv_heads": 1, "dim": 4, "scale": 0.3}
    h = torch.randn(1, 6, generator=g, dtype=F)
    key = h @ w["k"].T + w["k.b"]
    want = (key.repeat(1, 2) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T
    assert torch.allclose(plain.attention(h, m, w, "", 1e-5), want, atol=1e-12)


def test_plain_attention_head_by_head():
    g = torch.Generator().manual_seed(3)
    H, G, D, T = 4, 2, 3, 6
    w = attention_weights(g, H, G, D, 5)
    m = {"heads": H, "kv_heads": G, "dim": D, "scale": 0.6, "mask": {"size": 2}}
    h = torch.randn(T, 5, generator=g, dtype=F)
    got = plain.attention(h, m, w, "", 1e-5)
    out = torch.zeros(T, H * D, dtype=F)
    for hd in range(H):
        kv = hd // 2
        q = (h @ w["q"].T + w["q.b"])[:, hd * D:hd * D + D]
        k = (h @ w["k"].T + w["k.b"])[:, kv * D:kv * D + D]
        qn = q / (q.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * w["q.norm"]
        kn = k / (k.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * w["k.norm"]
        for i in range(T):
            js = [j for j in range(T) if 0 <= i - j < 2]
            e = torch.tensor([math.exp(float(qn[i] @ kn[j]) * 0.6 * float(w["temp"][hd])) for j in js], dtype=F)
            out[i, hd * D:hd * D + D] = sum(a * k[j] for a, j in zip(e / e.sum(), js))
    want = (out * torch.sigmoid(h @ w["g"].T)) @ w["o"].T
    assert torch.allclose(got, want, atol=1e-10)


def test_plain_hgrn2_as_a_sum_over_what_was_written():
    """o_t = sum_j (prod_(j < i <= t) f_i) (1 - f_j) q_t v_j, channel by channel."""
    g = torch.Generator().manual_seed(4)
    H, D, Dv, T = 2, 3, 4, 5
    w = {n: torch.randn(s, generator=g, dtype=F) for n, s in
         {"q": (H * D, 6), "f": (H * D, 6), "f.b": (H * D,), "v": (H * Dv, 6), "norm": (Dv,), "o": (6, H * Dv)}.items()}
    w["lower"] = torch.rand(H * D, generator=g, dtype=F)
    h = torch.randn(T, 6, generator=g, dtype=F)
    got = plain.hgrn2(h, {"heads": H, "dim": D, "vdim": Dv}, w, "", 1e-5)
    q = torch.nn.functional.silu(h @ w["q"].T).view(T, H, D)
    f = (w["lower"] + (1 - w["lower"]) * torch.sigmoid(h @ w["f"].T + w["f.b"])).view(T, H, D)
    v = (h @ w["v"].T).view(T, H, Dv)
    out = torch.zeros(T, H, Dv, dtype=F)
    for t in range(T):
        for j in range(t + 1):
            kept = f[j + 1:t + 1].prod(0) * (1 - f[j])                    # [H, D]
            out[t] += (q[t] * kept).sum(-1, keepdim=True) * v[j]
    out = out / (out.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * w["norm"]
    assert torch.allclose(got, out.reshape(T, -1) @ w["o"].T, atol=1e-10)
    assert torch.allclose(plain.forget_gate(torch.tensor([-60.0, 60.0], dtype=F), torch.tensor([0.3, 0.3], dtype=F)),
                          torch.tensor([0.3, 1.0], dtype=F))


def test_plain_borrowed_layers_run_the_owners_tensors():
    cfg = MODELS["C"]
    weights = make_weights(cfg, 3)
    toks = [5, 9, 100, 3, 77, 8]
    trace = []
    plain.forward(cfg, weights, toks, trace)
    w = {n: t.to(F) for n, t in weights.items()}
    x = trace[2]
    h = plain.stream_convolution(x, w["l0.canon1"])
    x = x + plain.rms_norm(plain.hgrn2(h, cfg["layers"][0]["mixer"], w, "l0.mix.", 1e-4), w["l0.norm1"], 1e-4)
    up = torch.relu(x @ w["l0.mlp.up"].T)
    x = x + plain.rms_norm((up * up) @ w["l0.mlp.down"].T, w["l0.norm2"], 1e-4)
    assert torch.allclose(x, trace[3], atol=1e-10)


@pytest.mark.parametrize("kind", MARKED_KINDS)
def test_the_marked_token_matters_exactly_where_it_is_seen(kind):
    cfg, weights = marked_token_model(kind)
    place = 64
    toks = make_requests(cfg["vocab"], [300], seed=8, avoid=(MARK,))["r0"]
    toks[place] = MARK
    other = list(toks)
    other[place] = MARK + 1
    d = (plain.forward(cfg, weights, toks) - plain.forward(cfg, weights, other)).abs().max(-1).values
    last = marked_reach(kind, place)
    assert float(d[:place].max()) == 0.0
    if last is None:
        assert float(d[place:].min()) > 0.3, float(d[place:].min())
    else:
        assert float(d[place:last + 1].min()) > 0.3, float(d[place:last + 1].min())
        assert float(d[last + 1:].max()) == 0.0


# ------------------------------------------------------------------ the engine's host side
@pytest.mark.parametrize("which", sorted(set(MODELS) - {"F"}))
@pytest.mark.parametrize("schedule", ["whole", "tail", "portions", "twos", "mixed"])
def test_every_way_of_cutting_gives_the_plain_logits(tmp_path, which, schedule):
    cfg = MODELS[which]
    folder, weights = write_folder(tmp_path, cfg, seed=11, tag=which)
    requests = make_requests(cfg["vocab"], [37, 1, 2, 49, 5, 26], seed=5)
    ref = reference(cfg, weights, requests)
    steps = {"whole": lambda: rs.whole(requests), "tail": lambda: rs.tail_decoded(requests, tail=12),
             "portions": lambda: rs.portions(requests),
             "twos": lambda: rs.portions(requests, sizes=(2, 2, 3, 2, 17, 2)),
             "mixed": lambda: rs.mixed(requests, {r: max(1, len(t) - 8) for r, t in requests.items()},
                                       max_live=3, seed=2)}[schedule]()
    out = str(tmp_path / "out")
    replay_in_process(folder, steps, out, "float32", rs.max_tokens_needed(steps),
                      ops=EmulatedOps(torch.float32), device="cpu", max_live=3)
    worst, where = compare(out, steps, ref, cfg["vocab"])
    bar = float32_bar(cfg, weights, requests, ref)
    assert worst < bar, f"max abs err {worst} at {where}, bar {bar}"


def test_slots_and_pages_that_held_another_request_start_afresh(tmp_path):
    """Two slots, seven requests: every slot and page serves several requests, and what the last one
    left there (last stream rows, memories, keys) must not reach the next."""
    cfg = MODELS["A"]
    folder, weights = write_folder(tmp_path, cfg, seed=12, tag="A")
    requests = make_requests(cfg["vocab"], [20, 3, 31, 1, 12, 2, 25], seed=6)
    ref = reference(cfg, weights, requests)
    steps = rs.mixed(requests, {r: len(t) // 2 for r, t in requests.items()}, max_live=2, seed=4, max_portion=7)
    out = str(tmp_path / "out")
    replay_in_process(folder, steps, out, "float32", rs.max_tokens_needed(steps), ops=EmulatedOps(torch.float32),
                      device="cpu", max_live=2)
    worst, where = compare(out, steps, ref, cfg["vocab"])
    assert worst < float32_bar(cfg, weights, requests, ref), f"max abs err {worst} at {where}"


def test_a_sequence_as_long_as_the_table_of_positions_and_no_longer(tmp_path):
    cfg = dict(MODELS["D"], max_positions=24)
    folder, weights = write_folder(tmp_path, cfg, seed=2, tag="short")
    requests = make_requests(cfg["vocab"], [24], seed=3)
    ref = reference(cfg, weights, requests)
    steps = rs.tail_decoded(requests, tail=6)
    out = str(tmp_path / "out")
    replay_in_process(folder, steps, out, "float32", 64, ops=EmulatedOps(torch.float32), device="cpu", max_live=1)
    assert compare(out, steps, ref, cfg["vocab"])[0] < float32_bar(cfg, weights, requests, ref)
    with pytest.raises(ValueError, match="exceed"):
        replay_in_process(folder, [{"step": 0, "entries": [{"id": "x", "tokens": [1] * 25, "want": []}], "end": []}],
                          out, "float32", 64, ops=EmulatedOps(torch.float32), device="cpu", max_live=1)
    assert np.isfinite(ref["r0"]).all()
