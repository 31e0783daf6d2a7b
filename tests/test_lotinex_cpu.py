"""Lotinex without a GPU: configuration and registry, declared tensors against a written checkpoint,
cache needs (chunks, pages that several layers read), the plain implementation's own mechanisms against
second closed forms, and the engine's host side (pages, state slots, run list, batching, replay) over the
kernel calls emulated in torch."""
import copy
import json
import math

import pytest
import torch

import plain_lotinex as plain
import replay_schedules as rs
from emulated_ops import EmulatedOps
from lotinex_models import (MARK, MARKED_KINDS, MODELS, YARN, float32_bar, make_requests, marked_reach, marked_token_model,
                            reference, tensor_shapes, write_folder)
from replay_harness import compare, replay_in_process
from servelab_amd import ConfigError, load_config
from servelab_amd.cache import CacheManager
from servelab_amd.config import LotinexConfig, resolve_architecture
from servelab_amd.parts import LayerNorm, PagedKVSpec, RMSNorm, Runtime, SideBySide, StateSpec
from servelab_amd.parts.model import LayerCall, build_model_spec
from servelab_amd.parts.norm import NormedDelta
from servelab_amd.weights.loader import Checkpoint, check_tensors

F = torch.float64


# ------------------------------------------------------------------ configuration
@pytest.mark.parametrize("which", sorted(MODELS))
def test_config_round_trip_and_declared_tensors(tmp_path, which):
    cfg = MODELS[which]
    folder, _ = write_folder(tmp_path, cfg, seed=1, tag=which)
    assert resolve_architecture(json.load(open(folder + "/config.json"))).name == "Lotinex"
    config = load_config(folder)
    assert isinstance(config, LotinexConfig)
    again = LotinexConfig.from_hf(config.to_hf())
    assert again.layers == config.layers and again.to_hf() == config.to_hf()
    assert (again.streams, again.embedding_scale, again.norm_eps) == (cfg["streams"], cfg["embedding"]["scale"], cfg["norm"]["eps"])
    spec = build_model_spec(config)
    check_tensors({n: s.shape for n, s in spec.param_specs().items()}, Checkpoint(folder).shapes())
    assert {n: tuple(s.shape) for n, s in spec.param_specs().items()} == tensor_shapes(cfg)
    assert spec.graph_safe


def test_missing_and_impossible_keys_name_themselves():
    base = MODELS["A"]
    for path, text in ((("width",), "width"), (("norm",), "norm"), (("embedding", "scale"), "scale"), (("streams",), "streams"),
                       (("layers", 0, "mixer", "kv_heads"), "kv_heads"), (("layers", 0, "mixer", "scale"), "scale"),
                       (("layers", 1, "mixer", "left"), "left"), (("layers", 1, "mixer", "right", "dt_rank"), "dt_rank"),
                       (("layers", 1, "mixer", "left", "rot", "base"), "base"), (("layers", 1, "mlp", "router", "top"), "top"),
                       (("layers", 1, "mlp", "expert"), "expert"), (("layers", 0, "mlp", "ff"), "ff"),
                       (("layers", 3, "mixer", "conv"), "conv"), (("layers", 0, "type"), "type")):
        cfg = copy.deepcopy(base)
        node = cfg
        for k in path[:-1]:
            node = node[k]
        del node[path[-1]]
        with pytest.raises(ConfigError, match=text):
            LotinexConfig.from_hf(cfg)
    for change, text in ((lambda c: c["layers"][0].update(type="rnn"), "attention, delta, parallel"),
                         (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"),
                         (lambda c: c["layers"][3]["mixer"].update(kv_heads=3), "kv_heads"),
                         (lambda c: c["layers"][1]["mlp"]["router"].update(top=6), "router.top"),
                         (lambda c: c["layers"][0]["mlp"].update(kind="gelu"), "dense, moe"),
                         (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "earlier attention"),
                         (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "earlier attention"),
                         (lambda c: c["layers"][2]["mixer"].update(vdim=16), "must be those of layer 0"),
                         (lambda c: c["layers"][2]["mixer"]["rot"].update(base=7.0), "must be those of layer 0"),
                         (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(scaling={"factor": 2.0, "original": 9, "low": 1, "high": 2}),
                          "fast"),
                         (lambda c: c.update(streams=0), "streams"), (lambda c: c.update(streams=17), "streams")):
        cfg = copy.deepcopy(base)
        change(cfg)
        with pytest.raises(ConfigError, match=text):
            LotinexConfig.from_hf(cfg)


def test_cache_needs_and_pages_that_several_layers_read():
    spec = build_model_spec(LotinexConfig.from_hf(MODELS["A"]))
    assert [(c.layer, c.streams, c.write) for c in spec.run] == \
        [(0, (0,), True), (1, (1, 2, 3), True), (2, (0,), False), (3, (4,), True)]
    streams = spec.stream_specs()
    # the owner's chunks of 12 and the reader's of 30 do not nest: the last 30 tokens serve both
    assert streams[0] == PagedKVSpec(2, 16, 30, value_dim=24)
    assert streams[1] == PagedKVSpec(3, 10, 9, value_dim=14)
    assert streams[2] == StateSpec((2 * (6 * 10 + 3 * 10 + 3 * 14),)) and streams[3] == StateSpec((56 * 6 + 3 * 56,))
    assert streams[4] == StateSpec((4 * 12 * 18 + 2 * (2 * 2 * 12 + 4 * 18),))
    # nested chunks keep the larger; one reader without chunks keeps every token
    f = copy.deepcopy(MODELS["F"])
    f["layers"][3]["mixer"]["mask"]["size"] = 300
    assert build_model_spec(LotinexConfig.from_hf(f)).stream_specs()[4] == PagedKVSpec(4, 32, value_dim=32, chunk=300)
    assert build_model_spec(LotinexConfig.from_hf(MODELS["C"])).stream_specs()[1] == PagedKVSpec(3, 32, value_dim=16)
    with pytest.raises(ValueError, match="different cache kind"):
        spec.run[2] = LayerCall(2, (1,), write=False)
        spec.stream_specs()


def test_pages_needed_by_a_chunk_and_by_two_needs_together():
    c = PagedKVSpec(1, 8, chunk=10)
    assert [c.first_needed(p) for p in (0, 9, 10, 19, 20)] == [0, 0, 10, 10, 20]
    both = PagedKVSpec(1, 8, window=4, chunk=10)
    assert [both.first_needed(p) for p in (0, 9, 10, 12, 19)] == [0, 6, 10, 10, 16]
    assert c.covering(PagedKVSpec(1, 8, chunk=30)) == PagedKVSpec(1, 8, chunk=30)
    assert c.covering(PagedKVSpec(1, 8, chunk=15, keep_first=3)) == PagedKVSpec(1, 8, window=15, keep_first=3)
    assert c.covering(PagedKVSpec(1, 8, window=25)) == PagedKVSpec(1, 8, window=25) == PagedKVSpec(1, 8, window=25).covering(c)
    assert both.covering(c) == PagedKVSpec(1, 8, window=10) and c.covering(PagedKVSpec(1, 8)) == PagedKVSpec(1, 8)
    assert c.covering(PagedKVSpec(1, 8, value_dim=4, chunk=10)) is None
    for a in (c, both, PagedKVSpec(1, 8, window=7), PagedKVSpec(1, 8, chunk=4)):
        for b in (c, both, PagedKVSpec(1, 8, window=7), PagedKVSpec(1, 8, chunk=4)):
            for p in range(50):
                assert a.covering(b).first_needed(p) <= min(a.first_needed(p), b.first_needed(p))


@pytest.mark.parametrize("page,chunk", [(16, 40), (16, 16), (32, 20), (16, 1)])
def test_a_chunk_group_holds_what_the_next_token_sees_and_no_page_more(page, chunk):
    m = CacheManager({0: PagedKVSpec(1, 8, chunk=chunk)}, 20, page, 2)
    m.open("r")
    done = 0
    for n in (3, 30, 1, 50, 1, 1, 1, 40, 7, 60):
        assert m.grow("r", done + n)
        done += n
        m.commit("r", done)
        m.check()
        held = [j for j, p in enumerate(m.block_table(0, "r")) if p >= 0]
        first = done // chunk * chunk // page
        assert held == list(range(first, -(-done // page))), (done, held)
    m.close("r")
    assert m.num_free_pages() == 20


# ------------------------------------------------------------------ the plain mechanisms
def test_plain_chunks_and_windows():
    seen = plain.sees_chunk(7, 3)
    assert [r.nonzero()[:, 0].tolist() for r in seen] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    assert [r.nonzero()[:, 0].tolist() for r in plain.sees_window(5, 2)] == [[0], [0, 1], [1, 2], [2, 3], [3, 4]]
    assert plain.sees_chunk(4, 0)[3].tolist() == [True] * 4 == plain.sees_window(4, 0)[3].tolist()


def test_plain_softmax_with_a_one_in_the_denominator():
    s = torch.tensor([[0.5, -2.0, 30.0], [-60.0, -70.0, 1.0]], dtype=F)
    seen = torch.tensor([[True, True, False], [True, True, False]])
    got = plain.softmax_plus_one(s, seen)
    for r in range(2):
        e = [math.exp(float(v)) for v in s[r, :2]]
        for j in range(2):
            assert abs(float(got[r, j]) - e[j] / (1 + sum(e))) <= 1e-15
    assert got[:, 2].tolist() == [0.0, 0.0]


def test_plain_blended_frequencies_at_their_ends():
    rot = {"base": 1000.0, "dims": 16, "scaling": dict(YARN)}
    f, mag = plain.frequencies(rot)
    base, _ = plain.frequencies({"base": 1000.0, "dims": 16})
    assert mag == 0.1 * math.log(YARN["factor"]) + 1.0 and f[0] == base[0]
    assert abs(f[-1] - base[-1] / YARN["factor"]) < 1e-15
    assert all(b / YARN["factor"] - 1e-15 <= a <= b for a, b in zip(f, base))


def test_plain_rotation_turns_halves_by_the_position():
    x = torch.randn(3, 1, 6, generator=torch.Generator().manual_seed(0), dtype=F)
    got = plain.rotate_halves(x, {"base": 10.0, "dims": 4})
    for t in range(3):
        for i in range(2):
            a = t * 10.0 ** (-2 * i / 4)
            u, v = float(x[t, 0, i]), float(x[t, 0, i + 2])
            assert abs(float(got[t, 0, i]) - (u * math.cos(a) - v * math.sin(a))) < 1e-12
            assert abs(float(got[t, 0, i + 2]) - (v * math.cos(a) + u * math.sin(a))) < 1e-12
    assert torch.equal(got[..., 4:], x[..., 4:])


def test_plain_streams_write_from_all_the_old_ones():
    g = torch.Generator().manual_seed(1)
    xs, y = torch.randn(3, 2, 4, generator=g, dtype=F), torch.randn(2, 4, generator=g, dtype=F)
    w = {"in": torch.randn(3, generator=g, dtype=F), "out": torch.randn(3, generator=g, dtype=F),
         "mix": torch.randn(3, 3, generator=g, dtype=F)}
    got = plain.write_streams(xs, y, w, "")
    for t in range(3):
        assert torch.allclose(got[t], sum(w["mix"][s, t] * xs[s] for s in range(3)) + w["out"][t] * y, atol=1e-12)
    assert torch.allclose(plain.read_streams(xs, w, ""), sum(w["in"][s] * xs[s] for s in range(3)), atol=1e-12)


def test_plain_delta_rule_with_orthogonal_keys_stores_and_replaces():
    """Unit keys, beta 1, no decay: what is read for a key is what was written for it last."""
    D, width = 4, 4
    w = {n: torch.zeros(4, 4, dtype=F) for n in ("q", "k", "v", "g")}
    for n in ("q", "k"):
        w[n] += 40.0 * torch.eye(4, dtype=F)
    w["v"] += torch.tensor([[1.0, 2, 3, 4], [5, 6, 7, 8], [9, 1, 2, 3], [4, 5, 6, 7]], dtype=F)
    w.update({n + ".conv": torch.tensor([[0.0, 1.0]] * 4, dtype=F) for n in ("q", "k", "v")})
    w.update({"b": torch.full((1, 4), 40.0, dtype=F), "a": torch.zeros(1, 4, dtype=F), "A_log": torch.tensor([-40.0], dtype=F),
              "dt_bias": torch.zeros(1, dtype=F), "norm": torch.ones(4, dtype=F), "o": torch.eye(4, dtype=F)})
    w["g"] += 1.0
    h = torch.eye(width, dtype=F)[[0, 1, 2, 0]]
    m = {"heads": 1, "kv_heads": 1, "dim": D, "vdim": 4}
    got = plain.gated_delta(h, m, w, "", 1e-12)
    for t in range(4):
        v = plain.silu(h[t] @ w["v"].T)
        want = v / v.pow(2).mean().sqrt() * plain.silu(h[t] @ w["g"].T)
        assert torch.allclose(got[t], want, atol=1e-5)


def test_plain_selective_scan_as_a_sum_over_what_was_written():
    g = torch.Generator().manual_seed(4)
    C, N, R, T, width = 3, 2, 2, 5, 6
    shapes = {"in": (2 * C, width), "conv": (C, 2), "conv.b": (C,), "x": (R + 2 * N, C), "dt": (C, R), "dt.b": (C,),
              "A_log": (C, N), "D": (C,), "o": (width, C)}
    w = {n: torch.randn(s, generator=g, dtype=F) for n, s in shapes.items()}
    h = torch.randn(T, width, generator=g, dtype=F)
    got = plain.selective_scan(h, {"inner": C, "state": N, "dt_rank": R}, w, "")
    xz = h @ w["in"].T
    x = plain.silu(plain.short_convolution(xz[:, :C], w["conv"], w["conv.b"]))
    p = x @ w["x"].T
    dt = torch.log1p(torch.exp(p[:, :R] @ w["dt"].T + w["dt.b"]))
    y = w["D"] * x
    for t in range(T):
        for j in range(t + 1):
            kept = torch.exp(-torch.exp(w["A_log"]) * dt[j + 1:t + 1].sum(0)[:, None])            # [C, N]
            y[t] += (kept * p[j, R:R + N] * p[t, R + N:]).sum(-1) * dt[j] * x[j]
    assert torch.allclose(got, (y * plain.silu(xz[:, C:])) @ w["o"].T, atol=1e-10)


def test_plain_experts_see_their_weighted_input():
    g = torch.Generator().manual_seed(5)
    w = {"router": torch.randn(3, 4, generator=g, dtype=F)}
    for e in range(3):
        w.update({f"e{e}.{n}": torch.randn(s, generator=g, dtype=F) for n, s in (("gate", (5, 4)), ("up", (5, 4)), ("down", (4, 5)))})
    h = torch.randn(2, 4, generator=g, dtype=F)
    got = plain.routed_ff(h, {"router": {"top": 2}}, w, "")
    for t in range(2):
        s = torch.sigmoid(w["router"] @ h[t])
        want = torch.zeros(4, dtype=F)
        for e in sorted(range(3), key=lambda e: -float(s[e]))[:2]:
            x = s[e] * h[t]
            want += w[f"e{e}.down"] @ (plain.silu(w[f"e{e}.gate"] @ x) * (w[f"e{e}.up"] @ x))
        assert torch.allclose(got[t], want, atol=1e-12)


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
    end = 300 if last is None else last + 1
    assert float(d[place:end].min()) > 0.3, float(d[place:end].min())
    if last is not None:
        assert float(d[end:].max()) == 0.0


# ------------------------------------------------------------------ parts in other arrangements
def test_norms_take_side_by_side_outputs_that_have_norms_of_their_own():
    """A pair of normed outputs ahead of a plain RMS or layer norm (with a bias): both join the stream first."""
    ops = EmulatedOps(torch.float32)
    rt = Runtime(ops, "cpu", torch.float32)
    g = torch.Generator().manual_seed(6)
    y1, y2, g1, g2, w, b = (torch.randn(s, generator=g) for s in ((3, 8), (3, 8), (8,), (8,), (8,), (8,)))
    resid = torch.randn(3, 8, generator=g)

    def joined():
        n = lambda y, gain: y / (y.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * gain
        return resid + n(y1, g1) + n(y2, g2)
    pair = (NormedDelta(y1, g1, 1e-5), NormedDelta(y2, g2, 1e-5))
    for norm, want in ((RMSNorm(8, 1e-5), lambda v: v / (v.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * w),
                       (LayerNorm(8, 1e-5, bias_name="b"), lambda v: (v - v.mean(-1, keepdim=True))
                        / (v.var(-1, unbiased=False, keepdim=True) + 1e-5).sqrt() * w + b)):
        norm.load({"weight": w, "b": b}.__getitem__, rt)
        x = resid.clone()
        assert torch.allclose(norm.forward(x, pair), want(joined()), atol=1e-5)
        assert torch.allclose(x, joined(), atol=1e-6)


def test_side_by_side_hands_every_side_its_own_bindings():
    class Side:
        graph_safe = True

        def __init__(self, needs):
            self.needs = needs

        def param_specs(self):
            return {}

        def load(self, tensors, rt):
            pass

    class Several(Side):
        def cache_specs(self):
            return [StateSpec((n,)) for n in self.needs]

        def forward(self, x, batch, caches, shared):
            assert caches == ["a", "b"][:len(self.needs)]
            return x

    class One(Side):
        def cache_spec(self):
            return StateSpec((self.needs,)) if self.needs else None

        def forward(self, x, batch, cache, shared):
            assert cache == ("c" if self.needs else None)
            return 2 * x
    for right, tail in ((One(7), ["c"]), (One(0), [])):
        both = SideBySide(Several([3, 4]), right, 1.0, 0.5)
        both.load(None, Runtime(EmulatedOps(torch.float32), "cpu", torch.float32))
        assert len(both.cache_specs()) == 2 + len(tail)
        assert torch.equal(both.forward(torch.ones(2, 3), None, ["a", "b"] + tail, {}), torch.full((2, 3), 2.0))


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
    left there (kept inputs, states, keys) must not reach the next."""
    cfg = MODELS["A"]
    folder, weights = write_folder(tmp_path, cfg, seed=12, tag="A")
    requests = make_requests(cfg["vocab"], [20, 3, 31, 1, 12, 2, 45], seed=6)
    ref = reference(cfg, weights, requests)
    steps = rs.mixed(requests, {r: len(t) // 2 for r, t in requests.items()}, max_live=2, seed=4, max_portion=7)
    out = str(tmp_path / "out")
    replay_in_process(folder, steps, out, "float32", rs.max_tokens_needed(steps), ops=EmulatedOps(torch.float32),
                      device="cpu", max_live=2)
    worst, where = compare(out, steps, ref, cfg["vocab"])
    assert worst < float32_bar(cfg, weights, requests, ref), f"max abs err {worst} at {where}"


def test_keys_read_by_a_later_layer_outlive_their_owners_chunk(tmp_path):
    """The marked token's key, seen through a layer whose chunks are three times as long as its owner's, with
    a page pool that holds no more than the sequence."""
    cfg, weights = marked_token_model("shared")
    folder, _ = write_folder(tmp_path, cfg, 1, "shared", weights)
    requests = make_requests(cfg["vocab"], [150], seed=8, avoid=(MARK,))
    requests["r0"][5] = MARK
    ref = reference(cfg, weights, requests)
    steps = rs.portions(requests, sizes=(33, 2, 1, 1, 30, 1))
    out = str(tmp_path / "out")
    replay_in_process(folder, steps, out, "float32", rs.max_tokens_needed(steps), ops=EmulatedOps(torch.float32),
                      device="cpu", max_live=1)
    assert compare(out, steps, ref, cfg["vocab"])[0] < float32_bar(cfg, weights, requests, ref)
