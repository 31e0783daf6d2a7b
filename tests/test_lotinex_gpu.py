"""Lotinex through the engine on the GPU against the plain implementation: whole prompts, decoding token
by token, portions down to two tokens, mixed batches over pools and state slots that are used again,
long decoding through captured graphs, layers whose output hangs on one marked token (far back, at
page borders, just inside and just outside a window or a chunk, through another layer's keys, in a
state), the replay program, and greedy generation through the entry point and its scheduler."""
import json

import numpy as np
import pytest
import torch

import plain_lotinex as plain
import replay_schedules as rs
from lotinex_models import (MARK, MARKED_KINDS, MODELS, float32_bar, make_requests, marked_reach, marked_token_model,
                            reference, write_folder)
from replay_harness import compare, replay_in_process, replay_program
from servelab_amd import CacheConfig, LLMEngine, SamplingParams, SchedulerConfig, load_config
from servelab_amd.engine import ModelRunner

pytestmark = pytest.mark.gpu


def emulated_error(tmp_path, folder, cfg, requests, ref):
    """The largest row error of a CPU computation that rounds to bfloat16 where the kernels do
    (tests/emulated_ops.py), every request whole: what rounding alone does to this model."""
    from emulated_ops import EmulatedOps
    steps = rs.whole(requests)
    out = str(tmp_path / "out_emulated")
    replay_in_process(folder, steps, out, "bfloat16", rs.max_tokens_needed(steps), ops=EmulatedOps(torch.bfloat16),
                      device="cpu", max_live=max(16, len(requests)))
    return compare(out, steps, ref, cfg["vocab"])[0]


class Case:
    """A model, its requests and the bars: float32 ``float32_bar``; bfloat16 twice what rounding alone does."""

    def __init__(self, tmp_path, cfg, requests, seed=11, weights=None):
        self.tmp, self.cfg, self.requests = tmp_path, cfg, requests
        self.folder, self.weights = write_folder(tmp_path, cfg, seed, "case", weights=weights)
        self.ref = reference(cfg, self.weights, requests)
        self.bars = {}

    def bar(self, dtype):
        if dtype not in self.bars:
            self.bars[dtype] = float32_bar(self.cfg, self.weights, self.requests, self.ref) if dtype == "float32" else \
                2.0 * emulated_error(self.tmp, self.folder, self.cfg, self.requests, self.ref) + 1e-3
        return self.bars[dtype]

    def check(self, steps, dtype, tag, **kw):
        out = str(self.tmp / f"out_{tag}_{dtype}")
        kw.setdefault("max_live", 4)
        replay_in_process(self.folder, steps, out, dtype, kw.pop("max_tokens", None) or rs.max_tokens_needed(steps), **kw)
        worst, where = compare(out, steps, self.ref, self.cfg["vocab"])
        assert worst < self.bar(dtype), f"{tag}: max abs err {worst} at {where}, bar {self.bar(dtype)}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", sorted(set(MODELS) - {"F"}))
def test_every_way_of_cutting_gives_the_plain_logits(tmp_path, which, dtype):
    case = Case(tmp_path, MODELS[which], make_requests(MODELS[which]["vocab"], [71, 1, 2, 40, 97, 23], seed=5))
    requests = case.requests
    case.check(rs.whole(requests), dtype, "whole")
    case.check(rs.tail_decoded(requests, tail=45), dtype, "decode")
    case.check(rs.portions(requests), dtype, "portions")
    case.check(rs.portions(requests, sizes=(2, 2, 3, 2, 64, 2)), dtype, "twos")
    prompt_lens = {rid: max(1, len(t) - 20) for rid, t in requests.items()}
    for seed in (1, 2):
        case.check(rs.mixed(requests, prompt_lens, max_live=3, seed=seed), dtype, f"mixed{seed}", max_live=3)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_of_the_widest_model(tmp_path, dtype):
    """Prompts of several hundred tokens: many pages a request, steps of enough rows for every product
    kernel, many segments of the selective scan, the attentions on the matrix cores in bfloat16, a window and
    chunks that release pages."""
    case = Case(tmp_path, MODELS["F"], make_requests(MODELS["F"]["vocab"], [613, 190], seed=12), seed=16)
    requests = case.requests
    case.check(rs.whole(requests), dtype, "whole")
    case.check(rs.tail_decoded(requests, tail=40), dtype, "decode")
    case.check(rs.portions(requests, sizes=(100, 2, 255, 64, 7)), dtype, "portions")
    steps = rs.mixed(requests, {rid: len(t) - 30 for rid, t in requests.items()}, max_live=2, seed=5, max_portion=130)
    case.check(steps, dtype, "mixed", max_live=2)


@pytest.mark.parametrize("page", [16, 32, 64])
def test_pages_and_slots_are_used_again(tmp_path, page):
    """A pool no larger than the live requests need at their peak and three state slots for ten requests:
    every page and slot serves several requests, one after the other and side by side."""
    case = Case(tmp_path, MODELS["A"], make_requests(MODELS["A"]["vocab"], [50, 33, 80, 5, 64, 17, 129, 48, 2, 70], seed=6))
    steps = rs.mixed(case.requests, {rid: len(t) // 2 for rid, t in case.requests.items()}, max_live=3, seed=3,
                     max_portion=40)
    case.check(steps, "float32", f"reuse{page}", max_tokens=rs.max_tokens_needed(steps, max(64, page)), block_size=page,
               max_live=3)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_through_captured_graphs(tmp_path, dtype, monkeypatch):
    """Two requests decoded for 330 tokens: the steps replay captured graphs whose capacity is outgrown
    twice; states, kept inputs and pages are carried from replay to replay, windows and chunks are passed."""
    monkeypatch.setattr(ModelRunner, "GRAPH_MIN_CONTEXT", 128)
    case = Case(tmp_path, MODELS["C"], make_requests(MODELS["C"]["vocab"], [350, 341], seed=7), seed=13)
    a, b = case.requests["r0"], case.requests["r1"]
    steps = [{"step": 0, "entries": [{"id": "r0", "tokens": a[:20], "want": [0, 19]},
                                     {"id": "r1", "tokens": b[:11], "want": [10]}], "end": []}]
    for i in range(330):
        steps.append({"step": i + 1, "entries": [{"id": "r0", "tokens": [a[20 + i]], "want": [0]},
                                                 {"id": "r1", "tokens": [b[11 + i]], "want": [0]}],
                      "end": ["r0", "r1"] if i == 329 else []})
    case.check(steps, dtype, "long")


def test_graphs_are_in_use_for_decode_steps(tmp_path):
    folder, _ = write_folder(tmp_path, MODELS["A"], seed=14, tag="A")
    from servelab_amd.engine import StepEntry
    from servelab_amd.engine.session import load_model_on_device, make_runner
    _, model = load_model_on_device(folder, "bfloat16", "cuda:0")
    runner = make_runner(model, 64, 16, max_num_seqs=4)
    assert model.spec.graph_safe and runner.use_graphs
    runner.step([StepEntry("a", [1, 2, 3], [2])])
    for t in range(6):
        runner.step([StepEntry("a", [t], [0])])
    assert runner.graph_replays >= 4


@pytest.mark.parametrize("kind", MARKED_KINDS)
@pytest.mark.parametrize("place", [0, 15, 16, 39, 40, 119, 200])
def test_a_marked_token_decides_the_logits(tmp_path, kind, place):
    """The marked token at the start, and just before, at and after the borders of pages and chunks; in a
    prompt, among decoded tokens, in two-token portions.  Behind a window or in a chunk, the last token that
    sees it and the first that does not are both checked: the plain logits differ by much at the one and
    not at all at the other."""
    cfg, weights = marked_token_model(kind)
    requests = make_requests(cfg["vocab"], [300], seed=8, avoid=(MARK,))
    requests["r0"][place] = MARK
    case = Case(tmp_path, cfg, requests, weights=weights)
    toks = list(requests["r0"])
    toks[place] = MARK + 1
    d = np.abs(case.ref["r0"] - reference(cfg, weights, {"r0": toks})["r0"]).max(-1)
    last = marked_reach(kind, place)
    shift = d[place:] if last is None else d[place:last + 1]
    assert shift.min() > 3 * case.bar("bfloat16"), (shift.min(), case.bar("bfloat16"))
    if last is not None:
        assert d[last + 1:].max() == 0.0
    for name, steps in (("whole", rs.whole(requests)), ("decode", rs.tail_decoded(requests, tail=260)),
                        ("twos", rs.portions(requests, sizes=(33, 2, 64, 2, 2)))):
        case.check(steps, "float32", name)
        case.check(steps, "bfloat16", name)


def test_the_first_tokens_and_the_narrowest_windows(tmp_path):
    """Sequences of one to five tokens (shorter than the convolutions and windows), model B's chunks of one
    token and model D's window of two, one by one and in portions of two."""
    for which in ("B", "D", "E"):
        case = Case(tmp_path, MODELS[which], make_requests(MODELS[which]["vocab"], [1, 2, 3, 4, 5, 1], seed=13), seed=17)
        case.check(rs.whole(case.requests), "float32", which + "whole")
        case.check(rs.tail_decoded(case.requests, tail=4), "float32", which + "ones")
        case.check(rs.portions(case.requests, sizes=(2,)), "float32", which + "twos")


def test_the_program_replays_a_trace(tmp_path):
    case = Case(tmp_path, MODELS["B"], make_requests(MODELS["B"]["vocab"], [30, 9], seed=9), seed=14)
    steps = rs.tail_decoded(case.requests, tail=5)
    out = str(tmp_path / "out_prog")
    replay_program(case.folder, steps, out, "float32", rs.max_tokens_needed(steps))
    worst, where = compare(out, steps, case.ref, case.cfg["vocab"])
    assert worst < case.bar("float32"), (worst, where)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "E"])
def test_greedy_generation_through_the_entry_point(tmp_path, which, dtype):
    """Every token generated is the plain implementation's best, or (rounding) within the bar of it."""
    requests = make_requests(MODELS[which]["vocab"], [30, 4, 77, 1, 12, 50], seed=10)
    case = Case(tmp_path, MODELS[which], requests, seed=15)
    prompts, new = list(requests.values()), 24
    for budget, blocks in ((256, 64), (8, 64), (64, 24)):
        engine = LLMEngine(load_config(case.folder), CacheConfig(num_blocks=blocks),
                           SchedulerConfig(max_num_seqs=3, max_num_batched_tokens=budget), dtype=dtype)
        outs = engine.generate(prompts, SamplingParams.greedy(new))
        engine.runner.manager.check()
        for p, o in zip(prompts, outs):
            toks = o.outputs[0].token_ids
            assert o.finished and len(toks) == new
            logits = plain.forward(case.cfg, case.weights, list(p) + toks).float()
            for i, t in enumerate(toks):
                row = logits[len(p) - 1 + i]
                assert row[t] >= row.max() - 4 * case.bar(dtype), (i, float(row.max() - row[t]))


def test_command_line_samples_from_a_random_model(tmp_path, capsys):
    from servelab_amd import cli
    path = tmp_path / "config.json"
    path.write_text(json.dumps(MODELS["B"]))
    assert cli.main(["--config", str(path), "--random-weights", "3", "--prompt-ids", "5,6,7,8", "--max-tokens", "9",
                     "--temperature", "0.8", "--top-k", "20", "--top-p", "0.9", "--max-num-seqs", "4"]) == 0
    assert "finish=length" in capsys.readouterr().out
