"""Vupelorn through the engine against the plain implementation (``plain_vupelorn.py``,
float64, whole sequences, one function per mechanism).

float32 runs are held to the plain logits row by row (root mean square of the difference
over the vocabulary, means taken off, relative to the logits' own spread); every schedule,
cut and batch is held to the same bound.  A bfloat16 run chooses experts from a rounded
input: where two scores are closer than that rounding a token goes to another expert than in
float64, so single rows may differ visibly.  bfloat16 rows are therefore held to the plain
logits by their median and their ninth decile, and only a few in a hundred may be far off; and
how a bfloat16 request was cut and batched must not show beyond rounding: every schedule is
held to the whole prompts' run in the same way."""

import copy
import json
import os
import subprocess
import sys

import pytest
import torch

import engine_util as eu
import plain_vupelorn as plain
import vupelorn_util as vu

pytestmark = pytest.mark.gpu

F32_BOUND = 1e-4
BF16_MEDIAN, BF16_DECILE = 0.04, 0.12
BF16_FAR, BF16_FAR_SHARE = 0.3, 0.03          # rows further off than this, and how many may be
BF16_BETWEEN_MEDIAN, BF16_BETWEEN_DECILE = 0.02, 0.06


def build(cfg, seed=0, dtype="float32", tensors=None):
    from zig_ai_amd.engine import DecoderModel
    d, tensors = vu.folder(cfg, seed, tensors)
    return DecoderModel.from_folder(d, dtype), tensors


def runner_for(model, page_size=4, tokens=256, slots=4, graphs=True):
    from zig_ai_amd.engine import ModelRunner
    return ModelRunner(model, page_size=page_size, num_pages=max(1, -(-tokens // page_size)),
                       num_slots=slots, use_graphs=graphs)


def plain_logits(cfg, tensors, prompts):
    return [plain.forward(cfg, tensors, p).float() for p in prompts]


def worst(got, want):
    return float(vu.row_error(got, want).max())


def assert_bfloat16_close(got, want, what=None):
    e = vu.row_error(got, want)
    found = (float(e.median()), float(e.quantile(0.9)), float((e > BF16_FAR).double().mean()))
    assert found[0] < BF16_MEDIAN and found[1] < BF16_DECILE and found[2] <= BF16_FAR_SHARE, \
        (what, found)


def assert_bfloat16_same_run(got, base, what=None):
    e = vu.row_error(got, base)
    found = (float(e.median()), float(e.quantile(0.9)))
    assert found[0] < BF16_BETWEEN_MEDIAN and found[1] < BF16_BETWEEN_DECILE, (what, found)


# ----------------------------------------------------------- each mechanism alone
SMALL = vu.gla(heads=1, dim=8, vdim=8, rank=4)
ALONE = {
    "gla": vu.one_layer("gla", vu.gla(), buckets=0),
    "gla, one root, keys wider than values": vu.one_layer("gla", vu.gla(3, 40, 8, 1.0, 12), buckets=0),
    "gla, values wider than keys, rank one": vu.one_layer("gla", vu.gla(2, 4, 72, 9.0, 1), buckets=0),
    "gla, wide heads": vu.one_layer("gla", vu.gla(2, 136, 132, 16.0, 16), buckets=0, width=64),
    "gla, sizes of nothing": vu.one_layer("gla", vu.gla(3, 7, 11, 2.5, 5), buckets=0),
    "halves, stretched": vu.one_layer("latent_attention", vu.latent(scaling=vu.yarn()), buckets=0),
    "halves, stretched far": vu.one_layer("latent_attention", vu.latent(
        heads=2, dim=8, vdim=16, kv_rank=24, q_rank=16, rot_dim=32, base=5e4,
        scaling=vu.yarn(32.0, 20, 4.0, 1.0)), buckets=0),
    "halves, not stretched": vu.one_layer("latent_attention", vu.latent(), buckets=0),
    "adjacent": vu.one_layer("latent_attention_2", vu.latent(), buckets=0),
    "adjacent, many heads": vu.one_layer("latent_attention_2", vu.latent(
        heads=40, dim=8, vdim=8, kv_rank=72, q_rank=16, rot_dim=8), buckets=0, width=64),
    "shared rows": vu.config([
        vu.layer("latent_attention_2", vu.latent()),
        vu.layer("latent_attention_2", vu.latent(heads=5, dim=8, vdim=16, q_rank=40, kv_from=0)),
        vu.layer("latent_attention_2", vu.latent(heads=1, scale=0.3, kv_from=0))], buckets=0),
    "experts": vu.one_layer("gla", SMALL, vu.moe(), buckets=0),
    "one expert of many, tight bound": vu.one_layer("gla", SMALL, vu.moe(16, 9, 1, 0.3), buckets=0),
    "all experts": vu.one_layer("gla", SMALL, vu.moe(8, 3, 3, 5.0), buckets=0),
    "pairs of tokens": vu.one_layer("gla", SMALL, buckets=53),
    "pairs of tokens, large factors": vu.one_layer("gla", SMALL, buckets=1009, mul_prev=2147483647,
                                                   mul_cur=2000000011),
    "one bucket": vu.one_layer("gla", SMALL, buckets=1, mul_prev=0, mul_cur=1),
}


@pytest.mark.parametrize("name", sorted(ALONE))
def test_mechanism_alone(name):
    cfg = ALONE[name]
    model, tensors = build(cfg, seed=3)
    prompts = [vu.tokens(70, cfg["vocab"], 1), vu.tokens(5, cfg["vocab"], 2)]
    lengths = [len(p) for p in prompts]
    want = plain_logits(cfg, tensors, prompts)
    # whole, and token by token from the first token on: the cache and the state alone
    for schedule in (eu.whole(lengths), eu.bulk_then_single(lengths, tail=10 ** 6),
                     eu.changing_portions(lengths, sizes=(2, 3, 2, 9))):
        got = eu.run_schedule(runner_for(model), prompts, schedule)
        for g, w in zip(got, want):
            assert worst(g, w) < F32_BOUND


def test_streams_after_every_layer():
    cfg = vu.TINY_ALL
    model, tensors = build(cfg, seed=3)
    from zig_ai_amd.engine import StepEntry
    prompt = vu.tokens(33, cfg["vocab"], 1)
    streams = []
    plain.forward(cfg, tensors, prompt, streams)
    runner = runner_for(model)
    runner.admit("a")
    taps = []
    runner.step([StepEntry("a", prompt, [])], taps=taps)
    assert len(taps) == 1 + len(streams)
    for got, want in zip(taps[1:], streams):
        assert float((got["stream"].cpu().double() - want).abs().max()) < 2e-4


def test_every_mechanism_counts():
    """The plain implementation without one mechanism is far from the one with it: the
    weights make each of them visible, so the comparisons above can fail."""
    cfg = vu.TINY_ALL
    tensors = vu.make_tensors(cfg, seed=3)
    prompt = vu.tokens(40, cfg["vocab"], 1)
    want = plain.forward(cfg, tensors, prompt).float()

    def changed(edit):
        c, t = copy.deepcopy(cfg), dict(tensors)
        edit(c, t)
        return worst(plain.forward(c, t, prompt).float(), want)

    def put(i, **kw):
        return lambda c, t: c["layers"][i]["mixer"].update(**kw)

    def own_rows(c, t):
        c["layers"][3]["mixer"].pop("kv_from")
        t["l3.mix.dkv"], t["l3.mix.dkv.norm"] = -t["l2.mix.dkv"], t["l2.mix.dkv.norm"]

    edits = {
        "stretching": lambda c, t: c["layers"][0]["mixer"]["rot"].pop("scaling"),
        "the ramp's start": lambda c, t: c["layers"][0]["mixer"]["rot"]["scaling"].update(fast=0.6),
        "base": lambda c, t: [c["layers"][i]["mixer"]["rot"].update(base=30.0) for i in (2, 3)],
        "pairing": lambda c, t: c["layers"][2].update(type="latent_attention"),
        "scale": put(2, scale=0.4), "root": put(1, tau=2.0), "shared rows": own_rows,
        "bound": lambda c, t: c["layers"][1]["mlp"]["expert"].update(limit=7.0),
        "how many experts": lambda c, t: c["layers"][0]["mlp"]["router"].update(top=1),
        "pairs of tokens": lambda c, t: c.pop("embedding"),
        "factor of the predecessor": lambda c, t: c["embedding"]["bigram"].update(mul_prev=30),
        "decay bias": lambda c, t: t.update({"l1.mix.a2.b": 0 * t["l1.mix.a2.b"]}),
        "norm of the read-out": lambda c, t: t.update({"l1.mix.norm": torch.ones(24)}),
        "first token's row": lambda c, t: t.update({"bigram": torch.cat(
            [t["bigram"][:-1], 0 * t["bigram"][-1:]])}),
    }
    for name, edit in edits.items():
        assert changed(edit) > 0.02, name


# ------------------------------- sizes that are multiples of nothing the kernels like
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_awkward_sizes(dtype):
    cfg = vu.config([
        vu.layer("latent_attention", vu.latent(heads=3, dim=12, vdim=20, kv_rank=28, q_rank=12,
                                               rot_dim=6, base=77.0, scaling=vu.yarn()),
                 vu.moe(ff=20, experts=7, top=3)),
        vu.layer("gla", vu.gla(heads=5, dim=9, vdim=13, tau=7.0, rank=3), vu.moe(ff=12, experts=2, top=1)),
        vu.layer("latent_attention_2", vu.latent(heads=70, dim=8, vdim=8, kv_rank=18, q_rank=14,
                                                 rot_dim=10)),
        vu.layer("latent_attention_2", vu.latent(heads=7, dim=10, vdim=6, kv_rank=18, q_rank=9,
                                                 rot_dim=10, kv_from=2)),
    ], width=36, vocab=53, buckets=31)
    cfg = vu.settled(cfg) if dtype == "bfloat16" else cfg
    model, tensors = build(cfg, seed=17, dtype=dtype)
    lengths = [50, 3, 21]
    prompts = [vu.tokens(n, cfg["vocab"], 30 + i) for i, n in enumerate(lengths)]
    want = plain_logits(cfg, tensors, prompts)
    base = None
    for name, schedule in (("whole", eu.whole(lengths)),
                           ("portions", eu.changing_portions(lengths, seed=2)),
                           ("mixed", eu.mixed(lengths, seed=3, max_live=3, decode_tail=8))):
        got = eu.run_schedule(runner_for(model, page_size=8, tokens=128, slots=3), prompts, schedule)
        if dtype == "float32":
            for g, w in zip(got, want):
                assert worst(g, w) < F32_BOUND, name
        else:
            assert_bfloat16_close(torch.cat(got), torch.cat(want), name)
            base = base or got
            assert_bfloat16_same_run(torch.cat(got), torch.cat(base), name)


# -------------------------------------------------------- schedules of whole models
LENGTHS = [150, 37, 9, 1, 75, 130, 2]


def schedules(lengths):
    return {
        "whole": eu.whole(lengths),
        "bulk + tail": eu.bulk_then_single(lengths, tail=40),
        "portions": eu.changing_portions(lengths, seed=1),
        "portions of two": eu.changing_portions(lengths, seed=0, sizes=(2, 2, 3, 2, 17)),
        "mixed": eu.mixed(lengths, seed=2, max_live=4, decode_tail=20),
        "mixed, three live": eu.mixed(lengths, seed=5, max_live=3, decode_tail=45),
    }


@pytest.mark.parametrize("which", ["all", "other"])
@pytest.mark.parametrize("page_size", [4, 16])
def test_schedules_float32(which, page_size):
    cfg = vu.TINY_ALL if which == "all" else vu.TINY_OTHER
    model, tensors = build(cfg, seed=11)
    prompts = [vu.tokens(n, cfg["vocab"], 20 + i) for i, n in enumerate(LENGTHS)]
    want = plain_logits(cfg, tensors, prompts)
    for name, schedule in schedules(LENGTHS).items():
        # a pool for the most tokens live at any time: pages and slots are used again
        peak = eu.peak_tokens(LENGTHS, schedule, round_to=max(16, page_size))
        runner = runner_for(model, page_size=page_size, tokens=peak, slots=4)
        got = eu.run_schedule(runner, prompts, schedule)
        for i, (g, w) in enumerate(zip(got, want)):
            assert worst(g, w) < F32_BOUND, (name, i)
        if "mixed" in name:
            assert runner.cache.pages_reused > 0
        assert len(runner.cache.requests) == 0


@pytest.mark.parametrize("which", ["all", "other"])
def test_schedules_bfloat16(which):
    cfg = vu.settled(vu.TINY_ALL if which == "all" else vu.TINY_OTHER)
    model, tensors = build(cfg, seed=11, dtype="bfloat16")
    prompts = [vu.tokens(n, cfg["vocab"], 20 + i) for i, n in enumerate(LENGTHS)]
    want = plain_logits(cfg, tensors, prompts)
    base = None
    for name, schedule in schedules(LENGTHS).items():
        peak = eu.peak_tokens(LENGTHS, schedule, round_to=16)
        got = eu.run_schedule(runner_for(model, page_size=16, tokens=peak, slots=4), prompts, schedule)
        assert_bfloat16_close(torch.cat(got), torch.cat(want), name)
        base = base or got
        assert_bfloat16_same_run(torch.cat(got), torch.cat(base), name)


# ------------------------------------------------ configurations drawn at random
@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(seed):
    cfg = vu.random_config(seed)
    lengths = [70, 1, 33, 12, 2]
    prompts = [vu.tokens(n, cfg["vocab"], 90 + i) for i, n in enumerate(lengths)]
    model, tensors = build(cfg, seed=seed)
    want = plain_logits(cfg, tensors, prompts)
    for name, schedule in (("whole", eu.whole(lengths)),
                           ("portions", eu.changing_portions(lengths, seed=seed)),
                           ("mixed", eu.mixed(lengths, seed=seed, max_live=3, decode_tail=9))):
        peak = eu.peak_tokens(lengths, schedule, round_to=16)
        runner = runner_for(model, page_size=4 if seed % 2 else 16, tokens=peak, slots=3)
        got = eu.run_schedule(runner, prompts, schedule)
        for i, (g, w) in enumerate(zip(got, want)):
            assert worst(g, w) < 3 * F32_BOUND, (name, i, cfg)
    # the same model in bfloat16 runs (odd widths fall back to 32-bit weights) and agrees
    # with itself across schedules
    model16, _ = build(cfg, seed=seed, dtype="bfloat16")
    base = None
    for schedule in (eu.whole(lengths), eu.mixed(lengths, seed=seed, max_live=3, decode_tail=9)):
        got = eu.run_schedule(runner_for(model16, page_size=16, tokens=256, slots=3), prompts, schedule)
        assert all(torch.isfinite(g).all() for g in got)
        base = base or got
        assert_bfloat16_same_run(torch.cat(got), torch.cat(base), cfg)


# --------------------- the recurrence's chunks: portions around their edges, long memory
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_chunk_edges(dtype):
    from zig_ai_amd.kernels import ops
    C = ops.CHANNEL_CHUNKS[1]
    # (the second layer's many heads take the longer chunks, the first the shorter)
    cfg = vu.config([vu.layer("gla", vu.gla(heads=2, dim=20, vdim=24, tau=4.0)),
                     vu.layer("gla", vu.gla(heads=86, dim=4, vdim=72, tau=1.0, rank=3))], buckets=19)
    assert [ops.channel_chunk(3, 1, *hv) for hv in ((2, 24), (86, 72))] == list(ops.CHANNEL_CHUNKS)
    model, tensors = build(cfg, seed=6, dtype=dtype)
    lengths = [2 * C + 45, C - 1, C, C + 1, C + 2, 3]
    prompts = [vu.tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate(lengths)]
    want = plain_logits(cfg, tensors, prompts)
    edges = [[2, C, 1, C + 1, 10 ** 6], [C - 1], [C - 1, 1], [C, 1], [C, 2], [3]]
    cut = []
    for i, sizes in enumerate(edges):
        at = 0
        for size in sizes:
            to = min(lengths[i], at + size)
            if to > at:
                cut.append(([(i, at, to)], [i] if to == lengths[i] else []))
            at = to
    together = [([(i, 0, n) for i, n in enumerate(lengths)], list(range(len(lengths))))]
    # one request's long portion beside others' single tokens
    beside = [([(1, 0, C - 2), (4, 0, C + 1)], []),
              ([(1, C - 2, C - 1), (0, 0, 2 * C + 40), (4, C + 1, C + 2)], [1, 4]),
              ([(0, 2 * C + 40, 2 * C + 45), (2, 0, 1)], [0]), ([(2, 1, C)], [2]),
              ([(3, 0, C + 1), (5, 0, 2)], [3]), ([(5, 2, 3)], [5])]
    for name, schedule in (("whole", eu.whole(lengths)), ("cut", cut), ("together", together),
                           ("beside", beside)):
        got = eu.run_schedule(runner_for(model, page_size=16, tokens=8 * C, slots=6), prompts, schedule)
        for i, (g, w) in enumerate(zip(got, want)):
            if dtype == "float32":
                assert worst(g, w) < F32_BOUND, (name, i)
            else:
                assert_bfloat16_close(g, w, (name, i))


def lasting(cfg, tensors, i):
    """Layer ``i``'s decays all but one, so that its state keeps every token."""
    b = tensors[f"l{i}.mix.a2.b"]
    tensors[f"l{i}.mix.a2"] = 0 * tensors[f"l{i}.mix.a2"]
    tensors[f"l{i}.mix.a2.b"] = torch.full_like(b, 12.0)


def test_far_tokens_reach_the_end_through_the_state():
    cfg = vu.one_layer("gla", vu.gla(heads=2, dim=16, vdim=16, tau=16.0), buckets=0)
    tensors = vu.make_tensors(cfg, seed=9)
    lasting(cfg, tensors, 0)
    model, tensors = build(cfg, tensors=tensors)
    n = 600
    a = [t % 3 for t in vu.tokens(n, cfg["vocab"], 3)]
    # 24 of the first tokens are another one: the last rows still tell the two prompts apart
    b = [cfg["vocab"] - 1] * 24 + a[24:]
    wa, wb = plain_logits(cfg, tensors, [a, b])
    assert worst(wb[-8:], wa[-8:]) > 0.01
    for prompt, want in ((a, wa), (b, wb)):
        for schedule in (eu.whole([n]), eu.bulk_then_single([n], tail=40),
                         eu.changing_portions([n], sizes=(33, 2, 64, 17, 290))):
            got = eu.run_schedule(runner_for(model, tokens=640), [prompt], schedule)[0]
            assert worst(got, want) < F32_BOUND
    # nothing is left in a slot that is taken again
    runner = runner_for(model, tokens=640, slots=1)
    for prompt, want in ((a, wa), (b, wb), (a, wa)):
        got = eu.run_schedule(runner, [prompt], eu.bulk_then_single([n], tail=5))[0]
        assert worst(got, want) < F32_BOUND


def test_a_token_that_wipes_the_state():
    """Decays of nearly zero in the middle of a chunk: what came before is gone, and the
    products of decays behind it neither overflow nor lose what came after."""
    cfg = vu.one_layer("gla", vu.gla(heads=2, dim=16, vdim=16, tau=0.05, rank=8), buckets=0)
    tensors = vu.make_tensors(cfg, seed=12)
    model, tensors = build(cfg, tensors=tensors)
    h = plain.embed(list(range(cfg["vocab"])), tensors, None)
    a = plain.decays(h, tensors, "l0.mix.", 0.05)
    assert float(a.min()) < 1e-30 and float((a > 0.9).double().mean()) > 0.02
    n = 520
    prompt = vu.tokens(n, cfg["vocab"], 1)
    want = plain_logits(cfg, tensors, [prompt])[0]
    for schedule in (eu.whole([n]), eu.bulk_then_single([n], tail=100),
                     eu.changing_portions([n], sizes=(100, 2, 300))):
        got = eu.run_schedule(runner_for(model, tokens=640), [prompt], schedule)[0]
        assert worst(got, want) < F32_BOUND


# ---------------------------------------- the first tokens, and the token ahead of a portion
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_token_pairs_across_portions(dtype):
    """The token ahead of a portion's first comes from the request's state, whatever stood
    in the slot before: portions of every small size, requests that pause, slots taken again
    by a request whose first token must take the last row."""
    cfg = vu.one_layer("latent_attention_2", vu.latent(), buckets=41)
    tensors = vu.make_tensors(cfg, seed=5)
    tensors["bigram"] = 2.0 * tensors["bigram"]
    model, tensors = build(cfg, tensors=tensors, dtype=dtype)
    lengths = [24, 17, 1, 2, 9]
    prompts = [vu.tokens(n, cfg["vocab"], 10 + i) for i, n in enumerate(lengths)]
    want = plain_logits(cfg, tensors, prompts)
    # (the test can see a portion that takes its first token for a request's first)
    broken = plain.forward(cfg, tensors, prompts[0][2:]).float()
    assert worst(broken[:1], want[0][2:3]) > 0.3
    plans = {
        "two": eu.changing_portions(lengths, sizes=(2,)), "one": eu.changing_portions(lengths, sizes=(1,)),
        "one two three": eu.changing_portions(lengths, sizes=(1, 2, 3)),
        "paused": [([(0, 0, 3)], []), ([(1, 0, 16)], []), ([(0, 3, 4), (2, 0, 1)], [2]),
                   ([(3, 0, 2)], [3]), ([(0, 4, 24), (1, 16, 17)], [0, 1]), ([(4, 0, 1)], []),
                   ([(4, 1, 2)], []), ([(4, 2, 9)], [4])]}
    for name, schedule in plans.items():
        runner = runner_for(model, tokens=64, slots=3)
        for _ in range(2):
            got = eu.run_schedule(runner, prompts, schedule)
            for g, w in zip(got, want):
                if dtype == "float32":
                    assert worst(g, w) < F32_BOUND, name
                else:
                    assert float(vu.row_error(g, w).max()) < 0.1, name


# --------------------------------- the causal edge, with scores that stand out
def sharp_cfg(kind, reader=False):
    # a scale that makes the softmax all but choose one key: a key wrongly seen or wrongly
    # hidden then takes or loses nearly all of a query's weight
    mixer = vu.latent(heads=2, dim=16, vdim=16, kv_rank=24, q_rank=16, rot_dim=8, base=100.0,
                      scale=2.0, scaling=vu.yarn() if kind == "latent_attention" else None)
    layers = [vu.layer(kind, mixer)]
    if reader:
        layers.append(vu.layer(kind, dict(mixer, heads=3, kv_from=0)))
    return vu.config(layers, buckets=0)


def plain_with_reach(cfg, tensors, prompt, reach):
    """The plain model with every query seeing one key fewer (-1: not itself) or one more
    (+1: its successor too) than it should."""
    real = plain.latent_attention
    plain.latent_attention = lambda *a, **k: real(*a, reach=reach, **k)
    try:
        return plain.forward(cfg, tensors, prompt).float()
    finally:
        plain.latent_attention = real


@pytest.mark.parametrize("kind,reader", [("latent_attention", False), ("latent_attention_2", False),
                                         ("latent_attention_2", True)])
def test_causal_edge(kind, reader):
    cfg = sharp_cfg(kind, reader)
    model, tensors = build(cfg, seed=5)
    n = 90
    prompts = [vu.tokens(n, cfg["vocab"], 7)]
    want = plain_logits(cfg, tensors, prompts)[0]
    # the test can see an edge that is one token off (the first row has no key fewer to see)
    for reach in (-1, 1):
        off = plain_with_reach(cfg, tensors, prompts[0], reach)
        assert worst(off[1:], want[1:]) > 0.05
    for page_size in (4, 16):
        for name, schedule in (("whole", eu.whole([n])),
                               ("decoded", eu.bulk_then_single([n], tail=n - 3)),
                               ("portions", eu.changing_portions([n], sizes=(5, 2, 16, 3, 17, 15, 1)))):
            got = eu.run_schedule(runner_for(model, page_size=page_size, tokens=128), prompts,
                                  schedule)[0]
            assert worst(got, want) < 1e-3, (name, page_size)


# ----------------------------------------------------------------- far keys count
def far_prompt(cfg, tensors, n, place):
    """A prompt of ``n`` tokens and the same with another token at ``place``, made so that the
    last rows of the plain logits differ clearly: the body repeats three ids, the token at
    ``place`` occurs nowhere else, and the last eight tokens are one id whose queries it
    draws (both found by trying the ids kept aside for this)."""
    V = cfg["vocab"]
    body = [t % 3 for t in vu.tokens(n, V, 3)]
    best = None
    for tail in range(V - 16, V - 8):
        for cand in range(V - 8, V):
            a = list(body)
            a[-8:] = [tail] * 8
            b = list(a)
            a[place] = cand
            wa, wb = plain.forward(cfg, tensors, a).float(), plain.forward(cfg, tensors, b).float()
            d = worst(wb[-8:], wa[-8:])
            if best is None or d > best[0]:
                best = (d, a, b, wa, wb)
            if d > 0.1:
                return best
    return best


@pytest.mark.parametrize("kind,reader", [("latent_attention", False), ("latent_attention_2", True)])
def test_far_tokens_reach_the_end_through_the_cache(kind, reader):
    cfg = sharp_cfg(kind, reader)
    tensors = vu.make_tensors(cfg, seed=9)
    model, tensors = build(cfg, tensors=tensors)
    n = 600
    d, a, b, wa, wb = far_prompt(cfg, tensors, n, place=1)
    assert d > 0.02           # the second token still shows at the end, among hundreds
    for prompt, want in ((a, wa), (b, wb)):
        for page_size, schedule in ((16, eu.whole([n])), (4, eu.bulk_then_single([n], tail=40)),
                                    (16, eu.changing_portions([n], sizes=(33, 2, 64, 17, 200)))):
            got = eu.run_schedule(runner_for(model, page_size=page_size, tokens=640), [prompt],
                                  schedule)[0]
            assert worst(got, want) < 3 * F32_BOUND
    # nothing is left of a request whose pages are taken again: b after a in the same pool
    runner = runner_for(model, page_size=16, tokens=640, slots=1)
    for prompt, want in ((a, wa), (b, wb), (a, wa)):
        got = eu.run_schedule(runner, [prompt], eu.bulk_then_single([n], tail=5))[0]
        assert worst(got, want) < 3 * F32_BOUND
    assert runner.cache.pages_reused > 0


# ------------------------------------- long contexts in ranges of keys, long decoding
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_context_in_ranges(dtype):
    mixer = vu.latent(heads=2, dim=16, vdim=16, kv_rank=64, q_rank=16, rot_dim=16, base=1e4)
    cfg = vu.config([vu.layer("latent_attention_2", mixer),
                     vu.layer("latent_attention", dict(mixer, rot=dict(
                         mixer["rot"], scaling=vu.yarn(8.0, 200, 16.0, 1.0)))),
                     vu.layer("latent_attention_2", dict(mixer, heads=3, kv_from=0))])
    model, tensors = build(cfg, seed=4, dtype=dtype)
    n = 1500
    prompts = [vu.tokens(n, cfg["vocab"], 1), vu.tokens(30, cfg["vocab"], 2)]
    want = plain_logits(cfg, tensors, prompts)
    runner = runner_for(model, page_size=16, tokens=1600, graphs=False)
    wants = [list(range(n - 90, n)), list(range(30))]
    steps = [([(0, 0, n - 80)], [])]
    # the long request decodes beside the short one's portions and single tokens
    steps += [([(0, n - 80 + i, n - 79 + i)] + ([(1, 3 * i, 3 * i + 3)] if i < 10 else []),
               [1] if i == 9 else []) for i in range(80)]
    steps[-1] = (steps[-1][0], [0])
    got = eu.run_schedule(runner, prompts, steps, wants=wants)
    if dtype == "float32":
        assert worst(got[0], want[0][n - 90:]) < F32_BOUND
        assert worst(got[1], want[1]) < F32_BOUND
    else:
        assert_bfloat16_close(torch.cat(got), torch.cat([want[0][n - 90:], want[1]]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    cfg = vu.settled(vu.TINY_ALL) if dtype == "bfloat16" else vu.TINY_ALL
    model, tensors = build(cfg, seed=21, dtype=dtype)
    n = 330
    prompts = [vu.tokens(n, cfg["vocab"], 5)]
    want = plain_logits(cfg, tensors, prompts)[0]
    runner = runner_for(model, page_size=16, tokens=512)       # decode steps replay from graphs
    got = eu.run_schedule(runner, prompts, eu.bulk_then_single([n], tail=300))[0]
    assert runner.graphs.replays > 200
    if dtype == "float32":
        assert worst(got, want) < F32_BOUND
    else:
        assert_bfloat16_close(got, want)


# ------------------------------------------- unequal requests together and alone
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_batch_against_each_alone(dtype):
    cfg = vu.settled(vu.TINY_ALL) if dtype == "bfloat16" else vu.TINY_ALL
    model, tensors = build(cfg, seed=2, dtype=dtype)
    lengths = [64, 3, 41, 17]
    prompts = [vu.tokens(n, cfg["vocab"], 40 + i) for i, n in enumerate(lengths)]
    alone = eu.run_schedule(runner_for(model, tokens=256), prompts, eu.whole(lengths))
    together = [([(i, 0, n) for i, n in enumerate(lengths)], list(range(len(lengths))))]
    got = eu.run_schedule(runner_for(model, tokens=256), prompts, together)
    if dtype == "float32":
        assert worst(torch.cat(got), torch.cat(alone)) < F32_BOUND
    else:
        assert_bfloat16_same_run(torch.cat(got), torch.cat(alone))


# ----------------------------------- sizes at which the products run on the matrix cores
def test_wider_model_bfloat16():
    mixer = vu.latent(heads=8, dim=32, vdim=48, kv_rank=128, q_rank=96, rot_dim=32, base=1e5)
    cfg = vu.config([vu.layer("latent_attention_2", mixer, vu.moe(ff=64, experts=6, top=3, limit=1.5)),
                     vu.layer("gla", vu.gla(heads=4, dim=64, vdim=96, tau=16.0, rank=16),
                              vu.moe(ff=128, experts=8, top=2, limit=2.0)),
                     vu.layer("latent_attention_2", dict(mixer, kv_from=0, heads=4)),
                     vu.layer("latent_attention", vu.latent(
                         heads=4, dim=64, vdim=32, kv_rank=256, q_rank=64, rot_dim=64, base=1e4,
                         scaling=vu.yarn(8.0, 64, 8.0, 1.0)))], width=256, vocab=300, buckets=500)
    model, tensors = build(cfg, seed=6, dtype="bfloat16")
    lengths = [300, 70, 3]
    prompts = [vu.tokens(n, cfg["vocab"], 50 + i) for i, n in enumerate(lengths)]
    want = plain_logits(cfg, tensors, prompts)
    base = None
    for name, schedule in (("whole", eu.whole(lengths)),
                           ("bulk + tail", eu.bulk_then_single(lengths, tail=60)),
                           ("portions", eu.changing_portions(lengths, seed=3)),
                           ("mixed", eu.mixed(lengths, seed=1, max_live=3, decode_tail=30))):
        runner = runner_for(model, page_size=16, tokens=512, slots=3)
        got = eu.run_schedule(runner, prompts, schedule)
        assert_bfloat16_close(torch.cat(got), torch.cat(want), name)
        base = base or got
        assert_bfloat16_same_run(torch.cat(got), torch.cat(base), name)


# ------------------------------------------- generation through engine and scheduler
def test_greedy_generation():
    from zig_ai_amd.engine import Engine
    cfg = vu.TINY_ALL
    d, tensors = vu.folder(cfg, seed=8)
    engine = Engine(d, dtype="float32", page_size=4, num_pages=64, max_num_seqs=3,
                    max_num_batched_tokens=48, chunk_size=20, max_model_len=256)
    prompts = [vu.tokens(n, cfg["vocab"], 60 + i) for i, n in enumerate([33, 5, 70, 12, 1])]
    outs = engine.generate(prompts, max_new_tokens=40, temperature=0.0)
    assert all(len(o) == 40 for o in outs)
    for p, o in zip(prompts, outs):
        # every chosen token is the plain implementation's choice for the same history
        logits = plain.forward(cfg, tensors, p + o)
        for j, tok in enumerate(o):
            row = logits[len(p) + j - 1]
            assert float(row.max() - row[tok]) <= 1e-3 * float(row.abs().max()), (j, tok)
    assert len(engine.runner.cache.requests) == 0
    engine.runner.cache.check()


def test_generation_with_preempted_requests():
    """A pool so small that requests lose their pages and start over: their states, and the
    token ahead of their portions, start over with them."""
    from zig_ai_amd.engine import Engine
    cfg = vu.TINY_ALL
    d, tensors = vu.folder(cfg, seed=8)
    engine = Engine(d, dtype="float32", page_size=4, num_pages=24, max_num_seqs=3,
                    max_num_batched_tokens=32, chunk_size=16, max_model_len=90, multi_step=1)
    prompts = [vu.tokens(n, cfg["vocab"], 30 + i) for i, n in enumerate([30, 21, 26])]
    outs = engine.generate(prompts, max_new_tokens=30, temperature=0.0)
    assert engine.stats()["preemptions"] > 0
    for p, o in zip(prompts, outs):
        logits = plain.forward(cfg, tensors, p + o)
        for j, tok in enumerate(o):
            row = logits[len(p) + j - 1]
            assert float(row.max() - row[tok]) <= 1e-3 * float(row.abs().max()), (j, tok)


def test_generation_bfloat16_runs_through_graphs():
    from zig_ai_amd.engine import Engine
    cfg = vu.TINY_OTHER
    d, tensors = vu.folder(cfg, seed=8)
    engine = Engine(d, dtype="bfloat16", page_size=16, num_pages=64, max_num_seqs=4,
                    max_model_len=256)
    assert engine.runner.graphs is not None        # every part can be recorded
    prompts = [vu.tokens(n, cfg["vocab"], 80 + i) for i, n in enumerate([40, 7, 19])]
    outs = engine.generate(prompts, max_new_tokens=24, temperature=0.0)
    assert all(len(o) == 24 for o in outs)
    good = total = 0
    for p, o in zip(prompts, outs):
        logits = plain.forward(cfg, tensors, p + o)
        for j, tok in enumerate(o):
            row = logits[len(p) + j - 1]
            spread = float(row.max() - row.min())
            good += float(row.max() - row[tok]) <= 0.1 * spread
            total += 1
    # (a token routed to another expert than in float64 may pick another word; rare)
    assert good >= 0.9 * total, (good, total)


def test_trace_replay_and_command_line(tmp_path):
    import numpy as np
    cfg = vu.TINY_ALL
    d, tensors = vu.folder(cfg, seed=8)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompt, other = vu.tokens(40, cfg["vocab"], 3), vu.tokens(11, cfg["vocab"], 4)
    want = plain.forward(cfg, tensors, prompt).float()
    want_other = plain.forward(cfg, tensors, other).float()
    # portions of one request beside another's, single tokens, a step in which nothing is asked
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": prompt[:25], "want": [3, 24]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": prompt[25:27], "want": []},
                                     {"id": "b", "tokens": other[:10], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": other[10:], "want": [0]},
                                     {"id": "a", "tokens": prompt[27:], "want": [12]}], "end": ["a", "b"]}]
    out = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d,
                          "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "128"],
                         input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
                         capture_output=True, timeout=600)
    assert out.returncode == 0, out.stderr[-2000:]
    assert [l for l in out.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    first = torch.from_numpy(np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, -1))
    last = torch.from_numpy(np.fromfile(tmp_path / "2.f32", dtype="<f4").reshape(2, -1))
    assert not (tmp_path / "1.f32").exists()
    assert worst(torch.cat([first, last[1:]]), want[[3, 24, 39]]) < F32_BOUND
    assert worst(last[:1], want_other[[10]]) < F32_BOUND
    gen = subprocess.run([sys.executable, "-m", "zig_ai_amd", "--model", d, "--dtype", "float32",
                          "--prompt-ids", ",".join(map(str, prompt[:9])), "-n", "5",
                          "--temperature", "0", "--json"], cwd=root, text=True, capture_output=True,
                         timeout=600)
    assert gen.returncode == 0, gen.stderr[-2000:]
    outputs = json.loads(gen.stdout.strip().split("\n")[-1])["outputs"]
    assert len(outputs) == 1 and len(outputs[0]) == 5
    logits = plain.forward(cfg, tensors, prompt[:9] + outputs[0])
    for j, tok in enumerate(outputs[0]):
        row = logits[9 + j - 1]
        assert float(row.max() - row[tok]) <= 1e-3 * float(row.abs().max()), (j, tok)


# ------------------------------------------------------------------ kernels alone
@pytest.mark.parametrize("H,dk,dv", [(2, 16, 16), (3, 20, 70), (1, 64, 128), (2, 130, 9), (1, 7, 3)])
def test_channel_recurrence_kernels(H, dk, dv):
    """The blocks and the chunks against float64, from states that are not zero, with decays
    from one down to exactly zero; then single tokens, which are walked one by one."""
    from zig_ai_amd.engine.batch import _make_items
    from zig_ai_amd.kernels import ops
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(H + dk + dv)
    lens = [300, 1, 513, 70, 256]
    T, hk, hv = sum(lens), H * dk, H * dv
    q, k, v = (torch.randn(T, n, generator=g) for n in (hk, hk, hv))
    q *= dk ** -0.5
    a = torch.rand(T, hk, generator=g) ** 0.05
    a[torch.rand(T, hk, generator=g) < 0.01] = 0.0
    a[:, ::3] = 1.0 - 1e-3 * a[:, ::3]
    width = -(-(3 * hk + hv) // 4) * 4
    vectors = torch.zeros(T, width)
    vectors[:, :3 * hk + hv] = torch.cat([q, k, a, v], dim=1)
    pad = 5                                   # floats before the state in a slot
    slots = [3, 0, 5, 1, 4]
    state = torch.randn(6, pad + hk * dv, generator=g)
    start = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), dtype=torch.int32, device=dev)
    slot_id = torch.tensor(slots, dtype=torch.int32, device=dev)
    want, after = torch.zeros(T, hv, dtype=torch.float64), state.double().clone()
    row = 0
    for n, s in zip(lens, slots):
        S = state[s, pad:].double().view(H, dv, dk).transpose(1, 2).clone()
        for t in range(row, row + n):
            S = a[t].double().view(H, dk, 1) * S + k[t].double().view(H, dk, 1) * v[t].double().view(H, 1, dv)
            want[t] = (S * q[t].double().view(H, dk, 1)).sum(dim=1).reshape(-1)
        after[s, pad:] = S.transpose(1, 2).reshape(-1)
        row += n
    mk = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)
    for chunked in (0,) + ops.CHANNEL_CHUNKS:
        st, vec = state.to(dev), vectors.to(dev)
        if chunked:
            seq, row0, cnt = _make_items(lens, chunked)
            got = ops.channel_recurrence_chunked(vec, st, pad, slot_id, (mk(seq), mk(row0), mk(cnt), len(seq)),
                                                 chunked, H, dk, dv)
        else:
            got = ops.channel_recurrence(vec, st, pad, start, slot_id, H, dk, dv)
        scale = float(want.abs().max())
        assert float((got.cpu().double() - want).abs().max()) < 1e-5 * scale, chunked
        assert float((st.cpu().double() - after).abs().max()) < 1e-5 * float(after.abs().max()), chunked
    # the first token of every request, as a step of single tokens
    first = [int(r) for r in start[:-1]]
    st = state.to(dev)
    got = ops.channel_recurrence(vectors[first].contiguous().to(dev), st, pad,
                                 mk(list(range(len(lens) + 1))), slot_id, H, dk, dv)
    assert float((got.cpu().double() - want[first]).abs().max()) < 1e-5 * scale


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,dk,dv,rank", [(2, 16, 24, 8), (3, 100, 8, 5), (1, 8, 300, 1), (4, 64, 64, 300)])
def test_channel_decay_prepare_kernel(dtype, H, dk, dv, rank):
    from zig_ai_amd.kernels import ops
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(dk + dv)
    T, hk, hv, root = 21, H * dk, H * dv, 3.5
    proj = torch.randn(T, 2 * hk + hv + 7 + rank, generator=g).to(dtype)
    up = (torch.randn(hk, rank, generator=g) * 6 * rank ** -0.5).to(dtype)
    bias = torch.randn(hk, generator=g) * 20
    got = ops.channel_decay_prepare(proj.to(dev), 0, hk, 2 * hk, 2 * hk + hv + 7, up.to(dev),
                                    bias.to(dev), root, 0.25, H, dk, dv).cpu().double()
    p = proj.double()
    a = torch.sigmoid(p[:, 2 * hk + hv + 7:] @ up.double().T + bias.double()) ** (1 / root)
    want = torch.cat([p[:, :hk] * 0.25, p[:, hk:2 * hk], a, p[:, 2 * hk:2 * hk + hv]], dim=1)
    assert float((got[:, :want.shape[1]] - want).abs().max()) < 2e-6 * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("width", [40, 37, 1024, 4096, 5000])
def test_normed_addition_kernel(width):
    from zig_ai_amd.kernels import ops
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(width)
    T = 19
    stream, w = torch.randn(T, width, generator=g) * 3, torch.randn(width, generator=g)
    for shape, dtype in (((T, width), torch.float32), ((T, width), torch.bfloat16),
                         ((5, T, width), torch.float32), ((11, T, width), torch.float32)):
        y = (torch.randn(*shape, generator=g) * 2).to(dtype)
        total = y.double().sum(dim=0) if y.dim() == 3 else y.double()
        want = stream.double() + 0.7 * plain.rms_norm(total, w.double(), 1e-3)
        for copy_dtype in (None, torch.bfloat16, torch.float32):
            res = stream.to(dev).clone()
            out = ops.normed_add_(res, y.to(dev), w.to(dev), 1e-3, 0.7, copy_dtype)
            assert float((res.cpu().double() - want).abs().max()) < 2e-5
            if copy_dtype is None:
                assert out is res
            else:
                assert torch.equal(out, res.to(copy_dtype))


@pytest.mark.parametrize("magnitude", [1.0, 1.37])
@pytest.mark.parametrize("adjacent", [False, True])
def test_rotation_kernels(adjacent, magnitude):
    from zig_ai_amd.kernels import ops
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(4)
    T, H, dr, dims, Rq, R = 11, 3, 12, 8, 16, 24
    rot = {"dims": dims, "base": 40.0}
    inv = torch.tensor(plain.frequencies(rot)[0], dtype=torch.float32)
    pos = torch.tensor([0, 1, 2, 7, 9, 33, 100, 101, 400, 5, 6], dtype=torch.int32)
    src = torch.randn(T, H, 5 + dr, generator=g)

    def turned(x):
        y = plain.rotate(x.double(), pos, rot, adjacent)
        y[..., :dims] *= magnitude
        return y

    dst = torch.zeros(T, H, 20 + dr, device=dev)
    ops.rotate_part_(src.to(dev), 5, dst, 20, dr, pos.to(dev), inv.to(dev), dims, adjacent, magnitude)
    assert float((dst.cpu().double()[..., 20:] - turned(src[..., 5:])).abs().max()) < 1e-4
    down = torch.randn(T, Rq + R + dr, generator=g)
    qw, cw = torch.randn(Rq, generator=g), torch.randn(R, generator=g)
    plane = torch.zeros(4, 1, 4, R + dr, device=dev)
    slots = torch.randperm(16, generator=g)[:T].to(torch.int32)
    cq = ops.latent_prepare(down.to(dev), 0, Rq, Rq, R, dr, qw.to(dev), cw.to(dev), 1e-4, pos.to(dev),
                            slots.to(dev), inv.to(dev), dims, adjacent, plane, magnitude)
    rows = plane.view(16, R + dr)[slots.long().to(dev)].cpu().double()
    d = down.double()
    assert float((cq.cpu().double() - plain.rms_norm(d[:, :Rq], qw.double(), 1e-4)).abs().max()) < 1e-5
    assert float((rows[:, :R] - plain.rms_norm(d[:, Rq:Rq + R], cw.double(), 1e-4)).abs().max()) < 1e-5
    # (an angle of some hundred is good to 3e-5 in 32-bit)
    assert float((rows[:, R:] - turned(down[:, Rq + R:])).abs().max()) < 1e-4
    # rows that hold a query latent only: nothing is written
    cq2 = ops.latent_prepare(down[:, :Rq].contiguous().to(dev), 0, Rq, Rq, R, dr, qw.to(dev), None, 1e-4,
                             pos.to(dev), None, inv.to(dev), dims, adjacent, None, magnitude)
    assert torch.equal(cq, cq2)


@pytest.mark.parametrize("inter", [24, 13])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_bounded_gate_with_weights_on_the_input(inter, dtype):
    from zig_ai_amd.kernels import ops
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(inter)
    gu = (torch.randn(31, 2 * inter, generator=g) * 3).to(dtype)
    w = torch.rand(31, generator=g)
    got = ops.clamped_glu(gu.to(dev), 0.8, 1.702, 1.0, w.to(dev)).cpu().double()
    x = gu.double() * w.double()[:, None]
    a, u = x[:, :inter].clamp(max=0.8), x[:, inter:].clamp(-0.8, 0.8)
    want = a * torch.sigmoid(1.702 * a) * (u + 1.0)
    assert float((got - want).abs().max()) < (1e-5 if dtype == torch.float32 else 1e-2)
