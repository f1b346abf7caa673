"""Torisun through the engine against the plain implementation (``plain_torisun.py``,
float64, one function per mechanism).

float32 runs are held to the plain logits row by row (root mean square of the difference
over the vocabulary, relative to the logits' own spread) under every schedule, cut and batch.
bfloat16 rows are held to the plain logits by their median, their ninth decile and the share
of rows that are far off (the weights are drawn sharp on purpose, and a token whose scores lie
within rounding of each other goes to another expert: such a row is far off), and every
schedule to the whole prompts' run: how a request was cut and batched must not show beyond
rounding."""

import copy
import math

import pytest
import torch

import engine_util as eu
import plain_torisun as plain
import torisun_util as tu

pytestmark = pytest.mark.gpu

F32_BOUND = 1e-4
BF16_MEDIAN, BF16_DECILE, BF16_WORST = 0.04, 0.1, 0.5
BF16_FAR_SHARE = 0.03            # of rows beyond BF16_WORST
BF16_BETWEEN_MEDIAN, BF16_BETWEEN_WORST = 0.02, 0.2


def build(cfg, seed=0, dtype="float32", tensors=None):
    from zig_ai_amd.engine import DecoderModel
    d, tensors = tu.folder(cfg, seed, tensors)
    return DecoderModel.from_folder(d, dtype), tensors


def runner_for(model, page_size=4, tokens=256, slots=4, graphs=True):
    from zig_ai_amd.engine import ModelRunner
    return ModelRunner(model, page_size=page_size, num_pages=max(1, -(-tokens // page_size)),
                       num_slots=slots, use_graphs=graphs)


def plain_logits(cfg, tensors, prompts):
    return [plain.forward(cfg, tensors, p).float() for p in prompts]


def worst(got, want):
    return float(tu.row_error(got, want).max())


def assert_bfloat16_close(got, want, what=None):
    e = tu.row_error(got, want)
    found = (float(e.median()), float(e.quantile(0.9)), float((e > BF16_WORST).double().mean()))
    assert found[0] < BF16_MEDIAN and found[1] < BF16_DECILE and found[2] <= BF16_FAR_SHARE, \
        (what, found)


def assert_bfloat16_same(got, base, what=None):
    """Two bfloat16 runs of the same requests, cut or batched differently."""
    e = tu.row_error(got, base)
    found = (float(e.median()), float((e > BF16_BETWEEN_WORST).double().mean()))
    assert found[0] < BF16_BETWEEN_MEDIAN and found[1] <= BF16_FAR_SHARE, (what, found)


# ----------------------------------------------------------- each mechanism alone
ALONE = {
    "window, no kept tokens": tu.one_layer(tu.attention(keep=0)),
    "window with kept tokens": tu.one_layer(tu.attention(window=7, keep=5)),
    "kept tokens beyond the window": tu.one_layer(tu.attention(window=4, keep=9)),
    "window of one": tu.one_layer(tu.attention(window=1, keep=1)),
    "no mask, no rotation": tu.one_layer(tu.attention(window=0, rot_dims=0)),
    "partial rotation, stretched": tu.one_layer(tu.attention(dim=24, rot_dims=10, scaling=tu.yarn())),
    "stretched by one": tu.one_layer(tu.attention(scaling=tu.yarn(1.0, 100, 4.0, 0.5))),
    "one head, values as wide as keys": tu.one_layer(tu.attention(heads=1, kv_heads=1, dim=8, vdim=8)),
    "forty heads on one key head": tu.one_layer(tu.attention(heads=40, kv_heads=1, dim=8, vdim=8)),
    "sixty-six heads on two key heads, odd widths": tu.one_layer(
        tu.attention(heads=66, kv_heads=2, dim=6, vdim=10, window=11)),
    "wide heads": tu.one_layer(tu.attention(heads=2, kv_heads=1, dim=200, vdim=144, scale=0.1)),
    "dense": tu.one_layer(tu.attention(), tu.dense()),
    "dense without bounds, odd width": tu.one_layer(tu.attention(), tu.dense(ff=44, limit=0)),
    "experts and a shared one": tu.one_layer(tu.attention(), tu.moe()),
    "experts, no shared one": tu.one_layer(tu.attention(), tu.moe(shared=0, scale=1.0)),
    "experts, one of one": tu.one_layer(tu.attention(), tu.moe(ff=40, experts=1, top=1)),
    "experts, all of four": tu.one_layer(tu.attention(), tu.moe(ff=12, experts=4, top=4, shared=8)),
    "a reader with another window": tu.config([
        tu.layer(tu.attention(window=6, keep=2)), tu.layer(tu.attention(window=15, keep=4, kv_from=0))]),
    "a reader of every key": tu.config([
        tu.layer(tu.attention(window=6, keep=2)), tu.layer(tu.attention(window=0, kv_from=0, scale=0.2))]),
}


@pytest.mark.parametrize("name", sorted(ALONE))
def test_mechanism_alone(name):
    cfg = ALONE[name]
    model, tensors = build(cfg, seed=3)
    prompts = [tu.tokens(70, cfg["vocab"], 1), tu.tokens(5, cfg["vocab"], 2)]
    lengths = [len(p) for p in prompts]
    want = plain_logits(cfg, tensors, prompts)
    runner = runner_for(model)
    # whole, then token by token from the first token on
    for schedule in (eu.whole(lengths), eu.bulk_then_single(lengths, tail=10 ** 6)):
        for g, w in zip(eu.run_schedule(runner, prompts, schedule), want):
            assert worst(g, w) < F32_BOUND
    model, _ = build(cfg, seed=3, dtype="bfloat16")
    runner = runner_for(model, page_size=16)
    base = None
    for schedule in (eu.whole(lengths), eu.bulk_then_single(lengths, tail=10 ** 6)):
        got = torch.cat(eu.run_schedule(runner, prompts, schedule))
        assert_bfloat16_close(got, torch.cat(want), name)
        base = got if base is None else base
        assert_bfloat16_same(got, base, name)


def test_streams_after_every_layer():
    cfg = tu.TINY_ALL
    model, tensors = build(cfg, seed=4)
    prompt = tu.tokens(61, cfg["vocab"], 3)
    streams = []
    plain.forward(cfg, tensors, prompt, streams)
    from zig_ai_amd.engine import StepEntry
    runner = runner_for(model)
    runner.admit("a")
    taps = []
    runner.step([StepEntry("a", prompt, [])], taps=taps)
    assert len(taps) == len(streams) + 1 == 6            # the embedding, then five layers
    for i, s in enumerate(streams):
        got = taps[i + 1]["stream"].double().cpu()
        assert float((got - s).abs().max()) < 1e-4 * float(s.abs().max()), i


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


CONFIGS = {"all": tu.TINY_ALL, "other": tu.TINY_OTHER}


@pytest.mark.parametrize("which", ["all", "other"])
@pytest.mark.parametrize("page_size", [4, 16])
def test_schedules_float32(which, page_size):
    cfg = CONFIGS[which]
    model, tensors = build(cfg, seed=11)
    prompts = [tu.tokens(n, cfg["vocab"], 20 + i) for i, n in enumerate(LENGTHS)]
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
        runner.cache.check()


@pytest.mark.parametrize("which", ["all", "other"])
def test_schedules_bfloat16(which):
    cfg = tu.settled(CONFIGS[which])
    model, tensors = build(cfg, seed=11, dtype="bfloat16")
    assert all(b.parts["mixer"].planes for b in model.blocks)
    prompts = [tu.tokens(n, cfg["vocab"], 20 + i) for i, n in enumerate(LENGTHS)]
    want = plain_logits(cfg, tensors, prompts)
    base = None
    for name, schedule in schedules(LENGTHS).items():
        peak = eu.peak_tokens(LENGTHS, schedule, round_to=16)
        got = eu.run_schedule(runner_for(model, page_size=16, tokens=peak), prompts, schedule)
        assert_bfloat16_close(torch.cat(got), torch.cat(want), name)
        base = base or got
        assert_bfloat16_same(torch.cat(got), torch.cat(base), name)


@pytest.mark.parametrize("page_size", [1, 2, 4, 8, 64])
def test_page_sizes_bfloat16(page_size):
    """Pages that the matrix-core kernels take in 16-byte pieces, in 8-byte pieces and not at
    all (the general kernel then runs)."""
    cfg = tu.settled(tu.TINY_ALL)
    model, tensors = build(cfg, seed=12, dtype="bfloat16")
    lengths = [60, 21]
    prompts = [tu.tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate(lengths)]
    want = plain_logits(cfg, tensors, prompts)
    for name, schedule in (("whole", eu.whole(lengths)), ("mixed", eu.mixed(lengths, seed=3, max_live=2,
                                                                           decode_tail=12))):
        got = eu.run_schedule(runner_for(model, page_size=page_size, tokens=256), prompts, schedule)
        assert_bfloat16_close(torch.cat(got), torch.cat(want), name)


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(seed):
    cfg = tu.random_config(seed)
    model, tensors = build(cfg, seed=seed)
    lengths = [90, 1, 23, 2]
    prompts = [tu.tokens(n, cfg["vocab"], 30 + i) for i, n in enumerate(lengths)]
    want = plain_logits(cfg, tensors, prompts)
    for name, schedule in (("whole", eu.whole(lengths)),
                           ("portions", eu.changing_portions(lengths, seed=seed)),
                           ("mixed", eu.mixed(lengths, seed=seed, max_live=3, decode_tail=15))):
        peak = eu.peak_tokens(lengths, schedule, round_to=16)
        got = eu.run_schedule(runner_for(model, page_size=4, tokens=peak, slots=3), prompts, schedule)
        for i, (g, w) in enumerate(zip(got, want)):
            assert worst(g, w) < F32_BOUND, (seed, name, i)


@pytest.mark.parametrize("seed", range(12, 20))
def test_random_configurations_bfloat16(seed):
    cfg = tu.settled(tu.random_config(seed))
    model, tensors = build(cfg, seed=seed, dtype="bfloat16")
    lengths = [90, 1, 23, 2]
    prompts = [tu.tokens(n, cfg["vocab"], 30 + i) for i, n in enumerate(lengths)]
    want = plain_logits(cfg, tensors, prompts)
    base = None
    for name, schedule in (("whole", eu.whole(lengths)),
                           ("mixed", eu.mixed(lengths, seed=seed, max_live=3, decode_tail=15))):
        peak = eu.peak_tokens(lengths, schedule, round_to=16)
        got = eu.run_schedule(runner_for(model, page_size=16, tokens=peak, slots=3), prompts, schedule)
        assert_bfloat16_close(torch.cat(got), torch.cat(want), (seed, name))
        base = base or got
        assert_bfloat16_same(torch.cat(got), torch.cat(base), (seed, name))


# ------------------------------------------------ a key just inside and just outside
SEEK, ASK = 299, 298        # the token to find, and the token that asks for it


def edge_model(dim, vdim, window, keep, heads=2, kv_heads=1, reader=False):
    """A model whose asking query puts all but all of its weight on ONE key: the token to find
    wherever it stands.  A key that is wrongly seen, or wrongly not seen, moves the result by
    its whole size.  The key's LAST element (not rotated) reads the stream's first channel,
    where only that token is not zero; the queries' last elements read the second channel,
    where only the asking one is not zero.  ``reader``: a second layer with a window of one
    makes nothing of its own sight, and a third reads the first layer's keys and asks."""
    # (the score that stands out is 20, all others spread over a few units)
    mixer = tu.attention(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
                         scale=20.0 / (2.25 * dim), window=window, keep=keep, rot_dims=2, base=1e6)
    layers = [tu.layer(mixer)]
    if reader:
        layers = [tu.layer(dict(copy.deepcopy(mixer), mask={"size": 1, "keep_first": 0})),
                  tu.layer(dict(copy.deepcopy(mixer), kv_from=0))]
    cfg = tu.config(layers, width=64, vocab=300)
    t = tu.make_tensors(cfg, seed=7)
    t["embed.norm"] = torch.ones_like(t["embed.norm"])
    t["embed"][:, :2] = 0.0
    for tok, ch in ((SEEK, 0), (ASK, 1)):
        t["embed"][tok] = 0.0
        t["embed"][tok, ch] = 8.0
    for i in range(len(layers)):
        p = f"l{i}.mix."
        t[p + "q"][:, 1] = 0.0
        t[p + "q"][dim - 1::dim] = 0.0
        t[p + "q"][dim - 1::dim, 1] = 3.0
        t[p + "q.norm"] = torch.full_like(t[p + "q.norm"], 1.5)
        t[p + "sink"] = torch.zeros_like(t[p + "sink"])
        if p + "k" in t:
            t[p + "k"][:, 0] = 0.0
            t[p + "k"][dim - 1::dim] = 0.0
            t[p + "k"][dim - 1::dim, 0] = 3.0
            t[p + "k.norm"] = torch.full_like(t[p + "k.norm"], 1.5)
            # the token to find carries a value of its own
            t[p + "v"][:, 0] = t[p + "v"][:, 0] * 4.0
    if reader:
        # the first layer leaves the channels alone that the second one's queries read
        t["l0.norm1"][:2] = 0.0
    return cfg, {k: v.to(torch.bfloat16).float() for k, v in t.items()}


EDGE_SIZES = [("float32", 16, 24), ("bfloat16", 16, 24), ("bfloat16", 64, 64), ("bfloat16", 96, 40),
              ("bfloat16", 128, 128), ("bfloat16", 128, 64), ("bfloat16", 200, 136)]


@pytest.mark.parametrize("dtype,dim,vdim", EDGE_SIZES)
@pytest.mark.parametrize("reader", [False, True])
def test_edges_of_window_and_kept_tokens(dtype, dim, vdim, reader):
    window, keep = 70, 18
    cfg, tensors = edge_model(dim, vdim, window, keep, reader=reader)
    model, _ = build(cfg, tensors=tensors, dtype=dtype)
    n, asks = 230, 180                       # the window of the asking token: 111..180
    for place, seen in ((0, True), (1, True), (15, True), (16, True), (17, True), (18, False),
                        (19, False), (63, False), (64, False), (109, False), (110, False),
                        (111, True), (112, True), (128, True), (179, True)):
        prompt = [t % 298 for t in tu.tokens(n, 298, place)]
        prompt[place], prompt[asks] = SEEK, ASK
        other = list(prompt)
        other[place] = 5                                  # the same prompt without the key
        want = plain.forward(cfg, tensors, prompt).float()
        moved = worst(plain.forward(cfg, tensors, other).float()[asks:asks + 1], want[asks:asks + 1])
        assert (moved > 0.3) == seen, (place, moved)
        for schedule in (eu.whole([n]), eu.bulk_then_single([n], tail=n - 175),
                         eu.changing_portions([n], sizes=(47, 2, 62, 3, 2, 17))):
            got = eu.run_schedule(runner_for(model, page_size=16, tokens=256), [prompt], schedule)[0]
            if dtype == "float32":
                assert worst(got, want) < F32_BOUND, place
            else:
                assert worst(got[asks:asks + 1], want[asks:asks + 1]) < 0.04, place
                assert worst(got, want) < BF16_WORST, place


@pytest.mark.parametrize("dtype,dim,vdim", [("float32", 16, 24), ("bfloat16", 64, 32), ("bfloat16", 128, 64)])
def test_edges_met_by_decoded_tokens(dtype, dim, vdim):
    """Every position of a window's passage decoded one by one: the key is found as long as
    it is inside, and not a step longer; a kept key for ever."""
    window, keep = 20, 4
    cfg, tensors = edge_model(dim, vdim, window, keep)
    model, _ = build(cfg, tensors=tensors, dtype=dtype)
    n = 75
    for place in (3, 4, 31):
        prompt = [ASK] * n                               # every token asks
        prompt[place] = SEEK
        want = plain.forward(cfg, tensors, prompt).float()
        # (one asking token without the key in sight gives the same row everywhere)
        gone = want[place + window:] - want[place + window - 1]
        if place >= keep:
            assert float(gone.abs().max()) > 0.1
        for first in (1, place, place + 2, place + window - 1):
            got = eu.run_schedule(runner_for(model, page_size=4, tokens=96), [prompt],
                                  eu.bulk_then_single([n], tail=n - first))[0]
            assert worst(got, want) < (F32_BOUND if dtype == "float32" else 0.05), (place, first)


@pytest.mark.parametrize("dtype,dim,vdim", [("float32", 16, 24), ("bfloat16", 64, 64), ("bfloat16", 96, 40),
                                            ("bfloat16", 128, 128), ("bfloat16", 256, 256)])
@pytest.mark.parametrize("window", [0, 600])
def test_a_far_key_is_found(dtype, dim, vdim, window):
    cfg, tensors = edge_model(dim, vdim, window, 2, heads=4, kv_heads=2)
    model, _ = build(cfg, tensors=tensors, dtype=dtype)
    n = 700
    for place in (0, 1, 15, 16, 64, 99, 100, 333):      # first tokens, page and tile borders
        prompt = [t % 298 for t in tu.tokens(n, 298, place)]
        prompt[place], prompt[-1] = SEEK, ASK
        other = list(prompt)
        other[place] = 5
        want = plain.forward(cfg, tensors, prompt).float()
        seen = not window or place < 2 or n - 1 - place < window
        moved = worst(plain.forward(cfg, tensors, other).float()[-1:], want[-1:])
        assert (moved > 0.3) == seen, place
        for schedule in (eu.whole([n]), eu.bulk_then_single([n], tail=3),
                         eu.changing_portions([n], sizes=(64, 2, 130, 17, 256))):
            got = eu.run_schedule(runner_for(model, page_size=16, tokens=1024), [prompt], schedule,
                                  wants=[[n - 1]])[0]
            assert worst(got, want[-1:]) < (F32_BOUND if dtype == "float32" else 0.04), place


# --------------------------------------------------------------- the sink's share
@pytest.mark.parametrize("dtype,dim,vdim", [("float32", 16, 24), ("bfloat16", 64, 64), ("bfloat16", 24, 16)])
def test_the_sink_counts_once_however_the_context_is_cut(dtype, dim, vdim):
    # sinks of about the logarithm of the number of keys take a good share of every head's
    # weight at 1,300 keys and nearly all of it at the first tokens: left out, or counted once
    # per range of a cut context, they would move every output by tens of percent
    cfg = tu.one_layer(tu.attention(heads=4, kv_heads=1, dim=dim, vdim=vdim, window=0, scale=0.02),
                       width=64, vocab=97)
    tensors = tu.make_tensors(cfg, seed=5)
    n = 1300
    prompt = tu.tokens(n, cfg["vocab"], 1)
    tensors["l0.mix.sink"] = torch.tensor([6.0, 7.0, 7.5, 8.0])
    # what the norm on the mixer's output would hide: the heads' shares differ, so their mix turns
    want = plain.forward(cfg, tensors, prompt).float()
    without = dict(tensors)
    without["l0.mix.sink"] = torch.full((4,), -30.0)
    assert worst(plain.forward(cfg, without, prompt).float()[-40:], want[-40:]) > 0.05
    twice = dict(tensors)
    twice["l0.mix.sink"] = tensors["l0.mix.sink"] + math.log(2.0)
    assert worst(plain.forward(cfg, twice, prompt).float()[-40:], want[-40:]) > 0.015
    model, _ = build(cfg, tensors=tensors, dtype=dtype)
    # one request decoding at 1,300 keys: its list of tiles is cut into ranges that are merged
    for schedule in (eu.whole([n]), eu.bulk_then_single([n], tail=40),
                     eu.changing_portions([n], sizes=(600, 2, 500, 64, 100, 3))):
        got = eu.run_schedule(runner_for(model, page_size=16, tokens=2048), [prompt], schedule)[0]
        for rows in (slice(-40, None), slice(0, 8)):             # far on, and the first tokens
            e = tu.row_error(got[rows], want[rows])
            assert float(e.max()) < (F32_BOUND if dtype == "float32" else 0.03)
            assert float(e.median()) < (F32_BOUND if dtype == "float32" else 0.01)


# ------------------------------------------------------------------- long decoding
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    cfg = tu.settled(tu.TINY_ALL)
    model, tensors = build(cfg, seed=21, dtype=dtype)
    n = 330
    prompts = [tu.tokens(n, cfg["vocab"], 5)]
    want = plain_logits(cfg, tensors, prompts)[0]
    runner = runner_for(model, page_size=16, tokens=512)       # decode steps replay from graphs
    assert runner.graphs is not None
    got = eu.run_schedule(runner, prompts, eu.bulk_then_single([n], tail=300))[0]
    if dtype == "float32":
        assert worst(got, want) < F32_BOUND
    else:
        assert_bfloat16_close(got, want)
    # the same steps issued kernel by kernel
    again = eu.run_schedule(runner_for(model, page_size=16, tokens=512, graphs=False), prompts,
                            eu.bulk_then_single([n], tail=300))[0]
    if dtype == "float32":
        assert worst(again, got) < 1e-5
    else:
        assert_bfloat16_same(again, got)


def test_pages_behind_the_window_serve_other_requests():
    """A pool far smaller than the requests are long: what the window leaves behind is used
    again, while the first tokens' pages stay with their request."""
    cfg = tu.config([tu.layer(tu.attention(window=12, keep=5), tu.dense()),
                     tu.layer(tu.attention(window=9, keep=2, kv_from=0), tu.moe())])
    model, tensors = build(cfg, seed=17)
    n = 160
    prompts = [tu.tokens(n, cfg["vocab"], 90 + i) for i in range(3)]
    want = plain_logits(cfg, tensors, prompts)
    steps = []
    for lo in range(0, n, 8):                            # all three together, eight tokens a step
        steps.append(([(i, lo, lo + 8) for i in range(3)], list(range(3)) if lo + 8 == n else []))
    runner = runner_for(model, page_size=4, tokens=96)
    got = eu.run_schedule(runner, prompts, steps)
    for g, w in zip(got, want):
        assert worst(g, w) < F32_BOUND
    assert runner.cache.pages_reused > 60
    assert runner.cache.groups[0].pool.high_water <= 24


# ------------------------------------------- unequal requests together and alone
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_batch_against_each_alone(dtype):
    cfg = tu.settled(tu.TINY_ALL)
    model, tensors = build(cfg, seed=2, dtype=dtype)
    lengths = [64, 3, 41, 17]
    prompts = [tu.tokens(n, cfg["vocab"], 40 + i) for i, n in enumerate(lengths)]
    alone = eu.run_schedule(runner_for(model, tokens=256), prompts, eu.whole(lengths))
    together = [([(i, 0, n) for i, n in enumerate(lengths)], list(range(len(lengths))))]
    got = eu.run_schedule(runner_for(model, tokens=256), prompts, together)
    if dtype == "float32":
        assert worst(torch.cat(got), torch.cat(alone)) < 1e-5
    else:
        assert_bfloat16_same(torch.cat(got), torch.cat(alone))


# --------------------------------------------------- at widths of real layers
@pytest.mark.parametrize("heads,kv,dim,vdim", [(8, 2, 64, 64), (4, 4, 128, 64), (6, 3, 96, 64), (4, 1, 192, 128)])
def test_wide_layers(heads, kv, dim, vdim):
    cfg = tu.config([
        tu.layer(tu.attention(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, window=100, keep=4,
                              scale=dim ** -0.5, rot_dims=dim // 2, base=1e4, scaling=tu.yarn()),
                 tu.dense(256, 3.0)),
        tu.layer(tu.attention(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, window=64, keep=70,
                              scale=dim ** -0.5, rot_dims=dim // 2, base=1e4, scaling=tu.yarn(),
                              kv_from=0), tu.moe(ff=64, experts=6, top=2, shared=128)),
    ], width=256, vocab=211)
    model, tensors = build(cfg, seed=6, dtype="bfloat16")
    lengths = [300, 70, 3]
    prompts = [tu.tokens(n, cfg["vocab"], 50 + i) for i, n in enumerate(lengths)]
    want = plain_logits(cfg, tensors, prompts)
    base = None
    for name, schedule in (("whole", eu.whole(lengths)),
                           ("bulk + tail", eu.bulk_then_single(lengths, tail=60)),
                           ("portions", eu.changing_portions(lengths, seed=3)),
                           ("mixed", eu.mixed(lengths, seed=1, max_live=3, decode_tail=30))):
        runner = runner_for(model, page_size=16, tokens=768, slots=3)
        got = eu.run_schedule(runner, prompts, schedule)
        assert_bfloat16_close(torch.cat(got), torch.cat(want), name)
        base = base or got
        assert_bfloat16_same(torch.cat(got), torch.cat(base), name)


# ------------------------------------------- generation through engine and scheduler
def test_greedy_generation():
    from zig_ai_amd.engine import Engine
    cfg = tu.TINY_ALL
    d, tensors = tu.folder(cfg, seed=8)
    engine = Engine(d, dtype="float32", page_size=4, num_pages=128, max_num_seqs=3,
                    max_num_batched_tokens=48, chunk_size=20, max_model_len=256)
    prompts = [tu.tokens(n, cfg["vocab"], 60 + i) for i, n in enumerate([33, 5, 70, 12, 1])]
    outs = engine.generate(prompts, max_new_tokens=20, temperature=0.0)
    assert all(len(o) == 20 for o in outs)
    for p, o in zip(prompts, outs):
        # every chosen token is the plain implementation's choice for the same history
        logits = plain.forward(cfg, tensors, p + o)
        for j, tok in enumerate(o):
            row = logits[len(p) + j - 1]
            assert float(row.max() - row[tok]) <= 1e-3 * float(row.abs().max()), (j, tok)
    assert len(engine.runner.cache.requests) == 0
    engine.runner.cache.check()


def test_generation_with_preemption():
    """A pool that cannot hold all requests: some are put back and computed again."""
    from zig_ai_amd.engine import Engine
    cfg = tu.one_layer(tu.attention(window=0), tu.moe())
    d, tensors = tu.folder(cfg, seed=9)
    engine = Engine(d, dtype="float32", page_size=4, num_pages=26, max_num_seqs=4,
                    max_num_batched_tokens=32, chunk_size=16, max_model_len=96)
    prompts = [tu.tokens(n, cfg["vocab"], 160 + i) for i, n in enumerate([20, 22, 18, 25])]
    outs = engine.generate(prompts, max_new_tokens=24, temperature=0.0)
    for p, o in zip(prompts, outs):
        logits = plain.forward(cfg, tensors, p + o)
        assert len(o) == 24
        for j, tok in enumerate(o):
            row = logits[len(p) + j - 1]
            assert float(row.max() - row[tok]) <= 1e-3 * float(row.abs().max()), (j, tok)


def test_generation_bfloat16_runs_through_graphs():
    from zig_ai_amd.engine import Engine
    cfg = tu.settled(tu.TINY_OTHER)
    d, tensors = tu.folder(cfg, seed=8)
    engine = Engine(d, dtype="bfloat16", page_size=16, num_pages=64, max_num_seqs=4,
                    max_model_len=256)
    assert engine.runner.graphs is not None        # every part can be recorded
    prompts = [tu.tokens(n, cfg["vocab"], 80 + i) for i, n in enumerate([40, 7, 19])]
    outs = engine.generate(prompts, max_new_tokens=24, temperature=0.0)
    for p, o in zip(prompts, outs):
        logits = plain.forward(cfg, tensors, p + o)
        for j, tok in enumerate(o):
            row = logits[len(p) + j - 1]
            spread = float(row.max() - row.min())
            assert float(row.max() - row[tok]) <= 0.1 * spread, (j, tok)


def test_trace_replay_and_command_line(tmp_path):
    import json
    import os
    import subprocess
    import sys
    cfg = tu.TINY_OTHER
    d, tensors = tu.folder(cfg, seed=12)
    prompt = tu.tokens(40, cfg["vocab"], 9)
    want = plain.forward(cfg, tensors, prompt).float()
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": prompt[:25], "want": [3, 24]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": prompt[25:27], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": prompt[27:], "want": [12]}], "end": ["a"]}]
    out = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d,
                          "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"],
                         input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
                         capture_output=True, timeout=600)
    assert out.returncode == 0, out.stderr[-2000:]
    assert [l for l in out.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    import numpy as np
    first = torch.from_numpy(np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, -1))
    last = torch.from_numpy(np.fromfile(tmp_path / "2.f32", dtype="<f4").reshape(1, -1))
    assert not (tmp_path / "1.f32").exists()
    assert worst(torch.cat([first, last]), want[[3, 24, 39]]) < F32_BOUND
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
def attention_case(dtype, nh, nkv, d, dv, requests, page_size, window, keep, chunk, seed, per_item):
    """Random keys and values in scattered pages and what attention over them is, row by row in
    float64.  ``requests``: (tokens in the cache before, new tokens).  Pages behind the window are
    not in the table, as after a commit."""
    g = torch.Generator().manual_seed(seed)
    S = len(requests)
    longest = max(c + n for c, n in requests)
    width = -(-longest // page_size) + 1
    n_pages = S * width + 2
    keys = torch.randn(n_pages, nkv, page_size, d, generator=g).to(dtype)
    values = torch.randn(n_pages, nkv, dv, page_size, generator=g).to(dtype)
    sink = torch.randn(nh, generator=g) + 1.0
    perm = torch.randperm(n_pages, generator=g)
    table = torch.full((S, width), -1, dtype=torch.int32)
    scale = 1.5 * d ** -0.5
    q = torch.randn(sum(n for _, n in requests), nh, d, generator=g).to(dtype)
    pos, want, iseq, irow, icnt = [], [], [], [], []
    row = 0
    for s, (ctx, n) in enumerate(requests):
        pages = perm[s * width:(s + 1) * width]
        used = -(-(ctx + n) // page_size)
        table[s, :used] = pages[:used].int()
        if window:
            for p in range(used):
                if (p + 1) * page_size <= ctx - window + 1 and p * page_size >= keep:
                    table[s, p] = -1
        k = keys[pages].permute(0, 2, 1, 3).reshape(width * page_size, nkv, d).double()
        v = values[pages].permute(0, 3, 1, 2).reshape(width * page_size, nkv, dv).double()
        for i in range(n):
            p = ctx + i
            pos.append(p)
            j = torch.arange(p + 1)
            inside = torch.ones(p + 1, dtype=torch.bool)
            if window:
                inside &= p - j < window
            if chunk:
                inside &= j // chunk == p // chunk
            inside |= j < keep
            out = torch.zeros(nh, dv, dtype=torch.float64)
            for h in range(nh):
                b = h // (nh // nkv)
                sc = k[:p + 1, b] @ q[row + i, h].double() * scale
                sc = torch.cat([sc[inside], sink[h:h + 1].double()])
                out[h] = torch.softmax(sc, dim=0)[:-1] @ v[:p + 1, b][inside]
            want.append(out)
        for lo in range(0, n, per_item):
            iseq.append(s)
            irow.append(row + lo)
            icnt.append(min(per_item, n - lo))
        row += n
    dev = torch.device("cuda")
    mk = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)
    # a page: the keys of all heads, then the values of all heads
    per_page = nkv * page_size * (d + dv)
    mem = torch.cat([keys.reshape(n_pages, -1), values.reshape(n_pages, -1)], dim=1).to(dev).contiguous()
    key_plane = mem[:, :nkv * page_size * d].unflatten(1, (nkv, page_size, d))
    value_plane = mem[:, nkv * page_size * d:per_page].unflatten(1, (nkv, page_size, dv))
    items = (mk(iseq), mk(irow), mk(icnt), len(iseq))
    return (q.to(dev), key_plane, value_plane, table.to(dev), mk(pos), items, scale, sink.to(dev),
            torch.stack(want))


SIZES = [(4, 2, 64, 64), (6, 6, 40, 24), (5, 1, 96, 40), (3, 3, 96, 96), (8, 2, 128, 64), (4, 1, 128, 96),
         (16, 1, 128, 128), (2, 2, 192, 72), (3, 1, 136, 128), (2, 1, 192, 192), (2, 1, 248, 128),
         (2, 1, 256, 256), (2, 2, 64, 32), (4, 2, 96, 64), (2, 2, 16, 160), (40, 2, 64, 64)]


@pytest.mark.parametrize("nh,nkv,d,dv", SIZES)
def test_planes_attention_kernels(nh, nkv, d, dv):
    from zig_ai_amd.kernels import ops
    G = nh // nkv
    cases = [(16, 0, 0, 0), (16, 50, 5, 0), (4, 1, 0, 0), (8, 33, 70, 0), (16, 0, 0, 48), (32, 130, 3, 0)]
    # prompt portions behind cached tokens, a first portion, single tokens, one token alone
    requests = [(70, 9), (0, 45), (233, 1), (0, 1), (131, 2)]
    per_item = max(1, ops.PLANES_ROWS // G)
    for page_size, window, keep, chunk in cases:
        q, kp, vp, table, pos, items, scale, sink, want = attention_case(
            torch.bfloat16, nh, nkv, d, dv, requests, page_size, window, keep, chunk, nh + d, per_item)
        shape = ops.ScoreShape(sink=sink, chunk=chunk, keep_first=keep)
        for tiles, nsplit in ((0, 1), (1, 3), (2, 2)):
            got = ops.planes_attention(q, kp, vp, table, pos, items, scale, window, tiles, nsplit,
                                       shape=shape).cpu().double()
            assert float((got - want).abs().max()) < 2.5e-2, (page_size, window, keep, chunk, nsplit)
    if G > ops.PLANES_DECODE_GROUP:
        return
    # single tokens only
    requests = [(200, 1), (0, 1), (63, 1), (64, 1), (700, 1)]
    for page_size, window, keep, chunk in cases:
        q, kp, vp, table, pos, items, scale, sink, want = attention_case(
            torch.bfloat16, nh, nkv, d, dv, requests, page_size, window, keep, chunk, d + dv, 1)
        shape = ops.ScoreShape(sink=sink, chunk=chunk, keep_first=keep)
        for tiles, nsplit in ((0, 1), (1, 5), (3, 2)):
            got = ops.planes_attention(q, kp, vp, table, pos, None, scale, window, tiles, nsplit,
                                       shape=shape).cpu().double()
            assert float((got - want).abs().max()) < 2.5e-2, (page_size, window, keep, chunk, nsplit)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh,nkv,d,dv", [(6, 2, 16, 24), (5, 1, 96, 40), (2, 1, 200, 136)])
def test_general_attention_with_kept_tokens(dtype, nh, nkv, d, dv):
    from zig_ai_amd.kernels import ops
    requests = [(70, 9), (0, 45), (233, 1), (0, 1), (131, 2)]
    per_item = max(1, ops.ATTENTION_MAX_ROWS // (nh // nkv))
    for page_size, window, keep, chunk in ((16, 50, 5, 0), (1, 1, 0, 0), (3, 33, 70, 0), (8, 130, 3, 0)):
        q, kp, vp, table, pos, items, scale, sink, want = attention_case(
            dtype, nh, nkv, d, dv, requests, page_size, window, keep, chunk, nh + d, per_item)
        shape = ops.ScoreShape(sink=sink, chunk=chunk, keep_first=keep)
        for keys, nsplit in ((0, 1), (64, 4)):
            got = ops.paged_attention_gated(q, kp, vp, table, pos, *items, scale, window, keys, nsplit,
                                            shape=shape).cpu().double()
            assert float((got - want).abs().max()) < (2e-5 if dtype == torch.float32 else 2e-2)


def test_kernels_that_know_no_kept_tokens_say_so():
    from zig_ai_amd.kernels import ops
    with pytest.raises(ops.KernelError):
        ops.ScoreShape(keep_first=3).args(4)
    with pytest.raises(ops.KernelError):
        ops.ScoreShape(keep_first=-1)
    assert not ops.planes_attention_supported(torch.bfloat16, 4, 2, 64, 64, shape=ops.ScoreShape(softcap=3.0))
    assert not ops.planes_attention_supported(torch.float32, 4, 2, 64, 64)
    assert not ops.planes_attention_supported(torch.bfloat16, 4, 2, 64, 64, page_size=2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh,nkv,d,dv,rot,adjacent,T", [(6, 2, 16, 24, 16, False, 11), (3, 3, 40, 8, 10, False, 150),
                                                        (16, 4, 128, 64, 128, False, 140),
                                                        (2, 1, 24, 24, 0, False, 5), (4, 2, 32, 16, 12, True, 9)])
def test_norm_over_all_heads_rotation_and_stores(dtype, nh, nkv, d, dv, rot, adjacent, T):
    from zig_ai_amd.kernels import ops
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(nh * d + T)
    stride = -(-((nh + nkv) * d + nkv * dv + 5) // 8) * 8
    qkv = (torch.randn(T, stride, generator=g) * 2).to(dtype)
    # (the last element of every head stands for one that was filled up: the mean leaves it out)
    qc, kc = nh * (d - 1), nkv * (d - 1)
    for h in range(nh + nkv):
        qkv[:, h * d + d - 1] = 0
    qw, kw = torch.randn(nh * d, generator=g), torch.randn(nkv * d, generator=g)
    inv = torch.rand(max(1, rot // 2), generator=g)
    mag, eps, page_size = 1.3, 1e-3, 8
    pos = torch.arange(37, 37 + T, dtype=torch.int32)
    n_pages = T // page_size + 3
    # most tokens side by side from a page's start on, a few elsewhere, one nowhere
    slots = torch.arange(8, 8 + T, dtype=torch.int32)
    slots[1], slots[-1] = -1, 3
    per_page = nkv * page_size * (d + dv)
    mem = torch.zeros(n_pages, per_page, dtype=dtype, device=dev)
    kp = mem[:, :nkv * page_size * d].unflatten(1, (nkv, page_size, d))
    vp = mem[:, nkv * page_size * d:].unflatten(1, (nkv, page_size, dv))
    args = (qkv.to(dev), pos.to(dev), slots.to(dev), qw.to(dev), kw.to(dev), inv.to(dev) if rot else None)
    q = ops.qk_norm_rope_kv_write_wide(*args, kp, vp, nh, nkv, d, dv, rot, adjacent, eps,
                                       magnitude=mag, row_norm=(qc, kc))

    def ready(cols, heads, w, count):
        x = cols.double()
        x = x / torch.sqrt((x * x).sum(dim=1, keepdim=True) / count + eps) * w.double()
        x = x.view(T, heads, d)
        out = x.clone()
        if rot:
            ang = pos.double()[:, None] * inv.double()[None, :]
            c, s = mag * torch.cos(ang)[:, None], mag * torch.sin(ang)[:, None]
            u, v = (slice(0, rot, 2), slice(1, rot, 2)) if adjacent else (slice(0, rot // 2), slice(rot // 2, rot))
            out[..., u] = x[..., u] * c - x[..., v] * s
            out[..., v] = x[..., v] * c + x[..., u] * s
        return out
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    want_q = ready(qkv[:, :nh * d], nh, qw, qc)
    assert float((q.cpu().double() - want_q).abs().max()) < tol * float(want_q.abs().max())
    want_k = ready(qkv[:, nh * d:(nh + nkv) * d], nkv, kw, kc)
    v = qkv[:, (nh + nkv) * d:(nh + nkv) * d + nkv * dv].view(T, nkv, dv)
    k_mem, v_mem = kp.cpu(), mem[:, nkv * page_size * d:].unflatten(1, (nkv, dv, page_size)).cpu()
    for t in range(T):
        if slots[t] < 0:
            continue
        page, off = int(slots[t]) // page_size, int(slots[t]) % page_size
        assert float((k_mem[page, :, off].double() - want_k[t]).abs().max()) < tol * float(want_k.abs().max())
        assert torch.equal(v_mem[page, :, :, off], v[t])
    # queries only: rows without keys and values, nothing stored
    rows = qkv[:, :nh * d].contiguous()
    alone = ops.qk_norm_rope_kv_write_wide(rows.to(dev), *args[1:2], None, args[3], None, args[5], None, None,
                                           nh, 0, d, dv, rot, adjacent, eps, write_kv=False,
                                           magnitude=mag, row_norm=(qc, kc))
    assert torch.equal(alone, q)
    # and the per-head norm of the same path with the factor on the rotation
    if rot == d:
        per_head = ops.qk_norm_rope_kv_write_wide(
            args[0], args[1], None, qw[:d].contiguous().to(dev), kw[:d].contiguous().to(dev), args[5],
            None, None, nh, nkv, d, dv, rot, adjacent, eps, write_kv=False, magnitude=mag)
        plainer = ops.qk_norm_rope_kv_write_wide(
            args[0], args[1], None, qw[:d].contiguous().to(dev), kw[:d].contiguous().to(dev), args[5],
            None, None, nh, nkv, d, dv, rot, adjacent, eps, write_kv=False)
        assert float((per_head.double() - mag * plainer.double()).abs().max()) < tol * float(plainer.abs().max())


@pytest.mark.parametrize("M,I,K", [(1, 40, 64), (8, 300, 512), (16, 128, 2048), (5, 72, 1000)])
def test_bounded_unit_in_the_product(M, I, K):
    from zig_ai_amd.kernels import ops
    g = torch.Generator().manual_seed(M + I)
    x = torch.randn(M, K, generator=g).to(torch.bfloat16)
    w = (torch.randn(2 * I, K, generator=g) * 1.5 * K ** -0.5).to(torch.bfloat16)
    for limit in (0.0, 0.8):
        got = ops.linear_swiglu(x.cuda(), w.cuda(), bounded=(limit, 1.702, 1.0)).cpu().double()
        gu = x.double() @ w.double().T
        a, u = gu[:, :I], gu[:, I:]
        if limit:
            a, u = a.clamp(max=limit), u.clamp(-limit, limit)
        want = a * torch.sigmoid(1.702 * a) * (u + 1.0)
        assert float((got - want).abs().max()) < 1e-2 * float(want.abs().max()), limit


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [36, 256, 3000])
def test_normed_rows_of_the_embedding(dtype, width):
    from zig_ai_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    table = (torch.randn(19, width, generator=g) * 3).to(dtype)
    w = torch.randn(width, generator=g)
    ids = torch.randint(0, 19, (7,), generator=g, dtype=torch.int32)
    want = plain.rms_norm(table[ids.long()].double(), w.double(), 1e-2)
    rows, copy = ops.embed_norm(ids.cuda(), table.cuda(), w.cuda(), 1e-2, torch.bfloat16)
    assert float((rows.cpu().double() - want).abs().max()) < 1e-5 * float(want.abs().max())
    assert torch.equal(copy, rows.to(torch.bfloat16))
    assert ops.embed_norm(ids.cuda(), table.cuda(), w.cuda(), 1e-2)[1] is None


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("E,top,N,K,T", [(5, 2, 24, 40, 3), (4, 3, 72, 64, 50), (3, 2, 200, 136, 300), (9, 1, 8, 24, 1)])
def test_grouped_products_with_gates_and_weights(dtype, E, top, N, K, T):
    """The gated unit on the product's own sums, weights an assignment ahead of it and behind
    the plain product, results written as planes of a given stack: decode batches, tiles of 64
    rows and tiles of 128."""
    from zig_ai_amd.kernels import ops
    dev = torch.device("cuda")
    g = torch.Generator().manual_seed(E * N + T)
    x = torch.randn(T, K, generator=g).to(dtype)
    w = (torch.randn(E, 2 * N, K, generator=g) * 1.5 * K ** -0.5).to(dtype)
    chosen = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).int()
    weight = torch.rand(T, top, generator=g) + 0.2
    lists, counts = ops.expert_lists(None, chosen.to(dev), T, E)
    sums = torch.stack([w[chosen[t, j]].double() @ x[t].double() for t in range(T) for j in range(top)])
    a, u = sums[:, :N], sums[:, N:]
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    r = weight.reshape(-1, 1).double()
    wants = {"silu": (a * torch.sigmoid(a) * u, dict(gate="silu")),
             "gelu": (torch.nn.functional.gelu(a, approximate="tanh") * u, dict(gate="gelu_tanh")),
             "bounded": ((lambda p, q: p * torch.sigmoid(1.7 * p) * (q + 0.5))(
                 (r * a).clamp(max=0.8), (r * u).clamp(-0.8, 0.8)),
                 dict(bounded=(0.8, 1.7, 0.5), row_weight=weight.to(dev)))}
    for name, (want, kw) in wants.items():
        for out_dtype in (dtype, torch.float32):
            got = ops.grouped_linear(x.to(dev), w.to(dev), lists, counts, T, per_token=True,
                                     out_dtype=out_dtype, **kw).cpu().double()
            assert float((got - want).abs().max()) < tol * float(want.abs().max()), (name, out_dtype)
    rows = torch.randn(T * top, K, generator=g).to(dtype)
    want = torch.stack([r[i] * (w[chosen.reshape(-1)[i]].double() @ rows[i].double()) for i in range(T * top)])
    stack = torch.full((top + 1, T, 2 * N), 7.0, dtype=torch.float32, device=dev)
    ops.grouped_linear(rows.to(dev), w.to(dev), lists, counts, T, per_token=False, stacked=True,
                       row_weight=weight.to(dev), out=stack[:top])
    got = stack[:top].permute(1, 0, 2).reshape(T * top, 2 * N).cpu().double()
    assert float((got - want).abs().max()) < tol * float(want.abs().max())
    assert bool((stack[top] == 7.0).all())
    # a plain product into the plane behind
    ops.linear(x.to(dev), w[0].contiguous().to(dev), out_dtype=torch.float32, into=stack[top])
    want = x.double() @ w[0].double().T
    assert float((stack[top].cpu().double() - want).abs().max()) < tol * float(want.abs().max())
