"""Torisun's configuration and description as parts (no GPU), and what pins the plain
implementation's mechanisms: identities that a consistent mistake would break."""

import copy
import math

import pytest
import torch

import plain_torisun as plain
import torisun_util as tu
from zig_ai_amd.config import ConfigError, config_from_dict, known_architectures, load_config
from zig_ai_amd.parts import lookup
from zig_ai_amd.parts.base import PagedNeed
from zig_ai_amd.weights.loader import expected_tensors


def test_registered_and_round_trip():
    assert "Torisun" in known_architectures()
    for cfg in (tu.TINY_ALL, tu.TINY_OTHER) + tuple(tu.random_config(s) for s in range(20)):
        typed = config_from_dict(cfg)
        assert config_from_dict(typed.to_dict()) == typed
        assert typed.to_dict() == cfg
        assert typed.hidden_size == cfg["width"] and typed.vocab_size == cfg["vocab"]


@pytest.mark.parametrize("cfg", [tu.TINY_ALL, tu.TINY_OTHER] + [tu.random_config(s) for s in range(6)])
def test_every_tensor_is_named_with_its_shape(cfg):
    tensors = tu.make_tensors(cfg)
    spec = config_from_dict(cfg).to_spec()
    expected = {e.names[0]: tuple(e.rule.shapes[0]) for e in expected_tensors(spec)}
    assert set(expected) == set(tensors)
    for name, shape in expected.items():
        assert tuple(tensors[name].shape) == shape, name


def test_what_a_config_may_leave_out():
    cfg = copy.deepcopy(tu.TINY_ALL)
    m = cfg["layers"][2]["mixer"]
    for key in ("kv_heads", "vdim", "scale", "mask"):
        del m[key]
    del cfg["layers"][1]["mlp"]["router"]["scale"]
    del cfg["layers"][0]["mixer"]["mask"]["keep_first"]
    typed = config_from_dict(cfg)
    s = typed.layers[2].attention
    assert (s.kv_heads, s.vdim, s.window, s.keep_first) == (4, 24, 0, 0)
    assert s.scale == 24 ** -0.5
    assert typed.layers[1].mlp.route_scale == 1.0
    assert typed.layers[0].attention.keep_first == 0 and typed.layers[0].attention.window == 20


def needs(spec):
    return [lookup("mixer", l.parts["mixer"].kind).cache_need(l.parts["mixer"].params)
            for l in spec.layers]


def test_run_order_and_what_the_cache_holds():
    spec = config_from_dict(tu.TINY_ALL).to_spec()
    assert [(c.layer, c.cache, c.writes_cache) for c in spec.schedule] == [
        (0, 0, True), (1, 0, False), (2, 2, True), (3, 0, False), (4, 4, True)]
    # the entry holds what its writer and its readers need together
    shared = PagedNeed(((2, 16), (2, 24)), 33, keep_first=7)
    got = needs(spec)
    assert got[0] == got[1] == got[3] == shared
    assert got[2] == PagedNeed(((4, 24), (4, 8)), 9) and got[4] == PagedNeed(((1, 8), (1, 40)))
    assert not spec.layers[1].parts["mixer"].params["makes_kv"]
    assert "k_proj.weight" not in spec.layers[1].parts["mixer"].tensors
    # a reader without a window keeps every key; head widths are filled up to multiples of 8
    other = config_from_dict(tu.TINY_OTHER).to_spec()
    got = needs(other)
    assert got[1] == got[2] == PagedNeed(((1, 16), (1, 32)))
    assert got[0] == PagedNeed(((1, 24), (1, 16)), 1, keep_first=2)


def test_constants_reach_the_parts():
    spec = config_from_dict(tu.TINY_ALL).to_spec()
    a = spec.layers[0].parts["mixer"].params
    assert (a["window"], a["keep_first"], a["qk_norm"], a["sink"]) == (20, 3, "row", True)
    assert a["position"].params == {"head_dim": 16, "rotary_dim": 16, "theta": 300.0,
                                    "pairing": "half", "scaling": dict(tu.yarn(), type="yarn")}
    b = spec.layers[1].parts["mixer"].params
    assert b["softmax_scale"] == 0.3 and (b["window"], b["keep_first"]) == (33, 7)
    c = spec.layers[2].parts["mixer"].params
    assert c["position"].params["rotary_dim"] == 10 and "scaling" not in c["position"].params
    assert spec.layers[4].parts["mixer"].params["position"] is None
    ff = spec.layers[0].parts["feed_forward"]
    assert ff.kind == "clamped_glu" and (ff.params["limit"], ff.params["alpha"], ff.params["up_offset"]) \
        == (0.9, 1.702, 1.0)
    ff = spec.layers[1].parts["feed_forward"].params
    assert (ff["experts"], ff["top"], ff["intermediate_size"], ff["shared_size"]) == (5, 2, 24, 40)
    assert ff["scores"] == "sigmoid" and ff["renormalize"] and ff["route_scale"] == 1.7
    assert ff["activation"] == "silu"
    assert spec.layers[3].parts["feed_forward"].params["shared_size"] == 0
    assert spec.layers[0].arrangement == "normed_output"
    assert spec.layers[2].arrangement == "normed_output_no_ff"
    assert spec.ignored_tensors == ("l2.norm2",)
    assert spec.lm_head.params["tied"] and spec.embedding.params["norm"]
    assert spec.embedding.tensors["norm.weight"] == ("embed.norm",)


@pytest.mark.parametrize("breakage", [
    lambda c: c["layers"][0].update(type="attention_2"),
    lambda c: c["layers"][0]["mixer"].pop("dim"),
    lambda c: c["layers"][0]["mixer"].update(kv_heads=4),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7),
    lambda c: c["layers"][0]["mixer"]["rot"].pop("base"),
    lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(scaling=3),
    lambda c: c["layers"][0]["mixer"].update(mask=5),
    lambda c: c["layers"][0]["mixer"]["mask"].update(size=0),
    lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=-1),
    lambda c: c["layers"][0]["mixer"].update(scale=0.0),
    lambda c: c["layers"][1]["mixer"].update(kv_from=1),
    lambda c: c["layers"][1]["mixer"].update(kv_from=9),
    lambda c: c["layers"][3]["mixer"].update(kv_from=1),        # no keys of its own there
    lambda c: c["layers"][3]["mixer"].update(kv_from=2),        # other heads
    lambda c: c["layers"][1]["mixer"].update(vdim=16),
    lambda c: c["layers"][1]["mixer"]["rot"].update(base=20.0),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=9),
    lambda c: c["layers"][1]["mlp"].pop("expert"),
    lambda c: c["layers"][1]["mlp"].update(shared=3),
    lambda c: c["layers"][0]["mlp"].update(kind="glu"),
    lambda c: c["layers"][0]["mlp"].pop("ff"),
    lambda c: c.pop("norm"),
    lambda c: c.update(layers=[]),
])
def test_malformed_configurations(breakage):
    cfg = copy.deepcopy(tu.TINY_ALL)
    breakage(cfg)
    with pytest.raises(ConfigError):
        config_from_dict(cfg)


def test_random_model_folder(tmp_path):
    from zig_ai_amd.weights.random_init import write_random_model
    from zig_ai_amd.weights.safetensors_io import Checkpoint
    write_random_model(tu.TINY_ALL, str(tmp_path), seed=3)
    ckpt = Checkpoint(str(tmp_path))
    assert set(ckpt.names()) == set(tu.make_tensors(tu.TINY_ALL))
    assert tuple(ckpt.shape("l0.mix.q.norm")) == (96,)
    assert load_config(str(tmp_path)) == config_from_dict(tu.TINY_ALL)


# ----------------------------------------------- what pins the plain implementation
def test_stretched_frequencies_by_hand():
    # pair(t) = 16 ln(1000 / (2 pi t)) / (2 ln 10000): 1.995 turns at t=16 -> lo 1; 4.40 -> hi 5
    rot = {"dims": 16, "base": 10000.0,
           "scaling": {"factor": 8.0, "original": 1000, "fast": 16.0, "slow": 1.0}}
    freq, magnitude = plain.frequencies(rot)
    base = [10000.0 ** (-2 * i / 16) for i in range(8)]
    for i, share in enumerate((0, 0, 0.25, 0.5, 0.75, 1, 1, 1)):
        assert abs(freq[i] - base[i] * (share / 8.0 + 1 - share)) < 1e-15
    assert abs(magnitude - (1 + 0.1 * math.log(8.0))) < 1e-15


def test_rotation_depends_on_distance_only():
    g = torch.Generator().manual_seed(1)
    rot = {"dims": 8, "base": 100.0, "scaling": tu.yarn()}
    q = torch.randn(1, 1, 12, generator=g, dtype=torch.float64)
    k = torch.randn(1, 1, 12, generator=g, dtype=torch.float64)

    def dot(pq, pk):
        return float((plain.rotate(q, torch.tensor([pq]), rot)
                      * plain.rotate(k, torch.tensor([pk]), rot)).sum())
    assert abs(dot(17, 5) - dot(112, 100)) < 1e-9
    m = plain.frequencies(rot)[1]
    q0, k0 = q[0, 0], k[0, 0]
    assert abs(dot(4, 4) - float(m * m * (q0 * k0)[:8].sum() + (q0 * k0)[8:].sum())) < 1e-9
    turned = plain.rotate(q, torch.tensor([3]), rot)[0, 0]
    assert abs(float(turned[0] ** 2 + turned[4] ** 2) - m * m * float(q0[0] ** 2 + q0[4] ** 2)) < 1e-9


def test_visible_keys_by_hand():
    sees = plain.visible(8, {"size": 3, "keep_first": 2})
    assert sees.int().tolist() == [
        [1, 0, 0, 0, 0, 0, 0, 0], [1, 1, 0, 0, 0, 0, 0, 0], [1, 1, 1, 0, 0, 0, 0, 0],
        [1, 1, 1, 1, 0, 0, 0, 0], [1, 1, 1, 1, 1, 0, 0, 0], [1, 1, 0, 1, 1, 1, 0, 0],
        [1, 1, 0, 0, 1, 1, 1, 0], [1, 1, 0, 0, 0, 1, 1, 1]]
    assert plain.visible(5, None).int().sum() == 15
    assert plain.visible(5, {"size": 1, "keep_first": 0}).int().equal(torch.eye(5, dtype=torch.int32))


def test_one_norm_over_all_heads():
    """Scaling one head's rows of the key projection changes what the other heads see."""
    cfg = tu.one_layer(tu.attention(rot_dims=0, window=0))
    t = tu.make_tensors(cfg, 2)
    m = cfg["layers"][0]["mixer"]
    h = torch.randn(4, cfg["width"], dtype=torch.float64, generator=torch.Generator().manual_seed(5))
    k, _ = plain.keys_values(h, t, "l0.mix.", m, 1e-5)
    raw = h @ t["l0.mix.k"].double().T
    for r in range(4):
        whole = math.sqrt(float((raw[r] ** 2).mean()) + 1e-5)
        assert torch.allclose(k[r].reshape(-1), raw[r] / whole * t["l0.mix.k.norm"].double())
    louder = dict(t)
    louder["l0.mix.k"] = t["l0.mix.k"].clone()
    louder["l0.mix.k"][:16] *= 10
    other, _ = plain.keys_values(h, louder, "l0.mix.", m, 1e-5)
    assert float((other[:, 1] - k[:, 1]).abs().max()) > 0.1 * float(k[:, 1].abs().max())


def test_sink_is_one_more_score_without_a_value():
    cfg = tu.one_layer(tu.attention(window=0))
    t = tu.make_tensors(cfg, 4)
    m = cfg["layers"][0]["mixer"]
    H, G, dv = m["heads"], m["kv_heads"], m["vdim"]
    h = torch.randn(7, cfg["width"], dtype=torch.float64, generator=torch.Generator().manual_seed(2))
    got, (k, v) = plain.attention(h, t, "l0.mix.", m, 1e-5)
    q = plain.rotate(plain.rms_norm(h @ t["l0.mix.q"].double().T, t["l0.mix.q.norm"].double(), 1e-5)
                     .view(7, H, -1), torch.arange(7), m["rot"])
    out = torch.zeros(7, H, dv, dtype=torch.float64)
    for i in range(7):
        for a in range(H):
            b = a // (H // G)
            s = torch.cat([k[:i + 1, b] @ q[i, a] * m["scale"], t["l0.mix.sink"][a:a + 1].double()])
            out[i, a] = torch.softmax(s, dim=0)[:-1] @ v[:i + 1, b]
    assert torch.allclose(got, out.reshape(7, -1) @ t["l0.mix.o"].double().T)


def test_chosen_weights_sum_to_the_scale():
    cfg = tu.one_layer(tu.attention(), tu.moe(experts=6, top=3, scale=0.8, shared=16))
    t = tu.make_tensors(cfg, 1)
    mlp = cfg["layers"][0]["mlp"]
    h = torch.randn(9, cfg["width"], dtype=torch.float64, generator=torch.Generator().manual_seed(3))
    chosen, weight = plain.route(h, t, "l0.mlp.", mlp["router"])
    assert torch.allclose(weight.sum(dim=1), torch.full((9,), 0.8, dtype=torch.float64))
    # the shared expert is added as it is
    y = plain.experts(h, t, "l0.mlp.", mlp)
    alone = sum(weight[:, j:j + 1] * torch.stack([plain.expert(h[r:r + 1], t, f"l0.mlp.e{int(e)}.")[0]
                                                  for r, e in enumerate(chosen[:, j])])
                for j in range(3))
    assert torch.allclose(y - alone, plain.expert(h, t, "l0.mlp.shared."))


def test_bounds_of_the_dense_feed_forward():
    cfg = tu.one_layer(tu.attention(), tu.dense(limit=0.5))
    t = tu.make_tensors(cfg, 1)
    h = torch.randn(5, cfg["width"], dtype=torch.float64, generator=torch.Generator().manual_seed(3))
    assert float(plain.dense(0 * h, t, "l0.mlp.", 0.5).abs().max()) == 0.0
    huge = plain.dense(1e6 * h, t, "l0.mlp.", 0.5)
    most = 0.5 * 1.5 * t["l0.mlp.down"].double().abs().sum(dim=1)
    assert bool((huge.abs() <= most[None, :]).all())


def test_every_mechanism_matters():
    """The plain implementation with one mechanism changed is far from itself: what the
    engine is held to would notice each of them."""
    cfg = tu.TINY_ALL
    tensors = tu.make_tensors(cfg, seed=4)
    prompt = tu.tokens(60, cfg["vocab"], 3)
    want = plain.forward(cfg, tensors, prompt).float()

    def changed(edit):
        c, t = copy.deepcopy(cfg), dict(tensors)
        edit(c, t)
        return float(tu.row_error(plain.forward(c, t, prompt).float(), want).max())

    def window(c, t): c["layers"][0]["mixer"]["mask"]["size"] += 1
    def kept(c, t): c["layers"][1]["mixer"]["mask"]["keep_first"] += 1
    def scaling(c, t): c["layers"][0]["mixer"]["rot"]["scaling"]["factor"] = 1.0
    def partial(c, t): c["layers"][2]["mixer"]["rot"]["dims"] = 24
    def sink(c, t): t["l3.mix.sink"] = t["l3.mix.sink"] - 2.0
    def source(c, t): t["l0.mix.v"] = -t["l0.mix.v"]
    def router_scale(c, t): c["layers"][1]["mlp"]["router"]["scale"] = 1.0
    def shared(c, t): t["l1.mlp.shared.down"] = 0 * t["l1.mlp.shared.down"]
    def limit(c, t): c["layers"][0]["mlp"]["limit"] = 100.0
    def embed_norm(c, t): t["embed.norm"] = torch.ones_like(t["embed.norm"])
    for edit in (window, kept, scaling, partial, sink, source, router_scale, shared, limit, embed_norm):
        assert changed(edit) > 0.02, edit.__name__
