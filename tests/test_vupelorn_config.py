"""Vupelorn's configuration and description as parts (no GPU), and what pins the plain
implementation's mechanisms: identities that a consistent mistake would break."""

import copy
import json
import math

import pytest
import torch

import plain_vupelorn as plain
import vupelorn_util as vu
from zig_ai_amd.config import ConfigError, config_from_dict, known_architectures, load_config
from zig_ai_amd.weights.loader import expected_tensors


def test_registered_and_round_trip():
    assert "Vupelorn" in known_architectures()
    for cfg in (vu.TINY_ALL, vu.TINY_OTHER) + tuple(vu.random_config(s) for s in range(20)):
        typed = config_from_dict(cfg)
        assert config_from_dict(typed.to_dict()) == typed
        assert typed.to_dict() == cfg
        assert typed.hidden_size == cfg["width"] and typed.vocab_size == cfg["vocab"]


@pytest.mark.parametrize("cfg", [vu.TINY_ALL, vu.TINY_OTHER] + [vu.random_config(s) for s in range(6)])
def test_every_tensor_is_named_with_its_shape(cfg):
    tensors = vu.make_tensors(cfg)
    spec = config_from_dict(cfg).to_spec()
    expected = {e.names[0]: tuple(e.rule.shapes[0]) for e in expected_tensors(spec)}
    assert set(expected) == set(tensors)
    for name, shape in expected.items():
        assert tuple(tensors[name].shape) == shape, name


def test_decay_ranks_come_from_the_tensors():
    d, tensors = vu.folder(vu.TINY_ALL)
    assert "decay_rank" not in json.load(open(d + "/config.json"))["layers"][1]["mixer"]
    read = load_config(d)
    assert read.layers[1].gla.decay_rank == 16            # the default, until tensors are seen
    read = read.with_shapes(lambda name: tuple(tensors[name].shape) if name in tensors else None)
    assert [l.gla.decay_rank for l in read.layers if l.gla is not None] == [8, 16]
    assert read == config_from_dict(vu.TINY_ALL)


def test_run_order_and_shared_rows():
    spec = config_from_dict(vu.TINY_ALL).to_spec()
    assert [(c.layer, c.cache, c.writes_cache) for c in spec.schedule] == [
        (0, 0, True), (1, 1, True), (2, 2, True), (3, 2, False), (4, 4, True)]
    assert not spec.layers[3].parts["mixer"].params["makes_rows"]
    assert "kv_down.weight" not in spec.layers[3].parts["mixer"].tensors
    other = config_from_dict(vu.TINY_OTHER).to_spec()
    assert [c.cache for c in other.schedule] == [0, 1, 1, 3, 1]
    assert [c.writes_cache for c in other.schedule] == [True, True, False, True, False]
    from zig_ai_amd.parts import lookup
    needs = [lookup("mixer", l.parts["mixer"].kind).cache_need(l.parts["mixer"].params)
             for l in spec.layers]
    assert needs[0].planes == ((1, 40),) and needs[2] == needs[3]
    assert needs[1].shape == (2 * 16 * 24,) and needs[1].dtype == torch.float32
    keeps = lookup("embedding", spec.embedding.kind).cache_need(spec.embedding.params)
    assert keeps.shape == (1,) and keeps.dtype == torch.int32
    assert lookup("embedding", other.embedding.kind).cache_need(other.embedding.params) is None


def test_constants_reach_the_parts():
    spec = config_from_dict(vu.TINY_ALL).to_spec()
    a = spec.layers[0].parts["mixer"].params
    assert a["gate"] is None and not a["sink"] and a["makes_rows"]
    assert a["position"].params == {"head_dim": 8, "rotary_dim": 8, "theta": 300.0,
                                    "pairing": "half", "scaling": dict(vu.yarn(), type="yarn")}
    b = spec.layers[3].parts["mixer"].params
    assert b["position"].params["pairing"] == "adjacent" and "scaling" not in b["position"].params
    assert b["softmax_scale"] == 0.17
    c = spec.layers[4].parts["mixer"]
    assert c.kind == "gated_linear" and c.params["decay_root"] == 16.0 and c.params["decay_rank"] == 16
    assert c.tensors["decay_up.bias"] == ("l4.mix.a2.b",)
    ff = spec.layers[1].parts["feed_forward"].params
    assert (ff["experts"], ff["top"], ff["intermediate_size"], ff["bound"]) == (3, 1, 16, 0.7)
    assert ff["scores"] == "sigmoid" and ff["weight_on"] == "input" and not ff["renormalize"]
    assert (ff["gate_slope"], ff["up_offset"]) == (1.702, 1.0)
    assert spec.layers[0].arrangement == "normed_output"
    assert spec.layers[2].arrangement == "normed_output_no_ff"
    assert spec.ignored_tensors == ("l2.norm2", "l4.norm2")
    assert spec.lm_head.params["tied"]
    assert spec.embedding.params["pair"] == {"buckets": 97, "mul_prev": 29, "mul_cur": 13}


@pytest.mark.parametrize("breakage", [
    lambda c: c["layers"][0].update(type="attention"),
    lambda c: c["layers"][0]["mixer"].pop("kv_rank"),
    lambda c: c["layers"][0]["mixer"].pop("rot"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7),
    lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(scaling=3),
    lambda c: c["layers"][3]["mixer"].update(kv_from=3),
    lambda c: c["layers"][3]["mixer"].update(kv_from=9),
    lambda c: c["layers"][3]["mixer"].update(kv_from=1),        # no latent there
    lambda c: c["layers"][3]["mixer"].update(kv_from=0),        # another rotation
    lambda c: c["layers"][3]["mixer"].update(kv_rank=16),
    lambda c: c["layers"][3]["mixer"]["rot"].update(base=20.0),
    lambda c: c["layers"].append(dict(c["layers"][3], mixer=dict(c["layers"][3]["mixer"], kv_from=3))),
    lambda c: c["layers"][1]["mixer"].pop("tau"),
    lambda c: c["layers"][1]["mixer"].update(tau=0.0),
    lambda c: c["layers"][0]["mlp"]["router"].update(top=9),
    lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"),
    lambda c: c["layers"][0]["mlp"].update(kind="dense"),
    lambda c: c["embedding"]["bigram"].pop("mul_cur"),
    lambda c: c["embedding"].update(bigram=5),
    lambda c: c.pop("norm"),
    lambda c: c.update(layers=[]),
])
def test_malformed_configurations(breakage):
    cfg = copy.deepcopy(vu.TINY_ALL)
    breakage(cfg)
    with pytest.raises(ConfigError):
        config_from_dict(cfg)


def test_random_model_folder(tmp_path):
    from zig_ai_amd.weights.random_init import write_random_model
    from zig_ai_amd.weights.safetensors_io import Checkpoint
    write_random_model(vu.TINY_ALL, str(tmp_path), seed=3)
    ckpt = Checkpoint(str(tmp_path))
    assert set(ckpt.names()) == set(vu.make_tensors(vu.TINY_ALL))
    assert tuple(ckpt.shape("bigram")) == (98, vu.TINY_ALL["width"])


# -------------------------------------------------- the stretched rotation's table
@pytest.mark.parametrize("dims,base,scaling", [(8, 300.0, vu.yarn()), (64, 1e4, vu.yarn(40.0, 4096, 32.0, 1.0)),
                                               (2, 10.0, vu.yarn(2.0, 16, 4.0, 1.0)),
                                               (32, 5e5, vu.yarn(16.0, 100, 3.0, 2.9)),
                                               (24, 50.0, vu.yarn(1.0, 64, 8.0, 0.5))])
def test_frequencies_of_the_part(dims, base, scaling):
    from zig_ai_amd.parts import lookup
    from zig_ai_amd.parts.base import Runtime
    part = lookup("position", "rope")({"head_dim": dims, "rotary_dim": dims, "theta": base,
                                       "scaling": dict(scaling, type="yarn")}, {},
                                      Runtime(torch.device("cpu"), torch.float32))
    freq, factor = plain.frequencies({"dims": dims, "base": base, "scaling": scaling})
    assert torch.allclose(part.inv_freq, torch.tensor(freq, dtype=torch.float32), rtol=1e-6)
    assert abs(part.magnitude - factor) < 1e-12
    if scaling["factor"] != 1.0:
        with pytest.raises(ValueError):
            part.without_magnitude()
    else:
        assert part.without_magnitude() is part


# ----------------------------------------------- what pins the plain implementation
def test_stretched_frequencies_by_hand():
    # the pairs that turn often keep their frequency, those that never finish a turn are
    # divided by the factor, and the ones between are mixed in equal steps
    rot = {"dims": 16, "base": 10000.0,
           "scaling": {"factor": 8.0, "original": 1000, "fast": 16.0, "slow": 1.0}}
    freq, magnitude = plain.frequencies(rot)
    # pair(t) = 16 ln(1000 / (2 pi t)) / (2 ln 10000): 1.995 turns at t=16 -> lo 1; 4.40 -> hi 5
    lo = 16 * math.log(1000 / (2 * math.pi * 16)) / (2 * math.log(10000))
    hi = 16 * math.log(1000 / (2 * math.pi)) / (2 * math.log(10000))
    assert (math.floor(lo), math.ceil(hi)) == (1, 5)
    base = [10000.0 ** (-2 * i / 16) for i in range(8)]
    for i, share in enumerate((0, 0, 0.25, 0.5, 0.75, 1, 1, 1)):
        assert abs(freq[i] - base[i] * (share / 8.0 + 1 - share)) < 1e-15
    assert abs(magnitude - (1 + 0.1 * math.log(8.0))) < 1e-15


@pytest.mark.parametrize("interleaved", [False, True])
def test_rotation_depends_on_distance_only(interleaved):
    g = torch.Generator().manual_seed(1)
    rot = {"dims": 8, "base": 100.0, "scaling": vu.yarn()}
    q = torch.randn(1, 12, generator=g, dtype=torch.float64)
    k = torch.randn(1, 12, generator=g, dtype=torch.float64)

    def dot(pq, pk):
        return float((plain.rotate(q, torch.tensor([pq]), rot, interleaved)
                      * plain.rotate(k, torch.tensor([pk]), rot, interleaved)).sum())
    assert abs(dot(17, 5) - dot(112, 100)) < 1e-9
    m = plain.frequencies(rot)[1]
    assert abs(dot(4, 4) - float(m * m * (q * k)[:, :8].sum() + (q * k)[:, 8:].sum())) < 1e-9
    turned = plain.rotate(q, torch.tensor([3]), rot, interleaved)
    i, j = (0, 1) if interleaved else (0, 4)
    assert abs(float(turned[0, i] ** 2 + turned[0, j] ** 2) - m * m * float(q[0, i] ** 2 + q[0, j] ** 2)) < 1e-9


def test_pair_rows_by_hand():
    assert plain.pair_rows([5, 7, 7, 0], 11, 3, 2) == [11, (15 + 14) % 11, (21 + 14) % 11, (21 + 0) % 11]
    assert plain.pair_rows([5], 11, 3, 2) == [11]


def test_recurrence_is_a_decayed_sum():
    """The read-out equals the sum over earlier tokens of their values, each weighted by a
    product of query, key and the decays in between, taken channel by channel."""
    cfg = vu.one_layer("gla", vu.gla())
    t = vu.make_tensors(cfg, 4)
    m = cfg["layers"][0]["mixer"]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    h = torch.randn(9, cfg["width"], dtype=torch.float64, generator=torch.Generator().manual_seed(2))
    w = {k: v.double() for k, v in t.items()}
    a = plain.decays(h, t, "l0.mix.", m["tau"]).view(9, H, d)
    q = (h @ w["l0.mix.q"].T).view(9, H, d) / math.sqrt(d)
    k = (h @ w["l0.mix.k"].T).view(9, H, d)
    v = (h @ w["l0.mix.v"].T).view(9, H, dv)
    o = torch.zeros(9, H, dv, dtype=torch.float64)
    for i in range(9):
        for j in range(i + 1):
            s = (q[i] * k[j] * a[j + 1:i + 1].prod(dim=0)).sum(dim=-1)
            o[i] += s[:, None] * v[j]
    o = plain.rms_norm(o, w["l0.mix.norm"], 1e-5).reshape(9, H * dv)
    want = (o * plain.silu(h @ w["l0.mix.g"].T)) @ w["l0.mix.o"].T
    assert float((plain.gla(h, t, "l0.mix.", m, 1e-5) - want).abs().max()) < 1e-10


def test_weight_multiplies_the_input_of_an_expert():
    cfg = vu.one_layer("gla", vu.gla(), vu.moe(experts=1, top=1, limit=0.5))
    t = vu.make_tensors(cfg, 1)
    h = torch.randn(5, cfg["width"], dtype=torch.float64, generator=torch.Generator().manual_seed(3))
    s = torch.sigmoid(h @ t["l0.mlp.router"].double().T)
    inside = plain.bounded_expert(s * h, t, "l0.mlp.e0.", 0.5)
    outside = s * plain.bounded_expert(h, t, "l0.mlp.e0.", 0.5)
    got = plain.experts(h, t, "l0.mlp.", cfg["layers"][0]["mlp"])
    assert float((got - inside).abs().max()) < 1e-12 and float((got - outside).abs().max()) > 0.05
    # inputs of zero give down(0 * (0 + 1)) = 0; a large input is held by the bounds
    assert float(plain.bounded_expert(0 * h, t, "l0.mlp.e0.", 0.5).abs().max()) == 0.0
    huge = plain.bounded_expert(1e6 * h, t, "l0.mlp.e0.", 0.5)
    most = 0.5 * 1.5 * t["l0.mlp.e0.down"].double().abs().sum(dim=1)
    assert bool((huge.abs() <= most[None, :]).all())
