"""Small Vupelorn configurations and weights for tests, made here: none of them is a model
anybody ships.  The weights are drawn so that faults show: attention scores spread over
several units, decays from nearly one down to a tenth, router scores far from flat, gates that
meet their bounds, a table of token pairs as large as the tokens' own."""

import json
import os
import tempfile

import torch

FOLDERS = {}


def yarn(factor=4.0, original=64, fast=8.0, slow=0.5):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def latent(heads=3, dim=16, vdim=24, kv_rank=32, q_rank=24, rot_dim=8, base=300.0, scale=None,
           scaling=None, kv_from=None):
    rot = {"dims": rot_dim, "base": base}
    if scaling is not None:
        rot["scaling"] = scaling
    out = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
           "scale": scale if scale is not None else 0.7 * (dim + rot_dim) ** -0.5,
           "rot_dim": rot_dim, "rot": rot}
    if kv_from is not None:
        out["kv_from"] = kv_from
    return out


def gla(heads=2, dim=16, vdim=24, tau=3.0, rank=8):
    """``decay_rank`` is not read where tensors say it; it is here for ``make_tensors``."""
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}


def moe(ff=24, experts=5, top=2, limit=1.1):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "top": top}}


def layer(kind, mixer, mlp=None):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def config(layers, width=48, vocab=131, eps=1e-5, buckets=97, mul_prev=29, mul_cur=13):
    out = {"architecture": "Vupelorn", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "layers": layers}
    if buckets:
        out["embedding"] = {"bigram": {"buckets": buckets, "mul_prev": mul_prev,
                                       "mul_cur": mul_cur}}
    return out


# every mixer, a layer that reads another's rows, a layer without feed-forward; sizes differ
# wherever two could be equal
TINY_ALL = config([
    layer("latent_attention", latent(scaling=yarn()), moe()),
    layer("gla", gla(), moe(ff=16, experts=3, top=1, limit=0.7)),
    layer("latent_attention_2", latent(heads=2, dim=24, vdim=16, kv_rank=40, q_rank=16, rot_dim=16,
                                       base=1e4), None),
    layer("latent_attention_2", latent(heads=5, dim=8, vdim=8, kv_rank=40, q_rank=32, rot_dim=16,
                                       base=1e4, kv_from=2, scale=0.17), moe(ff=8, experts=6, top=4,
                                                                            limit=3.0)),
    layer("gla", gla(heads=3, dim=24, vdim=8, tau=16.0, rank=16), None),
])

# another order and other sizes: two readers of one layer's rows, one head, all experts chosen,
# keys wider than values, no table of pairs, no stretched frequencies
TINY_OTHER = config([
    layer("gla", gla(heads=1, dim=40, vdim=16, tau=1.0, rank=24), None),
    layer("latent_attention_2", latent(heads=1, dim=8, vdim=40, kv_rank=16, q_rank=8, rot_dim=2,
                                       base=50.0), moe(ff=40, experts=2, top=2, limit=0.4)),
    layer("latent_attention_2", latent(heads=4, dim=16, vdim=8, kv_rank=16, q_rank=40, rot_dim=2,
                                       base=50.0, kv_from=1), None),
    layer("latent_attention", latent(heads=2, dim=16, vdim=32, kv_rank=24, q_rank=16, rot_dim=24),
          moe(ff=16, experts=4, top=1)),
    layer("latent_attention_2", latent(heads=2, dim=8, vdim=16, kv_rank=16, q_rank=24, rot_dim=2,
                                       base=50.0, kv_from=1), moe(ff=8, experts=1, top=1, limit=2.0)),
], width=40, vocab=67, eps=1e-6, buckets=0)


def settled(cfg):
    """The same with every expert chosen in all feed-forwards but the last.  In bfloat16 a token
    whose scores are close may go to another expert than in float64, and one such token early in
    the model shows in every later row; with this no early layer has a choice to make."""
    out = json.loads(json.dumps(cfg))
    mlps = [lay["mlp"] for lay in out["layers"] if lay["mlp"] is not None]
    for mlp in mlps[:-1]:
        mlp["router"]["top"] = mlp["router"]["experts"]
    return out


def one_layer(kind, mixer, mlp=None, **kw):
    return config([layer(kind, mixer, mlp)], **kw)


def make_tensors(cfg, seed=0):
    """name -> float32 tensor (values representable in bfloat16) for ``cfg``."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def normal(*shape, std=1.0, mean=0.0):
        t = torch.randn(*shape, generator=g) * std + mean
        return t.to(torch.bfloat16).to(torch.float32)

    out = {"embed": normal(V, W), "final.norm": normal(W, std=0.3, mean=1.0)}
    pair = (cfg.get("embedding") or {}).get("bigram")
    if pair:
        out["bigram"] = normal(pair["buckets"] + 1, W)
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        out[p + "norm1"] = normal(W, std=0.3, mean=1.0)
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if lay["type"] == "gla":
            r = m["decay_rank"]
            for name, rows in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv)):
                out[f"{p}mix.{name}"] = normal(rows, W, std=W ** -0.5)
            out[p + "mix.a1"] = normal(r, W, std=W ** -0.5)
            out[p + "mix.a2"] = normal(H * d, r, std=1.5 * r ** -0.5)
            # (decays from nearly one, with a memory of hundreds of tokens, to a tenth)
            out[p + "mix.a2.b"] = normal(H * d, std=3.0, mean=2.0)
            out[p + "mix.norm"] = normal(dv, std=0.3, mean=1.0)
        else:
            R, Rq, dr = m["kv_rank"], m["q_rank"], m["rot_dim"]
            out[p + "mix.dq"] = normal(Rq, W, std=W ** -0.5)
            out[p + "mix.dq.norm"] = normal(Rq, std=0.3, mean=1.0)
            out[p + "mix.uq"] = normal(H * (d + dr), Rq, std=1.5 * Rq ** -0.5)
            if m.get("kv_from") is None:
                out[p + "mix.dkv"] = normal(R + dr, W, std=W ** -0.5)
                out[p + "mix.dkv.norm"] = normal(R, std=0.3, mean=1.0)
            out[p + "mix.uk"] = normal(H * d, R, std=1.5 * R ** -0.5)
            out[p + "mix.uv"] = normal(H * dv, R, std=R ** -0.5)
        out[p + "mix.o"] = normal(W, H * dv, std=(H * dv) ** -0.5)
        mlp = lay["mlp"]
        if mlp is None:
            continue
        out[p + "norm2"] = normal(W, std=0.3, mean=1.0)
        F = mlp["expert"]["ff"]
        out[p + "mlp.router"] = normal(mlp["router"]["experts"], W, std=1.5 * W ** -0.5)
        for e in range(mlp["router"]["experts"]):
            out[f"{p}mlp.e{e}.gate"] = normal(F, W, std=W ** -0.5)
            out[f"{p}mlp.e{e}.up"] = normal(F, W, std=W ** -0.5)
            out[f"{p}mlp.e{e}.down"] = normal(W, F, std=F ** -0.5)
    return out


def folder(cfg, seed=0, tensors=None):
    """A model folder (config.json, model.safetensors in bfloat16) in a temporary place;
    returns (folder, tensors).  config.json does not hold the decay ranks: tensors do."""
    from safetensors.torch import save_file
    key = (json.dumps(cfg, sort_keys=True), seed) if tensors is None else None
    if key is not None and key in FOLDERS:
        return FOLDERS[key]
    if tensors is None:
        tensors = make_tensors(cfg, seed)
    stored = json.loads(json.dumps(cfg))
    for lay in stored["layers"]:
        lay["mixer"].pop("decay_rank", None)
    d = tempfile.mkdtemp(prefix="vupelorn_model_")
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(stored, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()},
              os.path.join(d, "model.safetensors"))
    if key is not None:
        FOLDERS[key] = (d, tensors)
    return d, tensors


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(5000 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def row_error(got, want):
    """Per row: the root mean square of the difference (means taken off) relative to the
    root mean square of the wanted logits over all rows."""
    got, want = got.double(), want.double()
    assert got.shape == want.shape, (got.shape, want.shape)
    assert torch.isfinite(got).all(), "non-finite logits"
    d = got - want
    d = d - d.mean(dim=1, keepdim=True)
    scale = (want - want.mean(dim=1, keepdim=True)).pow(2).mean().sqrt()
    return d.pow(2).mean(dim=1).sqrt() / scale


def random_config(seed):
    """A configuration drawn at random: layer order, every size and every constant."""
    import random
    rng = random.Random(seed)

    def pick(*values):
        return rng.choice(values)

    layers, sources = [], []
    for i in range(pick(1, 2, 3, 4, 5)):
        kind = pick("gla", "latent_attention", "latent_attention_2", "latent_attention_2")
        if kind == "gla":
            mixer = gla(heads=pick(1, 2, 3, 5), dim=pick(4, 8, 16, 24, 72), vdim=pick(8, 16, 40, 80),
                        tau=pick(0.5, 1.0, 4.0, 16.0), rank=pick(1, 4, 8, 20))
        else:
            mixer = latent(heads=pick(1, 2, 3, 6), dim=pick(8, 16, 24, 40), vdim=pick(8, 16, 24, 48),
                           kv_rank=pick(8, 24, 32, 72), q_rank=pick(8, 16, 56),
                           rot_dim=pick(2, 8, 16, 24), base=pick(10.0, 1000.0, 5e5),
                           scale=pick(0.1, 0.2, 0.4))
            if kind == "latent_attention" and pick(True, True, False):
                mixer["rot"]["scaling"] = yarn(pick(1.0, 2.0, 40.0), pick(16, 100, 4096),
                                               pick(4.0, 32.0), pick(0.5, 1.0))
            elif kind == "latent_attention_2" and sources and pick(True, False):
                j = pick(*sources)
                mixer.update({k: layers[j]["mixer"][k] for k in ("kv_rank", "rot_dim", "rot")},
                             kv_from=j)
            if kind == "latent_attention_2" and "kv_from" not in mixer:
                sources.append(i)
        mlp = None
        if pick(True, True, False):
            experts = pick(1, 2, 5, 9)
            mlp = moe(ff=pick(8, 16, 40), experts=experts, top=rng.randrange(1, min(experts, 4) + 1),
                      limit=pick(0.3, 1.0, 7.0))
        layers.append(layer(kind, mixer, mlp))
    return config(layers, width=pick(16, 24, 40, 64, 104), vocab=pick(11, 50, 203),
                  eps=pick(1e-6, 1e-5, 1e-3), buckets=pick(0, 1, 50, 1000), mul_prev=pick(0, 1, 31, 99991),
                  mul_cur=pick(1, 17, 70001))
