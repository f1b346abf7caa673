"""Small Torisun configurations and weights for tests, made here: none of them is a model
anybody ships.  The weights are drawn so that faults show: attention scores spread over
several units, sinks that take a good share of a row, router scores far from flat, gates that
meet their bounds."""

import json
import os
import tempfile

import torch

FOLDERS = {}


def yarn(factor=4.0, original=64, fast=8.0, slow=0.5):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def attention(heads=6, kv_heads=2, dim=16, vdim=24, window=20, keep=3, scale=None, rot_dims=None,
              base=300.0, scaling=None, kv_from=None):
    """``window`` 0: no mask; ``rot_dims`` 0: no rotation."""
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
           "scale": scale if scale is not None else 2.0 * dim ** -0.5}
    rot_dims = dim if rot_dims is None else rot_dims
    if rot_dims:
        out["rot"] = {"dims": rot_dims, "base": base}
        if scaling is not None:
            out["rot"]["scaling"] = scaling
    if window:
        out["mask"] = {"size": window, "keep_first": keep}
    if kv_from is not None:
        out["kv_from"] = kv_from
    return out


def dense(ff=56, limit=0.9):
    out = {"kind": "dense", "ff": ff}
    if limit:
        out["limit"] = limit
    return out


def moe(ff=24, experts=5, top=2, scale=1.7, shared=40):
    out = {"kind": "moe", "expert": {"ff": ff},
           "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp=None):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def config(layers, width=48, vocab=131, eps=1e-5):
    return {"architecture": "Torisun", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": layers}


def one_layer(mixer, mlp=None, **kw):
    return config([layer(mixer, mlp)], **kw)


# every mechanism; readers of a layer's keys whose windows are wider, narrower and absent; layers
# without feed-forward, without a shared expert, without rotation; sizes differ wherever two
# could be equal
TINY_ALL = config([
    layer(attention(scaling=yarn()), dense()),
    layer(attention(window=33, keep=7, scaling=yarn(), kv_from=0, scale=0.3), moe()),
    layer(attention(heads=4, kv_heads=4, dim=24, vdim=8, window=9, keep=0, rot_dims=10, base=5e3),
          None),
    layer(attention(window=5, keep=1, scaling=yarn(), kv_from=0), moe(ff=16, experts=7, top=3, scale=0.6,
                                                                     shared=0)),
    layer(attention(heads=3, kv_heads=1, dim=8, vdim=40, window=0, rot_dims=0), dense(ff=40, limit=2.5)),
])

# another order and other sizes: one head, widths that are multiples of nothing, a window of one,
# more kept tokens than the window is long, a reader without a window, all experts chosen
TINY_OTHER = config([
    layer(attention(heads=1, kv_heads=1, dim=20, vdim=12, window=1, keep=2, rot_dims=6), moe(
        ff=12, experts=3, top=3, scale=1.0, shared=20)),
    layer(attention(heads=5, kv_heads=1, dim=10, vdim=28, window=6, keep=11, rot_dims=10,
                    scaling=yarn(8.0, 30, 4.0, 1.0)), None),
    layer(attention(heads=5, kv_heads=1, dim=10, vdim=28, window=0, rot_dims=10,
                    scaling=yarn(8.0, 30, 4.0, 1.0), kv_from=1), dense(ff=44, limit=0)),
    layer(attention(heads=8, kv_heads=2, dim=32, vdim=16, window=50, keep=4, rot_dims=16, base=1e4),
          moe(ff=20, experts=1, top=1, scale=2.5, shared=12)),
], width=36, vocab=67, eps=1e-6)


def settled(cfg):
    """The same with every expert chosen in all feed-forwards but the last.  In bfloat16 a token
    whose scores are close may go to another expert than in float64, and one such token early in
    the model shows in every later row; with this no early layer has a choice to make."""
    out = json.loads(json.dumps(cfg))
    mlps = [lay["mlp"] for lay in out["layers"] if lay["mlp"] is not None and lay["mlp"]["kind"] == "moe"]
    for mlp in mlps[:-1]:
        mlp["router"]["top"] = mlp["router"]["experts"]
    return out


def make_tensors(cfg, seed=0):
    """name -> float32 tensor (values representable in bfloat16) for ``cfg``."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def normal(*shape, std=1.0, mean=0.0):
        t = torch.randn(*shape, generator=g) * std + mean
        return t.to(torch.bfloat16).to(torch.float32)

    out = {"embed": normal(V, W), "embed.norm": normal(W, std=0.3, mean=1.0),
           "final.norm": normal(W, std=0.3, mean=1.0)}
    for i, lay in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", lay["mixer"], lay["mlp"]
        out[p + "norm1"] = normal(W, std=0.3, mean=1.0)
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out[p + "mix.q"] = normal(H * d, W, std=W ** -0.5)
        out[p + "mix.q.norm"] = normal(H * d, std=0.3, mean=1.0)
        if m.get("kv_from") is None:
            out[p + "mix.k"] = normal(G * d, W, std=W ** -0.5)
            out[p + "mix.k.norm"] = normal(G * d, std=0.3, mean=1.0)
            out[p + "mix.v"] = normal(G * dv, W, std=W ** -0.5)
        out[p + "mix.sink"] = normal(H, std=1.5, mean=1.0)
        out[p + "mix.o"] = normal(W, H * dv, std=(H * dv) ** -0.5)
        if mlp is None:
            continue
        out[p + "norm2"] = normal(W, std=0.3, mean=1.0)

        def unit(name, F):
            out[f"{p}mlp.{name}gate"] = normal(F, W, std=W ** -0.5)
            out[f"{p}mlp.{name}up"] = normal(F, W, std=W ** -0.5)
            out[f"{p}mlp.{name}down"] = normal(W, F, std=F ** -0.5)
        if mlp["kind"] == "dense":
            unit("", mlp["ff"])
            continue
        out[p + "mlp.router"] = normal(mlp["router"]["experts"], W, std=1.5 * W ** -0.5)
        for e in range(mlp["router"]["experts"]):
            unit(f"e{e}.", mlp["expert"]["ff"])
        if mlp.get("shared"):
            unit("shared.", mlp["shared"]["ff"])
    return out


def folder(cfg, seed=0, tensors=None):
    """A model folder (config.json, model.safetensors in bfloat16) in a temporary place;
    returns (folder, tensors)."""
    from safetensors.torch import save_file
    key = (json.dumps(cfg, sort_keys=True), seed) if tensors is None else None
    if key is not None and key in FOLDERS:
        return FOLDERS[key]
    if tensors is None:
        tensors = make_tensors(cfg, seed)
    d = tempfile.mkdtemp(prefix="torisun_model_")
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()},
              os.path.join(d, "model.safetensors"))
    if key is not None:
        FOLDERS[key] = (d, tensors)
    return d, tensors


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(7000 + seed)
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
        if sources and pick(True, False):
            j = pick(*sources)
            mixer = json.loads(json.dumps(layers[j]["mixer"]))
            mixer["kv_from"] = j
            mixer["scale"] = pick(0.1, 0.3, 0.6)
            mixer.pop("mask", None)
            window = pick(0, 1, 4, 17, 70)
            if window:
                mixer["mask"] = {"size": window, "keep_first": pick(0, 1, 5, 30)}
        else:
            kv, dim = pick(1, 2, 3), pick(6, 8, 16, 20, 24, 40, 72)
            mixer = attention(heads=kv * pick(1, 2, 5), kv_heads=kv, dim=dim,
                              vdim=pick(4, 8, 16, 24, 36, dim), window=pick(0, 1, 3, 16, 33, 64, 300),
                              keep=pick(0, 1, 4, 16, 40), scale=pick(0.1, 0.3, 0.6),
                              rot_dims=pick(0, 2, dim // 2 // 2 * 2, dim), base=pick(10.0, 1e3, 5e5),
                              scaling=pick(None, yarn(), yarn(40.0, 4096, 32.0, 1.0), yarn(1.0, 16, 4.0, 2.0)))
            if "rot" in mixer and mixer["rot"]["dims"] == 0:
                mixer.pop("rot")
            sources.append(i)
        kind = pick("none", "dense", "moe", "moe")
        mlp = None
        if kind == "dense":
            mlp = dense(ff=pick(8, 20, 64), limit=pick(0, 0.5, 7.0))
        elif kind == "moe":
            experts = pick(1, 2, 5, 9)
            mlp = moe(ff=pick(8, 12, 40), experts=experts, top=rng.randrange(1, min(experts, 4) + 1),
                      scale=pick(0.5, 1.0, 2.5), shared=pick(0, 8, 28))
        layers.append(layer(mixer, mlp))
    return config(layers, width=pick(24, 36, 40, 64, 104), vocab=pick(11, 50, 203),
                  eps=pick(1e-6, 1e-5, 1e-3))
