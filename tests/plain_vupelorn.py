"""A plain, slow Vupelorn: whole sequences, no cache, no batching, one function per
mechanism, on the CPU in float64.  It shares no code with the engine: it takes the
config.json dictionary and a mapping from tensor names to tensors.  The attention forms
every head's keys and values (the engine folds the two expansions into the query and the
output), the recurrence is walked token by token (the engine walks long portions in chunks),
and an expert's input is multiplied by its weight (the engine multiplies the product).

Notation: ``h`` is a mixer's input ``[T, width]``; weights are ``[out, in]`` and applied
as ``h @ W.T``; positions count from 0.
"""

from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional, Tuple

import torch

DT = torch.float64


def _w(tensors: Mapping[str, torch.Tensor], name: str) -> torch.Tensor:
    return tensors[name].to(DT)


# ------------------------------------------------------------------ small pieces
def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * torch.sigmoid(x)


# --------------------------------------------------------------------- embedding
def pair_rows(token_ids: List[int], buckets: int, mul_prev: int, mul_cur: int) -> List[int]:
    """Which row of the table of token pairs every token takes: a hash of the token before
    it and itself; a sequence's first token has the row behind all buckets."""
    rows = [buckets]
    for before, this in zip(token_ids, token_ids[1:]):
        rows.append((before * mul_prev + this * mul_cur) % buckets)
    return rows[:len(token_ids)]


def embed(token_ids: List[int], tensors, pair: Optional[Mapping]) -> torch.Tensor:
    x = _w(tensors, "embed")[torch.tensor(token_ids)]
    if pair:
        rows = pair_rows(token_ids, int(pair["buckets"]), int(pair["mul_prev"]), int(pair["mul_cur"]))
        x = x + _w(tensors, "bigram")[torch.tensor(rows)]
    return x


# ------------------------------------------------------------- rotary positions
def frequencies(rot: Mapping) -> Tuple[List[float], float]:
    """(angle per position of every pair, factor on cosine and sine)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    scaling = rot.get("scaling")
    if not scaling:
        return freq, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def turns_at(t: float) -> float:
        # the (fractional) pair that makes t turns within the original length
        return dims * math.log(original / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(turns_at(float(scaling["fast"]))), 0)
    hi = min(math.ceil(turns_at(float(scaling["slow"]))), dims - 1)
    out = []
    for i, f in enumerate(freq):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x: torch.Tensor, positions: torch.Tensor, rot: Mapping, interleaved: bool) -> torch.Tensor:
    """``x``: [T, ..., width]; the first ``dims`` elements of the last axis turn."""
    dims = int(rot["dims"])
    freq, factor = frequencies(rot)
    ang = positions.to(DT)[:, None] * torch.tensor(freq, dtype=DT)[None, :]
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [dims // 2]
    c, s = (factor * torch.cos(ang)).view(shape), (factor * torch.sin(ang)).view(shape)
    out = x.clone()
    first, second = (slice(0, dims, 2), slice(1, dims, 2)) if interleaved \
        else (slice(0, dims // 2), slice(dims // 2, dims))
    u, v = x[..., first], x[..., second]
    out[..., first] = u * c - v * s
    out[..., second] = v * c + u * s
    return out


# ------------------------------------------------------------- latent attention
def latent(h: torch.Tensor, tensors, p: str, m: Mapping, eps: float, interleaved: bool,
           positions: torch.Tensor) -> Tuple[torch.Tensor, torch.Tensor]:
    """(normed latent [T, kv_rank], rotated key part [T, rot_dim]) of every token."""
    r = int(m["kv_rank"])
    down = h @ _w(tensors, p + "dkv").T
    c = rms_norm(down[:, :r], _w(tensors, p + "dkv.norm"), eps)
    return c, rotate(down[:, r:], positions, m["rot"], interleaved)


def latent_attention(h: torch.Tensor, tensors, p: str, m: Mapping, eps: float, interleaved: bool,
                     shared: Optional[Tuple[torch.Tensor, torch.Tensor]] = None,
                     reach: int = 0) -> Tuple[torch.Tensor, Tuple[torch.Tensor, torch.Tensor]]:
    """(output, what other layers may take over).  ``shared``: another layer's latent and
    rotated key part, for a layer that makes none.  ``reach`` is 0; tests that ask whether
    a mask that is one token off would show set it to -1 or 1."""
    T = h.shape[0]
    H, d, dv, dr = int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["rot_dim"])
    pos = torch.arange(T)
    c, k_rot = shared if shared is not None else latent(h, tensors, p, m, eps, interleaved, pos)
    cq = rms_norm(h @ _w(tensors, p + "dq").T, _w(tensors, p + "dq.norm"), eps)
    q = (cq @ _w(tensors, p + "uq").T).view(T, H, d + dr)
    q_rot = rotate(q[..., d:], pos, m["rot"], interleaved)
    k = (c @ _w(tensors, p + "uk").T).view(T, H, d)
    v = (c @ _w(tensors, p + "uv").T).view(T, H, dv)
    causal = pos[None, :] <= pos[:, None] + reach
    out = torch.zeros((T, H, dv), dtype=DT)
    for hh in range(H):
        s = (q[:, hh, :d] @ k[:, hh].T + q_rot[:, hh] @ k_rot.T) * float(m["scale"])
        out[:, hh] = torch.softmax(s.masked_fill(~causal, -math.inf), dim=-1) @ v[:, hh]
    return out.reshape(T, H * dv) @ _w(tensors, p + "o").T, (c, k_rot)


# ------------------------------------------------------- gated linear attention
def decays(h: torch.Tensor, tensors, p: str, tau: float) -> torch.Tensor:
    z = (h @ _w(tensors, p + "a1").T) @ _w(tensors, p + "a2").T + _w(tensors, p + "a2.b")
    return torch.sigmoid(z) ** (1.0 / tau)


def gla(h: torch.Tensor, tensors, p: str, m: Mapping, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ _w(tensors, p + "q").T).view(T, H, d) * d ** -0.5
    k = (h @ _w(tensors, p + "k").T).view(T, H, d)
    v = (h @ _w(tensors, p + "v").T).view(T, H, dv)
    a = decays(h, tensors, p, float(m["tau"])).view(T, H, d)
    S = torch.zeros((H, d, dv), dtype=DT)
    o = torch.zeros((T, H, dv), dtype=DT)
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(dim=1)
    o = rms_norm(o, _w(tensors, p + "norm"), eps).reshape(T, H * dv)
    return (o * silu(h @ _w(tensors, p + "g").T)) @ _w(tensors, p + "o").T


# ----------------------------------------------------------------- feed-forward
def bounded_expert(x: torch.Tensor, tensors, p: str, limit: float) -> torch.Tensor:
    g = (x @ _w(tensors, p + "gate").T).clamp(max=limit)
    u = (x @ _w(tensors, p + "up").T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ _w(tensors, p + "down").T


def route(h: torch.Tensor, tensors, p: str, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    s = torch.sigmoid(h @ _w(tensors, p + "router").T)
    best = s.topk(top, dim=-1)
    return best.indices, best.values


def experts(h: torch.Tensor, tensors, p: str, mlp: Mapping) -> torch.Tensor:
    limit = float(mlp["expert"]["limit"])
    chosen, weights = route(h, tensors, p, int(mlp["router"]["top"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(chosen[t].tolist(), weights[t]):
            out[t] += bounded_expert(w * h[t:t + 1], tensors, f"{p}e{e}.", limit)[0]
    return out


# ------------------------------------------------------------------- the model
def forward(config: Mapping, tensors: Mapping[str, torch.Tensor], token_ids: List[int],
            streams: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] in float64.  ``streams`` receives the residual stream after
    every layer."""
    eps = float(config["norm"]["eps"])
    x = embed(token_ids, tensors, (config.get("embedding") or {}).get("bigram"))
    kept: Dict[int, Tuple[torch.Tensor, torch.Tensor]] = {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        if layer["type"] == "gla":
            y = gla(x, tensors, p + "mix.", m, eps)
        elif layer["type"] in ("latent_attention", "latent_attention_2"):
            source = m.get("kv_from")
            y, kept[i] = latent_attention(x, tensors, p + "mix.", m, eps,
                                          layer["type"] == "latent_attention_2",
                                          None if source is None else kept[int(source)])
        else:
            raise ValueError(layer["type"])
        x = x + rms_norm(y, _w(tensors, p + "norm1"), eps)
        if layer.get("mlp") is not None:
            y = experts(x, tensors, p + "mlp.", layer["mlp"])
            x = x + rms_norm(y, _w(tensors, p + "norm2"), eps)
        if streams is not None:
            streams.append(x.clone())
    return rms_norm(x, _w(tensors, "final.norm"), eps) @ _w(tensors, "embed").T
