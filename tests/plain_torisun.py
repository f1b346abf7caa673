"""A plain, slow Torisun: whole sequences, no cache, no batching, one function per
mechanism, on the CPU in float64.  It shares no code with the engine: it takes the
config.json dictionary and a mapping from tensor names to tensors.

Notation: ``h`` is a sublayer's input ``[T, width]``; weights are ``[out, in]`` and applied
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


def embed(token_ids: List[int], tensors, eps: float) -> torch.Tensor:
    rows = _w(tensors, "embed")[torch.tensor(token_ids)]
    return rms_norm(rows, _w(tensors, "embed.norm"), eps)


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


def rotate(x: torch.Tensor, positions: torch.Tensor, rot: Optional[Mapping]) -> torch.Tensor:
    """``x``: [T, heads, width]; element ``i`` of the first ``dims`` turns with ``i + dims/2``."""
    if not rot or not int(rot["dims"]):
        return x
    dims = int(rot["dims"])
    freq, factor = frequencies(rot)
    ang = positions.to(DT)[:, None] * torch.tensor(freq, dtype=DT)[None, :]
    c, s = (factor * torch.cos(ang))[:, None, :], (factor * torch.sin(ang))[:, None, :]
    out = x.clone()
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    out[..., :dims // 2] = u * c - v * s
    out[..., dims // 2:dims] = v * c + u * s
    return out


# -------------------------------------------------------------------- attention
def visible(T: int, mask: Optional[Mapping], reach: int = 0, kept: int = 0) -> torch.Tensor:
    """[T, T]: whether query i sees key j.  ``reach`` and ``kept`` are 0; tests that ask whether
    a window (or the kept first tokens) one off would show set them to -1 or 1."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    if not mask or not int(mask.get("size") or 0):
        return j <= i
    return (j <= i) & ((i - j < int(mask["size"]) + reach)
                       | (j < int(mask.get("keep_first") or 0) + kept))


def keys_values(h: torch.Tensor, tensors, p: str, m: Mapping, eps: float
                ) -> Tuple[torch.Tensor, torch.Tensor]:
    """Keys (normed over all their rows at once, then rotated) and values of every token."""
    T, G, d, dv = h.shape[0], int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    k = rms_norm(h @ _w(tensors, p + "k").T, _w(tensors, p + "k.norm"), eps).view(T, G, d)
    return rotate(k, torch.arange(T), m.get("rot")), (h @ _w(tensors, p + "v").T).view(T, G, dv)


def attention(h: torch.Tensor, tensors, p: str, m: Mapping, eps: float,
              shared: Optional[Tuple[torch.Tensor, torch.Tensor]] = None, reach: int = 0,
              kept: int = 0) -> Tuple[torch.Tensor, Tuple[torch.Tensor, torch.Tensor]]:
    """(output, (keys, values)).  ``shared``: another layer's keys and values, for a layer
    that makes none."""
    T, H, G = h.shape[0], int(m["heads"]), int(m["kv_heads"])
    d, dv = int(m["dim"]), int(m["vdim"])
    k, v = shared if shared is not None else keys_values(h, tensors, p, m, eps)
    q = rms_norm(h @ _w(tensors, p + "q").T, _w(tensors, p + "q.norm"), eps).view(T, H, d)
    q = rotate(q, torch.arange(T), m.get("rot"))
    sees = visible(T, m.get("mask"), reach, kept)
    sink = _w(tensors, p + "sink")
    out = torch.zeros((T, H, dv), dtype=DT)
    for a in range(H):
        b = a // (H // G)
        s = (q[:, a] @ k[:, b].T * float(m["scale"])).masked_fill(~sees, -math.inf)
        top = torch.maximum(s.max(dim=-1).values, sink[a])
        e = torch.exp(s - top[:, None])
        out[:, a] = e @ v[:, b] / (e.sum(dim=-1) + torch.exp(sink[a] - top))[:, None]
    return out.reshape(T, H * dv) @ _w(tensors, p + "o").T, (k, v)


# ----------------------------------------------------------------- feed-forward
def dense(h: torch.Tensor, tensors, p: str, limit: float) -> torch.Tensor:
    """``limit`` 0: no bounds."""
    g, u = h @ _w(tensors, p + "gate").T, h @ _w(tensors, p + "up").T
    if limit:
        g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ _w(tensors, p + "down").T


def expert(h: torch.Tensor, tensors, p: str) -> torch.Tensor:
    g = h @ _w(tensors, p + "gate").T
    return (g * torch.sigmoid(g) * (h @ _w(tensors, p + "up").T)) @ _w(tensors, p + "down").T


def route(h: torch.Tensor, tensors, p: str, router: Mapping) -> Tuple[torch.Tensor, torch.Tensor]:
    s = torch.sigmoid(h @ _w(tensors, p + "router").T)
    best = s.topk(int(router["top"]), dim=-1)
    weight = best.values / (best.values.sum(dim=-1, keepdim=True) + 1e-20)
    return best.indices, weight * float(router.get("scale", 1.0))


def experts(h: torch.Tensor, tensors, p: str, mlp: Mapping) -> torch.Tensor:
    chosen, weights = route(h, tensors, p, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(chosen[t].tolist(), weights[t]):
            out[t] += w * expert(h[t:t + 1], tensors, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        out = out + expert(h, tensors, p + "shared.")
    return out


# ------------------------------------------------------------------- the model
def forward(config: Mapping, tensors: Mapping[str, torch.Tensor], token_ids: List[int],
            streams: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] in float64.  ``streams`` receives the residual stream after
    every layer."""
    eps = float(config["norm"]["eps"])
    x = embed(token_ids, tensors, eps)
    made: Dict[int, Tuple[torch.Tensor, torch.Tensor]] = {}
    for i, layer in enumerate(config["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        if layer["type"] != "attention":
            raise ValueError(layer["type"])
        source = m.get("kv_from")
        y, made[i] = attention(x, tensors, p + "mix.", m, eps,
                               None if source is None else made[int(source)])
        x = x + rms_norm(y, _w(tensors, p + "norm1"), eps)
        if mlp is not None:
            y = dense(x, tensors, p + "mlp.", float(mlp.get("limit", 0.0))) if mlp["kind"] == "dense" \
                else experts(x, tensors, p + "mlp.", mlp)
            x = x + rms_norm(y, _w(tensors, p + "norm2"), eps)
        if streams is not None:
            streams.append(x.clone())
    return rms_norm(x, _w(tensors, "final.norm"), eps) @ _w(tensors, "embed").T
