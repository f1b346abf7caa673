"""Rotary position encoding as a part.

``inv_freq[i] = theta^(-2i / rotary_dim)`` and ``angle = position * inv_freq[i]``
(/root/reference/src/transformer/rope.zig:29-43); the pair rotated by that angle
is ``(i, i + rotary_dim/2)`` for ``pairing="half"`` (what the reference's device
kernel does, /root/reference/src/cuda/layer_kernels.cu:353-365) or ``(2i, 2i+1)``
for ``pairing="adjacent"`` (rope.zig:46-53).  ``rotary_dim < head_dim`` rotates
only the leading elements.  The attention mixer applies the rotation inside its
fused query/key kernel; this part only owns the constants.

``scaling`` (optional; ``{"factor", "low", "high", "original"}``) rescales the frequencies
by wavelength ``l = 2 pi / f``, in three bands: ``l < original / high`` keeps ``f``;
``l > original / low`` takes ``f / factor``; between the two, with ``s = (original / l - low)
/ (high - low)``, ``(1 - s) f / factor + s f``.  The table is made once, in double
precision.

``scaling`` with ``"type": "yarn"`` (``{"factor", "fast", "slow", "original"}``) ramps over the
pairs instead: with ``pair(t) = rotary_dim * ln(original / (2 pi t)) / (2 ln theta)`` (the pair
that makes ``t`` turns within the original length), ``lo = max(floor(pair(fast)), 0)``, ``hi =
min(ceil(pair(slow)), rotary_dim - 1)`` and ``r_i = clamp((i - lo) / max(hi - lo, 0.001), 0,
1)``, pair ``i`` takes ``r_i f_i / factor + (1 - r_i) f_i``, and what is rotated also grows by
``magnitude = 0.1 ln(factor) + 1`` (cosine and sine are multiplied by it).  A mixer whose
kernels have no such factor calls ``without_magnitude``, which refuses it.
"""

from __future__ import annotations

import math

import torch

from .base import PositionEncoding, Runtime, register_position


class RotaryEmbedding(PositionEncoding):
    kind = "rope"
    kernel_sources = ("rope_kv",)
    fused_rotation = True   # the mixer's kernel rotates; ``apply`` is not called
    graph_safe = True       # constants only: nothing of a step is looked at on the host

    def __init__(self, params, tensors, runtime: Runtime):
        super().__init__(params, tensors, runtime)
        self.head_dim = int(params["head_dim"])
        self.rotary_dim = int(params.get("rotary_dim", self.head_dim))
        self.theta = float(params["theta"])
        self.pairing = str(params.get("pairing", "half"))
        if self.pairing not in ("half", "adjacent"):
            raise ValueError(f"rope pairing must be half or adjacent, got {self.pairing!r}")
        if self.rotary_dim % 2 or not 0 < self.rotary_dim <= self.head_dim:
            raise ValueError(f"rotary_dim {self.rotary_dim} must be even and within head_dim "
                             f"{self.head_dim}")
        i = torch.arange(0, self.rotary_dim // 2, dtype=torch.float64)
        inv = 1.0 / torch.pow(torch.tensor(self.theta, dtype=torch.float64),
                              2.0 * i / self.rotary_dim)
        scaling = params.get("scaling")
        self.magnitude = 1.0    # factor on the rotated elements
        if scaling and scaling.get("type") == "yarn":
            inv, self.magnitude = self._ramped(inv, scaling)
        elif scaling:
            inv = self._banded(inv, scaling)
        self.inv_freq = inv.to(torch.float32).to(runtime.device)

    @staticmethod
    def _banded(inv: torch.Tensor, scaling) -> torch.Tensor:
        factor, low, high, original = (float(scaling[k]) for k in
                                       ("factor", "low", "high", "original"))
        if factor <= 0.0 or high <= low or original <= 0.0:
            raise ValueError(f"rope scaling needs factor > 0, high > low and original > 0, "
                             f"got {dict(scaling)!r}")
        wave = 2.0 * math.pi / inv
        blend = (original / wave - low) / (high - low)
        middle = (1.0 - blend) * inv / factor + blend * inv
        return torch.where(wave < original / high, inv,
                           torch.where(wave > original / low, inv / factor, middle))

    def _ramped(self, inv: torch.Tensor, scaling):
        factor, fast, slow, original = (float(scaling[k]) for k in
                                        ("factor", "fast", "slow", "original"))
        if min(factor, fast, slow, original) <= 0.0 or self.theta <= 0.0 or self.theta == 1.0:
            raise ValueError(f"yarn scaling needs positive numbers and a base other than one, "
                             f"got {dict(scaling)!r} at base {self.theta}")
        dims = self.rotary_dim

        def pair(turns: float) -> float:
            return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(self.theta))

        lo = max(math.floor(pair(fast)), 0)
        hi = min(math.ceil(pair(slow)), dims - 1)
        i = torch.arange(0, dims // 2, dtype=torch.float64)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        return inv / factor * ramp + inv * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


register_position(RotaryEmbedding.kind, RotaryEmbedding)
