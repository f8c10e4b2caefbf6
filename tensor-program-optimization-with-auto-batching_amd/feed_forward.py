"""Feed-forward blocks: a dense one with a clipped gated product, and a mixture of experts."""
from __future__ import annotations

import dataclasses

import torch

from . import decoder_ops as D
from . import ops
from .decoder_ops import pad32, pad64, padded


@dataclasses.dataclass(frozen=True)
class ClippedGluSpec:
    ff: int
    limit: float
    alpha: float = 1.702      # slope inside the gate's sigmoid


@dataclasses.dataclass(frozen=True)
class MoeSpec:
    ff: int
    experts: int
    top: int


class ClippedGlu:
    """down(g sigmoid(alpha g) (u + 1)) with g = min(gate h, limit), u = clamp(up h, +-limit); h = gain * input."""

    def __init__(self, spec: ClippedGluSpec, w: dict, width: int, gain: float, dtype, device):
        self.spec, self.gain, self.dtype = spec, float(gain), dtype
        Hp = pad64(width)
        self.ffp = pad64(spec.ff)
        gu = torch.cat([padded(w[k].to(device, dtype), self.ffp, Hp) for k in ("gate", "up")])
        self.gate_up = D.weight(gu)
        self.gate_up_il = ops.interleave_gate_up(gu) if dtype != torch.float32 else None
        self.down_rows = padded(w["down"].to(device, dtype), Hp, self.ffp)      # the output projection, for the layer to place

    def hidden(self, x, out):
        s = self.spec
        return D.gate_up_clipglu(x, self.gate_up, self.gate_up_il, self.gain, s.limit, s.alpha, out)


class MoeRelu2:
    """sum over the chosen experts of weight * down max(up h, 0)^2; router softmax over the chosen logits; h = gain * input."""

    def __init__(self, spec: MoeSpec, w: dict, width: int, gain: float, dtype, device):
        """w: router [E, width], router_b [E], up: E x [ff, width], down: E x [width, ff]."""
        self.spec, self.gain, self.dtype = spec, float(gain), dtype
        E, self.Hp, self.ffp = spec.experts, pad64(width), pad64(spec.ff)
        self.router = D.weight(padded(w["router"].to(device, dtype), pad32(E), self.Hp))
        self.bias = w["router_b"].to(device, torch.float32).contiguous()
        stack = lambda ws, n, k: D.weight(torch.cat([padded(m.to(device, dtype), n, k) for m in ws]))
        self.up = stack(w["up"], self.ffp, self.Hp)
        self.down = stack(w["down"], self.Hp, self.ffp)

    def add_to(self, resid, x, x_row, parts=None, out=None):
        """resid [T, Hp] += pending partials and the output; x: the input as an activation, x_row: the same row-major; out: the
        sum as an activation."""
        s = self.spec
        logits = ops.linear(x, self.router, out_dtype=torch.float32)
        pick, wt = D.moe_route(logits, self.bias, self.gain, s.top, self.dtype)
        plan = D.MoePlan(pick, s.experts, self.dtype)
        mid = D.moe_linear(x_row, self.up, plan, self.ffp, self.Hp, D.MOE_UP, D.ACT_RELU2, self.gain)
        D.moe_combine(resid, D.moe_linear(mid, self.down, plan, self.Hp, self.ffp, D.MOE_DOWN), wt, parts, out)
