"""Feed-forward blocks: a dense one with a clipped gated product, and mixtures of experts, routed by a router or by token id."""
from __future__ import annotations

import dataclasses
from typing import Optional

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


@dataclasses.dataclass(frozen=True)
class TableMoeSpec:
    """Experts by token id, each of weight 1 / top, and a shared expert of width `shared` (None: none)."""
    ff: int
    experts: int
    top: int
    shared: Optional[int] = None

    @classmethod
    def from_config(cls, c: dict) -> "TableMoeSpec":
        shared = c.get("shared")
        return cls(int(c["expert"]["ff"]), int(c["router"]["experts"]), int(c["router"]["top"]), int(shared["ff"]) if shared else None)


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


class SiluGlu:
    """down(silu(gate h) * up h)."""

    def __init__(self, w: dict, ff: int, width: int, dtype, device):
        Hp, self.ffp, self.dtype = pad64(width), pad64(ff), dtype
        gu = torch.cat([padded(w[k].to(device, dtype), self.ffp, Hp) for k in ("gate", "up")])
        self.gate_up = D.weight(gu)
        self.gate_up_il = ops.interleave_gate_up(gu) if dtype != torch.float32 else None
        self.down = D.weight(padded(w["down"].to(device, dtype), Hp, self.ffp))

    def hidden(self, x):
        return D.gate_up_silu(x, self.gate_up, self.gate_up_il, D.activation(x.shape[0], self.ffp, self.dtype, x.device))


class TableMoe:
    """Experts down(silu(gate h) * up h) chosen by token id, and a shared one for every token."""

    def __init__(self, spec: TableMoeSpec, w: dict, width: int, dtype, device):
        """w: table [V, top], gate, up: E x [ff, width], down: E x [width, ff], shared: the same three, if there is one."""
        self.spec, self.dtype = spec, dtype
        self.Hp, self.ffp = pad64(width), pad64(spec.ff)
        self.table = w["table"].to(device, torch.int32).contiguous()
        if self.table.shape[1] != spec.top or int(self.table.min()) < 0 or int(self.table.max()) >= spec.experts:
            raise ValueError(f"expert table {tuple(self.table.shape)}: entries outside 0..{spec.experts - 1}, or not {spec.top} per token")
        cut = lambda m, n, k: padded(m.to(device, dtype), n, k)
        # per expert its gate rows, then its up rows
        self.gate_up = D.weight(torch.cat([cut(m, self.ffp, self.Hp) for g, u in zip(w["gate"], w["up"]) for m in (g, u)]))
        self.down = D.weight(torch.cat([cut(m, self.Hp, self.ffp) for m in w["down"]]))
        self.shared = SiluGlu(w["shared"], spec.shared, width, dtype, device) if spec.shared else None

    def __call__(self, x, x_row, plan, split):
        """x: the input as an activation, x_row: the same row-major -> (entry rows [T * top, Hp] of weight 1 / top, shared output fp32 or
        None, its pending partials)."""
        if self.dtype == torch.float32:
            gu = D.moe_linear(x_row, self.gate_up, plan, 2 * self.ffp, self.Hp, D.MOE_UP)
            mid = D.silu_mul(gu, torch.empty((gu.shape[0], self.ffp), dtype=gu.dtype, device=gu.device))
        else:
            mid = D.moe_linear(x_row, self.gate_up, plan, self.ffp, self.Hp, D.MOE_UP, D.ACT_GLU)
        rows = D.moe_linear(mid, self.down, plan, self.Hp, self.ffp, D.MOE_DOWN)
        if self.shared is None:
            return rows, None, None
        return (rows, *D.linear_sum(self.shared.hidden(x), self.shared.down, split))


class TableRouting:
    """The routing of a pass: which expert a token takes depends on its id alone, so the plans of all layers are made at once."""

    def __init__(self, blocks: dict, dtype):
        """blocks: layer -> TableMoe."""
        self.dtype, self.groups = dtype, {}
        for l, b in blocks.items():
            self.groups.setdefault((b.spec.experts, b.spec.top), []).append(l)
        self.tables = {k: torch.stack([blocks[l].table for l in ls]).contiguous() for k, ls in self.groups.items()}

    def plans(self, ids):
        out = {}
        for (E, top), layers in self.groups.items():
            out.update(zip(layers, D.MoePlan.of_tables(self.tables[E, top], ids, E, self.dtype)))
        return out
