"""Time mixing: a linear recurrence over a matrix state per head, with a decay per key channel that depends on the token.

Every projection reads its own mix of the token's row and the previous token's.  The equations stand in csrc/time_mix.hip.
"""
from __future__ import annotations

import dataclasses

import torch

from . import decoder_ops as D
from . import ops
from .decoder_ops import pad32, pad64, padded

MIXES = ("r", "k", "v", "g", "w")


@dataclasses.dataclass(frozen=True)
class TimeMixSpec:
    heads: int
    dim: int

    @classmethod
    def from_config(cls, c: dict) -> "TimeMixSpec":
        return cls(int(c["heads"]), int(c["dim"]))

    def cache_entry(self, n_pages, slots, page, width_p):
        """Shapes of what a layer run keeps (and whether in elements rather than fp32): matrix states, and previous tokens' rows."""
        return ((slots, self.heads, self.dim, self.dim), False), ((slots, width_p), False)


@dataclasses.dataclass
class Mixes:
    """The five mixes of a pass: activations that lie one after the other in one buffer."""
    parts: list
    data: torch.Tensor

    def room(self) -> dict:
        """What a stream step fills."""
        return {"out_row": self.data} if self.data.dtype == torch.float32 else {"out": self.all()}

    def all(self):
        """All of them as one activation (bfloat16)."""
        x = self.parts[0]
        return ops.FragActivation(x.T, x.K, x.device, self.data)


class TimeMix:
    """Weights of one layer in kernel order."""

    def __init__(self, spec: TimeMixSpec, w: dict, width: int, eps: float, dtype, device):
        """w: mu.r .. mu.w [width], r, k, v, g [H dim, width], w1 [rank, width], w2 [H dim, rank], w0 [H dim], u [H, dim],
        norm [H dim], o [width, H dim]."""
        self.spec, self.eps, self.dtype = spec, float(eps), dtype
        cols, Hp = spec.heads * spec.dim, pad64(width)
        self.out_cols = pad64(cols)
        t = lambda n: w[n].to(device, dtype)
        self.mu = torch.stack([padded(t("mu." + s), Hp) for s in MIXES]).contiguous()
        self.rank = w["w1"].shape[0]
        rows = [padded(t(s), self.out_cols, Hp) for s in "rkvg"] + [padded(t("w1"), pad32(self.rank), Hp)]
        if dtype == torch.float32:
            self.all, (*proj, self.w1) = None, [D.weight(m) for m in rows]
        else:                                                                    # one matrix for decode steps, and its parts
            self.all = D.weight(torch.cat(rows))
            *proj, self.w1 = (self.all.rows(i * self.out_cols, m.shape[0]) for i, m in enumerate(rows))
        self.proj = dict(zip("rkvg", proj))
        self.w2 = padded(t("w2"), cols, pad32(self.rank)).contiguous()
        self.w0 = w["w0"].to(device, torch.float32).contiguous()
        self.u = w["u"].to(device, torch.float32).reshape(-1).contiguous()
        self.norm = t("norm").contiguous()
        self.o = D.weight(padded(t("o"), Hp, self.out_cols))
        self.prompt_form = dtype != torch.float32 and D.time_mix_prompt_served(spec.dim)

    def mixes(self, T, width_p, device) -> Mixes:
        """Room for the five mixes of a pass."""
        if self.dtype == torch.float32:
            rows = torch.empty((len(MIXES), T, width_p), dtype=self.dtype, device=device)
            return Mixes(list(rows), rows)
        n = ops.lib_of(self.dtype).mlora_frag_activation_elems(T, width_p)
        data = torch.empty(len(MIXES) * n, dtype=self.dtype, device=device)
        return Mixes([ops.FragActivation(T, width_p, device, data[i * n:(i + 1) * n]) for i in range(len(MIXES))], data)

    def run(self, mixes: Mixes, state, segs, tok_seq, tok_pos, plan=None):
        """-> the gated outputs of the heads, an activation of out_cols columns; updates state.
        segs: the sequences of the pass (None: a decode step); plan: a TimeMixPlan of the pass for the prompt form."""
        parts = mixes.parts
        T, dev, n = parts[0].shape[0], parts[0].device, self.out_cols
        out = D.activation(T, n, self.dtype, dev)
        rest = (self.w2, self.w0, self.u, self.norm, self.eps, state)
        if plan is None and self.all is not None and T <= 256 and self.w1.N <= n:
            y, z = D.linear_groups(mixes.all(), self.all, n, self.w1.N)
            r, k, v, g = (y[:, i * n:(i + 1) * n] for i in range(4))
        else:
            r, k, v, g = (ops.linear(m, self.proj[s]) for m, s in zip(parts, "rkvg"))
            if plan is not None:
                return D.time_mix_prompt(plan, r, k, v, g, parts[4], self.w1, *rest, out)
            z = ops.linear(parts[4], self.w1, out_dtype=torch.float32)[None]
        return D.time_mix(r, k, v, g, z, self.rank, *rest, segs, tok_seq, tok_pos, out)
