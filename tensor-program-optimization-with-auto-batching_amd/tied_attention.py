"""Attention whose values are its keys before their norm: the cache holds one vector per token and key/value head.

A key is its value divided by the value's root mean square, times a weight shared by the heads.  The weight goes to the queries
and the divisor is kept as one number per token and head, so nothing but the values is stored or read.  Positions enter
through a distance bias per head and, optionally, a temperature of the queries.  Decode steps and short passes read the pages
as they are; prompts lay keys and transposed values of their contexts out in scratch memory once per pass.
"""
from __future__ import annotations

import dataclasses
from typing import Optional, Tuple

import torch

from . import decoder_ops as D
from .decoder_ops import pad32, pad64, padded


@dataclasses.dataclass(frozen=True)
class TiedSpec:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    q_temp: Optional[Tuple[float, float]] = None      # (coefficient, every)

    @classmethod
    def from_config(cls, c: dict) -> "TiedSpec":
        heads, dim, temp = int(c["heads"]), int(c["dim"]), c.get("q_temp")
        s = cls(heads, int(c.get("kv_heads") or heads), dim, float(c["scale"]), (float(temp["coef"]), float(temp["every"])) if temp else None)
        if int(c.get("vdim") or dim) != dim or heads % s.kv_heads:
            raise ValueError(f"tied attention needs values as wide as its keys and whole groups of heads: {c}")
        return s

    def cache_entry(self, n_pages, slots, page, width_p):
        """Shapes of what a layer run keeps (and whether in elements rather than fp32): pages of values, and key scales."""
        return ((n_pages, self.kv_heads, -(-self.dim // 32), 4, page, 8), True), ((n_pages, self.kv_heads, page), False)


def distance_slopes(heads: int) -> torch.Tensor:
    """2^(-8 (h + 1) / heads)."""
    return torch.pow(2.0, torch.arange(1, heads + 1, dtype=torch.float64) * (-8.0 / heads)).float()


class TiedAttention:
    """Weights of one layer.  `proj` is the fused input projection, rows: the query heads, then the key/value heads."""

    def __init__(self, spec: TiedSpec, w: dict, width: int, eps: float, dtype, device):
        """w: q [H dim, width], q_b, k [G dim, width], k_b, q_norm [dim], k_norm [dim], o [width, H dim]."""
        s, self.spec, self.eps, self.dtype = spec, spec, float(eps), dtype
        H, Hp = s.heads, pad64(width)
        f32 = lambda *names: torch.cat([w[n].to(device, torch.float32) for n in names]).contiguous()
        rows = torch.cat([w["q"], w["k"]]).to(device, dtype)
        self.proj = D.weight(padded(rows, pad32(rows.shape[0]), Hp))
        self.bias = f32("q_b", "k_b")
        self.q_norm = f32("q_norm") * f32("k_norm")
        self.slopes = distance_slopes(H).to(device)
        self.vp = pad32(s.dim)
        self.out_cols = H * self.vp if dtype == torch.float32 else pad64(H * self.vp)
        o = padded(w["o"].to(device, dtype).view(width, H, s.dim), Hp, H, self.vp).reshape(Hp, H * self.vp)
        self.o = D.weight(padded(o, Hp, self.out_cols))
        self.prompt_form = dtype != torch.float32 and D.tied_prefill_served(s.dim)

    def prompt_form_pays(self, seqs) -> bool:
        """Whether a pass (per sequence: appended tokens, context length) is cheaper over keys and values in scratch memory: it
        reads the context three times more, but once per 128 tokens instead of once per token."""
        if not self.prompt_form:
            return False
        s = self.spec
        line = s.kv_heads * self.vp * 2
        direct = sum(n * (c - n / 2) for n, c in seqs) * line * -(-s.heads // s.kv_heads // 16) / 8e12
        laid = sum(c * 3 + n * c / 128 * s.heads / s.kv_heads for n, c in seqs) * line / 4e12
        return laid + 1e-5 < direct

    def attend(self, y, pages, key_scale, block_table, tok_seq, tok_pos, max_ctx, plan=None):
        """y [T, proj rows] fp32: the projections; plan: a PrefillPlan of the pass for the prompt form."""
        s, T = self.spec, y.shape[0]
        q = torch.empty((T, s.heads, self.vp), dtype=self.dtype, device=y.device)
        D.tied_prep(q, pages, key_scale, y, self.bias, self.q_norm, self.eps, s.q_temp, block_table, tok_seq, tok_pos, s.heads, s.kv_heads, s.dim)
        out = D.activation(T, self.out_cols, self.dtype, y.device)
        heads = out
        if self.out_cols > s.heads * self.vp:                                    # a block of columns that no head writes
            out.data.zero_()
            heads = out.columns(0, s.heads * self.vp)
        if plan is not None:
            D.tied_prefill(plan, q, pages, key_scale, self.slopes, s.scale, s.kv_heads, s.dim, heads)
        else:
            D.tied_attn(q, pages, key_scale, block_table, tok_seq, tok_pos, self.slopes, s.scale, s.kv_heads, s.dim, max_ctx, heads)
        return out
