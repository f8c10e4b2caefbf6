"""Latent attention: every head's keys and values are linear images of one cached vector per token.

Two forms of the same sums.  Decode steps and short passes lift the queries into the latent space (W_uk transposed) and take
the context vectors out of it again (W_uv), so the attention kernel reads nothing but the cache.  Prompts make the heads'
keys and values once per pass and attend over those: fewer products per score.  The equations and the cache layout stand in
csrc/latent_attention.hip.
"""
from __future__ import annotations

import dataclasses
from typing import Optional

import torch

from . import decoder_ops as D
from .decoder_ops import pad32, pad64, padded
from .rotary import Rotation


@dataclasses.dataclass(frozen=True)
class LatentSpec:
    heads: int
    dim: int            # unrotated query/key dimensions per head
    rot_dim: int        # rotated ones
    vdim: int
    kv_rank: int
    scale: float
    rotation: Rotation
    kv_from: Optional[int] = None     # the layer whose latents this one reads instead of its own

    @classmethod
    def from_config(cls, c: dict) -> "LatentSpec":
        return cls(int(c["heads"]), int(c["dim"]), int(c["rot_dim"]), int(c["vdim"]), int(c["kv_rank"]), float(c["scale"]),
                   Rotation.from_config(c["rot"]), None if c.get("kv_from") is None else int(c["kv_from"]))


class LatentAttention:
    """Weights of one layer in kernel order.  `proj` is the fused input projection, rows: the heads' unrotated query parts
    (each padded to 32), their rotated parts, and - with an own cache - the latent and the shared key part; its input is the
    normed row without the norm's gain, which is applied behind it."""

    def __init__(self, spec: LatentSpec, w: dict, width: int, gain: float, eps: float, dtype, device):
        """w: q [H (dim + rot_dim), width], uk [H dim, kv_rank], uv [H vdim, kv_rank], sink [H], o [width, H vdim] and, without
        kv_from, dkv [kv_rank + rot_dim, width], dkv_norm [kv_rank]."""
        s, self.spec = spec, spec
        self.gain, self.eps, self.dtype = float(gain), float(eps), dtype
        H, R, Hp = s.heads, s.kv_rank, pad64(width)
        self.dp, self.vp, self.rank_p = pad32(s.dim), pad32(s.vdim), pad32(R)
        self.q_cols = self.rank_p + pad32(s.rot_dim)
        self.out_cols = H * self.vp
        t = lambda name: w[name].to(device, dtype)
        q = t("q").view(H, s.dim + s.rot_dim, width)
        rows = [padded(q[:, : s.dim], H, self.dp, width).reshape(H * self.dp, width), q[:, s.dim:].reshape(H * s.rot_dim, width)]
        self.off_rot = H * self.dp
        self.off_c = self.off_rot + H * s.rot_dim
        self.off_kr = self.off_c + R
        self.c_norm = None
        if s.kv_from is None:
            rows.append(t("dkv"))
            self.c_norm = t("dkv_norm").contiguous()
        proj = torch.cat(rows)
        self.proj_rows = pad32(proj.shape[0])
        self.proj = D.weight(padded(proj, self.proj_rows, Hp))
        uk = t("uk").view(H, s.dim, R)
        self.lift = D.weight(padded(uk.transpose(1, 2), H, self.rank_p, self.dp).reshape(H * self.rank_p, self.dp))
        self.uk = None                                                           # for the prompt form
        if dtype != torch.float32 and D.latent_prefill_served(s.dim, s.rot_dim, s.vdim):
            self.uk = D.weight(padded(uk, H, self.dp, self.rank_p).reshape(H * self.dp, self.rank_p))
        uv = t("uv").view(H, s.vdim, R)
        self.uv = D.weight(padded(uv, H, self.vp, self.rank_p).reshape(H * self.vp, self.rank_p))
        self.sink = w["sink"].to(device, torch.float32).contiguous()
        o = t("o").view(width, H, s.vdim)
        self.o_rows = padded(o, Hp, H, self.vp).reshape(Hp, self.out_cols)      # the output projection, for the layer to place

    def prompt_form_pays(self, seqs) -> bool:
        """Whether a pass (per sequence: appended tokens, context length) is cheaper with keys and values made: products on
        the matrix cores for that form, cache bytes through the second-level caches for the other (they are read once per
        token and 16 heads)."""
        if self.uk is None:
            return False
        H = self.spec.heads
        lifted = sum(n * (c - n / 2) for n, c in seqs) * -(-H // 16) * self.q_cols * 2 / 8e12
        made = sum(c * self.rank_p * (self.dp + self.vp) + n * c * (self.dp + self.q_cols - self.rank_p + 2 * self.vp) for n, c in seqs) * 2 * H / 4e14
        return made + 2e-5 < lifted

    def attend(self, qkv, pages, block_table, tok_seq, tok_pos, cos, sin, max_ctx, store, plan=None, out=None):
        """plan: a PrefillPlan of the pass for the prompt form, None for the lifted form."""
        s, T = self.spec, qkv.shape[0]
        H = s.heads
        if out is None:
            out = D.activation(T, self.out_cols, self.dtype, qkv.device)
        # the norm's gain on the queries is left to the scale of the scores
        scale = s.scale * self.gain
        prep = lambda q, q_off, lift=None: D.latent_prep(q, q_off, pages, qkv, self.off_rot, self.off_c, self.off_kr, self.gain,
                                                         self.c_norm if store else None, self.eps, block_table, tok_seq, tok_pos, cos, sin, H,
                                                         s.kv_rank, s.rot_dim, lift)
        if plan is not None:
            q_rot = torch.empty((T, H, self.q_cols - self.rank_p), dtype=self.dtype, device=qkv.device)
            prep(q_rot, 0)
            return D.latent_prefill(plan, qkv, q_rot, pages, self.uk, self.uv, self.sink, scale, s.kv_rank, s.dim, s.rot_dim, s.vdim, out)
        q = torch.empty((T, H, self.q_cols), dtype=self.dtype, device=qkv.device)
        cached = (pages, block_table, tok_seq, tok_pos, self.sink, scale, s.kv_rank, s.rot_dim)
        if self.dtype == torch.float32:
            prep(q, self.rank_p)
            D.head_linear(qkv, self.proj_rows, self.dp, self.lift, H, T, self.dp, self.rank_p, q, H * self.q_cols, self.q_cols)
        else:
            prep(q, self.rank_p, self.lift)
        splits = D.latent_attn_splits(T, H, max_ctx, self.dtype)
        if splits > 1:
            return D.latent_attn_out(q, *cached, splits, self.uv, self.vp, out)
        ctx = D.latent_attn(q, *cached, max_ctx, splits=splits)
        return D.head_linear(ctx, H * self.rank_p, self.rank_p, self.uv, H, T, self.rank_p, self.vp, out, self.out_cols, self.vp)
