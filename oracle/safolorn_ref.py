"""Plain numpy evaluation of a Safolorn decoder, one function per mechanism, float64 throughout.

Written from the design's equations and used by the tests only: every token attends by an explicit loop over its
prefix, nothing is cached, nothing is fused, and no code is shared with the package.  `P` is a dict of arrays by
tensor name, `cfg` the parsed configuration.
"""
from __future__ import annotations

import math

import numpy as np


def rms(x, eps):
    """x divided by its root mean square over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rotation_frequencies(rot):
    """(frequencies [dims/2], factor on cos and sin) of one rotation; YaRN when `scaling` is given."""
    dims, base = rot["dims"], float(rot["base"])
    i = np.arange(dims // 2, dtype=np.float64)
    f = base ** (-2.0 * i / dims)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def turn_dim(t):
        return dims * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(turn_dim(sc["fast"])), 0)
    hi = min(math.ceil(turn_dim(sc["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, pos, rot):
    """x [T, ..., n] at positions pos [T]: neighbouring pairs (2i, 2i+1) of the first `dims` entries turn."""
    f, m = rotation_frequencies(rot)
    y = np.array(x, dtype=np.float64)
    for t, p in enumerate(pos):
        for i, fi in enumerate(f):
            c, s = m * math.cos(p * fi), m * math.sin(p * fi)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            y[t, ..., 2 * i] = u * c - v * s
            y[t, ..., 2 * i + 1] = v * c + u * s
    return y


def latent(h, pos, mix, P, name, eps):
    """What a layer with its own W_dkv keeps per token: (normed latent, rotated shared key part)."""
    r = mix["kv_rank"]
    d = h @ P[name + ".mix.dkv"].T
    return rms(d[:, :r], eps) * P[name + ".mix.dkv.norm"], rotate(d[:, r:], pos, mix["rot"])


def sink_softmax(scores, sink):
    """Weights of the visible keys; the sink takes its share of the denominator."""
    m = max(float(np.max(scores)), float(sink))
    e = np.exp(scores - m)
    return e / (e.sum() + math.exp(sink - m))


def latent_attention(h, pos, mix, P, name, kv):
    """h [T, width] at consecutive positions from 0; kv = (c [T, r], k_rot [T, rot_dim])."""
    T, H, dim, rd, vd = h.shape[0], mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"]
    c, kr = kv
    q = (h @ P[name + ".mix.q"].T).reshape(T, H, dim + rd)
    qr = rotate(q[..., dim:], pos, mix["rot"])
    k = (c @ P[name + ".mix.uk"].T).reshape(T, H, dim)
    v = (c @ P[name + ".mix.uv"].T).reshape(T, H, vd)
    out = np.zeros((T, H, vd))
    for i in range(T):
        for a in range(H):
            s = (k[: i + 1, a] @ q[i, a, :dim] + kr[: i + 1] @ qr[i, a]) * mix["scale"]
            out[i, a] = sink_softmax(s, P[name + ".mix.sink"][a]) @ v[: i + 1, a]
    return out.reshape(T, H * vd) @ P[name + ".mix.o"].T


def dense_ff(h, mlp, P, name):
    lim = mlp["limit"]
    g = np.minimum(h @ P[name + ".mlp.gate"].T, lim)
    u = np.clip(h @ P[name + ".mlp.up"].T, -lim, lim)
    return (g / (1.0 + np.exp(-1.702 * g)) * (u + 1.0)) @ P[name + ".mlp.down"].T


def route(h, mlp, P, name):
    """(experts chosen per token, best first, and their weights)."""
    z = h @ P[name + ".mlp.router"].T + P[name + ".mlp.router.b"]
    pick = np.argsort(-z, axis=-1, kind="stable")[:, : mlp["router"]["top"]]
    zz = np.take_along_axis(z, pick, -1)
    w = np.exp(zz - zz.max(-1, keepdims=True))
    return pick, w / w.sum(-1, keepdims=True)


def moe_ff(h, mlp, P, name):
    pick, w = route(h, mlp, P, name)
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, we in zip(pick[t], w[t]):
            a = np.maximum(P[f"{name}.mlp.e{e}.up"] @ h[t], 0.0) ** 2
            y[t] += we * (P[f"{name}.mlp.e{e}.down"] @ a)
    return y


def token_side(x, tokens, l, cfg, P):
    d = cfg["token_side"]["dim"]
    e = P["side.embed"][tokens][:, l * d:(l + 1) * d]
    g = gelu_tanh(x @ P[f"l{l}.side.gate"].T) * e
    return x + rms(g @ P[f"l{l}.side.proj"].T, cfg["norm"]["eps"]) * P[f"l{l}.side.norm"]


def forward(tokens, cfg, P, layers_out=None):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer."""
    tokens = np.asarray(tokens, dtype=np.int64)
    pos = np.arange(len(tokens))
    eps = cfg["norm"]["eps"]
    x = P["embed"][tokens].astype(np.float64)
    kvs = {}
    for l, L in enumerate(cfg["layers"]):
        name, mix = f"l{l}", L["mixer"]
        h1 = rms(x, eps) * P[name + ".norm1"]
        src = mix.get("kv_from")
        if src is None:
            src = l
            kvs[l] = latent(h1, pos, mix, P, name, eps)
        y = latent_attention(h1, pos, mix, P, name, kvs[src])
        if L.get("mlp") is not None:
            h2 = rms(x, eps) * P[name + ".norm2"]
            y = y + (dense_ff if L["mlp"]["kind"] == "dense" else moe_ff)(h2, L["mlp"], P, name)
        x = x + y
        if cfg.get("token_side"):
            x = token_side(x, tokens, l, cfg, P)
        if layers_out is not None:
            layers_out.append(x.copy())
    return (rms(x, eps) * P["final.norm"]) @ P["head"].T
