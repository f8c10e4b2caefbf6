"""Plain numpy evaluation of a Dinasun decoder, one function per mechanism, float64 throughout.

Written from the design's equations and used by the tests only: recurrences run token by token, every token attends by an
explicit loop over its prefix, nothing is cached, nothing is fused, and no code is shared with the package.  `P` is a dict
of arrays by tensor name, `cfg` the parsed configuration.
"""
from __future__ import annotations

import math

import numpy as np


def rms(x, eps):
    """x divided by its root mean square over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def silu(z):
    return z / (1.0 + np.exp(-z))


def dynamic_tanh(x, P, name):
    """The norm of this design: no statistics."""
    return np.tanh(P[name + ".alpha"] * x) * P[name] + P[name + ".b"]


def token_shift(h):
    """The previous token's row, zeros ahead of the first."""
    return np.concatenate([np.zeros_like(h[:1]), h[:-1]])


def shift_mix(h, mu):
    return h + (token_shift(h) - h) * mu


def log_decay(mix_w, P, name):
    """Logarithm of the decay per channel: negative."""
    return -np.exp(np.tanh(mix_w @ P[name + ".w1"].T) @ P[name + ".w2"].T + P[name + ".w0"])


def wkv_scan(r, k, v, w, u, S=None):
    """r, k, v, w (decays) [T, H, D], u [H, D] -> (outputs [T, H, D], final state [H, D (key), D (value)])."""
    T, H, D = r.shape
    S = np.zeros((H, D, D)) if S is None else S.copy()
    o = np.zeros((T, H, D))
    for t in range(T):
        for a in range(H):
            kv = np.outer(k[t, a], v[t, a])
            o[t, a] = (S[a] + u[a][:, None] * kv).T @ r[t, a]
            S[a] = w[t, a][:, None] * S[a] + kv
    return o, S


def wkv(h, mix, P, name, eps):
    """Time mixing over a whole sequence h [T, width]."""
    T, H, D = h.shape[0], mix["heads"], mix["dim"]
    m = {s: shift_mix(h, P[f"{name}.mu.{s}"]) for s in "rkvgw"}
    r, k, v = ((m[s] @ P[f"{name}.{s}"].T).reshape(T, H, D) for s in "rkv")
    gate = silu(m["g"] @ P[name + ".g"].T)
    w = np.exp(log_decay(m["w"], P, name)).reshape(T, H, D)
    o, _ = wkv_scan(r, k, v, w, P[name + ".u"])
    return (rms(o, eps).reshape(T, H * D) * P[name + ".norm"] * gate) @ P[name + ".o"].T


def query_temperature(pos, temp):
    if not temp:
        return np.ones(len(pos))
    return 1.0 + temp["coef"] * np.log(np.floor((np.asarray(pos) + 1.0) / temp["every"]) + 1.0)


def slopes(H):
    return np.array([2.0 ** (-8.0 * (a + 1) / H) for a in range(H)])


def softmax(s):
    e = np.exp(s - s.max())
    return e / e.sum()


def attention(h, mix, P, name, eps):
    """Tied keys and values, grouped heads, distance bias."""
    T, H, G, D = h.shape[0], mix["heads"], mix["kv_heads"], mix["dim"]
    v = (h @ P[name + ".k"].T + P[name + ".k.b"]).reshape(T, G, D)
    q = (h @ P[name + ".q"].T + P[name + ".q.b"]).reshape(T, H, D)
    k = rms(v, eps) * P[name + ".k.norm"]
    q = rms(q, eps) * P[name + ".q.norm"] * query_temperature(range(T), mix.get("q_temp"))[:, None, None]
    m = slopes(H)
    out = np.zeros((T, H, D))
    for i in range(T):
        for a in range(H):
            g = a // (H // G)
            s = (k[: i + 1, g] @ q[i, a]) * mix["scale"] - m[a] * (i - np.arange(i + 1))
            out[i, a] = softmax(s) @ v[: i + 1, g]
    return out.reshape(T, H * D) @ P[name + ".o"].T


def glu(h, P, name):
    return (silu(h @ P[name + ".gate"].T) * (h @ P[name + ".up"].T)) @ P[name + ".down"].T


def table_moe(h, tokens, mlp, P, name):
    """Experts by token id, equal weights, and the shared one."""
    top = mlp["router"]["top"]
    y = np.zeros_like(h)
    for t, tok in enumerate(tokens):
        for e in P[name + ".table"][tok].astype(int):
            y[t] += glu(h[t], P, f"{name}.e{e}") / top
    if mlp.get("shared"):
        y = y + glu(h, P, name + ".shared")
    return y


def passes(cfg):
    """[(layers of the pass, whether the embedding comes in ahead)]: the loop's passes and what lies around them."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(range(n), False)]
    a, b = loop["start"], loop["stop"]
    return [(range(a), False)] + [(range(a, b), True)] * loop["times"] + [(range(b, n), False)]


def forward(tokens, cfg, P, layers_out=None):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer run."""
    tokens = np.asarray(tokens, dtype=np.int64)
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x0 = x = P["embed"][tokens].astype(np.float64) * cfg["embedding"]["scale"]
    for layers, entry in passes(cfg):
        if entry:
            x = np.concatenate([x, x0], -1) @ P["loop.in"].T
        for l in layers:
            n, L = f"l{l}", cfg["layers"][l]
            mixer = {"wkv": wkv, "attention": attention}[L["type"]]
            x = x + m * dynamic_tanh(mixer(dynamic_tanh(x, P, n + ".norm1"), L["mixer"], P, n + ".mix", eps), P, n + ".norm1b")
            if L.get("mlp"):
                x = x + m * dynamic_tanh(table_moe(dynamic_tanh(x, P, n + ".norm2"), tokens, L["mlp"], P, n + ".mlp"), P, n + ".norm2b")
            if layers_out is not None:
                layers_out.append(x.copy())
    return dynamic_tanh(x, P, "final.norm") @ P["embed"].T
