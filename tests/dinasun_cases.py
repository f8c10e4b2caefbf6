"""Small Dinasun configurations with random weights (values that bfloat16 holds exactly, so that every element type and the
oracle read the same numbers)."""
import numpy as np
import torch


def att(heads=6, kv_heads=2, dim=40, scale=0.2, temp=(0.4, 24), mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if temp:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def wkv(heads=3, dim=24, mlp=None):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "mlp": mlp}


def moe(ff=40, experts=5, top=2, shared=72):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def config(layers, vocab=330, width=104, eps=1e-5, scale=3.0, mult=0.7, loop=None):
    c = {"architecture": "Dinasun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "residual_mult": mult,
         "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


CONFIGS = {
    # odd sizes everywhere, a loop from the first layer on over both kinds of mixers, a layer without feed-forward
    "odd": config([att(mlp=moe()), wkv(mlp=moe(experts=7, top=3)), att(5, 5, 20, temp=None), wkv(2, 72, moe(24, 3, 1, None))], loop=(0, 3, 3)),
    # no loop, one head, one expert per token, nothing shared, whole residual
    "plain": config([wkv(1, 64, moe(32, 4, 1, None)), att(1, 1, 64, 0.125, (0.5, 16)), wkv(2, 32)], vocab=256, width=64, eps=1e-3, scale=1.0, mult=1.0),
    # a group of more heads than one matrix-core tile has columns, heads of more than 128, a loop that ends with the last layer
    "wide": config([att(36, 2, 96, 0.1, (0.3, 40), moe(64, 9, 9, 64)), wkv(1, 136, moe(64, 16, 4, 200))], vocab=512, width=128, scale=6.0, mult=0.4,
                   loop=(1, 2, 2)),
}


def weights(cfg, seed=0, sharp=1.0):
    """name -> float64 array.  sharp: factor on the queries' norm weights (peaked attention: single keys decide)."""
    rng = np.random.default_rng(seed)
    W, V = cfg["width"], cfg["vocab"]
    P = {}

    def put(name, shape, std, mean=0.0):
        P[name] = torch.from_numpy(np.asarray(rng.normal(mean, std, shape))).to(torch.bfloat16).double().numpy()

    def norm(name):
        put(name, (W,), 0.2, 1.0)
        put(name + ".b", (W,), 0.1)
        put(name + ".alpha", (), 0.05, 0.5)

    def glu(name, ff):
        for k in ("gate", "up"):
            put(f"{name}.{k}", (ff, W), 1.5 * W ** -0.5)
        put(name + ".down", (W, ff), 2 * ff ** -0.5)

    put("embed", (V, W), 0.5)
    if cfg.get("loop"):
        put("loop.in", (W, 2 * W), (2 * W) ** -0.5)
    for l, L in enumerate(cfg["layers"]):
        n, m, f = f"l{l}", L["mixer"], L.get("mlp")
        for k in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            norm(f"{n}.{k}")
        H, D, x = m["heads"], m["dim"], n + ".mix"
        if L["type"] == "attention":
            G = m["kv_heads"]
            for k, rows in (("q", H * D), ("k", G * D)):
                put(f"{x}.{k}", (rows, W), 2 * W ** -0.5)
                put(f"{x}.{k}.b", (rows,), 0.3)
            put(x + ".q.norm", (D,), 0.2 * sharp, sharp)
            put(x + ".k.norm", (D,), 0.2, 1.0)
        else:
            for s in "rkvgw":
                P[f"{x}.mu.{s}"] = torch.from_numpy(rng.uniform(0, 1, W)).to(torch.bfloat16).double().numpy()
            for s in "rkvg":
                put(f"{x}.{s}", (H * D, W), 1.5 * W ** -0.5)
            R = 5 + D // 4
            put(x + ".w1", (R, W), 1.5 * W ** -0.5)
            put(x + ".w2", (H * D, R), R ** -0.5)
            put(x + ".w0", (H * D,), 1.5, -2.0)        # decays from almost none to almost everything per token
            put(x + ".u", (H, D), 1.0)
            put(x + ".norm", (H * D,), 0.2, 1.0)
        put(x + ".o", (W, H * D), (H * D) ** -0.5)
        if f:
            E, top = f["router"]["experts"], f["router"]["top"]
            P[n + ".mlp.table"] = np.argsort(rng.random((V, E)), -1)[:, :top].astype(np.int32)
            for e in range(E):
                glu(f"{n}.mlp.e{e}", f["expert"]["ff"])
            if f.get("shared"):
                glu(n + ".mlp.shared", f["shared"]["ff"])
    norm("final.norm")
    return P


def tensors(P):
    def get(name):
        t = torch.from_numpy(np.asarray(P[name]))
        return t if t.dtype == torch.int32 else t.to(torch.bfloat16)
    return get
