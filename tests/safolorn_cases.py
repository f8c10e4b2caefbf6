"""Small Safolorn configurations with random weights (values that bfloat16 holds exactly, so that every element type and the
oracle read the same numbers)."""
import numpy as np
import torch


def rot(base=1000.0, dims=16, scaling=None):
    return {"base": base, "dims": dims, **({"scaling": scaling} if scaling else {})}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def mixer(heads=3, dim=40, rot_dim=24, vdim=48, kv_rank=72, scale=0.125, r=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
         "rot": r or rot(dims=rot_dim, scaling=YARN)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def dense(ff=88, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff=40, experts=6, top=2):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def layer(mix, mlp):
    return {"type": "latent_attention", "mixer": mix, "mlp": mlp}


def config(layers, vocab=330, width=104, eps=1e-5, side=20):
    c = {"architecture": "Safolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if side:
        c["token_side"] = {"dim": side}
    return c


CONFIGS = {
    # odd sizes everywhere, a shared cache that skips a layer, a layer without feed-forward
    "odd": config([layer(mixer(), dense()), layer(mixer(), moe()), layer(mixer(kv_from=0), moe(experts=7, top=3)),
                   layer(mixer(heads=5, dim=24, vdim=20, kv_from=1), None)]),
    # one head, one expert per token, plain rotation, layers of different geometry, no side input
    "plain": config([layer(mixer(heads=1, dim=32, rot_dim=8, vdim=32, kv_rank=32, r=rot(dims=8)), moe(experts=5, top=1)),
                     layer(mixer(heads=2, dim=16, rot_dim=40, vdim=64, kv_rank=160, r=rot(10000.0, 40)), dense(64, 0.5))],
                    vocab=256, width=64, eps=1e-3, side=0),
    # more heads than one matrix-core tile has columns, a latent wider than one output chunk
    "wide": config([layer(mixer(heads=18, dim=16, rot_dim=16, vdim=16, kv_rank=544, scale=0.2), dense(96, 4.0)),
                    layer(mixer(heads=18, dim=8, rot_dim=16, vdim=24, kv_rank=544, scale=0.2, kv_from=0), moe(64, 9, 9))],
                   vocab=512, width=128, side=32),
}


def weights(cfg, seed=0, sharp=1.0):
    """name -> float64 array.  sharp: factor on the query projections (peaked attention: single keys decide)."""
    rng = np.random.default_rng(seed)
    W = cfg["width"]
    P = {}

    def put(name, shape, std, mean=0.0):
        P[name] = torch.from_numpy(rng.normal(mean, std, shape)).to(torch.bfloat16).double().numpy()

    put("embed", (cfg["vocab"], W), 1.0)
    n_layers = len(cfg["layers"])
    sd = cfg["token_side"]["dim"] if cfg.get("token_side") else 0
    if sd:
        put("side.embed", (cfg["vocab"], sd * n_layers), 1.0)
    for l, L in enumerate(cfg["layers"]):
        n, m = f"l{l}", L["mixer"]
        put(n + ".norm1", (), 0.1, 1.3)
        H, d, r, v, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        put(n + ".mix.q", (H * (d + r), W), sharp * W ** -0.5)
        if m.get("kv_from") is None:
            put(n + ".mix.dkv", (R + r, W), W ** -0.5)
            put(n + ".mix.dkv.norm", (R,), 0.2, 1.0)
        put(n + ".mix.uk", (H * d, R), R ** -0.5)
        put(n + ".mix.uv", (H * v, R), R ** -0.5)
        put(n + ".mix.sink", (H,), 1.0)
        put(n + ".mix.o", (W, H * v), (H * v) ** -0.5)
        f = L.get("mlp")
        if f is not None:
            put(n + ".norm2", (), 0.1, 0.8)
            if f["kind"] == "dense":
                put(n + ".mlp.gate", (f["ff"], W), 1.5 * W ** -0.5)
                put(n + ".mlp.up", (f["ff"], W), 1.5 * W ** -0.5)
                put(n + ".mlp.down", (W, f["ff"]), f["ff"] ** -0.5)
            else:
                E, ff = f["router"]["experts"], f["expert"]["ff"]
                put(n + ".mlp.router", (E, W), 2.0 * W ** -0.5)
                put(n + ".mlp.router.b", (E,), 0.5)
                for e in range(E):
                    put(f"{n}.mlp.e{e}.up", (ff, W), W ** -0.5)
                    put(f"{n}.mlp.e{e}.down", (W, ff), ff ** -0.5)
        if sd:
            put(n + ".side.gate", (sd, W), W ** -0.5)
            put(n + ".side.proj", (W, sd), sd ** -0.5)
            put(n + ".side.norm", (W,), 0.2, 0.5)
    put("final.norm", (), 0.1, 1.1)
    put("head", (cfg["vocab"], W), W ** -0.5)
    return P


def tensors(P):
    return lambda name: torch.from_numpy(np.asarray(P[name])).to(torch.bfloat16)
