"""Host side of the Dinasun model: configuration, order of layer runs, state cache, argument checks - and the oracle itself."""
import ctypes

import numpy as np
import pytest
import torch

import dinasun_cases as C
from conftest import load_pkg
from oracle import dinasun_ref as R


def test_configuration_is_read_and_checked():
    m = load_pkg("dinasun")
    c = m.DinasunConfig.from_dict(C.CONFIGS["odd"])
    assert (c.vocab, c.width, c.embed_scale, c.residual_mult, len(c.layers), c.loop) == (330, 104, 3.0, 0.7, 4, (0, 3, 3))
    a, w = c.layers[0], c.layers[1]
    assert (a.mixer.heads, a.mixer.kv_heads, a.mixer.dim, a.mixer.q_temp) == (6, 2, 40, (0.4, 24.0)) and c.layers[2].mixer.q_temp is None
    assert (w.mixer.heads, w.mixer.dim, w.ff.experts, w.ff.top, w.ff.shared) == (3, 24, 7, 3, 72)
    assert c.layers[2].ff is None and c.layers[3].ff.shared is None
    bad = [C.config([{**C.wkv(), "type": "other"}]), C.config([C.wkv(mlp={"kind": "dense"})]), C.config([C.wkv()], loop=(0, 2, 1)),
           C.config([C.wkv()], loop=(0, 1, 0)), C.config([C.att(6, 4)])]
    vdim = C.att()
    vdim["mixer"]["vdim"] = 8
    for cfg in bad + [C.config([vdim])]:
        with pytest.raises(ValueError):
            m.DinasunConfig.from_dict(cfg)


@pytest.mark.parametrize("n,loop,want", [(3, None, [(0, 0), (1, 0), (2, 0)]), (3, (1, 3, 2), [(0, 0), (1, 1), (2, 0), (1, 1), (2, 0)]),
                                         (2, (0, 1, 3), [(0, 1), (0, 1), (0, 1), (1, 0)]), (3, (1, 2, 1), [(0, 0), (1, 1), (2, 0)])])
def test_layer_runs(n, loop, want):
    c = load_pkg("dinasun").DinasunConfig.from_dict(C.config([C.wkv()] * n, loop=loop))
    assert [(l, int(e)) for l, e in c.runs()] == want
    assert [l for l, _ in c.runs()] == [l for r, _ in R.passes(C.config([C.wkv()] * n, loop=loop)) for l in r]


def test_registry_knows_the_design():
    reg = load_pkg("registry")
    cls = reg.model_class(C.CONFIGS["plain"])
    assert cls.__name__ == "DinasunForCausalLM" and cls.dtypes == ("bfloat16", "float32")
    with pytest.raises(ValueError):
        cls._ids(cls(load_pkg("dinasun").DinasunConfig.from_dict(C.CONFIGS["odd"]), device="cpu"), 3, {0: (None, [1])})


def test_state_cache_bookkeeping():
    """One entry per layer run; segments and last tokens of a pass; none of them in a decode step."""
    c = load_pkg("dinasun").DinasunConfig.from_dict(C.CONFIGS["odd"])
    kv = load_pkg("kv_cache").PagedStateCache([c.layers[l].mixer for l, _ in c.runs()], 128, 8, max_seqs=3, max_blocks=4, max_pos=64, dtype=torch.float32,
                                              device="cpu")
    assert len(kv.entries) == 10 and kv.entries[0][0].shape == (8, 2, 2, 4, 16, 8) and kv.entries[0][1].shape == (8, 2, 16)
    assert kv.entries[1][0].shape == (3, 3, 24, 24) and kv.shift(1).shape == (3, 128) and kv.entries[9][0].shape == (3, 2, 72, 72)
    with pytest.raises(RuntimeError):
        kv._pass()
    for s in "ab":
        kv.add_sequence(s)
    kv.begin_forward(["b", "a"], [5, 2])
    m = kv._pass()
    assert m["segs"].tolist() == [[1, 0, 5, 0], [0, 5, 2, 0]] and m["last"].tolist() == [4] * 5 + [6] * 2 and kv._pass() is m
    kv.end_forward()
    kv.begin_forward(["a", "b"], [3, 1])
    assert kv._pass()["segs"].tolist() == [[0, 0, 3, 2], [1, 3, 1, 5]] and kv._pass()["last"].tolist() == [2, 2, 2, 3]
    kv.end_forward()
    kv.begin_forward(["a", "b"], [1, 1])
    assert kv._pass()["segs"] is None and kv.token_meta()[2] is None
    kv.end_forward()


def test_expert_tables_are_checked():
    ff = load_pkg("feed_forward")
    spec = ff.TableMoeSpec(8, 3, 2)
    for bad in ([[0, 3]], [[-1, 0]], [[0, 1, 2]]):
        with pytest.raises(ValueError):
            ff.TableMoe(spec, {"table": torch.tensor(bad, dtype=torch.int32)}, 16, torch.float32, "cpu")


def test_argument_validation():
    """Refused on the host before any launch (dummy pointers)."""
    load_pkg("build").ensure("bfloat16"), load_pkg("build").ensure("float32")
    lm = load_pkg("_lib")
    b, f = lm.lib("bfloat16"), lm.lib("float32")

    def step(lib, **kw):
        a = lm.StreamStep(**{**dict(T=4, Hp=64, x=16, out_row=16, ld_row=64), **kw})
        return lib.mlora_stream_step(ctypes.byref(a), None)
    assert step(b, Hp=40) == -2 and step(b, x=None) == -1 and step(b, n_part=1) == -1 and step(b, rows=16) == -1 and step(b, ld_row=32) == -1
    assert step(f, out_frag=16) == -2 and step(b, mu=16) == -1
    assert step(b, mu=16, shift=16, tok_seq=16, tok_pos=16, n_seq=1, y=16, x_out=16) == -1          # would update in place what neighbours read
    mix = lambda lib=b, lay=0, ld_y=64, D=32, R=8, segs=None, n=4: lib.mlora_time_mix(16, lay, ld_y, 16, 16, 16, 16, 64, 16, 1, 32, R, 16, 64, 16, 16, 16, 1e-5, 16,
                                                                                    2, segs, n, 16, 16, 4, 2, D, None)
    assert mix(D=33) == -2 and mix(R=300) == -2 and mix(f, lay=1) == -2 and mix(n=3) == -2 and mix(ld_y=128) == -2
    att = lambda lib, G=2, D=40, splits=1, ws=None, n=0: lib.mlora_tied_attn(16, 0, 16, 16, 16, 16, 4, 16, 16, 16, 0.1, 2, 6, G, D, 8, 2, splits, ws, n, None)
    assert att(b, G=4) == -2 and att(b, D=520) == -2 and att(b, splits=2) == -3 and att(f, splits=2) == -2
    assert b.mlora_tied_attn_splits(1, 8, 2, 100000) > 1 and f.mlora_tied_attn_splits(1, 8, 2, 100000) == 1
    pre = lambda D=64, pages=4, elems=1 << 30: b.mlora_tied_prefill(16, 0, 512, 16, 16, 16, 16, pages, 16, 1, 16, 0.1, 8, 8, 2, D, 8, 16, elems, None)
    assert pre(D=200) == -2 and pre(pages=6) == -2 and pre(elems=8) == -3
    assert b.mlora_moe_table_plan(16, 16, 16, 16, 16, 0, 5, 4, 3, 2, None) == -2
    ml = lambda **k: b.mlora_moe_linear(16, 16, 16, 16, 16, 16, 16, 4, 64, 4, 64, 64, 2, k.get("stage", 0), 2, k.get("alpha", 1.0), None, 0, None)
    assert ml(stage=1) == -2 and ml(alpha=2.0) == -2
    assert b.mlora_linear_ksplit_store(16, None, 2, 16, 16, 4, 1024, 64, None) == -1


# ------------------------------------------------------------------ the oracle by what the equations fix
def test_oracle_recurrence_unrolled():
    """A token's output is the sum over the tokens before it, decayed by everything between, and its own with the bonus."""
    rng = np.random.default_rng(0)
    T, H, D = 7, 2, 5
    r, k, v = (rng.normal(size=(T, H, D)) for _ in range(3))
    w, u = rng.uniform(0.1, 1, (T, H, D)), rng.normal(size=(H, D))
    o, S = R.wkv_scan(r, k, v, w, u)
    for t in range(T):
        want = np.einsum("hd,hd->h", r[t], u * k[t])[:, None] * v[t]
        for s in range(t):
            want += np.einsum("hd,hd->h", r[t], k[s] * w[s + 1:t].prod(0))[:, None] * v[s]
        assert np.allclose(o[t], want)
    assert np.allclose(R.wkv_scan(r[4:], k[4:], v[4:], w[4:], u, R.wkv_scan(r[:4], k[:4], v[:4], w[:4], u)[1])[0], o[4:])


def test_oracle_norm_temperature_and_slopes():
    P = {"n": np.array([2.0, 3.0]), "n.b": np.array([0.5, -1.0]), "n.alpha": 0.25}
    assert np.allclose(R.dynamic_tanh(np.array([4.0, -4.0]), P, "n"), [2 * np.tanh(1) + 0.5, -3 * np.tanh(1) - 1])
    t = R.query_temperature([0, 6, 7, 8, 15, 23], {"coef": 0.5, "every": 8})
    assert np.allclose(t, 1 + 0.5 * np.log([1, 1, 2, 2, 3, 4]))
    assert np.allclose(R.slopes(4), [0.25, 0.0625, 0.015625, 0.00390625])
    assert np.allclose(load_pkg("tied_attention").distance_slopes(6).numpy(), R.slopes(6), rtol=1e-7)


def test_oracle_causality_and_loop():
    cfg = C.CONFIGS["odd"]
    P = C.weights(cfg, 3)
    toks = np.random.default_rng(0).integers(0, cfg["vocab"], 12)
    lo = []
    full = R.forward(toks, cfg, P, lo)
    assert len(lo) == 10 and np.allclose(full[:7], R.forward(toks[:7], cfg, P))
    other = toks.copy()
    other[0] = (other[0] + 1) % cfg["vocab"]
    assert np.abs(R.forward(other, cfg, P)[-1] - full[-1]).max() > 1e-4
    once = C.config(cfg["layers"], loop=(0, 3, 1))
    assert np.abs(R.forward(toks, once, P) - full).max() > 1e-2
