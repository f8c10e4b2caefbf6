"""Host side of the Safolorn model: configuration, rotation tables, page bookkeeping, registry, ABI - and the oracle itself."""
import ctypes
import json
import os
import re

import numpy as np
import pytest

import safolorn_cases as C
from conftest import ROOT, load_pkg
from oracle import safolorn_ref as R


@pytest.mark.parametrize("c,width", [(C.rot(500.0, 12), 12), (C.rot(500.0, 12), 20), (C.rot(1000.0, 24, C.YARN), 24),
                                     (C.rot(1e6, 64, {"factor": 1.0, "original": 4096, "fast": 32.0, "slow": 1.0}), 64),
                                     (C.rot(100.0, 2, {"factor": 8.0, "original": 2048, "fast": 1.0, "slow": 1.0}), 2),
                                     (C.rot(30.0, 6, {"factor": 3.0, "original": 7, "fast": 64.0, "slow": 2.0}), 8)])
def test_rotation_tables(c, width):
    rotation = load_pkg("rotary").Rotation.from_config(c)
    cos, sin = rotation.tables(width, 50)
    x = np.random.default_rng(1).normal(size=(50, width))
    want = R.rotate(x, range(50), c)
    got = np.empty_like(x)
    got[:, 0::2] = x[:, 0::2] * cos - x[:, 1::2] * sin
    got[:, 1::2] = x[:, 1::2] * cos + x[:, 0::2] * sin
    assert np.abs(got - want).max() < 1e-6


def test_configuration_is_read_and_checked():
    m = load_pkg("safolorn")
    c = m.SafolornConfig.from_dict(C.CONFIGS["odd"])
    assert (c.vocab, c.width, c.side_dim, len(c.layers)) == (330, 104, 20, 4)
    assert c.layers[2].mixer.kv_from == 0 and c.layers[3].ff is None and c.layers[1].ff.top == 2 and c.layers[0].ff.limit == 1.5
    bad = lambda **kw: C.config([{**C.layer(C.mixer(), C.dense()), **kw}])
    for cfg in (bad(type="other"), bad(mlp={"kind": "other"}), C.config([C.layer(C.mixer(kv_from=0), None)]),
                C.config([C.layer(C.mixer(), None), C.layer(C.mixer(kv_from=0), None), C.layer(C.mixer(kv_from=1), None)])):
        with pytest.raises(ValueError):
            m.SafolornConfig.from_dict(cfg)


def test_pages_and_slots_are_given_back():
    kvm = load_pkg("kv_cache")
    t = kvm.PageTable(4, max_seqs=2, max_blocks=3, max_pos=48, device="cpu", free_pages=[2, 0, 3, 1])
    for sid, n in (("a", 17), ("b", 20)):
        t.add_sequence(sid)
        t.begin_forward([sid], [n])
        t.end_forward()
    assert t.pages_of("a") == [2, 0] and t.pages_of("b") == [3, 1] and not t.free
    with pytest.raises(RuntimeError):
        t.add_sequence("c")
    t.free_sequence("a")
    t.add_sequence("c")
    assert t.slot["c"] == 0
    t.begin_forward(["c", "b"], [2, 1])
    assert t.pages_of("c") == [2] and t.free == [0]
    with pytest.raises(RuntimeError):
        t.free_sequence("b")
    t.end_forward()
    assert t.lens == {"b": 21, "c": 2} and t.block_table.tolist() == [[2, -1, -1], [3, 1, -1]]
    with pytest.raises(RuntimeError):                  # out of pages, not out of blocks
        t.begin_forward(["c"], [40])


def test_registry_and_trace_refusal(tmp_path, capsys):
    reg, trace = load_pkg("registry"), load_pkg("trace")
    assert reg.model_class({"architectures": ["LlamaForCausalLM"]}).__name__ == "LlamaForCausalLM"
    assert reg.model_class(C.CONFIGS["plain"]).dtypes == ("bfloat16", "float32")
    with pytest.raises(ValueError):
        reg.model_class({"architecture": "nothing"})
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["LlamaForCausalLM"]}))
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "16"]) == 3
    assert "float16" in capsys.readouterr().err


def test_models_without_adapters_refuse_them():
    m = load_pkg("safolorn").SafolornForCausalLM
    assert m._ids(m, 3, {}) == {}
    with pytest.raises(ValueError):
        m._ids(m(load_pkg("safolorn").SafolornConfig.from_dict(C.CONFIGS["odd"]), device="cpu"), 3, {0: (None, [1])})
    with pytest.raises(KeyError):
        m.__getitem__(m(load_pkg("safolorn").SafolornConfig.from_dict(C.CONFIGS["odd"]), device="cpu"), "decode_a0")


def test_decoder_header_and_libraries_agree():
    lm, b = load_pkg("_lib"), load_pkg("build")
    text = re.sub(r"/\*.*?\*/", "", open(os.path.join(ROOT, "include", "mlora_decoder.h")).read(), flags=re.S)
    names = sorted(set(re.findall(r"\b(mlora_[a-z0-9_]+)\s*\(", text)))
    assert sorted(lm.DECODER_SIGNATURES) == names
    for dt in ("bfloat16", "float32"):
        b.ensure(dt)
        lib = ctypes.CDLL(lm.LIB_PATHS[dt])
        missing = [n for n in names if not hasattr(lib, n)]
        assert missing == ([] if dt == "bfloat16" else sorted(lm.MATRIX_CORE_ONLY))


def test_decoder_argument_validation():
    """Refused on the host before any launch (dummy pointers)."""
    load_pkg("build").ensure("bfloat16"), load_pkg("build").ensure("float32")
    lm = load_pkg("_lib")
    b, f = lm.lib("bfloat16"), lm.lib("float32")
    assert b.mlora_stream_norm(16, None, 16, None, 0, None, None, 1e-5, 1.0, 0, 4, 100, 100, None) == -2
    assert f.mlora_stream_norm(16, None, 16, None, 0, None, None, 1e-5, 1.0, 0, 4, 96, 96, None) == -2
    assert b.mlora_stream_norm(16, None, 16, None, 2, None, None, 1e-5, 1.0, 0, 4, 96, 96, None) == -1
    assert b.mlora_head_linear(16, 0, 64, 32, 16, 60, 32, 16, 2, 4, 32, 32, 1.0, None) == -2
    assert f.mlora_head_linear(16, 1, 64, 32, 16, 64, 32, 16, 2, 4, 32, 32, 1.0, None) == -2
    la = lambda lib, splits=1, ws=None, n=0: lib.mlora_latent_attn(16, 16, 16, 16, 4, 16, 16, None, 0.1, 2, 3, 72, 24, 8, 2, splits, ws, n, None)
    assert la(b, splits=2) == -3 and la(f, splits=2) == -2
    assert b.mlora_latent_attn_workspace_bytes(2, 3, 72, 2) == 2 * 2 * 3 * (96 + 2) * 4
    assert b.mlora_latent_attn_splits(4, 16, 100000) > 1 and b.mlora_latent_attn_splits(4096, 16, 100000) == 1 == f.mlora_latent_attn_splits(4, 16, 9999)
    assert b.mlora_moe_route(16, 16, 16, 8, 16, 1.0, 4, 8, 9, None) == -2
    for lib in (b, f):
        for T, E, top in ((1, 6, 2), (40, 6, 2), (1000, 64, 8)):
            rows = lib.mlora_moe_tile_rows(T, E, top)
            assert lib.mlora_moe_max_tiles(T, E, top) >= -(-T * top // rows) and lib.mlora_moe_max_places(T, E, top) >= T * top
    ml = lambda rows=32, K=64, stage=0, act=1, ws=16, n=1 << 20: b.mlora_moe_linear(16, 16, 16, 16, 16, 16, rows, 4, 64, 4, K, 64, 2, stage, act, 1.0, ws, n,
                                                                                     None)
    assert ml() == -2 and ml(rows=256, K=96) == -2 and ml(rows=256, act=0) == -2 and ml(rows=256, n=64) == -3 and ml(rows=16, K=40) == -2
    lp = lambda pages=4, dim=64, elems=1 << 30, sc=16: b.mlora_latent_prefill(16, 0, 64, 16, 64, 16, 16, 16, pages, 16, 1, 16, 16, None, 0.1, 8, 2, 64, dim, 16,
                                                                              64, 8, sc, elems, None)
    assert lp(pages=5) == -2 and lp(dim=256) == -2 and lp(elems=8) == -3 and lp(sc=None) == -1


# ------------------------------------------------------------------ the oracle by what the equations fix
def test_oracle_sink_and_causality():
    w = R.sink_softmax(np.array([1.0, 2.0]), 3.0)
    assert np.allclose(w, np.exp([1.0, 2.0]) / np.exp([1.0, 2.0, 3.0]).sum())
    assert np.allclose(R.sink_softmax(np.array([1.0, 2.0]), -1e9).sum(), 1.0)
    cfg = C.CONFIGS["odd"]
    P = C.weights(cfg, 3)
    toks = np.random.default_rng(0).integers(0, cfg["vocab"], 12)
    full = R.forward(toks, cfg, P)
    assert np.allclose(full[:7], R.forward(toks[:7], cfg, P))
    other = toks.copy()
    other[0] = (other[0] + 1) % cfg["vocab"]
    assert np.abs(R.forward(other, cfg, P)[-1] - full[-1]).max() > 1e-4


def test_oracle_scores_from_the_latent_side():
    """k . q through the keys equals c . (W_uk^T q)."""
    rng = np.random.default_rng(2)
    uk, q, c = rng.normal(size=(5, 9)), rng.normal(size=5), rng.normal(size=9)
    assert np.isclose((uk @ c) @ q, c @ (uk.T @ q))


def test_oracle_router_and_clipping():
    P = {"x.mlp.router": np.eye(3), "x.mlp.router.b": np.array([0.0, 0.5, -9.0])}
    pick, w = R.route(np.array([[1.0, 1.0, 2.0]]), {"router": {"top": 2}}, P, "x")
    assert pick.tolist() == [[1, 0]] and np.allclose(w, np.exp([[1.5, 1.0]]) / np.exp([1.5, 1.0]).sum())
    Q = {"x.mlp.gate": np.array([[5.0]]), "x.mlp.up": np.array([[-5.0]]), "x.mlp.down": np.array([[1.0]])}
    y = R.dense_ff(np.array([[1.0]]), {"limit": 2.0}, Q, "x")
    assert np.isclose(y[0, 0], 2.0 / (1 + np.exp(-1.702 * 2.0)) * (-2.0 + 1.0))
    y = R.dense_ff(np.array([[-1.0]]), {"limit": 2.0}, Q, "x")             # the gate has no lower bound
    assert np.isclose(y[0, 0], -5.0 / (1 + np.exp(1.702 * 5.0)) * (2.0 + 1.0))
