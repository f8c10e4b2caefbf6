"""The Dinasun model through the framework's cache, scheduler and front end against the numpy oracle."""
import io
import json

import numpy as np
import pytest
import torch

import dinasun_cases as C
from conftest import load_pkg
from oracle import dinasun_ref as R
from test_safolorn_gpu import cache, portions, rel, run, toks

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, B16 = torch.float32, torch.bfloat16


def build(cfg, dt, seed=0, sharp=1.0):
    P = C.weights(cfg, seed, sharp)
    return P, load_pkg("dinasun").DinasunForCausalLM.from_weights(cfg, C.tensors(P), dt, DEV)


def agrees(got, want, dt):
    """Nothing here flips a choice on rounding: experts go by token id."""
    return rel(got, want).max() < (2e-5 if dt == F32 else 6e-2)


@pytest.mark.parametrize("dt", [F32, B16])
@pytest.mark.parametrize("name", list(C.CONFIGS))
def test_prompt_layer_by_layer(name, dt):
    cfg = C.CONFIGS[name]
    P, m = build(cfg, dt, 1)
    t, lo, lw = toks(cfg, 75), [], []
    (got,) = run(m, cache(m), [("a", t)], lo)
    want = R.forward(t, cfg, P, lw)
    assert len(lo) == len(lw)
    for l, (a, b) in enumerate(zip(lo, lw)):
        assert np.abs(a.double().cpu().numpy() - b).max() / np.abs(b).max() < (1e-5 if dt == F32 else 4e-2), l
    assert agrees(got, want, dt)


@pytest.mark.parametrize("dt", [F32, B16])
@pytest.mark.parametrize("sizes", [[2], [1], [3, 2, 5], [16], [15, 17], [64, 1], [70], [33, 2]])
def test_portions_and_token_by_token(sizes, dt):
    """However a prompt is cut, also token by token, the logits are those of the whole (sharp attention: single keys decide)."""
    cfg = C.CONFIGS["odd"]
    P, m = build(cfg, dt, 2, sharp=3.0)
    t = toks(cfg, 101)
    kv = cache(m, free_pages=list(np.random.default_rng(0).permutation(68)))
    got = np.concatenate([run(m, kv, [("a", t[a:b])])[0] for a, b in portions(len(t), sizes)])
    assert agrees(got, R.forward(t, cfg, P), dt)


@pytest.mark.parametrize("name", ["odd", "wide"])
@pytest.mark.parametrize("prompt_form", [True, False])
def test_both_forms_of_the_attention(name, prompt_form, monkeypatch):
    """Keys and values laid out once per pass, and the pages read directly, each forced for all passes that are no decode steps."""
    cfg = C.CONFIGS[name]
    P, m = build(cfg, B16, 9, sharp=2.0)
    monkeypatch.setattr(load_pkg("tied_attention").TiedAttention, "prompt_form_pays", lambda self, seqs: prompt_form and self.prompt_form)
    a, b = toks(cfg, 150, 1), toks(cfg, 77, 2)
    kv = cache(m, free_pages=list(np.random.default_rng(0).permutation(68)))
    ga = [run(m, kv, [("a", a[:50])])[0]]
    x, y = run(m, kv, [("b", b[:70]), ("a", a[50:149])])
    ga.append(y)
    gb = [x] + [run(m, kv, [("b", b[i:j])])[0] for i, j in ((70, 72), (72, 77))]
    ga.append(run(m, kv, [("a", a[149:])])[0])
    assert agrees(np.concatenate(ga), R.forward(a, cfg, P), B16) and agrees(np.concatenate(gb), R.forward(b, cfg, P), B16)


@pytest.mark.parametrize("dt", [F32, B16])
def test_batches_of_unequal_requests(dt):
    cfg = C.CONFIGS["odd"]
    P, m = build(cfg, dt, 3)
    seqs = {"a": toks(cfg, 90, 1), "b": toks(cfg, 3, 2), "c": toks(cfg, 41, 3)}
    steps = [[("a", 0, 60), ("b", 0, 2)], [("c", 0, 17), ("a", 60, 61)], [("a", 61, 62), ("b", 2, 3), ("c", 17, 18)], [("c", 18, 41), ("a", 62, 90)]]
    kv, got = cache(m), {s: [] for s in seqs}
    for st in steps:
        for (s, _, _), g in zip(st, run(m, kv, [(s, seqs[s][a:b]) for s, a, b in st])):
            got[s].append(g)
    for s in seqs:
        assert agrees(np.concatenate(got[s]), R.forward(seqs[s], cfg, P), dt), s


@pytest.mark.parametrize("name", ["plain", "wide"])
def test_pages_and_slots_used_again(name):
    """Requests that come and go through a pool with room for few of them: neither pages nor states leave anything behind."""
    cfg = C.CONFIGS[name]
    P, m = build(cfg, F32, 4)
    kv = m.create_paged_kv_cache(2, 96, 96, 16, free_pages=[3, 0, 5, 1, 4, 2, 6, 7])
    live = []
    for i in range(6):
        t = toks(cfg, [40, 17, 64, 33, 1, 50][i], i)
        sid, n = f"s{i}", max(len(t) - 5, 1)
        got = [run(m, kv, [(sid, t[:n])])[0]] + [run(m, kv, [(sid, t[j:j + 1])])[0] for j in range(n, len(t))]
        assert rel(np.concatenate(got), R.forward(t, cfg, P)).max() < 2e-5, i
        live.append(sid)
        if len(live) == 2:
            kv.free_sequence(live.pop(i % 2))
    for s in live:
        kv.free_sequence(s)
    assert sorted(kv.free) == list(range(8)) and sorted(kv.free_slots) == [0, 1]


@pytest.mark.parametrize("dt", [F32, B16])
def test_far_keys_first_tokens_and_long_prompts(dt):
    """More than a thousand tokens in portions and decoded, attention sharp enough for single keys to decide, states carried all along."""
    cfg = C.config([C.att(4, 2, 16, 0.5, (0.2, 100)), C.wkv(2, 16, C.moe(16, 3, 2, 16))], vocab=64, width=32, loop=(0, 2, 2))
    P, m = build(cfg, dt, 5, sharp=2.0)
    t = toks(cfg, 1100)
    kv = cache(m, 1200)
    got = [run(m, kv, [("a", t[a:b])])[0] for a, b in ((0, 700), (700, 702), (702, 1060))]
    got += [run(m, kv, [("a", t[j:j + 1])])[0] for j in range(1060, 1100)]
    want = R.forward(t, cfg, P)
    assert agrees(np.concatenate(got), want, dt)
    (whole,) = run(m, kv, [("b", t[:100])])
    assert agrees(whole, want[:100], dt)


@pytest.mark.parametrize("dt", [F32, B16])
def test_long_decoding(dt):
    """A hundred decoded tokens behind a prompt of two, over page borders."""
    cfg = C.CONFIGS["plain"]
    P, m = build(cfg, dt, 12, sharp=3.0)
    t = toks(cfg, 102)
    kv = cache(m)
    got = [run(m, kv, [("a", t[:2])])[0]] + [run(m, kv, [("a", t[j:j + 1])])[0] for j in range(2, 102)]
    assert agrees(np.concatenate(got), R.forward(t, cfg, P), dt)


def test_many_tokens_take_the_large_tiles():
    """A pass of several long prompts: persistent GEMMs, grouped experts of 256-place tiles."""
    cfg = C.config([C.wkv(2, 64, C.moe(64, 3, 2, 64)), C.att(4, 2, 64, 0.2, (0.4, 100), C.moe(128, 2, 1, 96))], vocab=128, width=128, loop=(1, 2, 2))
    P, m = build(cfg, B16, 13)
    seqs = [toks(cfg, n, n) for n in (700, 333, 901, 17)]
    kv = cache(m, 2400)
    for t, g in zip(seqs, run(m, kv, list(enumerate(seqs)))):
        assert agrees(g, R.forward(t, cfg, P), B16)


def greedy_ok(tokens, prompt, cfg, P, tol):
    """Every generated token is the oracle's choice, or within `tol` of it at a near tie."""
    lg = R.forward(np.concatenate([prompt, tokens])[:-1], cfg, P)[len(prompt) - 1:]
    return all(row.max() - row[k] <= tol for row, k in zip(lg, tokens))


@pytest.mark.parametrize("dt,tol", [(F32, 1e-3), (B16, 0.6)])
def test_generation_through_the_front_end(dt, tol):
    """Requests of unequal prompts and limits through the auto-batching front end: prefill, batched graph-replayed decode that
    shrinks, more than a page of tokens."""
    xg, ab = load_pkg("llama_exec_graph"), load_pkg("auto_batcher")
    cfg = C.CONFIGS["odd"]
    P, m = build(cfg, dt, 6)
    b = ab.LlamaAutoBatcherClass()
    b.set_model(m)
    b.set_exec_config(xg.LlamaExecConfig(max_prompt_len=64, max_gen_len=40, page_size=16))
    prompts, limits = [toks(cfg, n, n) for n in (31, 5, 64)], [40, 17, 2]
    outs = [b.generate(b.create_var(p.astype(np.int32)), max_gen_len=n) for p, n in zip(prompts, limits)]
    b.compile()
    b.execute()
    for p, n, o in zip(prompts, limits, outs):
        assert len(o.var) == n and greedy_ok(np.asarray(o.var), p, cfg, P, tol)
    if dt == F32:                     # the same without graph and with batched prefill, token for token
        c = ab.LlamaAutoBatcherClass()
        c.set_model(m)
        c.set_exec_config(xg.LlamaExecConfig(max_prompt_len=64, max_gen_len=40, page_size=16, native_decode=False, batch_prefill=True))
        again = [c.generate(c.create_var(p.astype(np.int32)), max_gen_len=n) for p, n in zip(prompts, limits)]
        c.compile()
        c.execute()
        assert all(np.array_equal(a.var, o.var) for a, o in zip(again, outs))


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_graph_replays_equal_eager_steps(name):
    """Every replay of a captured decode step, with eager work between, gives the eager step's tokens."""
    ds = load_pkg("decode_session")
    cfg = C.CONFIGS[name]
    _, m = build(cfg, B16, 7)
    out = []
    for graph in (False, True):
        kv = cache(m)
        for s in range(3):
            run(m, kv, [(s, toks(cfg, 20 + 7 * s, s))])
        sess = ds.DecodeSession(m, kv, [0, 1, 2], {}, [1, 2, 3], use_graph=graph)
        got = []
        for i in range(40):
            got.append(sess.step().cpu().numpy().copy())
            if i % 10 == 5:
                run(m, cache(m), [("x", toks(cfg, 33, i))])
        out.append(np.stack(got))
    assert np.array_equal(out[0], out[1])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_folder_registry_and_trace(tmp_path, monkeypatch, capsys, dtype):
    from safetensors.torch import save_file
    cfg = C.CONFIGS["odd"]
    P = C.weights(cfg, 8)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: C.tensors(P)(k).contiguous() for k in P}, str(tmp_path / "model.safetensors"))
    t, u = toks(cfg, 40, 1).tolist(), toks(cfg, 9, 2).tolist()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:30], "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": u[:8], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": t[30:], "want": [9]}, {"id": "b", "tokens": u[8:], "want": [0]}], "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": u, "want": [8]}], "end": ["a"]}]
    out = tmp_path / "out"
    out.mkdir()
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    assert load_pkg("trace").main(["--model", str(tmp_path), "--dtype", dtype, "--out", str(out), "--max-tokens", "64"]) == 0
    assert [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    ra, rb = R.forward(t, cfg, P), R.forward(u, cfg, P)
    for n, want in ((0, ra[[0, 29]]), (2, np.stack([ra[39], rb[8]])), (3, rb[[8]])):
        got = np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert got.shape == want.shape and agrees(got, want, F32 if dtype == "float32" else B16)
