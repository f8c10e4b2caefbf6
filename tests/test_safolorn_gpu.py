"""The Safolorn model through the framework's cache, scheduler and front end against the numpy oracle."""
import io
import json

import numpy as np
import pytest
import torch

import safolorn_cases as C
from conftest import load_pkg
from oracle import safolorn_ref as R

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, B16 = torch.float32, torch.bfloat16


def build(cfg, dt, seed=0, sharp=1.0):
    P = C.weights(cfg, seed, sharp)
    return P, load_pkg("safolorn").SafolornForCausalLM.from_weights(cfg, C.tensors(P), dt, DEV)


def toks(cfg, n, seed=0):
    return np.random.default_rng(100 + seed).integers(0, cfg["vocab"], n)


def run(model, kv, entries, layer_outputs=None):
    """entries: [(sid, tokens)] of one pass -> logits of every token, per entry."""
    for sid, _ in entries:
        if sid not in kv.slot:
            kv.add_sequence(sid)
    lens = [len(t) for _, t in entries]
    kv.begin_forward([s for s, _ in entries], lens)
    h = model.embed(torch.from_numpy(np.concatenate([t for _, t in entries]).astype(np.int32)))
    out = model.forward(h, kv, None, **({} if layer_outputs is None else {"layer_outputs": layer_outputs}))
    kv.end_forward()
    torch.cuda.synchronize()
    return np.split(out.double().cpu().numpy(), np.cumsum(lens)[:-1])


def portions(n, sizes):
    out, at, i = [], 0, 0
    while at < n:
        out.append((at, min(n, at + sizes[i % len(sizes)])))
        at, i = out[-1][1], i + 1
    return out


def cache(model, n_tokens=1024, seqs=4, **kw):
    return model.create_paged_kv_cache(seqs, n_tokens, n_tokens, 16, **kw)


def rel(got, want):
    """rms difference per position over the rms of the logits (means removed)."""
    d, w = got - want, want - want.mean(-1, keepdims=True)
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((w * w).mean())


def agrees(got, want, dt):
    e = rel(got, want)
    if dt == F32:
        return e.max() < 2e-5
    # bfloat16 flips a close choice of experts here and there; most positions are close
    return np.quantile(e, 0.8) < 3e-2


@pytest.mark.parametrize("dt", [F32, B16])
@pytest.mark.parametrize("name", list(C.CONFIGS))
def test_prompt_layer_by_layer(name, dt):
    cfg = C.CONFIGS[name]
    P, m = build(cfg, dt, 1)
    t, lo, lw = toks(cfg, 75), [], []
    (got,) = run(m, cache(m), [("a", t)], lo)
    want = R.forward(t, cfg, P, lw)
    for l, (a, b) in enumerate(zip(lo, lw)):
        e = np.abs(a.double().cpu().numpy() - b).max(-1) / np.abs(b).max()
        assert (e.max() < 1e-5) if dt == F32 else (np.quantile(e, 0.8) < 2e-2), l
    assert agrees(got, want, dt)


@pytest.mark.parametrize("dt", [F32, B16])
@pytest.mark.parametrize("sizes", [[2], [1], [3, 2, 5], [16], [15, 17], [64, 1], [70]])
def test_portions_and_token_by_token(sizes, dt):
    """However a prompt is cut, also token by token, the logits are those of the whole (sharp attention: single keys decide)."""
    cfg = C.CONFIGS["odd"]
    P, m = build(cfg, dt, 2, sharp=4.0)
    t = toks(cfg, 101)
    kv = cache(m, free_pages=list(np.random.default_rng(0).permutation(40)))
    got = np.concatenate([run(m, kv, [("a", t[a:b])])[0] for a, b in portions(len(t), sizes)])
    want = R.forward(t, cfg, P)
    assert agrees(got, want, dt)


@pytest.mark.parametrize("name", list(C.CONFIGS))
@pytest.mark.parametrize("prompt_form", [True, False])
def test_both_forms_of_the_attention(name, prompt_form, monkeypatch):
    """The prompt form and the lifted form, each forced for all passes that are no decode steps, portions and batches included."""
    cfg = C.CONFIGS[name]
    P, m = build(cfg, B16, 9, sharp=2.0)
    att = load_pkg("latent_attention").LatentAttention
    calls = []
    monkeypatch.setattr(att, "prompt_form_pays", lambda self, seqs: calls.append(prompt_form and self.uk is not None) or calls[-1])
    a, b = toks(cfg, 150, 1), toks(cfg, 77, 2)
    kv = cache(m, free_pages=list(np.random.default_rng(0).permutation(40)))
    ga = [run(m, kv, [("a", a[:50])])[0]]
    x, y = run(m, kv, [("b", b[:70]), ("a", a[50:149])])
    ga.append(y)
    gb = [x] + [run(m, kv, [("b", b[i:j])])[0] for i, j in ((70, 72), (72, 77))]
    ga.append(run(m, kv, [("a", a[149:])])[0])
    assert any(calls) == prompt_form
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


def test_pages_and_slots_used_again():
    """Requests that come and go through a pool with room for few of them."""
    cfg = C.CONFIGS["wide"]
    P, m = build(cfg, F32, 4)
    kv = m.create_paged_kv_cache(2, 96, 96, 16, free_pages=[3, 0, 5, 1, 4, 2, 6, 7])
    live = []
    for i in range(6):
        t = toks(cfg, [40, 17, 64, 33, 16, 50][i], i)
        sid = f"s{i}"
        run(m, kv, [(sid, t[:-5])])
        got = np.concatenate([run(m, kv, [(sid, t[j:j + 1])])[0] for j in range(len(t) - 5, len(t))])
        assert rel(got, R.forward(t, cfg, P)[-5:]).max() < 2e-5, i
        live.append(sid)
        if len(live) == 2:
            kv.free_sequence(live.pop(i % 2))
    for s in live:
        kv.free_sequence(s)
    assert sorted(kv.free) == list(range(8)) and sorted(kv.free_slots) == [0, 1]


@pytest.mark.parametrize("dt", [F32, B16])
def test_far_keys_first_tokens_and_long_prompts(dt):
    """More than a thousand tokens, attention sharp enough for single keys to decide."""
    cfg = C.config([C.layer(C.mixer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=32, scale=0.5, r=C.rot(1e5, 8)), C.dense(32)),
                    C.layer(C.mixer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=32, scale=0.5, r=C.rot(1e5, 8), kv_from=0), None)],
                   vocab=64, width=32, side=8)
    P, m = build(cfg, dt, 5, sharp=3.0)
    t = toks(cfg, 1100)
    kv = cache(m, 1200)
    (got,) = run(m, kv, [("a", t[:1060])])
    tail = np.concatenate([run(m, kv, [("a", t[j:j + 1])])[0] for j in range(1060, 1100)])
    got = np.concatenate([got, tail])
    assert agrees(got, R.forward(t, cfg, P), dt)


def greedy_ok(tokens, prompt, cfg, P, tol):
    """Every generated token is the oracle's choice, or within `tol` of it at a near tie."""
    seq = np.concatenate([prompt, tokens])
    lg = R.forward(seq[:-1], cfg, P)[len(prompt) - 1:]
    return all(row.max() - row[k] <= tol for row, k in zip(lg, tokens))


@pytest.mark.parametrize("dt,tol", [(F32, 1e-4), (B16, 0.3)])
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
    # the same without graph and batched prefill, token for token in fp32
    if dt == F32:
        c = ab.LlamaAutoBatcherClass()
        c.set_model(m)
        c.set_exec_config(xg.LlamaExecConfig(max_prompt_len=64, max_gen_len=40, page_size=16, native_decode=False, batch_prefill=True))
        again = [c.generate(c.create_var(p.astype(np.int32)), max_gen_len=n) for p, n in zip(prompts, limits)]
        c.compile()
        c.execute()
        assert all(np.array_equal(a.var, o.var) for a, o in zip(again, outs))


def test_graph_replays_equal_eager_steps():
    """Every replay of a captured decode step, with eager work between, gives the eager step's tokens."""
    ds = load_pkg("decode_session")
    cfg = C.CONFIGS["odd"]
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
                other = cache(m)
                run(m, other, [("x", toks(cfg, 33, i))])
        out.append(np.stack(got))
    assert np.array_equal(out[0], out[1])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_folder_registry_and_trace(tmp_path, monkeypatch, capsys, dtype):
    from safetensors.torch import save_file
    cfg = C.CONFIGS["plain"]
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
    assert sorted(p.name for p in out.iterdir()) == ["0.f32", "2.f32", "3.f32"]
    ra, rb = R.forward(t, cfg, P), R.forward(u, cfg, P)
    dt = F32 if dtype == "float32" else B16
    for n, want in ((0, ra[[0, 29]]), (2, np.stack([ra[39], rb[8]])), (3, rb[[8]])):
        got = np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert got.shape == want.shape and rel(got, want).max() < (2e-5 if dt == F32 else 0.1)


def test_llama_from_a_folder(tmp_path):
    """The registry serves the Llama model from a checkpoint folder, with the weights of the synthetic loader."""
    from safetensors.torch import save_file
    S, reg, llama = load_pkg("synth"), load_pkg("registry"), load_pkg("llama")
    shape = S.LlamaShape(hidden_size=128, intermediate_size=256, num_attention_heads=2, num_key_value_heads=2, num_hidden_layers=2, head_dim=64,
                         vocab_size=256)
    a = llama.LlamaForCausalLM.from_synthetic(1, shape, [], DEV)
    w = {}
    for l in range(2):
        for k, v in S.layer_weights(1, shape, l, torch.float16, "cpu").items():
            p = k.split(".", 2)[2]
            block = {"q": "self_attn.", "k": "self_attn.", "v": "self_attn.", "o": "self_attn.", "g": "mlp.", "u": "mlp.", "d": "mlp."}.get(p[0], "") \
                if p.endswith("_proj") else ""
            w[f"model.layers.{l}.{block}{p}.weight"] = v.contiguous()
    w["model.embed_tokens.weight"] = S.normal(1, "embed_tokens", (256, 128), 0.02, torch.float16, "cpu")
    w["lm_head.weight"] = S.normal(1, "lm_head", (256, 128), 0.02, torch.float16, "cpu")
    w["model.norm.weight"] = torch.ones(128, dtype=torch.float16)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["LlamaForCausalLM"], "hidden_size": 128, "intermediate_size": 256,
                                                      "num_attention_heads": 2, "num_hidden_layers": 2, "head_dim": 64, "vocab_size": 256,
                                                      "rms_norm_eps": shape.rms_norm_eps, "rope_theta": shape.rope_theta}))
    b = reg.load_model(str(tmp_path))
    outs = []
    for m in (a, b):
        kv = m.create_paged_kv_cache(1, 64, 64, 16)
        outs.append(run(m, kv, [(0, toks({"vocab": 256}, 20))])[0])
    assert np.array_equal(*outs)
