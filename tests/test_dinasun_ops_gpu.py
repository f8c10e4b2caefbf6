"""Every kernel of the time-mixing / tied-attention decoders alone, in both element types, against float64 numpy."""
import numpy as np
import pytest
import torch

from conftest import load_pkg
from oracle import dinasun_ref as R
from test_safolorn_ops_gpu import DEV, DTYPES, D, err, f64, rnd, rows_of, tol   # noqa: F401

pytestmark = pytest.mark.gpu
i32 = lambda a: torch.as_tensor(np.asarray(a, np.int32)).to(DEV)


# ------------------------------------------------------------------ residual stream
def stream_case(D, rng, dt, T, W):
    Hp = D.pad64(W)
    z = lambda *s, std=1.0: D.padded(rnd(rng, *s, W, std=std), *s, Hp).contiguous()
    norm = lambda: D.ElementwiseNorm(rnd(rng, W), rnd(rng, W, std=0.3), float(rng.uniform(0.3, 1.2)), Hp, dt, DEV)
    ref = lambda n, x: np.tanh(n.alpha * x) * f64(n.w)[:W] + f64(n.b)[:W]
    return Hp, z, norm, ref


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,W", [(1, 30), (17, 104), (70, 2100), (5, 5000), (300, 64), (33, 4096)])
def test_stream_steps(D, ops, dt, T, W):
    """Branch with partials and entry rows, norms on both sides; a raw step; a replaced stream."""
    rng = np.random.default_rng(T + W)
    Hp, z, norm, ref = stream_case(D, rng, dt, T, W)
    x, y, parts, rows = z(T, std=2.0), z(T), z(2, T), D.padded(rnd(rng, 3 * T, W, dt=dt), 3 * T, Hp).contiguous()
    post, pre = norm(), norm()
    s = D.ResidualStream(x.clone(), dt, 0.6)
    s.branch(y, ops.KSplitParts(parts, 3, Hp), post, rows, 0.25)
    frag = ops.FragActivation(T, Hp, DEV, dtype=dt) if dt == torch.bfloat16 else None
    row = torch.empty((T, Hp), dtype=dt, device=DEV)
    s.step(pre, out=frag, out_row=row)
    torch.cuda.synchronize()
    cut = lambda a: f64(a)[..., :W]
    want = cut(x) + 0.6 * ref(post, cut(y) + cut(parts).sum(0) + 0.25 * cut(rows).reshape(T, 3, W).sum(1))
    assert err(s.x[:, :W], want) < 3e-6 and float(s.x[:, W:].abs().sum()) == 0
    assert err(row[:, :W], ref(pre, want)) < tol(dt, f32=4e-6, b16=5e-3) and float(row[:, W:].abs().sum()) == 0
    assert frag is None or torch.equal(frag.unpack(), row)
    s.branch(None, None, post, rows, 1 / 3)                          # entry rows alone, the sum kept as it is into half of a wider row
    wide = torch.zeros((T, 2 * Hp), dtype=dt, device=DEV)
    s.step(out_row=wide[:, Hp:])
    torch.cuda.synchronize()
    want = want + 0.6 * ref(post, cut(rows).reshape(T, 3, W).mean(1))
    assert err(s.x[:, :W], want) < 5e-6 and torch.equal(wide[:, Hp:], s.x.to(dt)) and float(wide[:, :Hp].abs().sum()) == 0
    s.replace(y, ops.KSplitParts(parts, 3, Hp))
    s.step()
    torch.cuda.synchronize()
    assert err(s.x[:, :W], cut(y) + cut(parts).sum(0)) < 1e-6


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("W,segs", [(104, [(5, 0), (1, 3), (30, 0), (2, 9), (19, 4)]), (2100, [(1, 0)]), (64, [(700, 0), (1200, 6), (300, 1)]),
                                    (96, [(1, 7), (1, 0), (1, 1), (1, 30)]), (130, [(16, 1), (16, 0), (48, 2)])])
@pytest.mark.parametrize("pending", [True, False])
def test_stream_step_with_mixes(D, ops, dt, W, segs, pending):
    """segs: (tokens, position of the first) per sequence of the pass: the previous token comes from the pass, from the state or
    is none; the state takes the last token's row.  Slots hold garbage that a first token must not see."""
    rng = np.random.default_rng(W)
    T, n = sum(s for s, _ in segs), len(segs)
    Hp, z, norm, ref = stream_case(D, rng, dt, T, W)
    slots = rng.permutation(n + 2)[:n]
    x, y, rows = z(T, std=2.0), z(T), D.padded(rnd(rng, 2 * T, W, dt=dt), 2 * T, Hp).contiguous()
    shift0 = z(n + 2, std=5.0)
    shift = shift0.clone()
    post, pre = norm(), norm()
    mu = D.padded(torch.from_numpy(rng.uniform(0, 1, (5, W))).to(torch.bfloat16).to(dt).to(DEV), 5, Hp).contiguous()
    s = D.ResidualStream(x.clone(), dt, 0.6)
    if pending:
        s.branch(y, None, post, rows, 0.5)
    room = {"out": ops.FragActivation(T, Hp, DEV, torch.empty(5 * ops.FragActivation(T, Hp, DEV, dtype=dt).data.numel(), dtype=dt, device=DEV))} \
        if dt == torch.bfloat16 else {"out_row": torch.empty((5, T, Hp), dtype=dt, device=DEV)}
    seq = np.repeat(slots, [c for c, _ in segs])
    pos = np.concatenate([p + np.arange(c) for c, p in segs])
    ends = np.cumsum([c for c, _ in segs])
    last = None if all(c == 1 for c, _ in segs) else i32(np.repeat(ends - 1, [c for c, _ in segs]))
    s.step(pre, mu=mu, shift=shift, tokens=(i32(seq), i32(pos), last), **room)
    torch.cuda.synchronize()
    cut = lambda a: f64(a)[..., :W]
    xw = cut(x) + (0.6 * ref(post, cut(y) + 0.5 * cut(rows).reshape(T, 2, W).sum(1)) if pending else 0)
    h = ref(pre, xw)
    prev = np.concatenate([np.zeros((1, W)), h[:-1]])
    for (c, p), e, sl in zip(segs, ends, slots):
        prev[e - c] = cut(shift0)[sl] if p > 0 else 0
    assert err(s.x[:, :W], xw) < 3e-6
    got = room["out_row"] if dt == torch.float32 else \
        torch.stack([ops.FragActivation(T, Hp, DEV, d).unpack() for d in room["out"].data.view(5, -1)])
    for i in range(5):
        assert err(got[i][:, :W], h + (prev - h) * cut(mu)[i]) < tol(dt, f32=4e-6, b16=5e-3), i
        assert float(got[i][:, W:].abs().sum()) == 0
    want = cut(shift0).copy()
    want[slots] = h[ends - 1]
    assert np.abs(cut(shift) - want).max() < 2e-5


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,H", [(1, 64), (20, 96), (300, 1088)])
def test_embed_scaled(D, ops, dt, T, H):
    rng = np.random.default_rng(T)
    table, ids = rnd(rng, 50, H, dt=dt), rng.integers(0, 50, T)
    ids[-1] = 55
    if dt == torch.bfloat16:
        entry = ops.FragActivation(T, 2 * H, DEV, dtype=dt)
        entry.data.zero_()
        x = D.embed_scaled(table, i32(ids), 2.5, entry.columns(H, H))
        got = entry.unpack()
    else:
        got = torch.zeros((T, 2 * H), device=DEV)
        x = D.embed_scaled(table, i32(ids), 2.5, got[:, H:])
    want = 2.5 * f64(table)[np.minimum(ids, 49)]
    want[-1] = 0
    assert np.array_equal(f64(x), want.astype(np.float32)) and torch.equal(got[:, H:], x.to(dt)) and float(got[:, :H].abs().sum()) == 0


# ------------------------------------------------------------------ time mixing
def mix_case(D, rng, dt, T, H, Dm, Rk):
    ld = D.pad64(H * Dm)
    t = {s: D.padded(rnd(rng, T, H * Dm, dt=dt), T, ld).contiguous() for s in "rkvg"}
    z = D.padded(rnd(rng, T, Rk), T, D.pad32(Rk)).contiguous()[None]
    w2 = rnd(rng, H * Dm, Rk, std=Rk ** -0.5, dt=dt)
    w0 = rnd(rng, H * Dm, std=1.5) - 2.0
    u, norm = rnd(rng, H * Dm), rnd(rng, H * Dm, dt=dt)
    w = np.exp(-np.exp(np.tanh(f64(z)[0, :, :Rk]) @ f64(w2).T + f64(w0)))
    cut = lambda a: f64(a)[:, : H * Dm].reshape(T, H, Dm)
    return t, z, D.padded(w2, H * Dm, D.pad32(Rk)).contiguous(), w0, u, norm, (cut(t["r"]), cut(t["k"]), cut(t["v"]), w.reshape(T, H, Dm)), f64(u).reshape(H, Dm)


def mix_prompt(D, ops, plan, t, z, Rk, *rest):
    """The prompt form on given projections: the low-rank product is with the identity."""
    z = z[0]
    n = z.shape[1]
    eye = torch.zeros((n, n), dtype=torch.bfloat16, device=DEV)
    eye[:Rk, :Rk] = torch.eye(Rk)
    return D.time_mix_prompt(plan, t["r"], t["k"], t["v"], t["g"], ops.FragActivation.pack(z.to(torch.bfloat16)), D.weight(eye), *rest)


def mix_want(ref, u, gate, norm, H, Dm, eps, S):
    o, S = R.wkv_scan(*ref, u, S)
    return R.rms(o, eps).reshape(-1, H * Dm) * norm * R.silu(gate), S


MIX_SEGS = [[(1, 0)], [(40, 0), (1, 5), (2, 0), (17, 9), (3, 1)], [(1, 4), (1, 0), (1, 9)], [(200, 0), (333, 7), (64, 16), (65, 0)]]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,Dm,Rk", [(3, 24, 5), (1, 64, 70), (2, 40, 16), (2, 128, 33), (1, 136, 20), (4, 64, 64), (2, 16, 8)])
@pytest.mark.parametrize("case", range(len(MIX_SEGS)))
def test_time_mix(D, ops, dt, H, Dm, Rk, case):
    """Segments of all lengths in one pass, from a state and from the start (where the slot's old state must not show)."""
    segs = MIX_SEGS[case]
    rng = np.random.default_rng(H * Dm + case)
    T, n = sum(c for c, _ in segs), len(segs)
    t, z, w2, w0, u, norm, ref, uu = mix_case(D, rng, dt, T, H, Dm, Rk)
    slots = rng.permutation(n + 1)[:n]
    state0 = rnd(rng, n + 1, H, Dm, Dm, std=3.0)
    state = state0.clone()
    out = D.activation(T, D.pad64(H * Dm), dt, DEV)
    starts = np.cumsum([0] + [c for c, _ in segs])[:-1]
    decode = all(c == 1 for c, _ in segs)
    seg = None if decode else i32([(s, a, c, p) for s, a, (c, p) in zip(slots, starts, segs)])
    seq, pos = np.repeat(slots, [c for c, _ in segs]), np.concatenate([p + np.arange(c) for c, p in segs])
    D.time_mix(t["r"], t["k"], t["v"], t["g"], z, Rk, w2, w0, u, norm, 1e-4, state, seg, i32(seq), i32(pos), out)
    torch.cuda.synchronize()
    got = rows_of(out)
    assert float(got[:, H * Dm:].abs().sum()) == 0
    for s, a, (c, p) in zip(slots, starts, segs):
        part = [x[a:a + c] for x in ref]
        want, S = mix_want(part, uu, f64(t["g"])[a:a + c, : H * Dm], f64(norm), H, Dm, 1e-4, f64(state0)[s] if p else None)
        assert err(got[a:a + c, : H * Dm], want) < tol(dt, f32=2e-5, b16=6e-3), (c, p)
        assert err(state[s], S) < 2e-5, (c, p)
    idle = [s for s in range(n + 1) if s not in slots]
    assert torch.equal(state[idle], state0[idle])


@pytest.mark.parametrize("H,Dm,Rk", [(3, 24, 5), (1, 64, 70), (2, 40, 16), (2, 128, 33), (1, 30, 8), (4, 64, 64), (2, 16, 130), (1, 100, 20)])
@pytest.mark.parametrize("case", range(len(MIX_SEGS)))
@pytest.mark.parametrize("tokens", [None, 16, 48])
def test_time_mix_prompt(D, ops, H, Dm, Rk, case, tokens):
    """The chunked form: the same segments, in ranges side by side (cut where the plan cuts them, and shorter)."""
    segs, dt = MIX_SEGS[case], torch.bfloat16
    rng = np.random.default_rng(H * Dm + case)
    T, n = sum(c for c, _ in segs), len(segs)
    t, z, w2, w0, u, norm, ref, uu = mix_case(D, rng, dt, T, H, Dm, Rk)
    slots = [int(s) for s in rng.permutation(n + 1)[:n]]
    state0 = rnd(rng, n + 1, H, Dm, Dm, std=3.0)
    state, out = state0.clone(), D.activation(T, D.pad64(H * Dm), dt, DEV)
    starts = np.cumsum([0] + [c for c, _ in segs])[:-1].tolist()
    plan = D.TimeMixPlan([(s, a, c, p) for s, a, (c, p) in zip(slots, starts, segs)], H, DEV, tokens)
    mix_prompt(D, ops, plan, t, z, Rk, w2, w0, u, norm, 1e-4, state, out)
    torch.cuda.synchronize()
    got = rows_of(out)
    assert float(got[:, H * Dm:].abs().sum()) == 0
    for s, a, (c, p) in zip(slots, starts, segs):
        part = [x[a:a + c] for x in ref]
        want, S = mix_want(part, uu, f64(t["g"])[a:a + c, : H * Dm], f64(norm), H, Dm, 1e-4, f64(state0)[s] if p else None)
        assert err(got[a:a + c, : H * Dm], want) < 6e-3, (c, p)
        assert err(state[s], S) < 4e-6, (c, p)
    idle = [s for s in range(n + 1) if s not in slots]
    assert torch.equal(state[idle], state0[idle])


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sizes", [[2], [1], [70, 3], [64], [65, 31, 128]])
def test_time_mix_in_portions(D, ops, dt, sizes):
    """However a sequence is cut, outputs and final state are those of the whole."""
    H, Dm, Rk, T = 2, 64, 12, 300
    rng = np.random.default_rng(7)
    t, z, w2, w0, u, norm, ref, uu = mix_case(D, rng, dt, T, H, Dm, Rk)
    want, S = mix_want(ref, uu, f64(t["g"])[:, : H * Dm], f64(norm), H, Dm, 1e-4, None)
    state, at, i, outs = rnd(rng, 2, H, Dm, Dm), 0, 0, []
    while at < T:
        c = min(sizes[i % len(sizes)], T - at)
        sl = lambda a: a[at:at + c].contiguous()
        out = D.activation(c, D.pad64(H * Dm), dt, DEV)
        zz = torch.stack([sl(z[0]) * 0.25, sl(z[0]) * 0.75])                      # partial sums
        D.time_mix(sl(t["r"]), sl(t["k"]), sl(t["v"]), sl(t["g"]), zz, Rk, w2, w0, u, norm, 1e-4, state, None if c == 1 else i32([[1, 0, c, at]]),
                   i32([1] * c), i32(at + np.arange(c)), out)
        outs.append(rows_of(out))
        at, i = at + c, i + 1
    torch.cuda.synchronize()
    assert err(torch.cat(outs)[:, : H * Dm], want) < tol(dt, f32=2e-5, b16=6e-3) and err(state[1], S) < 2e-5


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("w0", [-30.0, -3.0, 1.5, 4.0])
def test_time_mix_decays_of_any_strength(D, ops, dt, w0):
    """From none (everything is kept) to total within a token: no overflow, no loss of what is kept."""
    H, Dm, Rk, T = 1, 64, 4, 400
    rng = np.random.default_rng(3)
    t, z, w2, _, u, norm, ref, uu = mix_case(D, rng, dt, T, H, Dm, Rk)
    w0 = torch.full((H * Dm,), w0, device=DEV) + rnd(rng, H * Dm, std=0.5)
    w = np.exp(-np.exp(np.tanh(f64(z)[0, :, :Rk]) @ f64(w2)[:, :Rk].T + f64(w0))).reshape(T, H, Dm)
    want, S = mix_want((*ref[:3], w), uu, f64(t["g"])[:, : H * Dm], f64(norm), H, Dm, 1e-4, None)
    state, out = rnd(rng, 1, H, Dm, Dm), D.activation(T, H * Dm, dt, DEV)
    D.time_mix(t["r"], t["k"], t["v"], t["g"], z, Rk, w2, w0, u, norm, 1e-4, state, i32([[0, 0, T, 0]]), i32([0] * T), i32(np.arange(T)), out)
    torch.cuda.synchronize()
    assert err(rows_of(out), want) < tol(dt, f32=2e-5, b16=6e-3) and err(state[0], S) < 2e-5
    if dt == torch.bfloat16:
        state, out = rnd(rng, 1, H, Dm, Dm), D.activation(T, H * Dm, dt, DEV)
        mix_prompt(D, ops, D.TimeMixPlan([(0, 0, T, 0)], H, DEV), t, z, Rk, w2, w0, u, norm, 1e-4, state, out)
        torch.cuda.synchronize()
        assert err(rows_of(out), want) < 6e-3 and err(state[0], S) < 6e-6


@pytest.mark.parametrize("dt,prompt", [(torch.float32, False), (torch.bfloat16, False), (torch.bfloat16, True)])
def test_time_mix_far_tokens(D, ops, dt, prompt):
    """One token's key stands out in a channel of its own that hardly decays: its value comes back wherever a later token asks for
    that channel, over chunk edges and portions, and not to the tokens before it."""
    H, Dm, Rk, T = 1, 64, 4, 300
    rng = np.random.default_rng(11)
    t, z, w2, w0, u, norm, ref, uu = mix_case(D, rng, dt, T, H, Dm, Rk)
    spots = [0, 1, 15, 16, 31, 32, 63, 64, 127, 128, 200]
    w0 = torch.full((H * Dm,), -3.0, device=DEV)
    w0[: len(spots)] = -12.0
    t["k"][:, : len(spots)] = 0
    t["r"][:, : len(spots)] = 0
    for c, j in enumerate(spots):
        t["k"][j, c] = 8.0
    asks = {int(q): int(rng.integers(len(spots))) for q in range(2, T, 3)}
    for q, c in asks.items():
        t["r"][q] = 0
        t["r"][q, c] = 8.0
    z.zero_()
    w = np.exp(-np.exp(f64(w0)))[None].repeat(T, 0).reshape(T, H, Dm)
    cut = lambda s: f64(t[s])[:, : H * Dm].reshape(T, H, Dm)
    want, S = mix_want((cut("r"), cut("k"), cut("v"), w), uu, f64(t["g"])[:, :Dm], f64(norm), H, Dm, 1e-4, None)
    state, outs = torch.zeros((1, H, Dm, Dm), device=DEV), []
    for a, b in ((0, 130), (130, 132), (132, 300)):
        out = D.activation(b - a, Dm, dt, DEV)
        part, zs = {s: x[a:b].contiguous() for s, x in t.items()}, z[:, a:b].contiguous()
        if prompt:
            mix_prompt(D, ops, D.TimeMixPlan([(0, 0, b - a, a)], H, DEV, 32), part, zs, Rk, w2, w0, u, norm, 1e-4, state, out)
        else:
            D.time_mix(*(part[s] for s in "rkvg"), zs, Rk, w2, w0, u, norm, 1e-4, state, i32([[0, 0, b - a, a]]), i32([0] * (b - a)),
                       i32(np.arange(a, b)), out)
        outs.append(rows_of(out))
    torch.cuda.synchronize()
    got, gate = f64(torch.cat(outs)), R.silu(f64(t["g"])[:, :Dm]) * f64(norm)
    assert np.abs(got - want).max() / np.abs(want).max() < tol(dt, f32=2e-5, b16=6e-3)
    for q, c in asks.items():
        if q > spots[c]:                                  # nothing but that value
            v = cut("v")[spots[c], 0]
            assert np.abs(got[q] - R.rms(v, 0) * gate[q]).max() < (1e-3 if dt == torch.float32 else 3e-2) * np.abs(gate[q]).max() + 1e-3, (q, c)
        elif q < spots[c]:
            assert np.abs(want[q]).max() < 1e-6 and np.abs(got[q]).max() < 1e-5


# ------------------------------------------------------------------ tied attention
def tied_case(D, dt, ctxs, H, G, dim, seed=0, n_extra=3):
    """Pages filled through tied_prep: (values float64 per sequence, pages, scales, block table, rng); unused pages are poisoned."""
    rng = np.random.default_rng(seed)
    need = [-(-c // 16) for c in ctxs]
    n_pages = sum(need) + n_extra
    order, k = rng.permutation(n_pages), 0
    bt = np.full((len(ctxs) + 1, max(need) + 1), -1, np.int32)
    for i, c in enumerate(need):
        bt[i + 1, :c] = order[k:k + c]
        k += c
    RB = D.pad32(dim) // 32
    pages = torch.full((n_pages, G, RB, 4, 16, 8), 50.0, dtype=dt, device=DEV)
    scales = torch.full((n_pages, G, 16), 3.0, device=DEV)
    vals = [torch.from_numpy(rng.normal(size=(c, G, dim))).to(torch.bfloat16).double().numpy() for c in ctxs]
    return vals, pages, scales, i32(bt), rng


def put_values(D, vals, pages, scales, bt, H, G, dim, eps):
    """Stores the values at their positions (the queries of these launches are thrown away)."""
    for i, v in enumerate(vals):
        n = len(v)
        y = torch.zeros((n, D.pad32((H + G) * dim)), device=DEV)
        y[:, H * dim:(H + G) * dim] = torch.from_numpy(v.reshape(n, G * dim)).float()
        q = torch.empty((n, H, D.pad32(dim)), dtype=pages.dtype, device=DEV)
        D.tied_prep(q, pages, scales, y, torch.zeros((H + G) * dim, device=DEV), torch.ones(dim, device=DEV), eps, None, bt, i32([i + 1] * n),
                    i32(np.arange(n)), H, G, dim)


def tied_want(vals, q, seq, pos, slopes, scale, eps):
    """q: queries with both norms' weights applied."""
    T, H, dim = q.shape
    out = np.zeros((T, H, dim))
    for t in range(T):
        v = vals[seq[t]][: pos[t] + 1]
        gs = H // v.shape[1]
        for h in range(H):
            s = R.rms(v[:, h // gs], eps) @ q[t, h] * scale - slopes[h] * (pos[t] - np.arange(pos[t] + 1))
            out[t, h] = R.softmax(s) @ v[:, h // gs]
    return out


def put_q(D, q, dt):
    return D.padded(torch.from_numpy(q).to(dt).to(DEV), q.shape[0], q.shape[1], D.pad32(q.shape[2])).contiguous()


GEOMETRY = [(1, 1, 32), (6, 2, 40), (36, 2, 96), (4, 4, 64), (8, 2, 128), (3, 1, 200), (2, 1, 300)]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim", GEOMETRY)
def test_tied_attention_decode(D, ops, dt, H, G, dim):
    ctxs = [1, 2, 15, 16, 17, 33, 200, 517]
    vals, pages, scales, bt, rng = tied_case(D, dt, ctxs, H, G, dim, seed=H)
    put_values(D, vals, pages, scales, bt, H, G, dim, 1e-5)
    seq, pos = list(range(len(ctxs))), [c - 1 for c in ctxs]
    q = torch.from_numpy(rng.normal(size=(len(ctxs), H, dim))).to(torch.bfloat16).double().numpy()
    slopes, scale = R.slopes(H).astype(np.float32), 3.0 * dim ** -0.5
    want = tied_want(vals, q, seq, pos, slopes, scale, 1e-5)
    args = (put_q(D, q, dt), pages, scales, bt, i32([s + 1 for s in seq]), i32(pos), torch.from_numpy(slopes).to(DEV), scale, G, dim, max(ctxs))
    rd = H * D.pad32(dim)
    for splits in ([1, 2, 5, 32] if dt == torch.bfloat16 else [1]):
        outs = [torch.empty((len(ctxs), rd), dtype=dt, device=DEV)] + ([ops.FragActivation(len(ctxs), rd, DEV, dtype=dt)] if dt == torch.bfloat16 else [])
        for out in outs:
            got = rows_of(D.tied_attn(*args, out, splits=splits)).view(len(ctxs), H, -1)
            torch.cuda.synchronize()
            assert err(got[..., :dim], want) < tol(dt, b16=6e-3), splits
            assert float(got[..., dim:].abs().sum()) == 0


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("steep", [False, True])
def test_tied_attention_single_keys_far_and_at_page_borders(D, dt, steep):
    """One key stands out for one query; its value is what comes back - wherever it lies, and not one token later - until the
    distance bias has eaten its lead."""
    G, dim, n, H = 1, 64, 1100, 2
    vals, pages, scales, bt, rng = tied_case(D, dt, [n], H, G, dim, seed=5)
    spots = [0, 1, 15, 16, 17, 31, 32, 159, 160, 255, 256, 511, 512, 1023, 1024, 1098, 1099]
    for c, j in enumerate(spots):
        vals[0][j] = 0
        vals[0][j, 0, c] = 8.0
    vals[0][[j for j in range(n) if j not in spots], 0, : len(spots)] = 0
    put_values(D, vals, pages, scales, bt, H, G, dim, 1e-5)
    toks = [(j, p) for j in spots for p in (j - 1, j, j + 1, j + 200, n - 1) if 0 <= p < n]
    q = np.zeros((len(toks), H, dim))
    for t, (j, _) in enumerate(toks):
        q[t, :, spots.index(j)] = 8.0
    slopes = np.array([0.5, 0.004] if steep else [0.02, 0.004], np.float32)
    got = torch.empty((len(toks), H * dim), dtype=dt, device=DEV)
    D.tied_attn(put_q(D, q, dt), pages, scales, bt, i32([1] * len(toks)), i32([p for _, p in toks]), torch.from_numpy(slopes).to(DEV), 0.7, G, dim, n, got)
    torch.cuda.synchronize()
    want = tied_want(vals, q, [0] * len(toks), [p for _, p in toks], slopes, 0.7, 1e-5)
    assert err(got, want.reshape(len(toks), -1)) < tol(dt, b16=6e-3)
    for t, (j, p) in enumerate(toks):
        e = np.abs(f64(got)[t, dim:] - vals[0][j, 0]).max()
        assert (e < 0.1) if p >= j else (e > 0.5), (j, p)


@pytest.mark.parametrize("H,G,dim", [g for g in GEOMETRY if g[2] <= 128])
@pytest.mark.parametrize("scale,layout", [(1.0, "frag"), (-0.7, "rows")])
def test_tied_prefill(D, ops, H, G, dim, scale, layout):
    """Whole prompts, portions in the middle of one, several sequences, scattered pages; sharp scores, so that a key too many or
    too few shows."""
    parts = [(200, 200), (5, 5), (130, 517), (1, 64), (33, 65), (2, 18)]          # (new tokens, context after them)
    dt, eps = torch.bfloat16, 1e-5
    vals, pages, scales, bt, rng = tied_case(D, dt, [c for _, c in parts], H, G, dim, seed=H)
    put_values(D, vals, pages, scales, bt, H, G, dim, eps)
    T, vp = sum(n for n, _ in parts), D.pad32(dim)
    q = torch.from_numpy(rng.normal(size=(T, H, dim))).to(dt).double().numpy()
    slopes = R.slopes(H).astype(np.float32)
    pl = [[int(p) for p in bt[i + 1].tolist() if p >= 0] for i in range(len(parts))]
    plan = D.PrefillPlan([(pl[i], n, c) for i, (n, c) in enumerate(parts)], DEV)
    out = ops.FragActivation(T, H * vp, DEV, dtype=dt) if layout == "frag" else torch.empty((T, H * vp), dtype=dt, device=DEV)
    D.tied_prefill(plan, put_q(D, q, dt), pages, scales, torch.from_numpy(slopes).to(DEV), scale, G, dim, out)
    torch.cuda.synchronize()
    seq = np.repeat(np.arange(len(parts)), [n for n, _ in parts])
    pos = np.concatenate([np.arange(c - n, c) for n, c in parts])
    got, want = f64(rows_of(out)).reshape(T, H, vp), tied_want(vals, q, seq, pos, slopes, scale, eps)
    # a key whose 16-bit rounding falls to the other side moves a sharp softmax a little
    e = np.abs(got[..., :dim] - want) / np.abs(want).max()
    assert np.quantile(e, 0.999) < 2e-2 and e.max() < 8e-2 and np.abs(got[..., dim:]).max(initial=0) == 0


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,dim,temp", [(6, 2, 40, (0.4, 7.0)), (3, 3, 64, None), (2, 1, 300, (-0.3, 2.0)), (8, 2, 128, (0.7, 16.0))])
def test_tied_prep(D, dt, H, G, dim, temp):
    """Biases, norms and temperature of the queries; what lands in the pages, and that nothing else changes there."""
    vals, pages, scales, bt, rng = tied_case(D, dt, [40, 25], H, G, dim)
    T, eps = 21, 1e-3
    seq = np.array([1] * 12 + [2] * 9, np.int32)
    pos = np.array(list(range(14, 26)) + list(range(16, 25)), np.int32)
    y, bias = rnd(rng, T, D.pad32((H + G) * dim)), rnd(rng, (H + G) * dim)
    w = rnd(rng, dim)
    q = torch.full((T, H, D.pad32(dim)), 9.0, dtype=dt, device=DEV)
    p0, s0 = pages.clone(), scales.clone()
    D.tied_prep(q, pages, scales, y, bias, w, eps, temp, bt, i32(seq), i32(pos), H, G, dim)
    torch.cuda.synchronize()
    z = (f64(y)[:, : (H + G) * dim] + f64(bias)).reshape(T, H + G, dim)
    t = R.query_temperature(pos, {"coef": temp[0], "every": temp[1]} if temp else None)
    assert err(q[..., :dim], R.rms(z[:, :H], eps) * f64(w) * t[:, None, None]) < tol(dt, b16=5e-3) and float(q[..., dim:].abs().sum()) == 0
    rows = f64(pages.permute(0, 4, 1, 2, 3, 5).reshape(pages.shape[0], 16, G, -1))
    at = np.array([int(bt[s, p // 16]) for s, p in zip(seq, pos)])
    assert np.abs(rows[at, pos % 16][..., :dim] - z[:, H:]).max() < tol(dt, b16=2e-2) * 8
    k = f64(scales)[at, :, pos % 16][..., None] * z[:, H:]
    assert np.abs(k - R.rms(z[:, H:], eps)).max() < 1e-5
    slots = lambda a, b: int((a != b).permute(0, 4, 1, 2, 3, 5).reshape(a.shape[0], 16, -1).any(-1).sum())
    assert slots(pages, p0) == T and int((scales != s0).permute(0, 2, 1).any(-1).sum()) == T


# ------------------------------------------------------------------ experts by token id
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,E,top,shared", [(1, 1, 1, None), (1, 6, 3, 24), (9, 70, 70, 40), (37, 5, 1, 100), (64, 130, 8, None), (700, 6, 4, 40),
                                            (900, 16, 3, 64), (1100, 3, 2, None)])
def test_experts_by_token_id(D, ops, dt, T, E, top, shared):
    rng = np.random.default_rng(T + E)
    ff = load_pkg("feed_forward")
    Wd, F, V = 72, 40, 23
    Hp = D.pad64(Wd)
    P, layers = {}, []

    def glu(name, n):
        out = {}
        for k in ("gate", "up", "down"):
            out[k] = rnd(rng, *((Wd, n) if k == "down" else (n, Wd)), std=1.5 * (n if k == "down" else Wd) ** -0.5)
            P[f"{name}.{k}"] = f64(out[k])
        return out
    for l in range(3):                                    # several layers' plans are made together
        n = f"l{l}.mlp"
        P[n + ".table"] = np.argsort(rng.random((V, E)), -1)[:, :top]
        w = [glu(f"{n}.e{e}", F) for e in range(E)]
        w = {k: [x[k] for x in w] for k in ("gate", "up", "down")}
        w["table"] = torch.from_numpy(P[n + ".table"])
        if shared:
            w["shared"] = glu(n + ".shared", shared)
        layers.append(ff.TableMoe(ff.TableMoeSpec(F, E, top, shared), w, Wd, dt, DEV))
    ids = rng.integers(0, V, T)
    plans = ff.TableRouting(dict(enumerate(layers)), dt).plans(i32(ids))
    x = D.padded(rnd(rng, T, Wd, dt=dt), T, Hp).contiguous()
    act = ops.FragActivation.pack(x) if dt == torch.bfloat16 else x
    for l, m in enumerate(layers):
        p = plans[l]
        torch.cuda.synchronize()
        tiles, perm, used = p.tiles.view(-1, 4).cpu().numpy()[: int(p.n_tiles[0])], p.perm.cpu().numpy(), int(p.n_tiles[1])
        flat = P[f"l{l}.mlp.table"][ids].reshape(-1)
        assert used <= p.places and sorted(q for q in perm[:used] if q >= 0) == list(range(T * top)) and tiles[:, 2].sum() == T * top
        for e, first, n, _ in tiles:
            assert 0 < n <= p.tile_rows and first % 16 == 0 and (flat[perm[first:first + n]] == e).all()
        for split in (True, False):
            rows, y, parts = m(act, x, p, split)
            torch.cuda.synchronize()
            got = f64(rows).reshape(T, top, Hp).mean(1)
            if y is not None:
                got = got + f64(y) + (f64(parts.part.view(parts.ks - 1, T, Hp)).sum(0) if parts is not None else 0)
            want = R.table_moe(f64(x)[:, :Wd], ids, {"router": {"top": top}, "shared": shared}, P, f"l{l}.mlp")
            assert np.abs(got[:, :Wd] - want).max() / np.abs(want).max() < tol(dt, f32=5e-6) and np.abs(got[:, Wd:]).max() < 1e-6


@pytest.mark.parametrize("T,K,N", [(1, 32, 20), (5, 3072, 160), (40, 4096, 1024), (64, 1600, 96), (100, 4096, 160), (200, 2048, 512), (600, 64, 224)])
def test_linear_sum(D, ops, T, K, N):
    rng = np.random.default_rng(T)
    x, W = rnd(rng, T, K, dt=torch.bfloat16), rnd(rng, N, K, std=K ** -0.5, dt=torch.bfloat16)
    want = f64(x) @ f64(W).T
    for split in (True, False):
        y, parts = D.linear_sum(ops.FragActivation.pack(x), ops.PackedWeight(W), split)
        torch.cuda.synchronize()
        got = f64(y) + (f64(parts.part.view(parts.ks - 1, T, N)).sum(0) if parts is not None else 0)
        assert np.abs(got - want).max() < 2e-5


@pytest.mark.parametrize("T,K,ff", [(1, 64, 64), (20, 96, 224), (64, 64, 96), (100, 64, 160), (4096, 64, 2048)])
def test_gate_up_silu(D, ops, T, K, ff):
    rng = np.random.default_rng(T)
    dt = torch.bfloat16
    gu, x = rnd(rng, 2 * ff, K, std=K ** -0.5, dt=dt), rnd(rng, T, K, std=2.0, dt=dt)
    out = D.gate_up_silu(ops.FragActivation.pack(x), D.weight(gu), ops.interleave_gate_up(gu), D.activation(T, ff, dt, DEV))
    torch.cuda.synchronize()
    z = f64(x) @ f64(gu).T
    assert err(out.unpack(), R.silu(z[:, :ff]) * z[:, ff:]) < 1.2e-2


@pytest.mark.parametrize("T,K,rows,ext", [(1, 64, 64, 32), (16, 96, 128, 64), (30, 1056, 64, 32), (64, 128, 2048, 64), (32, 64, 4096, 32), (5, 4096, 1024, 160),
                                          (65, 96, 64, 32), (128, 64, 4096, 64), (200, 160, 1024, 32), (256, 64, 4096, 64)])
def test_linear_groups(D, ops, T, K, rows, ext):
    """Four row groups and a narrow last one, each on activations of its own, in one launch."""
    rng = np.random.default_rng(T)
    dt = torch.bfloat16
    xs, W = [rnd(rng, T, K, dt=dt) for _ in range(5)], rnd(rng, 4 * rows + ext, K, std=K ** -0.5, dt=dt)
    data = torch.cat([ops.FragActivation.pack(x).data for x in xs])
    Wp = ops.PackedWeight(W)
    y, y2 = D.linear_groups(ops.FragActivation(T, K, DEV, data), Wp, rows, ext)
    torch.cuda.synchronize()
    for i in range(4):
        assert err(y[:, i * rows:(i + 1) * rows], f64(xs[i]) @ f64(W[i * rows:(i + 1) * rows]).T) < 4e-3
        assert torch.equal(Wp.rows(i * rows, rows).unpack(), W[i * rows:(i + 1) * rows])
    assert y2.shape[0] == (1 if T > 64 else 8 if K >= 2048 else max(K // 256, 1))
    assert err(y2.sum(0), f64(xs[4]) @ f64(W[4 * rows:]).T) < 2e-6
