"""Every kernel of the latent-attention decoders alone, in both element types, against float64 numpy."""
import numpy as np
import pytest
import torch

import safolorn_cases as C
from conftest import load_pkg
from oracle import safolorn_ref as R

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.bfloat16, torch.float32]


@pytest.fixture(scope="module")
def D(ops):
    return load_pkg("decoder_ops")


def tol(dt, f32=2e-6, b16=1.2e-2):
    return f32 if dt == torch.float32 else b16


def rnd(rng, *shape, std=1.0, dt=torch.float32):
    return torch.from_numpy(rng.normal(0, std, shape)).to(torch.bfloat16).to(dt).to(DEV)


def f64(t):
    return t.double().cpu().numpy()


def err(got, want):
    return float(np.abs(f64(got) - want).max() / np.abs(want).max())


def rows_of(act):
    return act if isinstance(act, torch.Tensor) else act.unpack()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,H,Hp", [(1, 30, 32), (17, 104, 128), (70, 2100, 2112), (5, 5000, 5024), (3, 9000, 9024)])
def test_stream_norm(D, ops, dt, T, H, Hp):
    rng = np.random.default_rng(T)
    x, y, parts = (torch.zeros((*s, Hp), device=DEV) for s in ((T,), (T,), (2, T)))
    for t in (x, y, parts):
        t[..., :H] = rnd(rng, *t.shape[:-1], H, std=3.0)
    w = torch.zeros(Hp, dtype=dt, device=DEV)
    w[:H] = rnd(rng, H, dt=dt)
    x0 = f64(x)
    kp = ops.KSplitParts(parts.contiguous(), 3, Hp) if dt == torch.bfloat16 else None
    want = x0[:, :H] + (f64(parts).sum(0)[:, :H] if kp else 0) + R.rms(f64(y)[:, :H], 1e-3) * f64(w)[:H]
    frag = ops.FragActivation(T, Hp, DEV, dtype=dt) if dt == torch.bfloat16 else None
    row = torch.empty((T, Hp), dtype=dt, device=DEV)
    D.stream_norm(x, H, 1e-3, 1.7, kp, (y, w), out=frag, out_row=row)
    torch.cuda.synchronize()
    assert err(x[:, :H], want) < 2e-6 and float(x[:, H:].abs().sum()) == 0
    assert err(row[:, :H], R.rms(want, 1e-3) * 1.7) < tol(dt, b16=4e-3) and float(row[:, H:].abs().sum()) == 0
    if frag is not None:
        assert torch.equal(frag.unpack(), row)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,width,dim", [(1, 40, 5), (33, 104, 20), (300, 96, 20), (300, 96, 40), (4100, 72, 250), (16, 200, 70)])
def test_token_gate(D, ops, dt, T, width, dim):
    rng = np.random.default_rng(T)
    Hp, N, V = D.pad32(width), D.pad32(dim), 50
    x = torch.zeros((T, Hp), device=DEV)
    x[:, :width] = rnd(rng, T, width)
    Wr = rnd(rng, dim, width, std=2 * width ** -0.5, dt=dt)
    table = rnd(rng, V, 3 * dim, dt=dt)
    ids = torch.from_numpy(rng.integers(0, V, T).astype(np.int32)).to(DEV)
    xs, xa = f64(x)[:, :width], x
    if dt == torch.bfloat16:                              # the stream rounded to 16 bits, with what is pending added to it
        part = torch.zeros((2, T, Hp), device=DEV)
        part[..., :width] = rnd(rng, 2, T, width)
        xs = xs + f64(part).sum(0)[:, :width]
        xa = ops.FragActivation(T, Hp, DEV, dtype=dt)
        D.stream_norm(x, width, 1e-5, parts=ops.KSplitParts(part, 3, Hp), out=xa, raw=True)
        assert err(x[:, :width], xs) < 1e-6 and torch.equal(xa.unpack(), x.to(dt))
    out = rows_of(D.token_gate(xa, D.weight(D.padded(Wr, N, Hp)), table, dim, dim, ids))
    torch.cuda.synchronize()
    want = R.gelu_tanh(xs @ f64(Wr).T) * f64(table)[f64(ids).astype(int)][:, dim:2 * dim]
    assert err(out[:, :dim], want) < tol(dt) and float(out[:, dim:].abs().sum()) == 0


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,K,ff", [(1, 64, 64), (20, 96, 224), (64, 64, 96), (100, 64, 160), (4096, 64, 2048)])
def test_clipped_glu(D, ops, dt, T, K, ff):
    """T <= 64: the product as the GEMV's epilogue; 4096: as the persistent GEMM's; between: a launch of its own."""
    rng = np.random.default_rng(T)
    g, u = rnd(rng, ff, K, std=K ** -0.5, dt=dt), rnd(rng, ff, K, std=K ** -0.5, dt=dt)
    x = rnd(rng, T, K, std=2.0, dt=dt)
    gu = torch.cat([g, u])
    frag = dt == torch.bfloat16
    out = D.activation(T, ff, dt, DEV)
    D.gate_up_clipglu(ops.FragActivation.pack(x) if frag else x, D.weight(gu), ops.interleave_gate_up(gu) if frag else None, 1.5, 1.25, 1.702, out)
    torch.cuda.synchronize()
    gs, us = np.minimum(1.5 * f64(x) @ f64(g).T, 1.25), np.clip(1.5 * f64(x) @ f64(u).T, -1.25, 1.25)
    assert err(rows_of(out), gs / (1 + np.exp(-1.702 * gs)) * (us + 1)) < tol(dt)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,H,K,N", [(1, 3, 32, 32), (18, 2, 64, 96), (50, 5, 96, 32), (300, 2, 64, 288)])
def test_head_linear(D, ops, dt, T, H, K, N):
    rng = np.random.default_rng(T)
    x = rnd(rng, T, H * K + 32, dt=dt)
    W = rnd(rng, H, N, K, std=K ** -0.5, dt=dt)
    out = torch.full((T, H, N + 32), 7.0, dtype=dt, device=DEV)
    D.head_linear(x, H * K + 32, K, D.weight(W.view(H * N, K)), H, T, K, N, out, H * (N + 32), N + 32, 0.5)
    want = 0.5 * np.einsum("thk,hnk->thn", f64(x)[:, : H * K].reshape(T, H, K), f64(W))
    torch.cuda.synchronize()
    assert err(out[..., :N], want) < tol(dt, b16=5e-3) and bool((out[..., N:] == 7.0).all())
    if dt == torch.bfloat16:
        f = ops.FragActivation(T, H * N, DEV, dtype=dt)
        D.head_linear(x, H * K + 32, K, D.weight(W.view(H * N, K)), H, T, K, N, f, 0, N, 0.5)
        assert torch.equal(f.unpack(), out[..., :N].reshape(T, H * N))


def latent_case(D, dt, ctxs, H, rank, rot, seed=0, n_extra=3):
    """A cache whose sequences have ctxs[i] tokens, pages scattered and the unused ones poisoned with large values."""
    rng = np.random.default_rng(seed)
    need = [-(-c // 16) for c in ctxs]
    n_pages = sum(need) + n_extra
    NB = D.pad32(rank) // 32 + D.pad32(rot) // 32
    order = rng.permutation(n_pages)
    bt = np.full((len(ctxs) + 1, max(need) + 1), -1, np.int32)
    lat = [rng.normal(size=(c, rank + rot)) for c in ctxs]
    dense = np.full((n_pages, 16, NB * 32), 1e4)
    dense[:, :, rank:D.pad32(rank)] = 0
    dense[:, :, D.pad32(rank) + rot:] = 0
    k = 0
    for i, c in enumerate(ctxs):
        lat[i] = torch.from_numpy(lat[i]).to(torch.bfloat16).double().numpy()
        for b in range(need[i]):
            p = bt[i + 1, b] = order[k]
            k += 1
            n = min(16, c - 16 * b)
            dense[p, :n, :rank] = lat[i][16 * b:16 * b + n, :rank]
            dense[p, :n, D.pad32(rank):D.pad32(rank) + rot] = lat[i][16 * b:16 * b + n, rank:]
    pages = torch.from_numpy(dense).to(dt).to(DEV).view(n_pages, 16, NB, 4, 8).permute(0, 2, 3, 1, 4).contiguous()
    return lat, pages, torch.from_numpy(bt).to(DEV), rng


def attn_want(lat, q, seq, pos, sink, scale, rank):
    T, H, _ = q.shape
    out = np.zeros((T, H, rank))
    for t in range(T):
        kv = lat[seq[t]][: pos[t] + 1]
        for h in range(H):
            s = kv @ q[t, h] * scale
            w = R.sink_softmax(s, sink[h]) if sink is not None else np.exp(s - s.max()) / np.exp(s - s.max()).sum()
            out[t, h] = w @ kv[:, :rank]
    return out


def put_queries(D, q, rank, rot, dt):
    T, H, _ = q.shape
    full = torch.zeros((T, H, D.pad32(rank) + D.pad32(rot)), dtype=dt, device=DEV)
    full[..., :rank] = torch.from_numpy(q[..., :rank]).to(dt)
    full[..., D.pad32(rank):D.pad32(rank) + rot] = torch.from_numpy(q[..., rank:]).to(dt)
    return full


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,rank,rot", [(1, 32, 8), (3, 72, 24), (16, 128, 40), (18, 256, 64), (20, 544, 16)])
@pytest.mark.parametrize("sunk", [True, False])
def test_latent_attention_decode(D, dt, H, rank, rot, sunk):
    ctxs = [1, 2, 15, 16, 17, 33, 200, 517]
    lat, pages, bt, rng = latent_case(D, dt, ctxs, H, rank, rot, seed=H)
    seq = list(range(len(ctxs)))
    q = torch.from_numpy(rng.normal(size=(len(ctxs), H, rank + rot))).to(torch.bfloat16).double().numpy()
    sink = rng.normal(2.0, 1.0, H).astype(np.float32) if sunk else None
    scale = 3.0 * (rank + rot) ** -0.5
    args = (put_queries(D, q, rank, rot, dt), pages, bt, torch.tensor([s + 1 for s in seq], dtype=torch.int32, device=DEV),
            torch.tensor([c - 1 for c in ctxs], dtype=torch.int32, device=DEV), torch.from_numpy(sink).to(DEV) if sunk else None, scale, rank, rot)
    want = attn_want(lat, q, seq, [c - 1 for c in ctxs], sink, scale, rank)
    for splits in ([1, 2, 5, 32] if dt == torch.bfloat16 else [1]):
        got = D.latent_attn(*args, max_ctx=max(ctxs), splits=splits)
        torch.cuda.synchronize()
        assert err(got[..., :rank], want) < tol(dt, b16=5e-3), splits
        assert float(got[..., rank:].abs().sum()) == 0
        if splits > 1:                                    # the same, merged on the way through W_uv
            uv = rnd(rng, H, 64, rank, std=rank ** -0.5, dt=dt)
            y = load_pkg("ops").FragActivation(len(ctxs), H * 64, DEV, dtype=dt)
            D.latent_attn_out(*args, splits, D.weight(D.padded(uv, H, 64, D.pad32(rank)).reshape(H * 64, D.pad32(rank))), 64, y)
            torch.cuda.synchronize()
            assert err(y.unpack().view(-1, H, 64), np.einsum("thr,hvr->thv", want, f64(uv))) < 8e-3, splits


@pytest.mark.parametrize("dt", DTYPES)
def test_latent_attention_single_keys_far_and_at_page_borders(D, dt):
    """One key stands out by its rotated part; its latent is what comes back - wherever it lies, and not one token later."""
    rank, rot, H, n = 64, 16, 2, 300
    lat, pages, bt, rng = latent_case(D, dt, [n], H, rank, rot, seed=5)
    spots = [0, 1, 15, 16, 17, 31, 32, 159, 160, 255, 256, 298, 299]
    NBr = D.pad32(rank)
    for j in spots:                                       # key j: rotated part 0 except one coordinate of its own
        v = np.zeros(rot)
        v[spots.index(j)] = 8.0
        lat[0][j, rank:] = v
        p = int(bt[1, j // 16])
        for d in range(rot):
            pages[p, (NBr + d) // 32, (NBr + d) % 32 // 8, j % 16, (NBr + d) % 8] = float(v[d])
    toks = [(j, pos) for j in spots for pos in (j - 1, j, j + 1, n - 1) if 0 <= pos < n]
    q = np.zeros((len(toks), H, rank + rot))
    for t, (j, _) in enumerate(toks):
        q[t, :, rank + spots.index(j)] = 8.0
    got = D.latent_attn(put_queries(D, q, rank, rot, dt), pages, bt, torch.ones(len(toks), dtype=torch.int32, device=DEV),
                        torch.tensor([p for _, p in toks], dtype=torch.int32, device=DEV), None, 1.0, rank, rot, max_ctx=n)
    torch.cuda.synchronize()
    for t, (j, pos) in enumerate(toks):
        e = float(np.abs(f64(got)[t, 0] - lat[0][j, :rank]).max())
        assert (e < 1e-2) if pos >= j else (e > 0.5), (j, pos)
    assert err(got[..., :rank], attn_want(lat, q, [0] * len(toks), [p for _, p in toks], None, 1.0, rank)) < tol(dt, b16=6e-3)


@pytest.mark.parametrize("H,rank,dim,rot,vdim", [(1, 32, 32, 8, 32), (3, 72, 40, 24, 48), (4, 512, 128, 64, 128), (2, 96, 100, 16, 64), (5, 64, 16, 40, 100)])
@pytest.mark.parametrize("scale,layout", [(1.0, "frag"), (-0.7, "rows")])
def test_latent_prefill(D, ops, H, rank, dim, rot, vdim, scale, layout):
    """Keys and values made from the latents: whole prompts, portions in the middle of one, several sequences, scattered pages;
    sharp scores, so that a key too many or too few shows."""
    parts = [(200, 200), (5, 5), (130, 517), (1, 64), (33, 65), (2, 18)]          # (new tokens, context after them)
    dt = torch.bfloat16
    lat, pages, bt, rng = latent_case(D, dt, [c for _, c in parts], H, rank, rot, seed=H)
    dp, vp, rp = D.pad32(dim), D.pad32(vdim), D.pad32(rank)
    T = sum(n for n, _ in parts)
    uk, uv = rnd(rng, H, dim, rank, std=2 * rank ** -0.5), rnd(rng, H, vdim, rank, std=rank ** -0.5)
    qkv = torch.zeros((T, D.pad32(H * dp + 7)), dtype=dt, device=DEV)
    qn = rnd(rng, T, H, dim)
    qkv[:, : H * dp] = D.padded(qn, T, H, dp).reshape(T, H * dp).to(dt)
    qr = rnd(rng, T, H, rot, std=0.5)
    sink = rng.normal(1.0, 1.0, H).astype(np.float32)
    pl = [[int(p) for p in bt[i + 1].tolist() if p >= 0] for i in range(len(parts))]
    plan = D.PrefillPlan([(pl[i], n, c) for i, (n, c) in enumerate(parts)], DEV)
    out = ops.FragActivation(T, H * vp, DEV, dtype=dt) if layout == "frag" else torch.empty((T, H * vp), dtype=dt, device=DEV)
    D.latent_prefill(plan, qkv, D.padded(qr, T, H, D.pad32(rot)).to(dt), pages, D.weight(D.padded(uk, H, dp, rp).reshape(H * dp, rp).to(dt)),
                     D.weight(D.padded(uv, H, vp, rp).reshape(H * vp, rp).to(dt)), torch.from_numpy(sink).to(DEV), scale, rank, dim, rot, vdim, out)
    torch.cuda.synchronize()
    got = f64(rows_of(out)).reshape(T, H, vp)
    bf = lambda a: torch.from_numpy(a).to(dt).double().numpy()
    want, t = np.zeros((T, H, vdim)), 0
    for i, (n, c) in enumerate(parts):
        for h in range(H):
            k, v = bf(lat[i][:, :rank] @ f64(uk)[h].T), bf(lat[i][:, :rank] @ f64(uv)[h].T)   # stored in 16 bits
            for j in range(n):
                pos = c - n + j
                s = (k[: pos + 1] @ f64(qn)[t + j, h] + lat[i][: pos + 1, rank:] @ f64(qr)[t + j, h]) * scale
                want[t + j, h] = R.sink_softmax(s, sink[h]) @ v[: pos + 1]
        t += n
    # a key whose 16-bit rounding falls to the other side moves a sharp softmax a little
    e = np.abs(got[..., :vdim] - want) / np.abs(want).max()
    assert np.quantile(e, 0.999) < 1e-2 and e.max() < 6e-2 and np.abs(got[..., vdim:]).max(initial=0) == 0


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("scaling", [None, C.YARN])
def test_latent_prep(D, dt, scaling):
    """Rotation of queries and key part, norm of the latent, and where they land; token rows of several sequences."""
    H, dim, rank, rot, T = 3, 40, 72, 24, 21
    c = C.rot(1000.0, 20, scaling)
    lat, pages, bt, rng = latent_case(D, dt, [40, 25], H, rank, rot)
    rotation = load_pkg("rotary").Rotation.from_config(c)
    cos, sin = (torch.from_numpy(t).to(DEV) for t in rotation.tables(rot, 64))
    seq = np.array([1] * 12 + [2] * 9, np.int32)
    pos = np.array(list(range(14, 26)) + list(range(16, 25)), np.int32)
    dp = 64
    ld = D.pad32(H * dp + H * rot + rank + rot)
    qkv = rnd(rng, T, ld, dt=dt)
    w = rnd(rng, rank, dt=dt)
    q = torch.full((T, H, D.pad32(rank) + 32), 9.0, dtype=dt, device=DEV)
    off = H * dp
    before = pages.clone()
    D.latent_prep(q, D.pad32(rank), pages, qkv, off, off + H * rot, off + H * rot + rank, 1.25, None, 1e-5, bt, torch.from_numpy(seq).to(DEV), torch.from_numpy(pos).to(DEV),
                  cos, sin, H, rank, rot)
    torch.cuda.synchronize()
    assert torch.equal(pages, before)                     # a layer that reads another layer's latents stores nothing
    D.latent_prep(q, D.pad32(rank), pages, qkv, off, off + H * rot, off + H * rot + rank, 1.25, w, 1e-5, bt, torch.from_numpy(seq).to(DEV), torch.from_numpy(pos).to(DEV),
                  cos, sin, H, rank, rot)
    torch.cuda.synchronize()
    x = 1.25 * f64(qkv)
    wq = R.rotate(f64(qkv)[:, off:off + H * rot].reshape(T, H, rot), pos, c)     # the gain is left to the scores' scale
    assert err(q[..., D.pad32(rank):D.pad32(rank) + rot], wq) < tol(dt, b16=5e-3)
    assert float(q[..., D.pad32(rank) + rot:].abs().sum()) == 0 and bool((q[..., :D.pad32(rank)] == 9.0).all())
    cw = R.rms(x[:, off + H * rot:off + H * rot + rank], 1e-5) * f64(w)
    kw = R.rotate(x[:, off + H * rot + rank:off + H * rot + rank + rot], pos, c)
    rows = pages.permute(0, 3, 1, 2, 4).reshape(pages.shape[0], 16, -1)
    at = np.array([int(bt[s, p // 16]) for s, p in zip(seq, pos)])
    got = f64(rows)[at, pos % 16]
    assert np.abs(got[:, :rank] - cw).max() < tol(dt, b16=1e-2) * 2 and np.abs(got[:, D.pad32(rank):D.pad32(rank) + rot] - kw).max() < tol(dt, b16=1e-2) * 2
    if dt == torch.bfloat16:                              # the same with the unrotated parts lifted beside it
        W = rnd(rng, H, D.pad32(rank), dp, std=dp ** -0.5, dt=dt)
        q2, p2 = torch.empty_like(q), before.clone()
        D.latent_prep(q2, D.pad32(rank), p2, qkv, off, off + H * rot, off + H * rot + rank, 1.25, w, 1e-5, bt, torch.from_numpy(seq).to(DEV),
                      torch.from_numpy(pos).to(DEV), cos, sin, H, rank, rot, D.weight(W.view(H * D.pad32(rank), dp)))
        torch.cuda.synchronize()
        assert torch.equal(p2, pages) and torch.equal(q2[..., D.pad32(rank):], q[..., D.pad32(rank):])
        assert err(q2[..., :D.pad32(rank)], np.einsum("thk,hrk->thr", f64(qkv)[:, :off].reshape(T, H, dp), f64(W))) < 5e-3
    changed = (pages != before).permute(0, 3, 1, 2, 4).reshape(pages.shape[0], 16, -1).any(-1).sum()
    assert int(changed) == T                              # every token one slot, no other slot


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,E,top", [(1, 1, 1), (1, 6, 3), (9, 70, 70), (37, 5, 1), (64, 130, 8), (700, 6, 4), (900, 16, 3)])
def test_experts(D, ops, dt, T, E, top):
    rng = np.random.default_rng(T + E)
    Wd, ff = 72, 40
    Hp = D.pad64(Wd)
    P = {"x.mlp.router": f64(rnd(rng, E, Wd, std=Wd ** -0.5)), "x.mlp.router.b": f64(rnd(rng, E))}
    for e in range(E):
        P[f"x.mlp.e{e}.up"], P[f"x.mlp.e{e}.down"] = f64(rnd(rng, ff, Wd, std=Wd ** -0.5)), f64(rnd(rng, Wd, ff, std=ff ** -0.5))
    x = torch.zeros((T, Hp), dtype=dt, device=DEV)
    x[:, :Wd] = rnd(rng, T, Wd, dt=dt)
    spec = load_pkg("feed_forward").MoeSpec(ff, E, top)
    t = lambda n: torch.from_numpy(P["x.mlp." + n])
    m = load_pkg("feed_forward").MoeRelu2(spec, {"router": t("router"), "router_b": t("router.b"), "up": [t(f"e{e}.up") for e in range(E)],
                                                 "down": [t(f"e{e}.down") for e in range(E)]}, Wd, 1.5, dt, DEV)
    # routing on given logits: exact choice, ties to the lower index
    z = torch.from_numpy(np.round(rng.normal(size=(T, D.pad32(E))) * 4) / 4).float().to(DEV)
    pick, w = D.moe_route(z, torch.zeros(E, device=DEV), 1.0, top, dt)
    zz = f64(z)[:, :E]
    order = np.argsort(-zz, -1, kind="stable")[:, :top]
    assert np.array_equal(pick.cpu().numpy(), order)
    ex = np.exp(np.take_along_axis(zz, order, -1))
    assert np.abs(f64(w) - ex / ex.sum(-1, keepdims=True)).max() < 1e-6
    # the plan covers every entry once, tiles hold one expert
    plan = D.MoePlan(pick, E, dt)
    torch.cuda.synchronize()
    tiles, perm = plan.tiles.view(-1, 4).cpu().numpy()[: int(plan.n_tiles[0])], plan.perm.cpu().numpy()
    used = int(plan.n_tiles[1])
    assert used <= plan.places and used % 16 == 0 and sorted(p for p in perm[:used] if p >= 0) == list(range(T * top))
    assert len(tiles) <= plan.max_tiles and tiles[:, 2].sum() == T * top
    flat = order.reshape(-1)
    for e, first, n, _ in tiles:
        assert 0 < n <= plan.tile_rows and first % 16 == 0 and (flat[perm[first:first + n]] == e).all()
    # the whole block; in bf16 on the router's own fp32 logits of the rounded input, so that choices agree
    resid = rnd(rng, T, Hp)
    before, kp, sums = f64(resid), None, None
    if dt == torch.bfloat16:
        part, sums = rnd(rng, 1, T, Hp), ops.FragActivation(T, Hp, DEV, dtype=dt)
        kp, before = ops.KSplitParts(part, 2, Hp), before + f64(part)[0]
    m.add_to(resid, ops.FragActivation.pack(x) if dt == torch.bfloat16 else x, x, kp, sums)
    torch.cuda.synchronize()
    assert sums is None or torch.equal(sums.unpack(), resid.to(dt))
    want = R.moe_ff(1.5 * f64(x)[:, :Wd], {"router": {"top": top}}, P, "x")
    gap = np.sort(1.5 * f64(x)[:, :Wd] @ P["x.mlp.router"].T + P["x.mlp.router.b"], -1)[:, ::-1]
    clear = np.ones(T, bool) if top == E else gap[:, top - 1] - gap[:, top] > 1e-3
    got = f64(resid) - before
    assert clear.mean() > 0.9 and np.abs(got[clear, :Wd] - want[clear]).max() / np.abs(want).max() < tol(dt, f32=5e-6)
    assert np.abs(got[:, Wd:]).max() < 1e-6


@pytest.mark.parametrize("T,K,N", [(1, 32, 20), (5, 96, 160), (40, 160, 72), (64, 64, 8224), (100, 96, 160), (300, 64, 224), (4096, 64, 4096), (16, 3072, 256)])
def test_bf16_linear(ops, T, K, N):
    """The linear kernels of the bfloat16 library: every shape class of the fp16 ones."""
    rng = np.random.default_rng(T)
    x, W = rnd(rng, T, K, dt=torch.bfloat16), rnd(rng, N, K, std=K ** -0.5, dt=torch.bfloat16)
    want = f64(x) @ f64(W).T
    Wp, xf = ops.PackedWeight(W), ops.FragActivation.pack(x)
    assert torch.equal(Wp.unpack(), W) and torch.equal(xf.unpack(), x)
    for y in (ops.linear(xf, Wp, out_dtype=torch.float32), ops.linear(x, Wp, out_dtype=torch.float32)):
        assert err(y, want) < 2e-6
    assert err(ops.linear(xf, Wp), want) < 4e-3
    acc = rnd(rng, T, N)
    a0 = f64(acc)
    parts = ops.linear_acc_ksplit(xf, Wp, acc, torch.empty(3 * T * N, device=DEV))
    tot = f64(acc) + (f64(parts.part[: (parts.ks - 1) * T * N].view(parts.ks - 1, T, N)).sum(0) if parts is not None else 0)
    assert np.abs(tot - a0 - want).max() < 2e-5


@pytest.mark.parametrize("T,K,N", [(1, 32, 20), (70, 96, 130), (200, 160, 64)])
def test_fp32_linear(ops, T, K, N):
    rng = np.random.default_rng(T)
    x, W = (torch.from_numpy(rng.normal(size=s)).float().to(DEV) for s in ((T, K), (N, K)))
    want = f64(x) @ f64(W).T
    assert err(ops.linear(x, W), want) < 1e-6
    acc = torch.from_numpy(rng.normal(size=(T, N))).float().to(DEV)
    a0 = f64(acc)
    ops.linear(x, W, out=acc, accumulate=True)
    assert err(acc, a0 + want) < 1e-6
