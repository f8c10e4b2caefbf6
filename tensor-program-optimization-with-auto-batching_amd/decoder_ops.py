"""Operators of include/mlora_decoder.h, and the choice of layout that goes with an element type: bfloat16 works on
fragment-ordered activations and packed weights, fp32 on plain row-major tensors.  No CPU path.
"""
from __future__ import annotations

import ctypes

import torch

from . import ops
from ._lib import ACT_GLU, ACT_NONE, ACT_RELU2, FRAG, MOE_DOWN, MOE_UP, ROWMAJOR, StreamStep   # noqa: F401
from .ops import FragActivation, PackedWeight, _dev, _stream, check, lib_of


def pad32(n: int) -> int:
    return -(-n // 32) * 32


def pad64(n: int) -> int:
    """Row widths: the matrix-core kernels for many tokens take K in steps of 64."""
    return -(-n // 64) * 64


def padded(w: torch.Tensor, *shape) -> torch.Tensor:
    """`w` with zeros behind its rows / columns up to `shape`."""
    if tuple(w.shape) == tuple(shape):
        return w
    out = torch.zeros(shape, dtype=w.dtype, device=w.device)
    out[tuple(slice(0, n) for n in w.shape)] = w
    return out


def weight(w: torch.Tensor):
    """A linear weight [N, K] (K % 32 == 0) in the form the linears of its type take."""
    return w.contiguous() if w.dtype == torch.float32 else PackedWeight(w.contiguous())


def activation(T: int, K: int, dtype, device):
    """An activation block [T, K] in the order the linears of its type read."""
    if dtype == torch.float32:
        return torch.empty((T, K), dtype=dtype, device=device)
    return FragActivation(T, K, device, dtype=dtype)


def _wptr(w) -> int:
    return w.data.data_ptr() if isinstance(w, PackedWeight) else _dev(w)


def _ptr(t) -> int:
    return None if t is None else t.data_ptr()


def _parts(parts):
    """(pointer, blocks) of pending K-split partials."""
    return (parts.part.data_ptr(), parts.ks - 1) if parts is not None else (None, 0)


def stream_norm(x, H, eps, gain=1.0, parts=None, branch=None, out=None, out_row=None, raw=False):
    """x [T, Hp] fp32 (+= pending K-split partials, += branch[0] / rms * branch[1], in place); out (FragActivation) and / or
    out_row [T, Hp] = x / rms(x) * gain, or x itself with `raw`.  H: columns that count."""
    if out is None and out_row is None and parts is None and branch is None:
        return
    T, Hp = x.shape
    dt = out.dtype if out is not None else out_row.dtype if out_row is not None else branch[1].dtype if branch is not None else torch.bfloat16
    check(lib_of(dt).mlora_stream_norm(out.data.data_ptr() if out is not None else None, _ptr(out_row), _dev(x, torch.float32), *_parts(parts),
                                       _ptr(branch[0]) if branch is not None else None, _ptr(branch[1]) if branch is not None else None,
                                       float(eps), float(gain), int(raw), T, H, Hp, _stream()), dt)


def embed_scaled(table, ids, scale, out=None):
    """table[ids] * scale in fp32; out: an activation that takes the same in the table's type."""
    V, H = table.shape
    T = ids.numel()
    x = torch.empty((T, H), dtype=torch.float32, device=table.device)
    frag = out.data.data_ptr() if isinstance(out, FragActivation) else None
    row, ld = (out.data_ptr(), out.stride(0)) if isinstance(out, torch.Tensor) else (None, 0)
    check(lib_of(table.dtype).mlora_embed_scaled(_dev(x), frag, row, ld, _dev(table), _dev(ids, torch.int32), scale, T, H, V, _stream()), table.dtype)
    return x


class ElementwiseNorm:
    """tanh(alpha v) w + b, without statistics (weights [Hp], zero behind the width)."""

    def __init__(self, w, b, alpha, width_p, dtype, device):
        self.w, self.b = (padded(t.to(device, dtype), width_p).contiguous() for t in (w, b))
        self.alpha = float(alpha)

    def fill(self, f):
        f.w, f.b, f.alpha = self.w.data_ptr(), self.b.data_ptr(), self.alpha


class ResidualStream:
    """The fp32 stream x [T, Hp] of a pass with a branch that is still to be added: x + mult post(branch), where the branch is
    a sum of K-split partials and of entry rows of a mixture of experts.  Every step of a sublayer is one launch that adds
    what is pending and norms for the next sublayer."""

    def __init__(self, x, dtype, mult=1.0):
        self.x, self.dtype, self.mult = x, dtype, float(mult)
        self.shape, self.device = x.shape, x.device
        self.spare = None
        self.pending = None           # (y or None, KSplitParts or None, rows or None, row weight, norm or None, replaces x)

    def branch(self, y, parts=None, norm=None, rows=None, row_weight=1.0):
        assert self.pending is None
        self.pending = (y, parts, rows, row_weight, norm, False)

    def replace(self, y, parts=None):
        """x becomes y (+ its partials)."""
        assert self.pending is None
        self.pending = (y, parts, None, 1.0, None, True)

    def step(self, norm=None, out=None, out_row=None, mu=None, shift=None, tokens=None):
        """Adds what is pending; out (FragActivation) and / or out_row (rows, any stride): norm(x), or x itself without norm.
        mu [5, Hp], shift (state), tokens = (sequence, position, last token or None) per token: five mixes, stacked in out /
        out_row."""
        if out is None and out_row is None and self.pending is None:
            return
        T, Hp = self.shape
        a = StreamStep(T=T, Hp=Hp, x=self.x.data_ptr(), mult=self.mult, row_weight=1.0)
        if self.pending is not None:
            y, parts, rows, a.row_weight, post, new = self.pending
            if y is not None:
                a.y = _dev(y, torch.float32)
            if parts is not None:
                a.part, a.n_part = parts.part.data_ptr(), parts.ks - 1
            if rows is not None:
                a.rows, a.top = _dev(rows, self.dtype), rows.shape[0] // T
            if post is not None:
                post.fill(a.post)
            if new:
                a.x, a.mult = None, 1.0
            x = self.x
            if mu is not None or new:                     # a neighbour reads the old stream
                if self.spare is None:
                    self.spare = torch.empty_like(self.x)
                x, self.spare = self.spare, self.x
            a.x_out = x.data_ptr()
            self.x, self.pending = x, None
        if norm is not None:
            norm.fill(a.pre)
        if out is not None:
            a.out_frag, a.mix_stride = out.data.data_ptr(), out.data.numel() // 5
        if out_row is not None:
            a.out_row, a.ld_row = out_row.data_ptr(), out_row.stride(-2)
            if mu is not None:
                a.mix_stride = out_row.stride(0)
        if mu is not None:
            seq, pos, last = tokens
            a.mu, a.shift, a.n_seq = _dev(mu, self.dtype), _dev(shift, torch.float32), shift.shape[0]
            a.tok_seq, a.tok_pos, a.tok_last = _dev(seq, torch.int32), _dev(pos, torch.int32), _ptr(last)
        check(lib_of(self.dtype).mlora_stream_step(ctypes.byref(a), _stream()), self.dtype)


def linear_sum(x, W, split=True):
    """x @ W.T as (y fp32, K-split partials still to be added to it, or None)."""
    if not split or not isinstance(x, FragActivation):
        return ops.linear(x, W, out_dtype=torch.float32), None
    T, K = x.shape
    N = W.shape[0]
    L = lib_of(W.dtype)
    ks = L.mlora_gemv_ksplit(T, K, N)
    y = torch.empty((T, N), dtype=torch.float32, device=x.device)
    part = torch.empty((ks - 1) * T * N, dtype=torch.float32, device=x.device) if ks > 1 else None
    check(L.mlora_linear_ksplit_store(y.data_ptr(), _ptr(part), ks, x.data.data_ptr(), W.data.data_ptr(), T, K, N, _stream()), W.dtype)
    return y, ops.KSplitParts(part, ks, N) if ks > 1 else None


def linear_groups(x, W, group_rows, ext):
    """W's row groups of group_rows applied to activations of their own, the blocks of the FragActivation x one after the other: ->
    (all groups' results [T, rows], those of the last `ext` rows, a group of their own, as partial sums [n, T, ext] fp32)."""
    T, K = x.shape
    n, L = W.shape[0] - ext, lib_of(W.dtype)
    y = torch.empty((T, n), dtype=W.dtype, device=x.device)
    stride = x.data.numel() // (n // group_rows + 1)
    if T > 64:
        y2 = torch.empty((1, T, ext), dtype=torch.float32, device=x.device)
        check(L.mlora_gemm_frag_groups(_dev(y), x.data.data_ptr(), stride, group_rows, W.data.data_ptr(), T, K, n, _stream()), W.dtype)
        check(L.mlora_narrow_linear(_dev(y2), x.data[x.data.numel() - stride:].data_ptr(), W.rows(n, ext).data.data_ptr(), T, K, ext, _stream()), W.dtype)
        return y, y2
    y2 = torch.empty((L.mlora_gemv_groups_parts(K), T, ext), dtype=torch.float32, device=x.device)
    check(L.mlora_gemv_frag_groups(_dev(y), _dev(y2), x.data.data_ptr(), stride, group_rows, W.data.data_ptr(), T, K, n, ext, _stream()), W.dtype)
    return y, y2


def _cols(t, dtype):
    """(pointer, row stride) of a column range of a row-major tensor."""
    if not t.is_cuda or t.dtype != dtype or t.stride(1) != 1:
        raise ValueError("column ranges of GPU tensors of one type")
    return t.data_ptr(), t.stride(0) if t.shape[0] > 1 else max(t.shape[1], t.stride(0))


def token_gate(x, W, table, col0, dim, ids):
    """gelu_tanh(W x) * table[ids, col0 : col0 + dim] (x: an activation) as the activation of the following linear, its width
    W's padded row count."""
    T = x.shape[0]
    N, K = W.shape
    V, ld = table.shape
    if x.shape[1] != K or ids.shape != (T,):
        raise ValueError(f"token_gate: x{tuple(x.shape)} W{tuple(W.shape)} ids{tuple(ids.shape)}")
    out = activation(T, N, W.dtype, x.device)
    L = lib_of(W.dtype)
    if W.dtype == torch.float32:
        z = ops.linear(x, W)
        check(L.mlora_token_gate_mul(_dev(out), _dev(z), _dev(table, W.dtype), ld, col0, dim, _dev(ids, torch.int32), V, T, N, _stream()), W.dtype)
        return out
    check(L.mlora_token_gate(out.data.data_ptr(), x.data.data_ptr(), _wptr(W), _dev(table, W.dtype), ld, col0, dim, _dev(ids, torch.int32),
                             V, T, K, N, _stream()), W.dtype)
    return out


def clipglu_mul(gate_up, scale, limit, alpha, out):
    """The clipped gated product of gate_up [T, 2I] (gate columns first) into `out` (activation [T, I])."""
    T, I2 = gate_up.shape
    dt = gate_up.dtype
    frag = isinstance(out, FragActivation)
    p = _dev(gate_up)
    check(lib_of(dt).mlora_clipglu_mul(out.data.data_ptr() if frag else _dev(out), FRAG if frag else ROWMAJOR, p,
                                       p + I2 // 2 * gate_up.element_size(), I2, T, I2 // 2, scale, limit, alpha, _stream()), dt)
    return out


def gate_up_clipglu(x, W, W_il, scale, limit, alpha, out):
    """clipped gated product of x @ W.T (W [2I, K], gate rows first; W_il: its tiles interleaved) into `out` - the product as
    the epilogue of the linear where a kernel has that, else behind it."""
    T, K = x.shape
    I2 = W.shape[0]
    if isinstance(x, FragActivation):
        L = lib_of(x.dtype)
        args = (T, K, I2 // 2, scale, limit, alpha, _stream())
        if T <= 64:
            check(L.mlora_gemv_frag_clipglu(out.data.data_ptr(), x.data.data_ptr(), W_il.data.data_ptr(), *args), x.dtype)
            return out
        if L.mlora_gemm_frag_preferred(T, K, I2):
            check(L.mlora_linear_frag_clipglu(out.data.data_ptr(), x.data.data_ptr(), W.data.data_ptr(), *args), x.dtype)
            return out
    return clipglu_mul(ops.linear(x, W), scale, limit, alpha, out)


def silu_mul(gate_up, out):
    """silu(gate) * up of gate_up [T, 2I] (gate columns first) into `out` (activation [T, I])."""
    T, I2 = gate_up.shape
    dt = gate_up.dtype
    frag = isinstance(out, FragActivation)
    p = _dev(gate_up)
    check(lib_of(dt).mlora_silu_mul(out.data.data_ptr() if frag else _dev(out), FRAG if frag else ROWMAJOR, p, p + I2 // 2 * gate_up.element_size(), I2,
                                    T, I2 // 2, _stream()), dt)
    return out


def gate_up_silu(x, W, W_il, out):
    """silu(gate) * up of x @ W.T (W [2I, K], gate rows first; W_il: its tiles interleaved) into `out` - the product as the
    epilogue of the linear where a kernel has that, else behind it."""
    T, K = x.shape
    I2 = W.shape[0]
    if isinstance(x, FragActivation):
        L = lib_of(x.dtype)
        if T <= 64:
            check(L.mlora_gemv_frag_silu(out.data.data_ptr(), x.data.data_ptr(), W_il.data.data_ptr(), T, K, I2 // 2, _stream()), x.dtype)
            return out
        if L.mlora_gemm_frag_preferred(T, K, I2):
            check(L.mlora_linear_frag_silu(out.data.data_ptr(), x.data.data_ptr(), W.data.data_ptr(), T, K, I2 // 2, None, 0, None, 0, _stream()),
                  x.dtype)
            return out
    return silu_mul(ops.linear(x, W), out)


def time_mix(r, k, v, g, z, R, w2, w0, u, norm, eps, state, segs, tok_seq, tok_pos, out):
    """The recurrence of time mixing (csrc/time_mix.hip) over a pass: r, k, v, g [T, >= H * D] of one row stride, z [n, T, >= R] fp32 (partial sums), state
    [n, H, D, D] fp32 (updated), segs [n][4] int32 or None (a decode step) -> out, an activation [T, H * D rounded up]."""
    T = r.shape[0]
    (r_p, ld), (k_p, _), (v_p, _), (g_p, _) = (_cols(t, r.dtype) for t in (r, k, v, g))
    n_seq, H, D, _ = state.shape
    frag = isinstance(out, FragActivation)
    check(lib_of(r.dtype).mlora_time_mix(out.data.data_ptr() if frag else _dev(out, r.dtype), FRAG if frag else ROWMAJOR, out.shape[1],
                                         r_p, k_p, v_p, g_p, ld, _dev(z, torch.float32), z.shape[0], z.shape[2], R,
                                         _dev(w2, r.dtype), w2.shape[1], _dev(w0, torch.float32), _dev(u, torch.float32), _dev(norm, r.dtype), eps,
                                         _dev(state, torch.float32), n_seq, _ptr(segs), T if segs is None else segs.shape[0],
                                         _dev(tok_seq, torch.int32), _dev(tok_pos, torch.int32), T, H, D, _stream()), r.dtype)
    return out


class TimeMixPlan:
    """Ranges of a pass for `time_mix_prompt`: segs, per sequence (slot, first token, tokens, position of the first); tokens: of a
    range (chosen by the size of the pass)."""

    def __init__(self, segs, heads, device, tokens=None):
        if tokens is None:                                           # about four workgroups per compute unit
            tokens = min(max(1 << max(sum(n for _, _, n, _ in segs) * heads // 1024, 1).bit_length() - 1, 64), 256)
        ranges, seqs, self.n_states = [], [], 0
        for slot, first, n, pos in segs:
            parts = -(-n // tokens)
            if parts > 1:
                seqs.append((slot, pos, self.n_states, parts))
            for c in range(parts):
                at, end = c * tokens, c == parts - 1
                ranges.append((slot, first + at, min(tokens, n - at), pos + at, self.n_states + c if parts > 1 else -1, -1 if end else self.n_states + c, int(end), 0))
            if parts > 1:
                self.n_states += parts
        self.n_ranges, self.n_seqs = len(ranges), len(seqs)
        both = torch.tensor([x for t in (*ranges, *seqs) for x in t], dtype=torch.int32).to(device)
        self.ranges, self.seqs = both[: 8 * len(ranges)], both[8 * len(ranges):]


def time_mix_prompt_served(dim) -> bool:
    return bool(lib_of(torch.bfloat16).mlora_time_mix_prompt_served(dim))


def time_mix_prompt(plan, r, k, v, g, mix, w1, w2, w0, u, norm, eps, state, out):
    """time_mix for a pass over prompts; mix: the activation that the decay's low-rank projection w1 takes."""
    T, ld = r.shape
    n_seq, H, D, _ = state.shape
    L = lib_of(r.dtype)
    N = w1.shape[0]
    zp = torch.empty((T, 3, N), dtype=r.dtype, device=r.device)
    check(L.mlora_tanh_parts(zp.data_ptr(), mix.data.data_ptr(), _wptr(w1), T, mix.shape[1], N, _stream()), r.dtype)
    n = plan.n_states * H * D * (D + 1)
    scratch = torch.empty(n, dtype=torch.float32, device=r.device) if n else None
    frag = isinstance(out, FragActivation)
    check(L.mlora_time_mix_prompt(out.data.data_ptr() if frag else _dev(out, r.dtype), FRAG if frag else ROWMAJOR, out.shape[1], _dev(r), _dev(k, r.dtype),
                                  _dev(v, r.dtype), _dev(g, r.dtype), ld, zp.data_ptr(), N, _dev(w2, r.dtype), _dev(w0, torch.float32),
                                  _dev(u, torch.float32), _dev(norm, r.dtype), eps, _dev(state, torch.float32), n_seq, plan.ranges.data_ptr(),
                                  plan.n_ranges, plan.seqs.data_ptr(), plan.n_seqs, _ptr(scratch), n, plan.n_states, T, H, D, _stream()), r.dtype)
    return out


def tied_prep(q, pages, key_scale, y, bias, q_norm, eps, temp, block_table, tok_seq, tok_pos, H, G, dim):
    """Queries [T, H, pad32(dim)] from the projections y [T, >= (H + G) dim] fp32, and their values and key scales into the pages.
    temp: (coefficient, every) of the queries' temperature, or None."""
    n_seq, max_blocks = block_table.shape
    T, ld = y.shape
    coef, every = temp or (0.0, 0.0)
    check(lib_of(q.dtype).mlora_tied_prep(_dev(q), _dev(pages, q.dtype), _dev(key_scale, torch.float32), _dev(y, torch.float32), ld,
                                          _dev(bias, torch.float32), _dev(q_norm, torch.float32), eps, coef, every, _dev(block_table, torch.int32),
                                          max_blocks, _dev(tok_seq, torch.int32), _dev(tok_pos, torch.int32), T, H, G, dim, pages.shape[0], n_seq,
                                          _stream()), q.dtype)


def tied_attn(q, pages, key_scale, block_table, tok_seq, tok_pos, slopes, scale, G, dim, max_ctx, out, splits=None):
    """Causal attention over pages whose values are its keys -> out, an activation [T, H * pad32(dim)]."""
    T, H, _ = q.shape
    n_seq, max_blocks = block_table.shape
    L = lib_of(q.dtype)
    if splits is None:
        splits = L.mlora_tied_attn_splits(T, H, G, max_ctx)
    nb = L.mlora_latent_attn_workspace_bytes(T, H, dim, splits)
    ws = torch.empty(nb // 4, dtype=torch.float32, device=q.device) if nb else None
    frag = isinstance(out, FragActivation)
    check(L.mlora_tied_attn(out.data.data_ptr() if frag else _dev(out, q.dtype), FRAG if frag else ROWMAJOR, _dev(q), _dev(pages, q.dtype),
                            _dev(key_scale, torch.float32), _dev(block_table, torch.int32), max_blocks, _dev(tok_seq, torch.int32),
                            _dev(tok_pos, torch.int32), _dev(slopes, torch.float32), scale, T, H, G, dim, pages.shape[0], n_seq, splits, _ptr(ws), nb,
                            _stream()), q.dtype)
    return out


def tied_prefill_served(dim) -> bool:
    return bool(lib_of(torch.bfloat16).mlora_tied_prefill_served(dim))


def tied_prefill(plan, q, pages, key_scale, slopes, scale, G, dim, out):
    """The same for a pass over prompts (plan: PrefillPlan), with keys and transposed values laid out in scratch memory."""
    T, H, _ = q.shape
    L = lib_of(q.dtype)
    n = L.mlora_tied_prefill_scratch_elems(plan.pages, G, dim)
    scratch = torch.empty(n, dtype=q.dtype, device=q.device)
    frag = isinstance(out, FragActivation)
    check(L.mlora_tied_prefill(out.data.data_ptr() if frag else _dev(out, q.dtype), FRAG if frag else ROWMAJOR, out.shape[1], _dev(q),
                               _dev(pages, q.dtype), _dev(key_scale, torch.float32), plan.phys.data_ptr(), plan.pages, plan.tiles.data_ptr(), plan.n_tiles,
                               _dev(slopes, torch.float32), scale, T, H, G, dim, pages.shape[0], scratch.data_ptr(), n, _stream()), q.dtype)
    return out


def head_linear(x, ldx, head_x, W, heads, T, K, N, out, ldy, head_y, alpha=1.0):
    """out[t, h] = alpha * W[h] x[t, h]: x a tensor with row stride ldx and head stride head_x (elements), W the heads'
    [N, K] matrices stacked, out likewise or a FragActivation [T, heads * head_y]."""
    dt = x.dtype
    frag = isinstance(out, FragActivation)
    check(lib_of(dt).mlora_head_linear(out.data.data_ptr() if frag else out.data_ptr(), FRAG if frag else ROWMAJOR, ldy, head_y, x.data_ptr(),
                                       ldx, head_x, _wptr(W), heads, T, K, N, alpha, _stream()), dt)
    return out


def latent_prep(q, q_off, pages, qkv, off_rot, off_c, off_kr, gain, c_norm, eps, block_table, tok_seq, tok_pos, cos, sin, H, R, rot,
                lift=None):
    """Rotates the query parts of qkv into q [T, H, q_ld] at column q_off and stores latent and key part (c_norm given); lift:
    also lifts the unrotated parts (the first columns of qkv) with these matrices, stacked [H * pad32(R), K per head]."""
    n_seq, max_blocks = block_table.shape
    T, ld = qkv.shape
    check(lib_of(qkv.dtype).mlora_latent_prep(_dev(q, qkv.dtype), q.shape[2], q_off, _dev(pages, qkv.dtype), _dev(qkv), ld, off_rot, off_c, off_kr,
                                              gain, _ptr(c_norm), eps, _dev(block_table, torch.int32), max_blocks, _dev(tok_seq, torch.int32),
                                              _dev(tok_pos, torch.int32), _dev(cos, torch.float32), _dev(sin, torch.float32), cos.shape[0], T, H, R,
                                              rot, pages.shape[0], n_seq, _wptr(lift) if lift is not None else None,
                                              lift.shape[1] if lift is not None else 0, _stream()), qkv.dtype)


class PrefillPlan:
    """Contexts and query tiles of a pass for `latent_prefill`: per sequence (cache pages of its whole context, tokens that
    the pass appends, context length after it), in pass order."""

    def __init__(self, seqs, device):
        L = lib_of(torch.bfloat16)
        n = L.mlora_latent_prefill_tile_tokens()
        phys, tiles, t0 = [], [], 0
        for pages, new, ctx in seqs:
            base = len(phys)
            used = -(-ctx // 16)
            phys += list(pages[:used]) + [-1] * (-used % 4)
            tiles += [(t0 + i, min(n, new - i), base, ctx - new + i) for i in range(0, new, n)]
            t0 += new
        tiles.sort(key=lambda t: -(t[1] + t[3]))                     # the longest key ranges start first
        self.T, self.pages, self.n_tiles = t0, len(phys), len(tiles)
        both = torch.tensor([x for t in tiles for x in t] + phys, dtype=torch.int32).to(device)
        self.tiles, self.phys = both[: 4 * len(tiles)], both[4 * len(tiles):]


def latent_prefill_served(dim, rot, vdim) -> bool:
    return bool(lib_of(torch.bfloat16).mlora_latent_prefill_served(dim, rot, vdim))


def latent_prefill(plan, q, q_rot, pages, uk, uv, sink, scale, R, dim, rot, vdim, out):
    """Attention of a pass over keys and values made from the latents; q [T, ld] (unrotated query parts, each padded to 32
    columns), q_rot [T, H, pad32(rot)]; out: FragActivation or tensor [T, H * pad32(vdim)]."""
    T, H, _ = q_rot.shape
    L = lib_of(q.dtype)
    n = L.mlora_latent_prefill_scratch_elems(plan.pages, H, dim, rot, vdim)
    scratch = torch.empty(n, dtype=q.dtype, device=q.device)
    frag = isinstance(out, FragActivation)
    check(L.mlora_latent_prefill(out.data.data_ptr() if frag else _dev(out, q.dtype), FRAG if frag else ROWMAJOR, out.shape[1], _dev(q), q.shape[1],
                                 _dev(q_rot, q.dtype), _dev(pages, q.dtype), plan.phys.data_ptr(), plan.pages, plan.tiles.data_ptr(), plan.n_tiles,
                                 _wptr(uk), _wptr(uv), _ptr(sink), scale, T, H, R, dim, rot, vdim, pages.shape[0], scratch.data_ptr(), n, _stream()),
          q.dtype)
    return out


def latent_attn_splits(T, H, max_ctx, dtype) -> int:
    """Shares of the context that attention over contexts up to max_ctx is cut into."""
    return lib_of(dtype).mlora_latent_attn_splits(T, H, max_ctx)


def latent_attn_out(q, pages, block_table, tok_seq, tok_pos, sink, scale, R, rot, splits, uv, vp, out):
    """latent_attn over splits > 1 shares of the context, taken through the heads' W_uv (stacked [H * vp, pad32(R)]) into `out`
    (activation [T, H * vp])."""
    T, H, _ = q.shape
    n_seq, max_blocks = block_table.shape
    L = lib_of(q.dtype)
    nb = L.mlora_latent_attn_workspace_bytes(T, H, R, splits)
    ws = torch.empty(nb // 4, dtype=torch.float32, device=q.device)
    frag = isinstance(out, FragActivation)
    check(L.mlora_latent_attn_out(out.data.data_ptr() if frag else _dev(out, q.dtype), FRAG if frag else ROWMAJOR, H * vp, _wptr(uv), vp, _dev(q),
                                  _dev(pages, q.dtype), _dev(block_table, torch.int32), max_blocks, _dev(tok_seq, torch.int32),
                                  _dev(tok_pos, torch.int32), _ptr(sink), scale, T, H, R, rot, pages.shape[0], n_seq, splits, _ptr(ws), nb,
                                  _stream()), q.dtype)
    return out


def latent_attn(q, pages, block_table, tok_seq, tok_pos, sink, scale, R, rot, max_ctx, out=None, splits=None):
    """Causal attention of q [T, H, blocks * 32] over the latent pages -> [T, H, pad32(R)].  max_ctx: the longest context of
    the call (chooses the number of context shares)."""
    T, H, _ = q.shape
    n_seq, max_blocks = block_table.shape
    L = lib_of(q.dtype)
    if splits is None:
        splits = L.mlora_latent_attn_splits(T, H, max_ctx)
    out = torch.empty((T, H, pad32(R)), dtype=q.dtype, device=q.device) if out is None else out
    nb = L.mlora_latent_attn_workspace_bytes(T, H, R, splits)
    ws = torch.empty(nb // 4, dtype=torch.float32, device=q.device) if nb else None
    check(L.mlora_latent_attn(_dev(out), _dev(q), _dev(pages, q.dtype), _dev(block_table, torch.int32), max_blocks, _dev(tok_seq, torch.int32),
                              _dev(tok_pos, torch.int32), _ptr(sink), scale, T, H, R, rot, pages.shape[0], n_seq, splits, _ptr(ws), nb, _stream()),
          q.dtype)
    return out


def moe_route(logits, bias, scale, top, dtype):
    """logits [T, >= E] fp32, bias [E] fp32 -> (pick [T, top] int32, weight [T, top] fp32)."""
    T, ld = logits.shape
    E = bias.shape[0]
    pick = torch.empty((T, top), dtype=torch.int32, device=logits.device)
    w = torch.empty((T, top), dtype=torch.float32, device=logits.device)
    check(lib_of(dtype).mlora_moe_route(_dev(pick), _dev(w), _dev(logits, torch.float32), ld, _dev(bias, torch.float32), scale, T, E, top, _stream()),
          dtype)
    return pick, w


class MoePlan:
    """The (token, choice) entries of a routing sorted by expert into places and cut into tiles."""

    def __init__(self, pick, E, dtype):
        self._sizes(*pick.shape, E, dtype)
        self.perm, self.tiles, self.n_tiles = self._room(1, pick.device)
        check(lib_of(dtype).mlora_moe_plan(self.perm.data_ptr(), self.tiles.data_ptr(), self.n_tiles.data_ptr(), _dev(pick, torch.int32), self.T, E,
                                           self.top, _stream()), dtype)

    def _sizes(self, T, top, E, dtype):
        L = lib_of(dtype)
        self.T, self.top = T, top
        self.tile_rows = L.mlora_moe_tile_rows(T, E, top)
        self.max_tiles = L.mlora_moe_max_tiles(T, E, top)
        self.places = L.mlora_moe_max_places(T, E, top)

    def _room(self, layers, dev):
        return tuple(torch.empty(layers * n, dtype=torch.int32, device=dev) for n in (self.places, 4 * self.max_tiles, 2))

    @classmethod
    def of_tables(cls, tables, ids, E, dtype):
        """Plans of all layers whose experts are looked up by token id (tables [layers, V, top] int32) in one launch."""
        n, V, top = tables.shape
        T = ids.numel()
        plans = [cls.__new__(cls) for _ in range(n)]
        for p in plans:
            p._sizes(T, top, E, dtype)
        room = plans[0]._room(n, ids.device)
        check(lib_of(dtype).mlora_moe_table_plan(*(r.data_ptr() for r in room), _dev(tables, torch.int32), _dev(ids, torch.int32), n, V, T, E, top,
                                                 _stream()), dtype)
        for p, perm, tiles, n_tiles in zip(plans, *(r.view(n, -1) for r in room)):
            p.perm, p.tiles, p.n_tiles = perm, tiles, n_tiles
        return plans


def moe_linear(x, W, plan, N, K, stage, act=ACT_NONE, alpha=1.0):
    """Expert linears over a plan: stage MOE_UP: x [T, K] token rows -> places (rows [places, N], or those in fragment order
    where the plan's tiles are large); MOE_DOWN: places -> entry rows [T * top, N].  W: the experts' [N, K] matrices stacked."""
    up = stage == MOE_UP
    y = torch.empty((plan.places if up else plan.T * plan.top, N), dtype=x.dtype, device=x.device)
    ws = torch.empty(plan.places * K, dtype=x.dtype, device=x.device) if up and plan.tile_rows == 256 else None
    check(lib_of(x.dtype).mlora_moe_linear(_dev(y), _dev(x), _wptr(W), plan.perm.data_ptr(), plan.tiles.data_ptr(), plan.n_tiles.data_ptr(),
                                           plan.tile_rows, plan.max_tiles, plan.places, plan.T, K, N, plan.top, stage, act, alpha, _ptr(ws),
                                           ws.numel() if ws is not None else 0, _stream()), x.dtype)
    return y


def moe_combine(x, y, w, parts=None, out=None):
    """x [T, N] fp32 += pending partials, then the sum over the choices of w * y (entry rows); out (FragActivation): the result
    rounded to the element type."""
    T, top = w.shape
    check(lib_of(y.dtype).mlora_moe_combine(_dev(x, torch.float32), *_parts(parts), _dev(y), _dev(w, torch.float32), T, top, x.shape[1],
                                            out.data.data_ptr() if out is not None else None, _stream()), y.dtype)
