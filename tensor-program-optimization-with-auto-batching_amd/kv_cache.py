"""Paged caches: host-side page bookkeeping around the HIP attention kernels.

Keeps the host protocol of the reference's cache object
(`tvm/llama_auto_batcher/llama_exec_graph.py:41-46,66,75-79,85,121-127`):
    add_sequence(sid) ; begin_forward(seq_ids, append_lens) ; attention_with_fused_qkv(layer, qkv, n_q_heads) ;
    end_forward()
with RoPE applied inside the cache operator (`llama_for_causal_lm.py:148-174`: rotary_dim = head_dim,
scale 1, no sliding window).  Keys are stored already rotated, which is equivalent to rotating them at
read time and saves the per-step re-rotation of the whole context.

A finished sequence gives its pages and its slot back with free_sequence(sid).

Device layout of PagedKVCache per layer: k [n_pages, Hkv, 16, D], v [n_pages, Hkv, D, 16] (fp16), one int32 block table
[max_seqs, max_blocks], fp32 RoPE tables [max_pos, D/2].
"""
from __future__ import annotations

import numpy as np
import torch

from . import ops
from .decoder_ops import PrefillPlan, TimeMixPlan

PAGE = 16


def rope_tables(head_dim: int, theta: float, max_pos: int):
    """cos/sin [max_pos, head_dim/2] float32 (float64 math, rounded once)."""
    inv_freq = theta ** (-(np.arange(0, head_dim, 2, dtype=np.float64) / head_dim))
    ang = np.arange(max_pos, dtype=np.float64)[:, None] * inv_freq[None, :]
    return np.cos(ang).astype(np.float32), np.sin(ang).astype(np.float32)


class PageTable:
    """The host side of a paged cache: which pages of the pool belong to which sequence, and the protocol of a forward
    pass.  What lies in a page is up to the subclass."""

    def __init__(self, n_pages, max_seqs, max_blocks, max_pos, device, free_pages=None, page_size=PAGE):
        if page_size != PAGE:
            raise ValueError(f"page_size must be {PAGE}")
        self.n_pages, self.max_seqs, self.max_blocks, self.max_pos = n_pages, max_seqs, max_blocks, max_pos
        self.device = torch.device(device)
        self.free = list(range(n_pages)) if free_pages is None else [int(p) for p in free_pages]
        if sorted(self.free) != list(range(n_pages)):
            raise ValueError("free_pages must be a permutation of range(n_pages)")
        # host mirrors (integer bookkeeping is host logic, as in the reference's runtime)
        self.table_h = np.full((max_seqs, max_blocks), -1, dtype=np.int32)
        self.lens = {}          # sid -> committed length
        self.slot = {}          # sid -> row of the block table
        self.free_slots = list(range(max_seqs))
        self.block_table = torch.from_numpy(self.table_h.copy()).to(self.device)
        self._dirty = False
        self._cur = None

    # ------------------------------------------------------------------ protocol
    def add_sequence(self, sid):
        if sid in self.slot:
            raise ValueError(f"sequence with id {sid} has already been added")
        if not self.free_slots:
            raise RuntimeError("paged KV cache: no sequence slot left")
        self.slot[sid] = self.free_slots.pop(0)
        self.lens[sid] = 0

    def free_sequence(self, sid):
        """Give back the pages and the slot of a finished sequence."""
        if self._cur is not None:
            raise RuntimeError("free_sequence between begin_forward and end_forward")
        row = self.slot.pop(sid)
        del self.lens[sid]
        self.free.extend(int(p) for p in self.table_h[row] if p >= 0)
        self.table_h[row] = -1
        self.free_slots.insert(0, row)
        self._dirty = True

    def begin_forward(self, seq_ids, append_lens, device_meta=None):
        """Reserve pages for the appended tokens and stage the per-token (sequence, position) arrays."""
        if self._cur is not None:
            raise RuntimeError("begin_forward called twice without end_forward")
        if len(seq_ids) != len(append_lens):
            raise ValueError("seq_ids and append_lens differ in length")
        for sid, n in zip(seq_ids, append_lens):
            row = self.slot[sid]
            new_len = self.lens[sid] + n
            if new_len > self.max_pos or -(-new_len // PAGE) > self.max_blocks:
                raise RuntimeError(f"sequence {sid}: length {new_len} exceeds the cache geometry")
            have = int((self.table_h[row] >= 0).sum())
            need = -(-new_len // PAGE)
            for j in range(have, need):
                if not self.free:
                    raise RuntimeError("paged KV cache out of pages")
                self.table_h[row, j] = self.free.pop(0)
                self._dirty = True
        if self._dirty:
            self.block_table.copy_(torch.from_numpy(self.table_h), non_blocking=False)
            self._dirty = False
        decode = all(n == 1 for n in append_lens)
        rows = np.asarray([self.slot[s] for s in seq_ids], dtype=np.int32)
        base = np.asarray([self.lens[s] for s in seq_ids], dtype=np.int32)
        if device_meta is not None:
            tok_seq, tok_pos, ctx = device_meta
        elif decode:
            tok_seq = torch.from_numpy(rows).to(self.device)
            tok_pos = torch.from_numpy(base).to(self.device)
            ctx = torch.from_numpy(base + 1).to(self.device)
        else:
            ts = np.repeat(rows, append_lens).astype(np.int32)
            tp = np.concatenate([b + np.arange(n, dtype=np.int32) for b, n in zip(base, append_lens)]).astype(np.int32)
            tok_seq = torch.from_numpy(ts).to(self.device)
            tok_pos = torch.from_numpy(tp).to(self.device)
            ctx = None
        self._cur = (list(seq_ids), list(append_lens), decode, tok_seq, tok_pos, ctx)

    def end_forward(self):
        seq_ids, append_lens = self._cur[0], self._cur[1]
        for sid, n in zip(seq_ids, append_lens):
            self.lens[sid] += n
        self._cur = None

    # ------------------------------------------------------------------ helpers
    def pages_of(self, sid):
        row = self.table_h[self.slot[sid]]
        return row[row >= 0].tolist()


class PagedKVCache(PageTable):
    def __init__(self, n_layers, n_pages, n_kv_heads, head_dim, max_seqs, max_blocks, rope_theta, max_pos,
                 device="cuda:0", free_pages=None, page_size=PAGE):
        super().__init__(n_pages, max_seqs, max_blocks, max_pos, device, free_pages, page_size)
        self.n_layers, self.Hkv, self.D = n_layers, n_kv_heads, head_dim
        if head_dim % 32:
            raise ValueError("head_dim must be a multiple of 32")
        # keys in matrix-core fragment order: element (token, d) of a page at [d // 32, (d % 32) // 8, token, d % 8]
        self.k = torch.zeros((n_layers, n_pages, n_kv_heads, head_dim // 32, 4, PAGE, 8), dtype=torch.float16, device=self.device)
        self.v = torch.zeros((n_layers, n_pages, n_kv_heads, head_dim, PAGE), dtype=torch.float16, device=self.device)
        cos, sin = rope_tables(head_dim, rope_theta, max_pos)
        self.rope_cos = torch.from_numpy(cos).to(self.device)
        self.rope_sin = torch.from_numpy(sin).to(self.device)

    def k_rowmajor(self, layer: int) -> torch.Tensor:
        """The layer's rotated keys as [n_pages, Hkv, 16, D] (a copy, for inspection)."""
        k = self.k[layer]
        return k.permute(0, 1, 4, 2, 3, 5).reshape(self.n_pages, self.Hkv, PAGE, self.D).contiguous()

    def attention_with_fused_qkv(self, layer, qkv, n_q_heads, out=None, frag=False, o_shrink=None):
        """qkv [T, Hq + 2 Hkv, D] (or [T, (Hq + 2 Hkv) * D]) fp16, token-major in begin_forward order.
        Rotates q in place, appends rotated k and v, attends causally; returns [T, Hq * D] fp16
        (frag=True: as a FragActivation ready for the o_proj product).  o_shrink (a decode step only): see
        ops.paged_attn_decode - the call then returns (attention output, head shares of the o projection's shrink)."""
        if self._cur is None:
            raise RuntimeError("attention_with_fused_qkv outside begin_forward/end_forward")
        _, append_lens, decode, tok_seq, tok_pos, ctx = self._cur
        T = sum(append_lens)
        qkv = qkv.view(T, n_q_heads + 2 * self.Hkv, self.D)
        ops.rope_kv_append(qkv, self.k[layer], self.v[layer], self.block_table, tok_seq, tok_pos,
                           self.rope_cos, self.rope_sin, n_q_heads, self.Hkv, self.D)
        if decode:
            return ops.paged_attn_decode(qkv, self.k[layer], self.v[layer], self.block_table, tok_seq, ctx,
                                         n_q_heads, self.Hkv, self.D, out=out, frag=frag, o_shrink=o_shrink)
        if o_shrink is not None:
            raise ValueError("attention_with_fused_qkv: o_shrink is for decode steps")
        return ops.paged_attn_prefill(qkv, self.k[layer], self.v[layer], self.block_table, tok_seq, tok_pos,
                                      n_q_heads, self.Hkv, self.D, out=out, frag=frag)

    def kv_bytes_read_per_step(self, seq_ids):
        """Algorithmic K+V bytes one decode step reads for these sequences, all layers."""
        per_pos = self.n_layers * 2 * self.Hkv * self.D * 2
        return int(sum(self.lens[s] + 1 for s in seq_ids)) * per_pos


class PagedLatentCache(PageTable):
    """Pages of latent attention: per layer one vector per token, the normed latent and the rotated key part, in the page
    layout of latent_attention.hip.  A layer may read another layer's pages instead of having its own."""

    def __init__(self, layers, n_pages, max_seqs, max_blocks, max_pos, dtype, device="cuda:0", free_pages=None, page_size=PAGE):
        """layers: per layer (kv_rank, rot_dim, rotation, owner): owner is the layer whose pages this one reads (itself,
        if it has its own); rotation: rotary.Rotation."""
        super().__init__(n_pages, max_seqs, max_blocks, max_pos, device, free_pages, page_size)
        self.dtype = dtype
        self.owner = [o for *_, o in layers]
        self.pages = []
        self.rope = []
        tables = {}
        for l, (rank, rot_dim, rotation, o) in enumerate(layers):
            blocks = -(-rank // 32) + -(-rot_dim // 32)
            # padding between and behind the two parts is read by the matrix cores: it stays zero
            self.pages.append(torch.zeros((n_pages, blocks, 4, PAGE, 8), dtype=dtype, device=self.device) if o == l else self.pages[o])
            key = (rotation, rot_dim)
            if key not in tables:
                tables[key] = tuple(torch.from_numpy(t).to(self.device) for t in rotation.tables(rot_dim, max_pos))
            self.rope.append(tables[key])
        self._plan = None

    def latents(self, layer, sid):
        """The cached vectors [length, blocks * 32] of a sequence (a copy, for inspection)."""
        n = self.lens[sid]
        p = self.pages[layer][torch.tensor(self.pages_of(sid), device=self.device, dtype=torch.int64)]
        return p.permute(0, 3, 1, 2, 4).reshape(-1, p.shape[1] * 32)[:n].contiguous()

    def latent_attention(self, layer, qkv, att, out=None):
        """The mixer of `layer` behind its input projection: qkv [T, att.proj_rows] in begin_forward order (att:
        latent_attention.LatentAttention) -> the heads' outputs, concatenated (`out`: an activation of att.out_cols
        columns)."""
        if self._cur is None:
            raise RuntimeError("latent_attention outside begin_forward/end_forward")
        seq_ids, append_lens, decode, tok_seq, tok_pos, _ = self._cur
        ctx = [self.lens[s] + n for s, n in zip(seq_ids, append_lens)]
        plan = None
        if not decode and att.prompt_form_pays(list(zip(append_lens, ctx))):
            if self._plan is None or self._plan[0] is not self._cur:         # one plan per pass serves all its layers
                self._plan = (self._cur, PrefillPlan([(self.pages_of(s), n, c) for s, n, c in zip(seq_ids, append_lens, ctx)], self.device))
            plan = self._plan[1]
        return att.attend(qkv, self.pages[layer], self.block_table, tok_seq, tok_pos, *self.rope[layer], max_ctx=max(ctx),
                          store=self.owner[layer] == layer, plan=plan, out=out)


class PagedStateCache(PageTable):
    """What the layers of a model with recurrent and attention layers keep per sequence, one entry per layer run (a layer that
    runs several times has one for every pass): pages of tied attention, or a state per slot.  A slot needs no clearing:
    kernels start a sequence's state from zero at its position 0."""

    def __init__(self, runs, width_p, n_pages, max_seqs, max_blocks, max_pos, dtype, device="cuda:0", free_pages=None, page_size=PAGE):
        """runs: per layer run the mixer's spec, whose cache_entry says what is kept; width_p: columns of the residual stream."""
        super().__init__(n_pages, max_seqs, max_blocks, max_pos, device, free_pages, page_size)
        self.dtype = dtype
        self.entries = [tuple(torch.zeros(shape, dtype=dtype if elements else torch.float32, device=self.device)
                              for shape, elements in s.cache_entry(n_pages, max_seqs, PAGE, width_p)) for s in runs]
        self._meta = None

    def values(self, run, sid):
        """The cached values [length, G, columns] of a sequence (a copy, for inspection)."""
        p = self.entries[run][0][torch.tensor(self.pages_of(sid), device=self.device, dtype=torch.int64)]
        return p.permute(0, 4, 1, 2, 3, 5).reshape(-1, p.shape[1], p.shape[2] * 32)[: self.lens[sid]].contiguous()

    def state(self, run, sid):
        """The matrix states [H, D, D] of a sequence (a view)."""
        return self.entries[run][0][self.slot[sid]]

    def shift(self, run):
        """The previous tokens' rows [slots, columns] of a recurrent layer run."""
        return self.entries[run][1]

    def _pass(self):
        """Of the current pass, made once for all its layers: {"last": the last token of every token's sequence, "segs": [n][4]
        {slot, first token, tokens, position}} - both None in a decode step - and the plans of the prompt forms, once taken."""
        if self._cur is None:
            raise RuntimeError("outside begin_forward/end_forward")
        if self._meta is None or self._meta[0] is not self._cur:
            seq_ids, lens, decode = self._cur[:3]
            m = {"last": None, "segs": None, "plan": None, "ranges": {}, "host": None}
            if not decode:
                ends = np.cumsum(lens)
                m["host"] = segs = [(self.slot[s], int(e) - n, n, self.lens[s]) for s, n, e in zip(seq_ids, lens, ends)]
                both = np.concatenate([np.asarray(segs, dtype=np.int32).reshape(-1), np.repeat(ends - 1, lens).astype(np.int32)])
                both = torch.from_numpy(both).to(self.device)
                m["segs"], m["last"] = both[: 4 * len(segs)].view(-1, 4), both[4 * len(segs):]
            self._meta = (self._cur, m)
        return self._meta[1]

    def token_meta(self):
        """(sequence, position, last token of its sequence in the pass) per token."""
        return self._cur[3], self._cur[4], self._pass()["last"]

    def time_mix(self, run, mixes, mixer):
        """The recurrence of a layer run on the five mixes of the pass (mixer: time_mix.TimeMix)."""
        m, plan, heads = self._pass(), None, mixer.spec.heads
        if m["host"] is not None and mixer.prompt_form:
            if heads not in m["ranges"]:
                m["ranges"][heads] = TimeMixPlan(m["host"], heads, self.device)
            plan = m["ranges"][heads]
        return mixer.run(mixes, self.entries[run][0], m["segs"], self._cur[3], self._cur[4], plan)

    def tied_attention(self, run, y, att):
        """The attention of a layer run behind its input projection y (att: tied_attention.TiedAttention)."""
        m = self._pass()
        seq_ids, append_lens, decode, tok_seq, tok_pos, _ = self._cur
        seqs = [(n, self.lens[s] + n) for s, n in zip(seq_ids, append_lens)]
        plan = None
        if not decode and att.prompt_form_pays(seqs):
            if m["plan"] is None:
                m["plan"] = PrefillPlan([(self.pages_of(s), n, c) for s, (n, c) in zip(seq_ids, seqs)], self.device)
            plan = m["plan"]
        return att.attend(y, *self.entries[run], self.block_table, tok_seq, tok_pos, max_ctx=max(c for _, c in seqs), plan=plan)
