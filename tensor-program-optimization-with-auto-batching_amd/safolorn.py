"""Safolorn: a decoder-only model of latent-attention layers whose mixer and feed-forward both read the same residual
stream (parallel block, one-number norms), with a per-token input of its own in every layer.

    x <- x + mixer(norm1 x) + ff(norm2 x)
    x <- x + rms_norm(proj(gelu(gate x) * side_embed[token, layer]))

Both norms of a layer divide by the same root mean square and differ in one number, so a layer norms once; the numbers are
applied behind the projections, in fp32.  With a dense feed-forward the two output projections are one matrix over
[attention | hidden].  The residual stream, norms, softmax, router and rotation are fp32; projections and stored
activations have the model's element type (bfloat16, or float32 throughout).
"""
from __future__ import annotations

import dataclasses
from typing import Optional, Tuple

import torch

from . import decoder_ops as D
from . import ops
from .decoder_ops import pad32, pad64, padded
from .feed_forward import ClippedGlu, ClippedGluSpec, MoeRelu2, MoeSpec
from .kv_cache import PagedLatentCache
from .latent_attention import LatentAttention, LatentSpec
from .model_base import CausalLM


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: LatentSpec
    ff: Optional[object]       # ClippedGluSpec, MoeSpec or None


@dataclasses.dataclass(frozen=True)
class SafolornConfig:
    vocab: int
    width: int
    eps: float
    side_dim: int              # width of the per-layer token input, 0 = none
    layers: Tuple[LayerSpec, ...]

    @classmethod
    def from_dict(cls, c: dict) -> "SafolornConfig":
        layers = []
        for i, L in enumerate(c["layers"]):
            if L["type"] != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer {L['type']!r}")
            mlp, ff = L.get("mlp"), None
            if mlp is not None:
                if mlp["kind"] == "dense":
                    ff = ClippedGluSpec(int(mlp["ff"]), float(mlp["limit"]))
                elif mlp["kind"] == "moe":
                    ff = MoeSpec(int(mlp["expert"]["ff"]), int(mlp["router"]["experts"]), int(mlp["router"]["top"]))
                else:
                    raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            mixer = LatentSpec.from_config(L["mixer"])
            if mixer.kv_from is not None and not (0 <= mixer.kv_from < i and layers[mixer.kv_from].mixer.kv_from is None):
                raise ValueError(f"layer {i}: kv_from {mixer.kv_from} is not an earlier layer with latents of its own")
            layers.append(LayerSpec(mixer, ff))
        side = c.get("token_side")
        return cls(int(c["vocab"]), int(c["width"]), float(c["norm"]["eps"]), int(side["dim"]) if side else 0, tuple(layers))


@dataclasses.dataclass
class TokenHidden:
    """Residual stream of a pass with the token ids that its layers look up."""
    x: torch.Tensor            # [T, pad64(width)] fp32
    ids: torch.Tensor          # [T] int32

    @property
    def shape(self):
        return self.x.shape


class SafolornForCausalLM(CausalLM):
    dtypes = ("bfloat16", "float32")

    def __init__(self, config: SafolornConfig, dtype=torch.bfloat16, device="cuda:0"):
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        self.layers = []
        self.width_p = pad64(config.width)
        self.embed_tokens = self.side_embed = self.head = None
        self.final_gain = 1.0

    # ------------------------------------------------------------------ weights
    @classmethod
    def from_weights(cls, config: dict, tensors, dtype=torch.bfloat16, device="cuda:0"):
        """config: the parsed config.json; tensors(name) -> tensor."""
        m = cls(SafolornConfig.from_dict(config), dtype, device)
        for l in range(len(m.config.layers)):
            m.load_layer(l, tensors)
        m.load_head(tensors)
        return m

    def load_layer(self, l: int, tensors):
        assert l == len(self.layers), "layers must be loaded in order"
        c, spec, n, dev, dt = self.config, self.config.layers[l], f"l{l}.", self.device, self.dtype
        names = {"q": "q", "uk": "uk", "uv": "uv", "sink": "sink", "o": "o"}
        if spec.mixer.kv_from is None:
            names.update(dkv="dkv", dkv_norm="dkv.norm")
        att = LatentAttention(spec.mixer, {k: tensors(f"{n}mix.{v}") for k, v in names.items()}, c.width, float(tensors(n + "norm1")), c.eps, dt, dev)
        L = {"att": att, "dense": None, "moe": None}
        out = att.o_rows
        if isinstance(spec.ff, ClippedGluSpec):
            w = {k: tensors(f"{n}mlp.{k}") for k in ("gate", "up", "down")}
            L["dense"] = ff = ClippedGlu(spec.ff, w, c.width, float(tensors(n + "norm2")), dt, dev)
            out = torch.cat([out, ff.down_rows], 1)
            del ff.down_rows
        elif isinstance(spec.ff, MoeSpec):
            e = range(spec.ff.experts)
            w = {"router": tensors(n + "mlp.router"), "router_b": tensors(n + "mlp.router.b"),
                 "up": [tensors(f"{n}mlp.e{i}.up") for i in e], "down": [tensors(f"{n}mlp.e{i}.down") for i in e]}
            L["moe"] = MoeRelu2(spec.ff, w, c.width, float(tensors(n + "norm2")), dt, dev)
        L["out"] = D.weight(out)
        del att.o_rows
        if c.side_dim:
            sp = pad32(c.side_dim)
            L["side_gate"] = D.weight(padded(tensors(n + "side.gate").to(dev, dt), sp, self.width_p))
            L["side_proj"] = D.weight(padded(tensors(n + "side.proj").to(dev, dt), self.width_p, sp))
            L["side_norm"] = padded(tensors(n + "side.norm").to(dev, dt), self.width_p).contiguous()
        self.layers.append(L)

    def load_head(self, tensors):
        c, dev, dt = self.config, self.device, self.dtype
        self.embed_tokens = padded(tensors("embed").to(dev, dt), c.vocab, self.width_p).contiguous()
        if c.side_dim:
            self.side_embed = tensors("side.embed").to(dev, dt).contiguous()
        self.head = D.weight(padded(tensors("head").to(dev, dt), -(-c.vocab // 16) * 16, self.width_p))
        self.final_gain = float(tensors("final.norm"))

    # ------------------------------------------------------------------ cache
    def create_paged_kv_cache(self, max_batch_size, max_total_seq_len, prefill_chunk_size, page_size, free_pages=None, max_seq_len=None):
        n_pages, max_blocks = self._cache_geometry(max_batch_size, max_total_seq_len, page_size, free_pages, max_seq_len)
        layers = [(L.mixer.kv_rank, L.mixer.rot_dim, L.mixer.rotation, l if L.mixer.kv_from is None else L.mixer.kv_from)
                  for l, L in enumerate(self.config.layers)]
        return PagedLatentCache(layers, n_pages, max_seqs=max_batch_size, max_blocks=max_blocks, max_pos=max_blocks * page_size,
                                dtype=self.dtype, device=self.device, free_pages=free_pages, page_size=page_size)

    # ------------------------------------------------------------------ forward
    def embed(self, input_ids: torch.Tensor) -> TokenHidden:
        ids = input_ids.reshape(-1).to(self.device, torch.int32).contiguous()
        return TokenHidden(ops.embed(self.embed_tokens, ids, out_dtype=torch.float32), ids)

    def _norm(self, x, parts=None, branch=None, gain=1.0, row=False):
        """-> (normed activation, the same row-major if asked for); adds what is pending to x."""
        frag = None if self.dtype == torch.float32 else ops.FragActivation(*x.shape, x.device, dtype=self.dtype)
        rows = torch.empty(x.shape, dtype=self.dtype, device=x.device) if row or frag is None else None
        D.stream_norm(x, self.config.width, self.config.eps, gain, parts, branch, out=frag, out_row=rows)
        return (rows if frag is None else frag), rows

    def _add_linear(self, a, W, x, split):
        """x += a @ W.T; returns K-split partials still to be added, or None."""
        if not split or not isinstance(a, ops.FragActivation):
            ops.linear(a, W, out=x, accumulate=True)
            return None
        return ops.linear_acc_ksplit(a, W, x, torch.empty(3 * x.numel(), dtype=torch.float32, device=x.device))

    def forward(self, hidden: TokenHidden, kv, tok_adapter=None, logits_rows=None, layer_outputs=None):
        """Tokens in kv.begin_forward order -> logits fp32 of all tokens or of `logits_rows` (hidden is updated in place).
        layer_outputs: a list that receives the residual stream after every layer."""
        if tok_adapter:
            raise ValueError("Safolorn has no adapters")
        x, ids = hidden.x, hidden.ids
        T, c, dev = x.shape[0], self.config, x.device
        split = T <= 256 or bool(kv._cur[2])          # short passes and decode steps split K of the narrow output projections
        frag = self.dtype != torch.float32
        parts = branch = None
        for l, L in enumerate(self.layers):
            att, dense, moe = L["att"], L["dense"], L["moe"]
            n, n_row = self._norm(x, parts, branch, row=moe is not None)
            parts = branch = None
            qkv = ops.linear(n, att.proj)
            if dense is not None:
                cat = D.activation(T, att.out_cols + dense.ffp, self.dtype, dev)
                if frag:
                    kv.latent_attention(l, qkv, att, out=cat.columns(0, att.out_cols))
                    dense.hidden(n, cat.columns(att.out_cols, dense.ffp))
                else:
                    cat[:, : att.out_cols] = kv.latent_attention(l, qkv, att)
                    cat[:, att.out_cols:] = dense.hidden(n, torch.empty((T, dense.ffp), dtype=self.dtype, device=dev))
            else:
                cat = kv.latent_attention(l, qkv, att)
            parts = self._add_linear(cat, L["out"], x, split)
            xa = ops.FragActivation(*x.shape, dev, dtype=self.dtype) if frag and c.side_dim else None
            if moe is not None:
                moe.add_to(x, n, n_row, parts, xa)
                parts = None
            elif xa is not None:
                D.stream_norm(x, c.width, c.eps, parts=parts, out=xa, raw=True)
                parts = None
            if c.side_dim:
                g = D.token_gate(xa if frag else x, L["side_gate"], self.side_embed, l * c.side_dim, c.side_dim, ids)
                branch = (ops.linear(g, L["side_proj"], out_dtype=torch.float32), L["side_norm"])
            if layer_outputs is not None:
                D.stream_norm(x, c.width, c.eps, parts=parts, branch=branch)
                parts = branch = None
                layer_outputs.append(x[:, : c.width].clone())
        if logits_rows is not None:
            if parts is not None or branch is not None:
                D.stream_norm(x, c.width, c.eps, parts=parts, branch=branch)
                parts = branch = None
            x = x[logits_rows].contiguous()
            if x.shape[0] == 0:
                return torch.empty((0, c.vocab), dtype=torch.float32, device=dev)
        n, _ = self._norm(x, parts, branch, gain=self.final_gain)
        logits = ops.linear(n, self.head, out_dtype=torch.float32)
        return logits if logits.shape[1] == c.vocab else logits[:, : c.vocab].contiguous()
