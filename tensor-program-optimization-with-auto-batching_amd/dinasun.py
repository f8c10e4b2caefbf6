"""Dinasun: a decoder-only model of time-mixing and tied-attention layers with experts by token id, part of whose layers
run several times over.

    x <- x + m norm1b(mixer(norm1 x));   x <- x + m norm2b(ff(norm2 x));   norm: tanh(alpha v) w + b

The norms need no statistics, so every sublayer is bounded by one elementwise launch on the fp32 residual stream (which also mixes
neighbouring tokens for the time mixing).  Layers start .. stop - 1 run `times` times with the same weights and a cache or
state of their own per pass; ahead of each pass x <- W_in [x; x0] with the embedding output x0.
"""
from __future__ import annotations

import dataclasses
from typing import Optional, Tuple

import torch

from . import decoder_ops as D
from . import ops
from .decoder_ops import ElementwiseNorm, pad64, padded
from .feed_forward import TableMoe, TableMoeSpec, TableRouting
from .kv_cache import PagedStateCache
from .model_base import CausalLM
from .tied_attention import TiedAttention, TiedSpec
from .time_mix import MIXES, TimeMix, TimeMixSpec


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    mixer: object              # TiedSpec or TimeMixSpec
    ff: Optional[TableMoeSpec]


@dataclasses.dataclass(frozen=True)
class DinasunConfig:
    vocab: int
    width: int
    eps: float
    embed_scale: float
    residual_mult: float
    layers: Tuple[LayerSpec, ...]
    loop: Optional[Tuple[int, int, int]] = None      # (start, stop, times)

    @classmethod
    def from_dict(cls, c: dict) -> "DinasunConfig":
        layers = []
        for i, L in enumerate(c["layers"]):
            kinds = {"attention": TiedSpec, "wkv": TimeMixSpec}
            if L["type"] not in kinds:
                raise ValueError(f"layer {i}: unknown mixer {L['type']!r}")
            mlp = L.get("mlp")
            if mlp is not None and mlp["kind"] != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            layers.append(LayerSpec(kinds[L["type"]].from_config(L["mixer"]), TableMoeSpec.from_config(mlp) if mlp is not None else None))
        loop = c.get("loop")
        if loop is not None:
            loop = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
            if not (0 <= loop[0] < loop[1] <= len(layers) and loop[2] >= 1):
                raise ValueError(f"loop {loop} over {len(layers)} layers")
        return cls(int(c["vocab"]), int(c["width"]), float(c["norm"]["eps"]), float(c["embedding"]["scale"]), float(c["residual_mult"]),
                   tuple(layers), loop)

    def runs(self):
        """(layer, whether a pass of the loop starts ahead of it) in the order in which layers run."""
        n = len(self.layers)
        start, stop, times = self.loop or (n, n, 0)
        return [(l, False) for l in range(start)] + [(l, l == start) for _ in range(times) for l in range(start, stop)] + \
            [(l, False) for l in range(stop, n)]


@dataclasses.dataclass
class LoopHidden:
    """Residual stream of a pass with what its layers come back to: the token ids, and the loop's input [x; x0]."""
    x: torch.Tensor            # [T, pad64(width)] fp32
    ids: torch.Tensor          # [T] int32
    entry: object              # activation [T, 2 pad64(width)], its second half set; None without a loop

    @property
    def shape(self):
        return self.x.shape


class DinasunForCausalLM(CausalLM):
    dtypes = ("bfloat16", "float32")

    def __init__(self, config: DinasunConfig, dtype=torch.bfloat16, device="cuda:0"):
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        self.width_p = pad64(config.width)
        self.runs = config.runs()
        self.layers = []
        self.embed_tokens = self.head = self.final_norm = self.loop_in = self.routing = None

    # ------------------------------------------------------------------ weights
    @classmethod
    def from_weights(cls, config: dict, tensors, dtype=torch.bfloat16, device="cuda:0"):
        """config: the parsed config.json; tensors(name) -> tensor."""
        m = cls(DinasunConfig.from_dict(config), dtype, device)
        for l in range(len(m.config.layers)):
            m.load_layer(l, tensors)
        m.load_head(tensors)
        return m

    def _norm(self, tensors, name):
        return ElementwiseNorm(tensors(name), tensors(name + ".b"), tensors(name + ".alpha"), self.width_p, self.dtype, self.device)

    def load_layer(self, l: int, tensors):
        assert l == len(self.layers), "layers must be loaded in order"
        c, spec, n = self.config, self.config.layers[l], f"l{l}."
        mix = lambda names: {k: tensors(f"{n}mix.{v}") for k, v in names.items()}
        if isinstance(spec.mixer, TimeMixSpec):
            names = ["r", "k", "v", "g", "w1", "w2", "w0", "u", "norm", "o"] + ["mu." + s for s in MIXES]
            mixer = TimeMix(spec.mixer, mix({k: k for k in names}), c.width, c.eps, self.dtype, self.device)
        else:
            names = {"q": "q", "q_b": "q.b", "k": "k", "k_b": "k.b", "q_norm": "q.norm", "k_norm": "k.norm", "o": "o"}
            mixer = TiedAttention(spec.mixer, mix(names), c.width, c.eps, self.dtype, self.device)
        L = {"mixer": mixer, "moe": None, "norm1": self._norm(tensors, n + "norm1"), "norm1b": self._norm(tensors, n + "norm1b")}
        if spec.ff is not None:
            three = ("gate", "up", "down")
            w = {k: [tensors(f"{n}mlp.e{e}.{k}") for e in range(spec.ff.experts)] for k in three}
            w["table"] = tensors(n + "mlp.table")
            if spec.ff.shared:
                w["shared"] = {k: tensors(f"{n}mlp.shared.{k}") for k in three}
            L["moe"] = TableMoe(spec.ff, w, c.width, self.dtype, self.device)
            L.update(norm2=self._norm(tensors, n + "norm2"), norm2b=self._norm(tensors, n + "norm2b"))
        self.layers.append(L)

    def load_head(self, tensors):
        c, dev, dt, Hp = self.config, self.device, self.dtype, self.width_p
        embed = tensors("embed").to(dev, dt)
        self.embed_tokens = padded(embed, c.vocab, Hp).contiguous()
        self.head = D.weight(padded(embed, -(-c.vocab // 16) * 16, Hp))
        self.final_norm = self._norm(tensors, "final.norm")
        if c.loop is not None:
            w = tensors("loop.in").to(dev, dt).view(c.width, 2, c.width)
            self.loop_in = D.weight(padded(w, Hp, 2, Hp).reshape(Hp, 2 * Hp))
        self.routing = TableRouting({l: L["moe"] for l, L in enumerate(self.layers) if L["moe"] is not None}, dt)

    # ------------------------------------------------------------------ cache
    def create_paged_kv_cache(self, max_batch_size, max_total_seq_len, prefill_chunk_size, page_size, free_pages=None, max_seq_len=None):
        n_pages, max_blocks = self._cache_geometry(max_batch_size, max_total_seq_len, page_size, free_pages, max_seq_len)
        return PagedStateCache([self.config.layers[l].mixer for l, _ in self.runs], self.width_p, n_pages, max_seqs=max_batch_size,
                               max_blocks=max_blocks, max_pos=max_blocks * page_size, dtype=self.dtype, device=self.device,
                               free_pages=free_pages, page_size=page_size)

    # ------------------------------------------------------------------ forward
    def embed(self, input_ids: torch.Tensor) -> LoopHidden:
        ids = input_ids.reshape(-1).to(self.device, torch.int32).contiguous()
        entry = half = None
        if self.loop_in is not None:
            Hp = self.width_p
            entry = D.activation(ids.numel(), 2 * Hp, self.dtype, self.device)
            half = entry[:, Hp:] if isinstance(entry, torch.Tensor) else entry.columns(Hp, Hp)
        return LoopHidden(D.embed_scaled(self.embed_tokens, ids, self.config.embed_scale, half), ids, entry)

    def _normed(self, stream, norm, row=False):
        """-> (normed activation, the same row-major if asked for)."""
        f32 = self.dtype == torch.float32
        act = None if f32 else ops.FragActivation(*stream.shape, stream.device, dtype=self.dtype)
        rows = torch.empty(stream.shape, dtype=self.dtype, device=stream.device) if row or f32 else None
        stream.step(norm, out=act, out_row=rows)
        return (rows if f32 else act), rows

    def forward(self, hidden: LoopHidden, kv, tok_adapter=None, logits_rows=None, layer_outputs=None):
        """Tokens in kv.begin_forward order -> logits fp32 of all tokens or of `logits_rows` (hidden is used up).
        layer_outputs: a list that receives the residual stream after every layer run."""
        if tok_adapter:
            raise ValueError("Dinasun has no adapters")
        c, ids, entry = self.config, hidden.ids, hidden.entry
        T, Hp = hidden.shape
        split = T <= 256 or bool(kv._cur[2])          # short passes and decode steps split K of the narrow output projections
        plans = self.routing.plans(ids) if T else {}
        stream = D.ResidualStream(hidden.x, self.dtype, c.residual_mult)
        for run, (l, enters) in enumerate(self.runs):
            L = self.layers[l]
            mixer, moe = L["mixer"], L["moe"]
            if enters:
                if isinstance(entry, torch.Tensor):
                    stream.step(out_row=entry[:, :Hp])
                else:
                    stream.step(out=entry.columns(0, Hp))
                stream.replace(*D.linear_sum(entry, self.loop_in, split))
            if isinstance(mixer, TimeMix):
                mixes = mixer.mixes(T, Hp, stream.device)
                stream.step(L["norm1"], mu=mixer.mu, shift=kv.shift(run), tokens=kv.token_meta(), **mixes.room())
                y = kv.time_mix(run, mixes, mixer)
            else:
                y = kv.tied_attention(run, ops.linear(self._normed(stream, L["norm1"])[0], mixer.proj, out_dtype=torch.float32), mixer)
            stream.branch(*D.linear_sum(y, mixer.o, split), norm=L["norm1b"])
            if moe is not None:
                n, n_row = self._normed(stream, L["norm2"], row=True)
                rows, y, parts = moe(n, n_row, plans[l], split)
                stream.branch(y, parts, L["norm2b"], rows, 1.0 / moe.spec.top)
            if layer_outputs is not None:
                stream.step()
                layer_outputs.append(stream.x[:, : c.width].clone())
        if logits_rows is not None:
            stream.step()
            x = stream.x[logits_rows].contiguous()
            if x.shape[0] == 0:
                return torch.empty((0, c.vocab), dtype=torch.float32, device=x.device)
            stream = D.ResidualStream(x, self.dtype)
        n, _ = self._normed(stream, self.final_norm)
        logits = ops.linear(n, self.head, out_dtype=torch.float32)
        return logits if logits.shape[1] == c.vocab else logits[:, : c.vocab].contiguous()
