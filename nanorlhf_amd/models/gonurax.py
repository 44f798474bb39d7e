"""Gonurax: a decoder of parallel blocks over retention, windowed-attention and
lightning mixers, with a 32-bit residual stream.

Block:  h = norm1(x);  x <- x + m (mixer(h) + ff(h)).

Both sublayers read h and their outputs are added, so a block is two GEMMs:
one input projection for all of the mixer's inputs and the feed-forward's gate
and up, and one output projection over [mixer output | feed-forward output]
side by side, whose sum over the columns is the addition.  The update of x is
left pending and fused into the next norm.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops
from .mixers import MIXERS

ALIGN = 8   # columns of a segment start at multiples of 16 bytes (bf16)


def _round_up(n: int) -> int:
    return (n + ALIGN - 1) // ALIGN * ALIGN


@dataclass
class GonuraxConfig:
    vocab_size: int
    hidden_size: int
    layers: list = field(default_factory=list)   # {"type", "mixer", "mlp"} each
    norm_groups: int = 1
    norm_eps: float = 1e-5
    residual_mult: float = 1.0
    dtype: str = "bfloat16"

    def __post_init__(self):
        if self.hidden_size % self.norm_groups:
            raise ValueError("width must be a multiple of norm.groups")
        for layer in self.layers:
            if layer["type"] not in MIXERS:
                raise ValueError(f"unknown mixer {layer['type']!r}; have {sorted(MIXERS)}")
            mlp = layer.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"unknown feed-forward {mlp['kind']!r}")

    @classmethod
    def from_json(cls, c: dict, **overrides) -> "GonuraxConfig":
        d = dict(vocab_size=c["vocab"], hidden_size=c["width"], layers=c["layers"],
                 norm_groups=c["norm"]["groups"], norm_eps=c["norm"]["eps"],
                 residual_mult=c["residual_mult"])
        d.update(overrides)
        return cls(**d)

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def cache_layers(self) -> list:
        return [MIXERS[l["type"]](l["mixer"], self.norm_eps).cache_spec for l in self.layers]


class ParallelBlock(nn.Module):
    def __init__(self, cfg: GonuraxConfig, layer: dict):
        super().__init__()
        W = cfg.hidden_size
        self.groups, self.eps = cfg.norm_groups, cfg.norm_eps
        self.norm1 = nn.Parameter(torch.ones(W))
        self.mixer = MIXERS[layer["type"]](layer["mixer"], cfg.norm_eps)
        mlp = layer.get("mlp")
        self.ff = mlp["ff"] if mlp is not None else 0
        # columns of the input projection
        self.cols, n = {}, 0
        widths = dict(self.mixer.inputs)
        if self.ff:
            widths.update(gate=self.ff, up=self.ff)
        for name, w in widths.items():
            self.cols[name] = (n, n + w)
            n += _round_up(w)
        self.in_proj = nn.Linear(W, n, bias=False)
        # columns of the output projection's input
        self.mix_out = self.mixer.out_width
        self.ff_start = _round_up(self.mix_out) if self.ff else self.mix_out
        self.out_width = self.ff_start + _round_up(self.ff)
        self.out_proj = nn.Linear(self.out_width, W, bias=False)

    def load(self, take) -> None:
        """take(name) -> tensor of this layer; padding rows and columns are 0."""
        with torch.no_grad():
            self.norm1.copy_(take("norm1"))
            self.in_proj.weight.zero_()
            self.out_proj.weight.zero_()
            for name, (a, b) in self.cols.items():
                part = "mlp." if name in ("gate", "up") else "mix."
                self.in_proj.weight[a:b].copy_(take(part + name))
            self.out_proj.weight[:, :self.mix_out].copy_(take("mix.o"))
            if self.ff:
                self.out_proj.weight[:, self.ff_start:self.ff_start + self.ff].copy_(
                    take("mlp.down"))
            for name, p in self.mixer.weights.items():
                p.copy_(take("mix." + name))

    def forward(self, h: torch.Tensor, ctx, cache) -> torch.Tensor:
        proj = self.in_proj(h)
        cat = torch.empty(h.shape[0], self.out_width, dtype=h.dtype, device=h.device)
        self.mixer(self.cols, proj, ctx, cache, cat[:, :self.mix_out])
        if self.ff:
            gate, up = (proj[:, slice(*self.cols[n])] for n in ("gate", "up"))
            pad = self.ff_start - self.mix_out
            ops.gelu_glu(gate, up, cat[:, self.mix_out:], pad,
                         self.out_width - self.ff_start - self.ff)
        return self.out_proj(cat)


class GonuraxLM(nn.Module):
    """Served through SamplerEngine like CausalLM: forward(ids, ctx) returns
    final normed hidden states, logits() applies the (tied) head."""

    extensions = ("_serve",)            # HIP extensions its forward needs
    kv_cache_dtypes = ("bf16",)         # "bf16" = pages in the model's dtype
    packed_prefill = False              # prompts run through step portions

    def __init__(self, cfg: GonuraxConfig):
        super().__init__()
        self.cfg = cfg
        self.embed = nn.Embedding(cfg.vocab_size, cfg.hidden_size)
        self.layers = nn.ModuleList(ParallelBlock(cfg, l) for l in cfg.layers)
        self.norm = nn.Parameter(torch.ones(cfg.hidden_size))
        nn.init.normal_(self.embed.weight, std=0.02)
        for b in self.layers:
            nn.init.normal_(b.in_proj.weight, std=0.02)
            nn.init.normal_(b.out_proj.weight, std=0.02)

    @property
    def lm_head_weight(self) -> torch.Tensor:
        return self.embed.weight

    def load(self, tensors: dict) -> None:
        used = set()

        def take(name):
            if name not in tensors:
                raise KeyError(f"checkpoint is missing tensor {name!r}")
            used.add(name)
            return tensors[name]

        with torch.no_grad():
            self.embed.weight.copy_(take("embed"))
            self.norm.copy_(take("final.norm"))
        for i, b in enumerate(self.layers):
            b.load(lambda n, i=i: take(f"l{i}.{n}"))
        extra = sorted(set(tensors) - used)
        if extra:
            raise RuntimeError(f"unmapped checkpoint tensors: {extra[:8]}")

    def forward(self, input_ids: torch.Tensor, ctx) -> torch.Tensor:
        if ctx.mode not in ("step", "decode"):
            raise NotImplementedError(f"Gonurax is served, not trained (mode {ctx.mode!r})")
        c = self.cfg
        x = torch.empty(input_ids.shape[0], c.hidden_size, dtype=torch.float32,
                        device=input_ids.device)
        delta = None
        for i, b in enumerate(self.layers):
            h = ops.residual_group_norm(
                x, b.norm1, c.norm_eps, groups=c.norm_groups, delta=delta,
                mult=c.residual_mult, embed=self.embed.weight if i == 0 else None,
                ids=input_ids if i == 0 else None)
            delta = b(h, ctx, ctx.kv_caches[i])
            if ctx.on_layer is not None:
                ctx.on_layer(i, x + c.residual_mult * delta.float())
        return ops.residual_group_norm(
            x, self.norm, c.norm_eps, groups=c.norm_groups, delta=delta, mult=c.residual_mult,
            embed=None if self.layers else self.embed.weight,
            ids=None if self.layers else input_ids)

    def logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.lm_head_weight)
