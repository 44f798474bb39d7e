"""Sequence mixers of the parallel-block models.

A mixer owns no GEMM: its block projects the normed input once for all of the
mixer's inputs and the feed-forward's, hands it the columns, and gives it
columns of the row that the block's one output GEMM reads.  A mixer says

    inputs       name -> width of the projections it reads
    out_width    width of what it writes
    cache_spec   what it keeps of a sequence (KVSpec or StateSpec)
    weights      its own small parameters: tensor name -> parameter

and computes forward(cols, proj, ctx, cache, out), where cols[name] is the
(first, last) column of an input in proj [T, ld].
"""
from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from .config import KVSpec, StateSpec


class LinearMixer(nn.Module):
    """Decayed linear attention: the two mixers below differ in what happens to
    q, k, v on the way in and to the output on the way out."""

    silu_inputs = False

    def __init__(self, m: dict, eps: float):
        super().__init__()
        self.heads, self.dim, self.vdim = m["heads"], m["dim"], m["vdim"]
        if len(m["decay"]) != self.heads:
            raise ValueError("one decay per head expected")
        self.decay = ops.DecayTable(m["decay"])
        self.eps = eps
        self.rotation = None
        self.kscale = 1.0
        qk, v = self.heads * self.dim, self.heads * self.vdim
        self.inputs = {"q": qk, "k": qk, "v": v, "g": v}
        self.out_width = v
        self.cache_spec = StateSpec(self.heads, self.dim, self.vdim)

    @property
    def weights(self) -> dict:
        return {}

    def _kw(self, ctx, a, b):
        kw = dict(silu=self.silu_inputs, kscale=self.kscale)
        if self.rotation is not None and self.rotation.dims:
            kw.update(cs=ctx.angles(self.rotation)[a:b], interleaved=self.rotation.interleaved)
        return kw

    def forward(self, cols, proj, ctx, state, out):
        q, k, v, g = (proj[:, cols[n][0]:cols[n][1]] for n in ("q", "k", "v", "g"))
        T, nd = proj.shape[0], ctx.n_decode
        if nd:
            kw = self._kw(ctx, 0, nd)
            self.run(lambda **f: ops.linear_attn_decode(
                q[:nd], k[:nd], v[:nd], self.decay, ctx.state_slots, ctx.seq_lens, state,
                **kw, **f), g[:nd], out[:nd])
        if ctx.portions is not None:
            kw = self._kw(ctx, nd, T)
            self.run(lambda **f: ops.linear_attn_chunked(
                q[nd:], k[nd:], v[nd:], self.decay, ctx.portions, state, **kw, **f),
                g[nd:], out[nd:])


class Retention(LinearMixer):
    """Rotated q and k, k / sqrt(dim); each head's output is divided by its
    root mean square and gated by silu."""

    def __init__(self, m: dict, eps: float):
        super().__init__(m, eps)
        self.rotation = ops.Rotation(m["rot"]["dims"], m["rot"]["base"])
        self.kscale = self.dim ** -0.5

    def run(self, attn, g, out):
        attn(gate=g, eps=self.eps, out=out)


class Lightning(LinearMixer):
    """SiLU on q, k and v; the heads' outputs are normed together, with a
    weight, and gated by a sigmoid."""

    silu_inputs = True

    def __init__(self, m: dict, eps: float):
        super().__init__(m, eps)
        self.norm = nn.Parameter(torch.ones(self.out_width))

    @property
    def weights(self):
        return {"norm": self.norm}

    def run(self, attn, g, out):
        ops.gated_norm(attn(), self.norm, g, out, self.eps, act="sigmoid")


class WindowAttention(nn.Module):
    """Softmax attention over a sliding window and the kept first tokens, with
    per-head query/key norms and rotated values."""

    def __init__(self, m: dict, eps: float):
        super().__init__()
        self.heads, self.kv_heads = m["heads"], m["kv_heads"]
        if self.heads % self.kv_heads:
            raise ValueError("query heads must be a multiple of key/value heads")
        self.dim, self.vdim, self.eps = m["dim"], m["vdim"], eps
        self.scale = m["scale"]
        self.size, self.keep = m["mask"]["size"], m["mask"]["keep_first"]
        rot = m["rot"]
        self.rotation = ops.Rotation(rot["dims"], rot["base"], interleaved=True)
        self.v_rotation = ops.Rotation(self.vdim, rot["base"], interleaved=True)
        self.q_norm = nn.Parameter(torch.ones(self.dim))
        self.k_norm = nn.Parameter(torch.ones(self.dim))
        self.inputs = {"q": self.heads * self.dim, "k": self.kv_heads * self.dim,
                       "v": self.kv_heads * self.vdim}
        self.out_width = self.heads * self.vdim
        self.cache_spec = KVSpec(self.kv_heads, ops.pad_head_dim(self.dim),
                                 ops.pad_head_dim(self.vdim))

    @property
    def weights(self):
        return {"q.norm": self.q_norm, "k.norm": self.k_norm}

    def forward(self, cols, proj, ctx, cache, out):
        k_cache, v_cache = cache
        cs_v = ctx.angles(self.v_rotation)
        q = ops.rotary_qkv(proj, tuple(cols[n][0] for n in ("q", "k", "v")), self.heads,
                           self.kv_heads, self.dim, self.vdim, ctx.slots, k_cache, v_cache,
                           q_norm=self.q_norm, k_norm=self.k_norm,
                           cs_qk=ctx.angles(self.rotation) if self.rotation.dims else None,
                           cs_v=cs_v, interleaved=True, eps=self.eps)
        ops.paged_attn(q, k_cache, v_cache, ctx, out, self.scale, size=self.size,
                       keep=self.keep, uncs=cs_v)


MIXERS = {"retention": Retention, "attention": WindowAttention, "lightning": Lightning}
