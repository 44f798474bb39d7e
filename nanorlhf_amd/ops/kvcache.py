"""Paged KV-cache primitives for the in-process sampler.

Replaces vLLM's paged attention.  The pool is two
tensors [num_pages, page_size, Hkv, D] (K and V) in bf16, sized against
288 GB HBM3E; sequences own page lists (block tables).

  * kv_append: scatter freshly-projected K/V rows into their page slots.
  * paged_attn_decode: one query token per sequence; HIP kernel does
    online-softmax attention over the sequence's pages, one workgroup per
    (sequence, kv-head) with the q-heads of that group held in registers
    (GQA), vectorized bf16 loads of KV lines, fp32 accumulation.
  * paged_attn: the batch of one engine step — single tokens and portions of
    prompts together — with an optional sliding window, kept first tokens and
    outputs turned back by their position.
  * rotary_qkv: norm, rotation and cache write of a layer's q, k and v.
"""
from __future__ import annotations

import torch

from . import serve_ext
from .rope import rotate_pairs


def kv_append(k: torch.Tensor, v: torch.Tensor, slots: torch.Tensor,
              k_cache: torch.Tensor, v_cache: torch.Tensor) -> None:
    """k/v: [T, Hkv, D] bf16; slots: [T] int64 flat slot index
    (page * page_size + offset).  K cache is [P, ps, Hkv, D]; V cache is
    d-major per page, [P, Hkv, D, ps]."""
    if k.is_cuda:
        serve_ext().kv_append(k.contiguous(), v.contiguous(), slots, k_cache, v_cache)
        return
    ps = k_cache.shape[1]
    kc = k_cache.view(-1, *k_cache.shape[2:])
    if k_cache.dtype == torch.float8_e4m3fn:
        # mirror the kernel's fragment-major fp8 K layout
        kc[slots] = k[..., _fp8_k_perm(k.shape[-1])].to(k_cache.dtype)
    else:
        kc[slots] = k
    pages = torch.div(slots, ps, rounding_mode="floor")
    offs = slots % ps
    # v_cache[page, h, d, off] = v[t, h, d]
    v_cache[pages, :, :, offs] = v


def _fp8_k_perm(D: int) -> torch.Tensor:
    """Fragment-major permutation for the fp8 K cache: stored index
    hi*(D/4) + c*8 + j holds logical element c*32 + hi*8 + j."""
    fwd = torch.empty(D, dtype=torch.long)
    for d in range(D):
        c, rem = divmod(d, 32)
        hi, j = divmod(rem, 8)
        fwd[hi * (D // 4) + c * 8 + j] = c * 32 + hi * 8 + j
    return fwd


def depermute_fp8_k(kc_float: torch.Tensor) -> torch.Tensor:
    """Undo the fragment-major byte permutation of the fp8 K cache
    (csrc/kvcache.hip kv_append)."""
    D = kc_float.shape[-1]
    idx = torch.empty(D, dtype=torch.long)
    for d in range(D):
        c, rem = divmod(d, 32)
        hi, j = divmod(rem, 8)
        idx[c * 32 + hi * 8 + j] = hi * (D // 4) + c * 8 + j
    return kc_float[..., idx.to(kc_float.device)]


def paged_attn_decode(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
                      block_tables: torch.Tensor, seq_lens: torch.Tensor,
                      scale: float) -> torch.Tensor:
    """q: [B, Hq, D] bf16 (one new token per sequence); block_tables [B, P] int32;
    seq_lens [B] int32 (length INCLUDING the new token, whose K/V are already
    appended).  Returns [B, Hq, D] bf16."""
    if q.is_cuda:
        return serve_ext().paged_attn_decode(q.contiguous(), k_cache, v_cache,
                                       block_tables.contiguous(), seq_lens.contiguous(),
                                       float(scale))
    # CPU reference.  On an fp8 cache this mirrors the native-fp8 kernel's
    # arithmetic (csrc/kvcache.hip): Q and the softmax P are ALSO e4m3 so
    # the whole QK^T/PV runs on mfma_..._fp8_fp8 — quantize them here too.
    fp8 = k_cache.dtype == torch.float8_e4m3fn
    B, Hq, D = q.shape
    page = k_cache.shape[1]
    Hkv = k_cache.shape[2]
    rep = Hq // Hkv
    out = torch.empty_like(q, dtype=torch.float32)
    kc = k_cache.view(-1, Hkv, D).float()
    if fp8:
        kc = depermute_fp8_k(kc)
    # V d-major [P, Hkv, D, ps] -> flat [P*ps, Hkv, D]
    vc = v_cache.permute(0, 3, 1, 2).reshape(-1, Hkv, D).float()

    def q8(x):
        return x.to(torch.float8_e4m3fn).float() if fp8 else x

    for b in range(B):
        L = int(seq_lens[b])
        pages = block_tables[b, : (L + page - 1) // page].long()
        slots = (pages.unsqueeze(1) * page + torch.arange(page)).reshape(-1)[:L]
        kk = kc[slots].repeat_interleave(rep, dim=1)  # [L, Hq, D]
        vv = vc[slots].repeat_interleave(rep, dim=1)
        att = torch.einsum("hd,lhd->hl", q8(q[b].float()), kk) * scale
        att = q8(torch.softmax(att, dim=-1))
        out[b] = torch.einsum("hl,lhd->hd", att, vv)
    return out.to(q.dtype)


HEAD_DIMS = (32, 64, 128, 256)   # head widths the attention kernels tile


def pad_head_dim(d: int) -> int:
    """Cache width of a head: the next width the kernels tile.  Pad columns
    are zero from the pool's creation and are never written."""
    for p in HEAD_DIMS:
        if d <= p:
            return p
    raise ValueError(f"head width {d} exceeds {HEAD_DIMS[-1]}")


def rotary_qkv(proj: torch.Tensor, offsets: tuple, heads: int, kv_heads: int,
               dim: int, vdim: int, slots: torch.Tensor, k_cache: torch.Tensor,
               v_cache: torch.Tensor, *, q_norm=None, k_norm=None, cs_qk=None,
               cs_v=None, interleaved: bool = False, eps: float = 1e-6) -> torch.Tensor:
    """q, k, v are the columns at `offsets` of proj [T, ld].  q and k are
    normed per head (if weights are given) and rotated over the first
    cs_qk.shape[1] dimensions; v is rotated over all its dimensions if cs_v is
    given.  k and v go to their cache slots; returns q [T, heads, padded dim]."""
    if proj.is_cuda:
        return serve_ext().rotary_qkv(proj, *offsets, q_norm, k_norm, cs_qk, cs_v, slots,
                                      k_cache, v_cache, heads, kv_heads, dim, vdim,
                                      interleaved, float(eps))
    T, ps = proj.shape[0], k_cache.shape[1]

    def part(off, n, d):
        return proj[:, off:off + n * d].reshape(T, n, d).float()

    def norm(x, w):
        if w is None:
            return x
        return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w.float()

    q = norm(part(offsets[0], heads, dim), q_norm)
    k = norm(part(offsets[1], kv_heads, dim), k_norm)
    v = part(offsets[2], kv_heads, vdim)
    if cs_qk is not None:
        q = rotate_pairs(q, cs_qk, interleaved)
        k = rotate_pairs(k, cs_qk, interleaved)
    if cs_v is not None:
        v = rotate_pairs(v, cs_v, interleaved)
    page, off = slots // ps, slots % ps
    k_cache[page, off, :, :dim] = k.to(k_cache.dtype)
    v_cache[page, :, :vdim, off] = v.to(v_cache.dtype)
    out = q.new_zeros(T, heads, k_cache.shape[3])
    out[..., :dim] = q
    return out.to(proj.dtype)


def _paged_attn_ref(q, k_cache, v_cache, row_seq, positions, block_tables, out, scale,
                    size, keep, uncs):
    ps, G = k_cache.shape[1], k_cache.shape[2]
    T, H, _ = q.shape
    V = out.shape[1] // H
    for t in range(T):
        pos = int(positions[t])
        j = torch.arange(pos + 1)
        j = j[(pos - j < size) | (j < keep)]
        pages = block_tables[int(row_seq[t])].long()[j // ps]
        k = k_cache[pages, j % ps].float().repeat_interleave(H // G, dim=1)
        v = v_cache[pages, :, :, j % ps].float()[..., :V].repeat_interleave(H // G, dim=1)
        p = torch.softmax(torch.einsum("hd,lhd->hl", q[t].float(), k) * scale, dim=-1)
        o = torch.einsum("hl,lhd->hd", p, v)
        if uncs is not None:
            o = rotate_pairs(o[None], uncs[t:t + 1], True, sign=-1.0)[0]
        out[t] = o.reshape(-1).to(out.dtype)


NO_WINDOW = 1 << 30


def paged_attn(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, ctx,
               out: torch.Tensor, scale: float, *, size: int = NO_WINDOW, keep: int = 0,
               uncs: torch.Tensor | None = None) -> None:
    """Attention of one engine step over the paged cache, which already holds
    the step's own keys and values.

    q [T, H, padded dim]: ctx.n_decode single tokens first, then the tokens of
    ctx.portions.  Position i sees j <= i if i - j < size or j < keep.  uncs
    [T, V] (cos | sin by position) turns the output's interleaved pairs back.
    Writes out [T, H * V], any row stride."""
    nd, por = ctx.n_decode, ctx.portions

    def cut(t, a, b):
        return None if t is None else t[a:b]

    T = q.shape[0]
    groups = []
    if nd:
        groups.append((0, nd, ctx.block_tables, None))
    if por is not None:
        groups.append((nd, T, por.block_tables, por))
    for a, b, bt, p in groups:
        args = (float(scale), int(size), int(keep), cut(uncs, a, b))
        if q.is_cuda and q.dtype == torch.bfloat16:
            if p is None:
                serve_ext().paged_attn_decode_window(q[a:b], k_cache, v_cache, bt,
                                                     ctx.seq_lens, out[a:b], *args)
            else:
                serve_ext().paged_attn_varlen(q[a:b], k_cache, v_cache, p.cu, p.seq_lens, bt,
                                              out[a:b], p.max_q, *args)
            continue
        row_seq = p.row_seq if p is not None else torch.arange(
            b - a, dtype=torch.int32, device=q.device)
        fn = serve_ext().paged_attn_plain if q.is_cuda else _paged_attn_ref
        fn(q[a:b], k_cache, v_cache, row_seq, ctx.positions[a:b], bt, out[a:b], *args)
