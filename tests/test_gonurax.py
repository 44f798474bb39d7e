"""Gonurax against a plain implementation (tests/gonurax_oracle.py): each
mechanism alone, then the model through the engine's step function and its
scheduler.  Every case runs on the CPU's reference operations and, marked gpu,
on the HIP kernels."""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import gonurax_oracle as orc  # noqa: E402

from nanorlhf_amd import ops  # noqa: E402
from nanorlhf_amd.models import GonuraxConfig, GonuraxLM, build_model, get_config, load_model  # noqa: E402
from nanorlhf_amd.models.qwen2 import AttnContext, Portions  # noqa: E402
from nanorlhf_amd.sampler import SamplerEngine, SamplingParams, SeqState  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.param("cuda", marks=pytest.mark.gpu)
devices = pytest.mark.parametrize("dev", ["cpu", GPU])
# (device, dtype, error allowed relative to the result's size)
kinds = pytest.mark.parametrize("dev,dtype,tol", [
    ("cpu", torch.float32, 2e-5),
    pytest.param("cuda", torch.float32, 2e-5, marks=pytest.mark.gpu),
    pytest.param("cuda", torch.bfloat16, 0.02, marks=pytest.mark.gpu)])


def close(got, want, tol):
    got, want = got.double().cpu(), want.double()
    assert got.shape == want.shape
    err = (got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt().clamp(min=1e-9)
    worst = (got - want).abs().max() / want.pow(2).mean().sqrt().clamp(min=1e-9)
    assert err < tol and worst < 12 * tol, (float(err), float(worst))


def rand(*shape, seed=0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g).to(torch.bfloat16).to(dtype)


# ------------------------------------------------------------ configurations
def retention(heads=3, dim=24, vdim=20, rot=16, base=1000.0, decay=None):
    return dict(type="retention", mixer=dict(
        heads=heads, dim=dim, vdim=vdim, rot=dict(dims=rot, base=base),
        decay=decay or [0.9, 1.0, 0.97][:heads]))


def lightning(heads=2, dim=16, vdim=36, decay=None):
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim,
                                             decay=decay or [0.5, 0.995]))


def attention(heads=4, kv=2, dim=40, vdim=24, rot=32, size=21, keep=3, base=700.0, scale=0.2):
    return dict(type="attention", mixer=dict(
        heads=heads, kv_heads=kv, dim=dim, vdim=vdim, rot=dict(dims=rot, base=base),
        scale=scale, mask=dict(size=size, keep_first=keep)))


def config(*layers, width=96, vocab=263, groups=3, eps=1e-4, mult=0.7, ff=88):
    return dict(architecture="Gonurax", vocab=vocab, width=width, residual_mult=mult,
                norm=dict(eps=eps, groups=groups),
                layers=[dict(l, mlp=l.get("mlp", dict(kind="dense", ff=ff))) for l in layers])


def no_mlp(layer):
    return dict(layer, mlp=None)


CONFIGS = {
    "uneven": config(attention(), lightning(), retention(), no_mlp(attention(kv=1, keep=0, size=7))),
    "odd-widths": config(retention(heads=1, dim=6, vdim=10, rot=4), lightning(heads=2, dim=10, vdim=6),
                         attention(heads=3, kv=3, dim=10, vdim=6, rot=10, size=5, keep=1),
                         width=50, groups=1, vocab=97, ff=30, mult=1.0),
    "one-head": config(no_mlp(lightning(heads=1, dim=64, vdim=64, decay=[0.9])),
                       attention(heads=1, kv=1, dim=32, vdim=32, rot=32, size=1, keep=2),
                       no_mlp(retention(heads=1, dim=32, vdim=32, rot=32)), width=64, groups=4),
    "wide-heads": config(attention(heads=34, kv=2, dim=16, vdim=8, rot=0, size=1000, keep=0),
                         attention(heads=2, kv=1, dim=160, vdim=136, rot=96, size=40, keep=50),
                         retention(heads=2, dim=136, vdim=160, rot=100),
                         lightning(heads=2, dim=72, vdim=132), width=128, groups=8),
}


def make(cfg, dev="cpu", dtype=torch.float32, seed=0):
    """(model, oracle) of the same random weights."""
    t = orc.random_tensors(cfg, seed)
    name = str(dtype).split(".")[1]
    model = GonuraxLM(GonuraxConfig.from_json(cfg, dtype=name)).to(dtype)
    model.load(t)
    return model.to(dev).eval(), orc.Oracle(cfg, t)


def tokens(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def engine(model, pool=512, slots=4, **kw):
    return SamplerEngine(model, kv_pool_tokens=pool, state_slots=slots, **kw)


def run(eng, plan):
    """plan: list of steps, each a list of (sequence, n).  Logits of every
    token of every sequence, in order."""
    out = {}
    for step in plan:
        hidden, starts = eng.step(step)
        logits = eng.model.logits(hidden)
        for (s, n), r in zip(step, starts):
            out.setdefault(s.uid, []).append(logits[r:r + n].float().cpu())
    return {u: torch.cat(x) for u, x in out.items()}


def cut(seq, sizes):
    """Steps that run one sequence alone in portions of changing size."""
    left, plan, i = len(seq.tokens), [], 0
    while left:
        n = min(sizes[i % len(sizes)], left)
        plan.append([(seq, n)])
        left -= n
        i += 1
    return plan


# ------------------------------------------------------------ each mechanism
@kinds
@pytest.mark.parametrize("W,groups", [(96, 3), (50, 2), (2560, 1), (4096, 2), (9000, 2), (64, 64)])
def test_residual_group_norm(dev, dtype, tol, W, groups):
    x = rand(5, W, seed=1).to(dev)
    d, w = rand(5, W, seed=2, dtype=dtype), rand(W, seed=3, dtype=dtype)
    want_x = x.cpu().double() + 0.3 * d.double()
    y = ops.residual_group_norm(x, w.to(dev), 1e-3, groups=groups, delta=d.to(dev), mult=0.3)
    close(x, want_x, 1e-6)
    close(y, orc.group_rms(want_x, w.double(), groups, 1e-3), tol)
    emb, ids = rand(7, W, seed=4, dtype=dtype), torch.tensor([3, 0, 6, 6, 1])
    y = ops.residual_group_norm(x, w.to(dev), 1e-3, groups=groups, embed=emb.to(dev),
                                ids=ids.to(dev))
    close(x, emb[ids].double(), 1e-9)
    close(y, orc.group_rms(emb[ids].double(), w.double(), groups, 1e-3), tol)
    y = ops.residual_group_norm(x, w.to(dev), 1e-3, groups=groups)
    close(y, orc.group_rms(emb[ids].double(), w.double(), groups, 1e-3), tol)


@kinds
def test_norm_eps_is_inside_the_root(dev, dtype, tol):
    x = torch.full((1, 8), 1e-3, device=dev)
    y = ops.residual_group_norm(x, torch.ones(8, dtype=dtype, device=dev), 1e-2)
    close(y, torch.full((1, 8), 1e-3 / math.sqrt(1e-6 + 1e-2)), tol)


@kinds
@pytest.mark.parametrize("groups,part,act,weight", [
    (3, 20, "silu", False), (1, 130, "sigmoid", True), (2, 700, "silu", True), (5, 6, "sigmoid", False)])
def test_gated_norm(dev, dtype, tol, groups, part, act, weight):
    W = groups * part
    x, wide = rand(4, W, seed=1, dtype=dtype), rand(4, W + 11, seed=2, dtype=dtype)
    w = rand(W, seed=3, dtype=dtype) if weight else None
    out = torch.zeros(4, W + 5, dtype=dtype, device=dev)
    ops.gated_norm(x.to(dev), None if w is None else w.to(dev), wide.to(dev)[:, 3:3 + W],
                   out[:, 2:2 + W], 1e-3, groups=groups, act=act)
    gate = wide[:, 3:3 + W].double()
    want = orc.group_rms(x.double(), 1.0 if w is None else w.double(), groups, 1e-3)
    want = want * (orc.silu(gate) if act == "silu" else torch.sigmoid(gate))
    close(out[:, 2:2 + W], want, tol)
    assert out[:, :2].abs().sum() == 0 and out[:, 2 + W:].abs().sum() == 0


@kinds
@pytest.mark.parametrize("ff,pad,tail", [(24, 0, 0), (30, 0, 2), (17, 3, 5), (64, 8, 0)])
def test_gelu_glu(dev, dtype, tol, ff, pad, tail):
    p = rand(5, 2 * ff + 8, seed=1, dtype=dtype) * 2
    out = torch.full((5, pad + ff + tail), 9.0, dtype=dtype, device=dev)
    pd = p.to(dev)
    ops.gelu_glu(pd[:, :ff], pd[:, ff:2 * ff], out, pad, tail)
    want = orc.gelu_tanh(p[:, :ff].double()) * p[:, ff:2 * ff].double()
    close(out[:, pad:pad + ff], want, tol)
    assert out[:, :pad].abs().sum() == 0 and out[:, pad + ff:].abs().sum() == 0


@devices
def test_angles_hold_far_away(dev):
    pos = torch.tensor([0, 1, 777, 100003, 2 ** 24 + 1])
    rot = ops.Rotation(12, 5000.0)
    a = orc.angles(pos, 5000.0, 12)
    close(rot.angles(pos.to(dev)), torch.cat([a.cos(), a.sin()], 1), 2e-7)


def one_portion(n, start, pages, dev, slot=0):
    """Context of one portion of n tokens at positions start.. ."""
    def i32(x):
        return torch.tensor(x, dtype=torch.int32, device=dev)
    chunk = [[0] * -(-n // 64), list(range(0, n, 64)), [min(64, n - r) for r in range(0, n, 64)]]
    pos = torch.arange(start, start + n)
    bt = torch.tensor(pages)
    ctx = AttnContext(mode="step", positions=pos.to(dev),
                      slots=(bt[pos // 16] * 16 + pos % 16).to(dev))
    ctx.portions = Portions(cu=i32([0, n]), seq_lens=i32([start + n]), block_tables=i32([pages]),
                            row_seq=i32([0] * n), state_slots=i32([slot]),
                            fresh=i32([int(start == 0)]), chunks=i32(chunk),
                            chunk_first=i32([0, len(chunk[0])]), max_q=n)
    return ctx


def attn_layer(x, dims, mask, rot, dev, dtype, sizes, norms=None, scale=0.3, eps=1e-4):
    """x [T, (H + G) D + G V] through rotary_qkv and paged_attn in portions of
    the given sizes, over pages in shuffled order.  [T, H V]."""
    H, G, D, V = dims
    T = x.shape[0]
    npages = (T + 15) // 16
    g = torch.Generator().manual_seed(5)
    pages = torch.randperm(npages + 3, generator=g)[:npages].tolist()
    DP, VP = ops.pad_head_dim(D), ops.pad_head_dim(V)
    kc = torch.zeros(npages + 3, 16, G, DP, dtype=dtype, device=dev)
    vc = torch.zeros(npages + 3, G, VP, 16, dtype=dtype, device=dev)
    qn, kn = norms if norms is not None else (None, None)
    rqk, rv = ops.Rotation(rot[0], rot[1], True), ops.Rotation(V, rot[1], True)
    outs, at, i = [], 0, 0
    while at < T:
        n = min(sizes[i % len(sizes)], T - at)
        ctx = one_portion(n, at, pages, dev)
        if n == 1:      # as the engine does: one token is a decode row
            p = ctx.portions
            ctx.block_tables, ctx.seq_lens, ctx.portions = p.block_tables, p.seq_lens, None
        csv = rv.angles(ctx.positions)
        q = ops.rotary_qkv(x[at:at + n].to(dev), (0, H * D, (H + G) * D), H, G, D, V, ctx.slots,
                           kc, vc, q_norm=qn, k_norm=kn,
                           cs_qk=rqk.angles(ctx.positions) if rot[0] else None, cs_v=csv,
                           interleaved=True, eps=eps)
        o = torch.empty(n, H * V, dtype=dtype, device=dev)
        ops.paged_attn(q, kc, vc, ctx, o, scale, size=mask[0], keep=mask[1], uncs=csv)
        outs.append(o)
        at, i = at + n, i + 1
    return torch.cat(outs)


def attn_oracle(x, dims, mask, rot, norms=None, scale=0.3, eps=1e-4):
    H, G, D, V = dims
    x, T = x.double(), x.shape[0]
    pos = torch.arange(T)
    q, k, v = x[:, :H * D].view(T, H, D), x[:, H * D:(H + G) * D].view(T, G, D), \
        x[:, (H + G) * D:].view(T, G, V)
    if norms is not None:
        q = orc.rms(q, eps) * norms[0].cpu().double()
        k = orc.rms(k, eps) * norms[1].cpu().double()
    q = orc.rotate_interleaved(q, pos, rot[1], rot[0])
    k = orc.rotate_interleaved(k, pos, rot[1], rot[0])
    v = orc.rotate_interleaved(v, pos, rot[1], V)
    o = orc.windowed_attention(q, k, v, scale, *mask)
    return orc.rotate_interleaved(o, pos, rot[1], V, sign=-1).reshape(T, -1)


@kinds
@pytest.mark.parametrize("dims,mask,rot", [
    ((8, 2, 56, 40), (33, 5), (56, 900.0)),
    ((6, 1, 24, 20), (1, 0), (16, 900.0)),       # sees itself alone
    ((3, 3, 32, 32), (10 ** 6, 0), (32, 10.0)),  # no window
    ((2, 1, 128, 128), (100, 130), (0, 900.0)),  # more kept tokens than window
    ((36, 2, 16, 128), (64, 64), (8, 900.0)),    # more than 16 query heads a group
    ((2, 2, 200, 256), (16, 1), (198, 900.0)),
])
@pytest.mark.parametrize("sizes", [[200], [1], [2, 37, 1, 64, 3]])
def test_attention(dev, dtype, tol, dims, mask, rot, sizes):
    H, G, D, V = dims
    T = 150 if sizes != [1] else 70
    x = rand(T, (H + G) * D + G * V, seed=7, dtype=dtype)
    norms = tuple((1 + rand(D, seed=s) / 4).to(dtype).to(dev) * 2 for s in (8, 9))
    close(attn_layer(x, dims, mask, rot, dev, dtype, sizes, norms),
          attn_oracle(x, dims, mask, rot, norms), tol)


@kinds
@pytest.mark.parametrize("D,V,rot", [(24, 20, 16), (64, 32, 64), (130, 34, 2), (10, 6, 6)])
def test_rotate_half_layout_of_q_k_v(dev, dtype, tol, D, V, rot):
    """The other layout of pairs through the same preparation step."""
    H, G, T = 3, 1, 37
    x = rand(T, (H + G) * D + G * V, seed=4, dtype=dtype)
    DP, VP = ops.pad_head_dim(D), ops.pad_head_dim(V)
    kc = torch.zeros(4, 16, G, DP, dtype=dtype, device=dev)
    vc = torch.zeros(4, G, VP, 16, dtype=dtype, device=dev)
    pos = torch.arange(3, 3 + T)
    slots = torch.arange(T - 1, -1, -1) + 5
    rk, rv = ops.Rotation(rot, 90.0), ops.Rotation(V, 90.0)
    q = ops.rotary_qkv(x.to(dev), (0, H * D, (H + G) * D), H, G, D, V, slots.to(dev), kc, vc,
                       cs_qk=rk.angles(pos.to(dev)), cs_v=rv.angles(pos.to(dev)))
    xd = x.double()
    want_q = orc.rotate_half(xd[:, :H * D].view(T, H, D), pos, 90.0, rot)
    want_k = orc.rotate_half(xd[:, H * D:(H + G) * D].view(T, G, D), pos, 90.0, rot)
    want_v = orc.rotate_half(xd[:, (H + G) * D:].view(T, G, V), pos, 90.0, V)
    close(q[..., :D], want_q, tol)
    close(kc.cpu()[slots // 16, slots % 16, :, :D], want_k, tol)
    close(vc.cpu()[slots // 16, :, :V, slots % 16], want_v, tol)
    assert q[..., D:].abs().sum() == 0 and kc[..., D:].abs().sum() == 0
    assert vc[:, :, V:].abs().sum() == 0


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("interleaved", [True, False])
def test_qkv_of_a_large_batch_equals_its_parts(dtype, interleaved):
    H, G, D, V, T, dev = 7, 2, 200, 96, 8192, "cuda"
    x = rand(T, (H + G) * D + G * V, seed=6, dtype=dtype).to(dev)
    w = tuple((1 + rand(D, seed=s) / 4).to(dtype).to(dev) for s in (1, 2))
    pos = torch.arange(T, device=dev)
    ck = ops.Rotation(192, 5e3, interleaved).angles(pos)
    cv = ops.Rotation(V, 5e3, interleaved).angles(pos)
    res = []
    for n in (T, 1000):
        kc = torch.zeros(T // 16, 16, G, 256, dtype=dtype, device=dev)
        vc = torch.zeros(T // 16, G, 128, 16, dtype=dtype, device=dev)
        q = torch.cat([ops.rotary_qkv(
            x[a:a + n], (0, H * D, (H + G) * D), H, G, D, V, pos[a:a + n], kc, vc, q_norm=w[0],
            k_norm=w[1], cs_qk=ck[a:a + n], cs_v=cv[a:a + n], interleaved=interleaved)
            for a in range(0, T, n)])
        res.append((q, kc, vc))
    for a, b in zip(*res):
        assert torch.equal(a, b)
    assert (res[0][1][..., :D] != 0).any(-1).all() and (res[0][2][:, :, :V] != 0).any(-1).all()


@kinds
@pytest.mark.parametrize("size,keep", [(17, 0), (64, 3), (48, 16), (128, 20), (5, 1)])
@pytest.mark.parametrize("sizes", [[300], [1], [2, 31, 64]])
def test_window_edges_show(dev, dtype, tol, size, keep, sizes):
    """One key stands out so far that whoever sees it copies its value: the
    window's last and first unseen position, page and tile borders, the kept
    first tokens and the next ones are told apart without doubt."""
    H = G = 1
    D = V = 32
    T = size + 40
    planted = sorted({0, max(keep - 1, 0), keep, 15, 16, 31, 32, size - 1} & set(range(T)))
    for j in planted:
        x = rand(T, 3 * D, seed=11, dtype=torch.float32) * 0.1
        x[:, 0] = 8.0                    # q: unit direction, no rotation used
        x[:, D:2 * D] = 0
        x[j, D] = 8.0                    # the key that stands out
        x = x.to(dtype)
        got = attn_layer(x, (H, G, D, V), (size, keep), (0, 50.0), dev, dtype, sizes, scale=0.5)
        close(got, attn_oracle(x, (H, G, D, V), (size, keep), (0, 50.0), scale=0.5), tol)
        # and it is seen exactly where the mask says
        v = orc.rotate_interleaved(x[:, 2 * D:].double().view(T, 1, V), torch.arange(T), 50.0, V)
        for i in (j, j + size - 1, j + size, j + size + 1):
            if i < T:
                own = orc.rotate_interleaved(v[j:j + 1], torch.tensor([i]), 50.0, V, sign=-1)
                near = (got[i].double().cpu() - own.view(-1)).abs().max() < 0.02
                assert bool(near) == orc.visible(i, j, size, keep), (i, j)


@kinds
@pytest.mark.parametrize("H,D,V,rot,silu", [
    (3, 24, 20, 16, False), (2, 64, 64, 64, False), (1, 6, 10, 0, True), (2, 128, 96, 0, True),
    (2, 136, 160, 100, False), (1, 32, 512, 32, False), (5, 16, 30, 2, True)])
@pytest.mark.parametrize("sizes", [[1000], [2, 63, 64, 65, 1], [1]])
def test_linear_attention(dev, dtype, tol, H, D, V, rot, silu, sizes):
    T = 200 if sizes != [1] else 40
    decay = [1.0, 0.05, 0.98, 0.7, 0.999][:H] if H > 1 else [0.95]
    x = rand(T, H * (2 * D + V) + 9, seed=3, dtype=dtype)
    x[T // 2:, :] *= 2
    kscale = D ** -0.5
    table, r = ops.DecayTable(decay), ops.Rotation(rot, 300.0)
    state = torch.full((3, H, D, V), 5.0, device=dev)       # what another request left
    xd = x.to(dev)
    cols = (slice(0, H * D), slice(H * D, 2 * H * D), slice(2 * H * D, 2 * H * D + H * V))
    got, at, i = [], 0, 0
    while at < T:
        n = min(sizes[i % len(sizes)], T - at)
        ctx = one_portion(n, at, [0] * (T // 16 + 1), dev, slot=1)
        q, k, v = (xd[at:at + n, c] for c in cols)
        kw = dict(silu=silu, kscale=kscale, cs=r.angles(ctx.positions) if rot else None)
        if n == 1:
            got.append(ops.linear_attn_decode(q, k, v, table, ctx.portions.state_slots,
                                              ctx.portions.seq_lens, state, **kw))
        else:
            got.append(ops.linear_attn_chunked(q, k, v, table, ctx.portions, state, **kw))
        at, i = at + n, i + 1
    q, k, v = (x[:, c].double().view(T, H, -1) for c in cols)
    if silu:
        q, k, v = orc.silu(q), orc.silu(k), orc.silu(v)
    pos = torch.arange(T)
    q = orc.rotate_half(q, pos, 300.0, rot)
    k = orc.rotate_half(k, pos, 300.0, rot) * kscale
    want, S = orc.decayed_sum(q, k, v, decay)
    close(torch.cat(got), want.reshape(T, -1), tol)
    close(state[1], S, max(tol / 4, 2e-5))
    assert (state[0] == 5.0).all() and (state[2] == 5.0).all()


@devices
def test_state_keeps_32_bits(dev):
    """A large old term must not swallow small new ones: half precision of the
    state or of the products with it would."""
    H, D, V, T = 1, 32, 32, 130
    x = torch.zeros(T, 3 * D)
    x[:, 0] = 1.0
    x[:, D] = 1.0
    x[0, 2 * D:] = 1024.0
    x[1:, 2 * D:] = rand(T - 1, V, seed=2) * 0.25
    x = x.to(torch.bfloat16)
    dtype = torch.bfloat16 if dev == "cuda" else torch.float32
    table = ops.DecayTable([1.0])
    want, S = orc.decayed_sum(*(x[:, c * D:(c + 1) * D].double().view(T, H, D) for c in range(3)),
                              [1.0])
    for sizes in ([T], [2, 64, 3], [1]):
        state = torch.full((1, H, D, V), 3.0, device=dev)
        at, i = 0, 0
        while at < T:
            n = min(sizes[i % len(sizes)], T - at)
            ctx = one_portion(n, at, [0] * 16, dev)
            q, k, v = (x.to(dtype).to(dev)[at:at + n, c * D:(c + 1) * D] for c in range(3))
            if n == 1:
                ops.linear_attn_decode(q, k, v, table, ctx.portions.state_slots,
                                       ctx.portions.seq_lens, state)
            else:
                ops.linear_attn_chunked(q, k, v, table, ctx.portions, state)
            at, i = at + n, i + 1
        assert (state[0].cpu().double()[:, 0] - S[:, 0]).abs().max() < 2e-3


# ----------------------------------------------------------- the whole model
@kinds
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_model_whole_prompt_and_layers(dev, dtype, tol, name):
    cfg = CONFIGS[name]
    model, oracle = make(cfg, dev, dtype)
    toks = tokens(cfg, 75)
    want, streams = oracle.forward(toks)
    s, got = SeqState(0, toks, 0), []
    eng = engine(model)
    hidden, _ = eng.step([(s, 75)], on_layer=lambda i, x: got.append(x.cpu()))
    for i, (g, w) in enumerate(zip(got, streams)):
        close(g, w, 3 * tol)
    assert len(got) == len(cfg["layers"])
    close(model.logits(hidden).float(), want, 4 * tol)


@kinds
@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("sizes", [[1], [2], [3, 1, 17, 64, 2], [64, 5]])
def test_portions_and_decoding(dev, dtype, tol, name, sizes):
    cfg = CONFIGS[name]
    model, oracle = make(cfg, dev, dtype)
    toks = tokens(cfg, 70 if min(sizes) < 3 else 150)
    s = SeqState(0, toks, 0)
    got = run(engine(model), cut(s, sizes))[0]
    close(got, oracle.forward(toks)[0], 4 * tol)


@kinds
def test_mixed_batches_and_reused_slots(dev, dtype, tol):
    """Unequal requests in one batch, some left out of steps, more requests
    than slots: each as if alone.  Freed pages and slots hold old contents."""
    cfg = CONFIGS["uneven"]
    model, oracle = make(cfg, dev, dtype)
    eng = engine(model, pool=16 * 16, slots=3)
    seqs = [SeqState(u, tokens(cfg, n, seed=u), 0) for u, n in enumerate((90, 1, 33, 64, 2, 50, 17))]
    pattern = [3, 1, 16, 2, 29, 1, 1, 40]
    waiting, live, logits, at = list(seqs), [], {}, 0
    while waiting or live:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        step = []
        for i, s in enumerate(live):
            if (at + i) % 4 == 3 and len(live) > 1:
                continue                        # left out of this step
            step.append((s, min(pattern[(at + 3 * i) % 8], len(s) - s.computed)))
        for u, x in run(eng, [step]).items():
            logits.setdefault(u, []).append(x)
        for s in list(live):
            if s.computed == len(s):
                eng.pool.release(s)
                live.remove(s)
        at += 1
    assert eng.pool.free_slots == 3 and eng.pool.free_pages == eng.pool.num_pages
    for s in seqs:
        close(torch.cat(logits[s.uid]), oracle.forward(s.tokens)[0], 4 * tol)


@devices
def test_pool_and_slots_run_out_loudly(dev):
    model, _ = make(CONFIGS["uneven"], dev)
    eng = engine(model, pool=64, slots=1)
    a = SeqState(0, [1] * 10, 0)
    eng.step([(a, 10)])
    with pytest.raises(RuntimeError, match="slot"):
        eng.step([(SeqState(1, [1, 2], 0), 2)])
    with pytest.raises(RuntimeError, match="exhausted"):
        a.tokens += [1] * 60
        eng.step([(a, 60)])
    with pytest.raises(ValueError):
        eng.step([(a, 61)])


def greedy_oracle(oracle, prompt, n):
    """Greedy continuation, and each step's margin over the runner-up."""
    toks, margins = list(prompt), []
    for _ in range(n):
        top = oracle.forward(toks)[0][-1].topk(2)
        margins.append(float(top.values[0] - top.values[1]))
        toks.append(int(top.indices[0]))
    return toks[len(prompt):], margins


@kinds
@pytest.mark.parametrize("kw", [dict(), dict(prefill_chunk_tokens=24), dict(use_graphs=False)])
def test_greedy_generation(dev, dtype, tol, kw):
    """Through generate(): admission, portions, decoding (graphs on the GPU),
    retirement; more prompts than state slots."""
    cfg = CONFIGS["uneven"]
    model, oracle = make(cfg, dev, dtype)
    eng = engine(model, pool=256, slots=2, compact_interval=8, **kw)
    prompts = [tokens(cfg, n, seed=n) for n in (30, 1, 47, 2, 18)]
    n = 40
    out, lps = eng.generate(prompts, SamplingParams(n=1, temperature=0.0, top_p=1.0, max_tokens=n),
                            return_logprobs=True)
    assert eng.pool.free_slots == 2 and eng.pool.free_pages == eng.pool.num_pages
    for r, p in enumerate(prompts):
        got = out[r].tolist()
        # follow what the engine chose: each choice is the oracle's best, or
        # within rounding of it
        logits = oracle.forward(p + got)[0][len(p) - 1:-1]
        best = logits.max(-1).values
        mine = logits.gather(1, torch.tensor(got)[:, None])[:, 0]
        size = logits.pow(2).mean().sqrt()
        assert ((best - mine) / size).max() < 8 * tol
        want_lp = torch.log_softmax(logits, -1).gather(1, torch.tensor(got)[:, None])[:, 0]
        assert (lps[r].double() - want_lp).abs().max() < 40 * tol * max(1, float(size))


@pytest.mark.gpu
def test_graph_replays_equal_eager_steps():
    cfg = CONFIGS["uneven"]
    model, _ = make(cfg, "cuda", torch.float32)
    prompts = [tokens(cfg, n, seed=n) for n in (30, 5, 12)]
    p = SamplingParams(n=2, temperature=0.8, top_p=0.9, max_tokens=60, seed=3)
    a = engine(model, pool=1024, slots=8, use_graphs=True)
    b = engine(model, pool=1024, slots=8, use_graphs=False)
    want = b.generate(prompts, p)
    for _ in range(3):
        assert torch.equal(a.generate(prompts, p), want)
        torch.cuda.synchronize()


@kinds
def test_long_decoding_forgets_and_keeps(dev, dtype, tol):
    """Far past the window; a slow decay and the kept tokens still reach back."""
    cfg = config(attention(size=9, keep=2), retention(decay=[0.9, 1.0, 0.9995]), lightning())
    model, oracle = make(cfg, dev, dtype)
    toks = tokens(cfg, 330)
    s = SeqState(0, toks, 0)
    got = run(engine(model), [[(s, 10)]] + [[(s, 1)]] * 320)[0]
    close(got, oracle.forward(toks)[0], 4 * tol)


# -------------------------------------------------- loading, registry, tools
def save(cfg, path, seed=0):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    t = orc.random_tensors(cfg, seed)
    save_file(t, os.path.join(path, "model.safetensors"))
    return t


def test_registry_loads_by_config(tmp_path):
    cfg = CONFIGS["odd-widths"]
    t = save(cfg, str(tmp_path))
    m = load_model(str(tmp_path), dtype="float32").eval()
    assert isinstance(m, GonuraxLM) and m.cfg.num_layers == 3
    toks = tokens(cfg, 20)
    s = SeqState(0, toks, 0)
    close(run(engine(m), cut(s, [20]))[0], orc.Oracle(cfg, t).forward(toks)[0], 1e-4)


def test_missing_extra_and_unknown_are_refused(tmp_path):
    cfg = CONFIGS["odd-widths"]
    t = orc.random_tensors(cfg)
    m = GonuraxLM(GonuraxConfig.from_json(cfg))
    with pytest.raises(KeyError, match="l1.mix.norm"):
        m.load({k: v for k, v in t.items() if k != "l1.mix.norm"})
    with pytest.raises(RuntimeError, match="unmapped"):
        m.load(dict(t, other=torch.zeros(1)))
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["type"] = "mystery"
    with pytest.raises(ValueError, match="mystery"):
        GonuraxConfig.from_json(bad)
    with open(tmp_path / "config.json", "w") as f:
        json.dump({"architecture": "Nobody"}, f)
    with pytest.raises(ValueError, match="Nobody"):
        load_model(str(tmp_path))
    with pytest.raises(ValueError, match="fp8"):
        SamplerEngine(m, kv_pool_tokens=64, kv_cache_dtype="fp8_e4m3", state_slots=1)


def test_cache_keeps_what_the_layers_need():
    cfg = get_config("gonurax-tiny")
    m = build_model(cfg)
    eng = SamplerEngine(m, kv_pool_tokens=64, max_num_seqs=5)
    kinds_ = [type(l) for l in eng.pool.layers]
    assert kinds_ == [torch.Tensor, tuple, torch.Tensor, torch.Tensor]
    assert eng.pool.num_slots == 5 and eng.pool.layers[0].dtype == torch.float32
    assert eng.pool.bytes_per_slot(cfg) == 3 * 2 * 32 * 48 * 4
    assert eng.pool.bytes_per_token(cfg) == 2 * (32 + 32) * 2


def test_serving_front_end_runs_it(tmp_path):
    pytest.importorskip("fastapi")
    import serve
    srv = serve.make_server(None, "gonurax-tiny", kv_pool_tokens=2048)
    assert len(srv.generate(["some text"], 5, 0.0, 1.0, 2)[0]) == 2
    save(CONFIGS["odd-widths"], str(tmp_path))
    srv = serve.make_server(str(tmp_path), "", kv_pool_tokens=2048)
    assert srv.tokenizer is None and srv.generate(["abc"], 4, 0.7, 0.9, 1)[0][0]


@pytest.mark.parametrize("dev,dtype", [("cpu", "float32"),
                                       pytest.param("cuda", "float32", marks=pytest.mark.gpu),
                                       pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)])
def test_trace_replay_program(tmp_path, dev, dtype):
    """bin/trace_run as a user runs it: a request that goes on after a pause,
    one that ends and makes room, logits only where wanted."""
    cfg = CONFIGS["uneven"]
    t = save(cfg, str(tmp_path / "m"))
    out = tmp_path / "out"
    out.mkdir()
    seqs = {n: tokens(cfg, k, seed=k) for n, k in
            (("a", 40), ("b", 33), ("c", 64), ("d", 3), ("e", 20))}
    plan = [[("a", 30), ("b", 1)], [("b", 31), ("c", 60), ("d", 2)], [("a", 1), ("c", 4), ("d", 1)],
            [("a", 9), ("e", 20)], [("b", 1)]]
    at, lines, want = {}, [], []
    for k, step in enumerate(plan):
        es, rows, end = [], [], []
        for n, c in step:
            lo = at.get(n, 0)
            at[n] = lo + c
            w = [0, c - 1] if c > 1 else [0]
            if k != 0:
                rows += [(n, lo + x) for x in w]
            es.append(dict(id=n, tokens=seqs[n][lo:lo + c], want=w if k != 0 else []))
            if at[n] == len(seqs[n]):
                end.append(n)
        lines.append(json.dumps(dict(step=k, entries=es, end=end)))
        want.append(rows)
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"),
                        "--dtype", dtype, "--out", str(out), "--max-tokens", "256",
                        "--device", dev], input="\n".join(lines) + "\n", capture_output=True,
                       text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.split("\n") if x.startswith("done")] == \
        [f"done {k}" for k in range(len(plan))]
    full = {n: orc.Oracle(cfg, t).forward(x)[0] for n, x in seqs.items()}
    assert not (out / "0.f32").exists()
    for k, rows in enumerate(want):
        if rows:
            got = torch.frombuffer(bytearray((out / f"{k}.f32").read_bytes()),
                                   dtype=torch.float32).view(len(rows), cfg["vocab"])
            close(got, torch.stack([full[n][p] for n, p in rows]),
                  1e-4 if dtype == "float32" else 0.08)


@pytest.mark.parametrize("dev", ["cpu", GPU])
def test_qwen2_runs_the_same_steps(dev):
    """The step function serves the attention-only model too: portions and
    mixed batches equal its packed forward."""
    from nanorlhf_amd.models import CausalLM, pack_sequences
    torch.manual_seed(0)
    cfg = get_config("tiny", dtype="bfloat16" if dev == "cuda" else "float32")
    m = CausalLM(cfg).to(getattr(torch, cfg.dtype)).to(dev).eval()
    toks = [torch.randint(2, 1000, (n,)).tolist() for n in (70, 25)]
    eng = SamplerEngine(m, kv_pool_tokens=256)
    a, b = SeqState(0, toks[0], 0), SeqState(1, toks[1], 1)
    got = run(eng, [[(a, 40), (b, 2)], [(a, 1), (b, 20)], [(a, 29)], [(b, 3)]])
    for u, x in enumerate(toks):
        ids, cu, mx, pos = pack_sequences([torch.tensor(x)], device=dev)
        with torch.no_grad():
            want = m.logits(m(ids, CausalLM.train_ctx(cu, mx, pos))).float().cpu()
        close(got[u], want, 2e-5 if dev == "cpu" else 0.03)
