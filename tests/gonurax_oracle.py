"""Plain, slow Gonurax: one function per mechanism, written from the design's
equations with ordinary torch operations.  It shares no code with the package
and is what the tests compare the package against.

`rnd` is applied wherever a half-precision implementation may round (linear
outputs and the operands of linears); the identity gives the exact model.
"""
import math

import torch


def angles(positions, base, dims):
    """[T, dims/2] rotation angles p * base^(-2i/dims), in float64."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    return positions.double()[:, None] * base ** (-2.0 * i / dims)[None, :]


def turn(u, v, a):
    """Rotate the pairs (u, v) by the angles a."""
    c, s = a.cos().to(u.dtype), a.sin().to(u.dtype)
    return u * c - v * s, v * c + u * s


def rotate_half(x, positions, base, dims):
    """x [T, heads, D]: dimension i pairs with i + dims/2; the rest passes."""
    a = angles(positions, base, dims)[:, None, :]
    h = dims // 2
    u, v = turn(x[..., :h], x[..., h:dims], a)
    return torch.cat([u, v, x[..., dims:]], -1)


def rotate_interleaved(x, positions, base, dims, sign=1):
    """x [T, heads, D]: dimension 2i pairs with 2i + 1; the rest passes."""
    a = angles(positions, base, dims)[:, None, :] * sign
    u, v = turn(x[..., 0:dims:2], x[..., 1:dims:2], a)
    out = x.clone()
    out[..., 0:dims:2] = u
    out[..., 1:dims:2] = v
    return out


def rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def group_rms(x, w, groups, eps):
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms(parts, eps).reshape(x.shape) * w


def visible(i, j, size, keep_first):
    return j <= i and (i - j < size or j < keep_first)


def visible_mask(n, size, keep_first):
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def windowed_attention(q, k, v, scale, size, keep_first):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    mask = visible_mask(T, size, keep_first)
    out = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h // rep].T) * scale
        s = s.masked_fill(~mask, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, h // rep]
    return out


def decayed_sum(q, k, v, decay, state=None):
    """Token by token: S <- decay S + k v^T, o = S^T q.
    q, k [T, H, D], v [T, H, V], decay [H] -> (o [T, H, V], S [H, D, V])."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    d = torch.as_tensor(decay, dtype=torch.float64).to(q.dtype)[:, None, None]
    out = []
    for t in range(T):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((q[t][:, :, None] * S).sum(1))
    return torch.stack(out), S


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


class Oracle:
    def __init__(self, config, tensors, dtype=torch.float64, rnd=lambda x: x):
        self.c = config
        self.w = {n: t.to(dtype) for n, t in tensors.items()}
        self.dtype = dtype
        self.rnd = rnd

    def lin(self, name, x):
        return self.rnd(self.rnd(x) @ self.w[name].T)

    def retention(self, p, m, h, pos):
        T, H = h.shape[0], m["heads"]
        q = self.lin(p + "q", h).view(T, H, m["dim"])
        k = self.lin(p + "k", h).view(T, H, m["dim"])
        v = self.lin(p + "v", h).view(T, H, m["vdim"])
        r = m["rot"]
        q = rotate_half(q, pos, r["base"], r["dims"])
        k = rotate_half(k, pos, r["base"], r["dims"]) * m["dim"] ** -0.5
        o, _ = decayed_sum(q, k, v, m["decay"])
        o = rms(o, self.c["norm"]["eps"]).reshape(T, -1)
        return self.lin(p + "o", o * silu(self.lin(p + "g", h)))

    def lightning(self, p, m, h, pos):
        T, H = h.shape[0], m["heads"]
        q = silu(self.lin(p + "q", h)).view(T, H, m["dim"])
        k = silu(self.lin(p + "k", h)).view(T, H, m["dim"])
        v = silu(self.lin(p + "v", h)).view(T, H, m["vdim"])
        o, _ = decayed_sum(q, k, v, m["decay"])
        o = rms(o.reshape(T, -1), self.c["norm"]["eps"]) * self.w[p + "norm"]
        return self.lin(p + "o", o * torch.sigmoid(self.lin(p + "g", h)))

    def attention(self, p, m, h, pos):
        T, eps, r = h.shape[0], self.c["norm"]["eps"], m["rot"]
        q = self.lin(p + "q", h).view(T, m["heads"], m["dim"])
        k = self.lin(p + "k", h).view(T, m["kv_heads"], m["dim"])
        v = self.lin(p + "v", h).view(T, m["kv_heads"], m["vdim"])
        q = rms(q, eps) * self.w[p + "q.norm"]
        k = rms(k, eps) * self.w[p + "k.norm"]
        q = self.rnd(rotate_interleaved(q, pos, r["base"], r["dims"]))
        k = self.rnd(rotate_interleaved(k, pos, r["base"], r["dims"]))
        v = self.rnd(rotate_interleaved(v, pos, r["base"], m["vdim"]))
        o = windowed_attention(q, k, v, m["scale"], m["mask"]["size"],
                               m["mask"]["keep_first"])
        o = rotate_interleaved(o, pos, r["base"], m["vdim"], sign=-1)
        return self.lin(p + "o", o.reshape(T, -1))

    def dense(self, p, h):
        return self.lin(p + "down", gelu_tanh(self.lin(p + "gate", h)) * self.lin(p + "up", h))

    def forward(self, tokens):
        """Logits [T, vocab] and the residual stream after every layer."""
        c = self.c
        pos = torch.arange(len(tokens))
        x = self.w["embed"][torch.tensor(tokens)]
        streams = []
        for i, layer in enumerate(c["layers"]):
            h = group_rms(x, self.w[f"l{i}.norm1"], c["norm"]["groups"], c["norm"]["eps"])
            y = getattr(self, layer["type"])(f"l{i}.mix.", layer["mixer"], h, pos)
            if layer["mlp"] is not None:
                y = y + self.dense(f"l{i}.mlp.", h)
            x = x + c["residual_mult"] * y
            streams.append(x)
        h = group_rms(x, self.w["final.norm"], c["norm"]["groups"], c["norm"]["eps"])
        return self.rnd(h) @ self.w["embed"].T, streams


def tensor_shapes(c):
    """Name -> shape of every weight of a configuration."""
    W, out = c["width"], {"embed": (c["vocab"], c["width"])}
    for i, layer in enumerate(c["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        H, D, V = m["heads"], m["dim"], m["vdim"]
        G = m.get("kv_heads", H)
        out[f"l{i}.norm1"] = (W,)
        out.update({p + "q": (H * D, W), p + "k": (G * D, W), p + "v": (G * V, W)})
        if layer["type"] == "attention":
            out.update({p + "q.norm": (D,), p + "k.norm": (D,)})
        else:
            out[p + "g"] = (H * V, W)
        if layer["type"] == "lightning":
            out[p + "norm"] = (H * V,)
        out[p + "o"] = (W, H * V)
        if layer["mlp"] is not None:
            F = layer["mlp"]["ff"]
            p = f"l{i}.mlp."
            out.update({p + "gate": (F, W), p + "up": (F, W), p + "down": (W, F)})
    out["final.norm"] = (W,)
    return out


def random_tensors(c, seed=0, sharp=2.0):
    """bfloat16 weights whose activations stay of order one; `sharp` scales
    queries and keys so that attention is not flat."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(c).items():
        x = torch.randn(*shape, generator=g)
        if len(shape) == 1:
            x = 1 + 0.2 * x
            if name.endswith((".q.norm", ".k.norm")):
                x = x * sharp
        elif name != "embed":
            x = x / math.sqrt(shape[1])
        out[name] = x.to(torch.bfloat16)
    return out
