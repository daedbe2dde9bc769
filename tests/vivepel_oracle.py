"""Plain, slow implementation of Vivepel, written straight from the equations:
one function per mechanism, one sequence at a time, one head at a time. Imports
nothing from the package under test. `h` is [tokens, width] and weights are
float tensors applied as h @ w.T.
"""
import torch

from hybrid_oracle import _under, rms


def group_norm(x, w, groups, eps):
    """Unit RMS of each of `groups` equal consecutive parts, times w."""
    n = x.shape[-1] // groups
    parts = [rms(x[..., g * n:(g + 1) * n], eps) for g in range(groups)]
    return torch.cat(parts, dim=-1) * w


def rotate_half(x, pos, base, dims):
    """Turn the pairs (i, i + dims / 2) of x [t, ..., d] by
    pos * base^(-2 i / dims)."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        a = pos.to(torch.float64) * base ** (-2 * i / dims)
        shape = [-1] + [1] * (x.dim() - 2)
        c = torch.cos(a).to(x.dtype).view(shape)
        s = torch.sin(a).to(x.dtype).view(shape)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def keys_of(v, w, pos, base, dims, eps):
    """Keys from values: normed, weighted, rotated."""
    return rotate_half(rms(v, eps) * w, pos, base, dims)


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap)


def same_chunk(t, n, size):
    """[t, n] bool: which keys the last t of n positions see."""
    return torch.tensor([[j <= i and i // size == j // size for j in range(n)]
                         for i in range(n - t, n)])


def softmax_plus_one(s, seen):
    """exp(s) / (1 + sum exp(s)) over the seen."""
    s = s.masked_fill(~seen, float("-inf"))
    m = s.max(-1, keepdim=True).values.clamp(min=0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def mix_heads(p, talk):
    """Weights of output heads from those of score heads; p [H, t, n]."""
    return torch.stack([sum(talk[h, g] * p[g] for g in range(p.shape[0]))
                        for h in range(p.shape[0])])


def attend(q, k, v, talk, scale, cap, size):
    """q [t, H, d] of the last t of n positions, k and v [n, G, d] ->
    [t, H, d]."""
    t, H, _ = q.shape
    n, G, _ = k.shape
    seen = same_chunk(t, n, size)
    p = torch.stack([softmax_plus_one(
        soft_cap(q[:, h] @ k[:, h * G // H].T * scale, cap), seen)
        for h in range(H)])
    wt = mix_heads(p, talk)
    return torch.stack([wt[h] @ v[:, h * G // H] for h in range(H)], dim=1)


def attention(h, w, c, eps):
    t, H, G, d = h.shape[0], c["heads"], c["kv_heads"], c["dim"]
    pos = torch.arange(t)
    base, dims = c["rot"]["base"], c["rot"]["dims"]
    q = (h @ w["q"].T + w["q.b"]).view(t, H, d)
    v = (h @ w["k"].T + w["k.b"]).view(t, G, d)
    out = attend(keys_of(q, w["q.norm"], pos, base, dims, eps),
                 keys_of(v, w["k.norm"], pos, base, dims, eps), v, w["talk"],
                 c["scale"], c["softcap"], c["mask"]["size"])
    return out.reshape(t, H * d) @ w["o"].T


def poly_norm(z, coef, eps):
    """Three normed powers and a constant."""
    return coef[3] + sum(coef[k] * rms(z ** (k + 1), eps) for k in range(3))


def dense_ff(h, w, eps):
    return poly_norm(h @ w["up"].T, w["act"], eps) @ w["down"].T


def forward(cfg, weights, tokens, dtype=torch.float64):
    """Logits [tokens, vocab] of one sequence, and the residual stream behind
    every layer [layers, tokens, width]."""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x, trail = W["embed"][torch.as_tensor(tokens)], []

    def norm(z, name):
        return group_norm(z, W[name], groups, eps)

    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = attention(norm(x, p + "norm1"), _under(W, p + "mix."),
                      layer["mixer"], eps)
        x = x + norm(y, p + "norm1b") * W[p + "ls1"]
        if layer["mlp"] is not None:
            y = dense_ff(norm(x, p + "norm2"), _under(W, p + "mlp."), eps)
            x = x + norm(y, p + "norm2b") * W[p + "ls2"]
        trail.append(x)
    return norm(x, "final.norm") @ W["head"].T, torch.stack(trail)


def random_weights(cfg, seed=0, dtype=torch.bfloat16):
    """Random weights with every tensor that `cfg` asks for."""
    g = torch.Generator().manual_seed(seed)

    def r(*shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        return (mean + torch.randn(shape, generator=g) * std).to(dtype)

    wd = cfg["width"]

    def one(n=wd):
        return r(n, mean=1.0, std=0.2)

    W = {"embed": r(cfg["vocab"], wd, std=1.0), "final.norm": one(),
         "head": r(cfg["vocab"], wd)}
    for n, layer in enumerate(cfg["layers"]):
        p, c, ml = f"l{n}.", layer["mixer"], layer["mlp"]
        H, G, d = c["heads"], c["kv_heads"], c["dim"]
        W |= {p + "norm1": one(), p + "norm1b": one(), p + "ls1": one(),
              p + "mix.q": r(H * d, wd), p + "mix.q.b": r(H * d, std=0.3),
              p + "mix.k": r(G * d, wd), p + "mix.k.b": r(G * d, std=0.3),
              p + "mix.q.norm": one(d), p + "mix.k.norm": one(d),
              p + "mix.talk": r(H, H, std=0.4), p + "mix.o": r(wd, H * d)}
        if ml is not None:
            W |= {p + "norm2": one(), p + "norm2b": one(), p + "ls2": one(),
                  p + "mlp.up": r(ml["ff"], wd),
                  p + "mlp.down": r(wd, ml["ff"]),
                  p + "mlp.act": r(4, std=0.5)}
    return W
