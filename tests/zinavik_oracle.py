"""Plain, slow implementation of Zinavik, written straight from the equations:
one function per mechanism, one sequence at a time, one head at a time, one
token at a time where a recurrence runs. Imports nothing from the package under
test. `h` is [tokens, width] and weights are float tensors applied as h @ w.T.
"""
import math

import torch

from hybrid_oracle import _under, rms


def yarn_frequencies(base, dims, scaling):
    """Angle per position of every pair, and the factor on cosines and
    sines."""
    f = [base ** (-2 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return f, 1.0

    def turns(t):               # the pair that turns t times in the old length
        return dims * math.log(scaling["original"] / (2 * math.pi * t)) / \
            (2 * math.log(base))
    lo = max(math.floor(turns(scaling["fast"])), 0)
    hi = min(math.ceil(turns(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / scaling["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1


def rotate(x, pos, rot):
    """Turn the neighbouring pairs of the first dims coordinates of
    x [t, ..., d]."""
    f, m = yarn_frequencies(rot["base"], rot["dims"], rot.get("scaling"))
    out = x.clone()
    for i, fi in enumerate(f):
        a = (pos.to(torch.float64) * fi).view([-1] + [1] * (x.dim() - 2))
        c, s = (m * torch.cos(a)).to(x.dtype), (m * torch.sin(a)).to(x.dtype)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def visible(t, n, size, keep):
    """[t, n] bool: which keys the last t of n positions see."""
    i, j = torch.arange(n - t, n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep))


def attend(q, k, v, scale, seen):
    """q [t, H, d], k [n, G, d], v [n, G, dv], seen [t, n] -> [t, H, dv]."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T * scale).masked_fill(~seen, float("-inf"))
        out.append(torch.softmax(s, -1) @ v[:, g])
    return torch.stack(out, dim=1)


def attention(h, w, c, eps):
    """Window attention up to the output projection: [t, H * vdim]."""
    t, H, G, d, dv = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    pos = torch.arange(t)
    q = rms(rotate((h @ w["q"].T).view(t, H, d), pos, c["rot"]), eps)
    k = rms(rotate((h @ w["k"].T).view(t, G, d), pos, c["rot"]), eps)
    v = (h @ w["v"].T).view(t, G, dv)
    seen = visible(t, t, c["mask"]["size"], c["mask"]["keep_first"])
    o = attend(q, k, v, c["scale"], seen).reshape(t, H * dv)
    return o * torch.sigmoid(h @ w["g"].T)


def silu(z):
    return z * torch.sigmoid(z)


def decaying_memory(q, k, v, decay):
    """q, k [t, H, d], v [t, H, dv] -> [t, H, dv], token by token."""
    S = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype)
    lam = torch.tensor(decay, dtype=torch.float64).to(q.dtype).view(-1, 1, 1)
    out = []
    for t in range(q.shape[0]):
        S = lam * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def lightning(h, w, c, eps):
    """Linear attention with constant decays up to the output projection."""
    t, H = h.shape[0], c["heads"]
    q, k, v = (silu(h @ w[n].T).view(t, H, -1) for n in "qkv")
    o = decaying_memory(q, k, v, c["decay"]).reshape(t, -1)
    return rms(o, eps) * w["norm"] * torch.sigmoid(h @ w["g"].T)


def parallel(h, w, c, eps):
    wl, wr = _under(w, "left."), _under(w, "right.")
    return c["left_scale"] * (attention(h, wl, c["left"], eps) @ wl["o"].T) + \
        c["right_scale"] * (lightning(h, wr, c["right"], eps) @ wr["o"].T)


def expert(h, w, limit):
    g = torch.clamp(h @ w["gate"].T, max=limit)
    u = torch.clamp(h @ w["up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w["down"].T


def choose(z, top):
    """Places of the `top` largest logits and their sigmoid scores."""
    s = torch.sigmoid(z)
    at = torch.topk(z, top, dim=-1).indices
    return at, s.gather(-1, at)


def routed(h, w, c):
    """Each token's chosen experts on its weighted input, and the shared expert
    on its plain one."""
    at, s = choose(h @ w["router"].T, c["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(c["router"]["experts"]):
        for t, k in (at == e).nonzero().tolist():
            out[t] = out[t] + expert(s[t, k] * h[t], _under(w, f"e{e}."),
                                     c["expert"]["limit"])
    if c.get("shared") is not None:
        ws = _under(w, "shared.")
        out = out + expert(h, ws, c["shared"]["limit"]) * \
            torch.sigmoid(h @ ws["sg"].T)
    return out


def sublayer(xs, w, norm, eps, fn):
    """xs [streams, t, width]: read by w['in'], apply fn to the normed sum,
    mix the streams and write its result back."""
    u = sum(w["in"][s] * xs[s] for s in range(len(xs)))
    y = fn(rms(u, eps) * norm)
    return torch.stack([
        sum(w["mix"][s, t] * xs[s] for s in range(len(xs))) + w["out"][t] * y
        for t in range(len(xs))])


def order_of(cfg):
    """Numbers of the layers in the order they run in."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return list(range(n))
    body = list(range(loop["start"], loop["stop"]))
    return list(range(loop["start"])) + body * loop["times"] + \
        list(range(loop["stop"], n))


def forward(cfg, weights, tokens, dtype=torch.float64):
    """Logits [tokens, vocab] of one sequence, and the sum of the streams
    behind every layer run [runs, tokens, width]."""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    xs, trail = torch.stack([x] * cfg["streams"]), []
    for i in order_of(cfg):
        p, ly = f"l{i}.", cfg["layers"][i]
        xs = sublayer(xs, _under(W, p + "hc1."), W[p + "norm1"], eps,
                      lambda h: parallel(h, _under(W, p + "mix."),
                                         ly["mixer"], eps))
        if ly["mlp"] is not None:
            xs = sublayer(xs, _under(W, p + "hc2."), W[p + "norm2"], eps,
                          lambda h: routed(h, _under(W, p + "mlp."),
                                           ly["mlp"]))
        trail.append(xs.sum(0))
    return rms(xs.sum(0), eps) * W["final.norm"] @ W["embed"].T, \
        torch.stack(trail)


def random_weights(cfg, seed=0, dtype=torch.bfloat16):
    """Random weights with every tensor that `cfg` asks for."""
    g = torch.Generator().manual_seed(seed)

    def r(*shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        return (mean + torch.randn(shape, generator=g) * std).to(dtype)

    wd, s = cfg["width"], cfg["streams"]

    def one(n=wd):
        return r(n, mean=1.0, std=0.2)

    def glu(p, ff):
        return {p + "gate": r(ff, wd), p + "up": r(ff, wd),
                p + "down": r(wd, ff, std=0.4 * ff ** -0.5)}

    W = {"embed": r(cfg["vocab"], wd, std=1 / cfg["embedding"]["scale"]),
         "final.norm": one()}
    for n, ly in enumerate(cfg["layers"]):
        p, a, b, ml = f"l{n}.", ly["mixer"]["left"], ly["mixer"]["right"], \
            ly["mlp"]
        ql, kl = a["heads"] * a["dim"], a["kv_heads"] * a["dim"]
        vl, ol = a["kv_heads"] * a["vdim"], a["heads"] * a["vdim"]
        qr, vr = b["heads"] * b["dim"], b["heads"] * b["vdim"]
        left, right = p + "mix.left.", p + "mix.right."
        W |= {left + "q": r(ql, wd), left + "k": r(kl, wd),
              left + "v": r(vl, wd), left + "g": r(ol, wd),
              left + "o": r(wd, ol), right + "q": r(qr, wd),
              right + "k": r(qr, wd), right + "v": r(vr, wd),
              right + "g": r(vr, wd), right + "o": r(wd, vr),
              right + "norm": one(vr)}
        for k in (1, 2) if ml is not None else (1,):
            W |= {f"{p}norm{k}": one(), f"{p}hc{k}.in": r(s, mean=0.6, std=0.2),
                  f"{p}hc{k}.out": r(s, mean=0.5, std=0.2),
                  f"{p}hc{k}.mix": (torch.eye(s) * 0.9 + r(s, s, std=0.15)
                                    ).to(dtype)}
        if ml is None:
            continue
        W[p + "mlp.router"] = r(ml["router"]["experts"], wd,
                                std=2 * wd ** -0.5)
        for e in range(ml["router"]["experts"]):
            W |= glu(f"{p}mlp.e{e}.", ml["expert"]["ff"])
        if ml.get("shared") is not None:
            W |= glu(p + "mlp.shared.", ml["shared"]["ff"])
            W[p + "mlp.shared.sg"] = r(1, wd)
    return W
