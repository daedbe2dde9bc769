"""Plain, slow implementation of the layer-list designs (Birepel), written
straight from the equations: one function per mechanism, one sequence at a
time, one token at a time where a recurrence runs. Imports nothing from the
package under test. `h` is [tokens, width] and weights are 2-D float tensors
applied as h @ w.T.
"""
import math

import torch


def rms(x, eps):
    """x divided by its root mean square over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def zero_centred_norm(x, w, eps):
    return rms(x, eps) * (1 + w)


def query_temperature(pos, coef, every):
    """Factor that grows with the logarithm of how many blocks of `every`
    positions lie behind the query."""
    steps = torch.div(pos + 1, every, rounding_mode="floor")
    return 1 + coef * torch.log(steps.to(torch.float64) + 1)


def attend(q, k, v, scale, sink=None):
    """Causal softmax attention of one sequence, a sink in the denominator.
    q [t, H, d], k [t, G, d], v [t, G, dv] -> [t, H, dv]."""
    t, H, _ = q.shape
    G, dv = k.shape[1], v.shape[2]
    pos = torch.arange(t)
    out = torch.zeros(t, H, dv, dtype=q.dtype)
    for hd in range(H):
        kv = hd // (H // G)
        s = q[:, hd] @ k[:, kv].T * scale
        s = s.masked_fill(pos[None, :] > pos[:, None], float("-inf"))
        top = s.max(-1).values
        if sink is not None:
            top = torch.maximum(top, sink[hd])
        e = torch.exp(s - top[:, None])
        den = e.sum(-1)
        if sink is not None:
            den = den + torch.exp(sink[hd] - top)
        out[:, hd] = (e @ v[:, kv]) / den[:, None]
    return out


def attention(h, w, c, eps):
    """Grouped causal attention: unit-RMS q and k, a query temperature, one
    extra sink term per head in the denominator, one output gate per head."""
    t = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = rms((h @ w["q"].T).view(t, H, d), eps)
    k = rms((h @ w["k"].T).view(t, G, d), eps)
    v = (h @ w["v"].T).view(t, G, dv)
    temp = query_temperature(torch.arange(t), c["q_temp"]["coef"],
                             c["q_temp"]["every"]).to(h.dtype)
    out = attend(q * temp.view(t, 1, 1), k, v, c["scale"], w["sink"])
    out = out * torch.sigmoid(h @ w["g"].T)[:, :, None]
    return out.reshape(t, H * dv) @ w["o"].T


def soft_cap(x, cap):
    return cap * torch.tanh(x / cap)


def mlstm_step(S, n, m, q, k, v, i, f):
    """One token of every head. S [H, dim, vdim], n [H, dim], m [H]; q already
    scaled; i and f are the logarithms of the gates. Returns o and the state."""
    m_new = torch.maximum(f + m, i)
    keep, put = torch.exp(f + m - m_new), torch.exp(i - m_new)
    S = keep[:, None, None] * S + put[:, None, None] * k[:, :, None] * v[:, None]
    n = keep[:, None] * n + put[:, None] * k
    den = torch.maximum((n * q).sum(-1).abs(), torch.exp(-m_new)) + 1e-6
    return (S * q[:, :, None]).sum(1) / den[:, None], S, n, m_new


def mlstm_run(q, k, v, i, f):
    """One sequence from a zero state. q, k [t, H, d], v [t, H, dv],
    log gates [t, H] -> o [t, H, dv]."""
    t, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    n = torch.zeros(H, d, dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    o = []
    for p in range(t):
        out, S, n, m = mlstm_step(S, n, m, q[p], k[p], v[p], i[p], f[p])
        o.append(out)
    return torch.stack(o)


def mlstm_log_gates(zi, zf, cap):
    return soft_cap(zi, cap), torch.nn.functional.logsigmoid(soft_cap(zf, cap))


def mlstm(h, w, c, eps):
    t = h.shape[0]
    H, d, dv = c["heads"], c["dim"], c["vdim"]
    i, f = mlstm_log_gates(h @ w["i"].T + w["i.b"], h @ w["f"].T + w["f.b"],
                           c["gate_cap"])
    o = mlstm_run((h @ w["q"].T).view(t, H, d) * d ** -0.5,
                  (h @ w["k"].T).view(t, H, d), (h @ w["v"].T).view(t, H, dv),
                  i, f)
    o = rms(o, eps).reshape(t, H * dv) * w["norm"]
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def clamped_glu(g, u, limit):
    """Gate capped from above, linear part clamped on both sides and moved
    by one; the gate's own sigmoid has slope 1.702."""
    g = g.clamp(max=limit)
    u = u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def dense_ff(h, w, c):
    return clamped_glu(h @ w["gate"].T, h @ w["up"].T, c["limit"]) @ w["down"].T


def squared_relu(x):
    return torch.relu(x) ** 2


def route(h, w_router, top):
    """Chosen experts and their weights: softmax over the chosen logits."""
    z = h @ w_router.T
    val, idx = torch.topk(z, top, dim=-1)
    return idx, torch.softmax(val, dim=-1)


def moe(h, w, c):
    idx, wt = route(h, w["router"], c["router"]["top"])
    out = torch.zeros_like(h)
    for p in range(h.shape[0]):
        for j in range(idx.shape[1]):
            e = int(idx[p, j])
            y = squared_relu(h[p] @ w[f"e{e}.up"].T) @ w[f"e{e}.down"].T
            out[p] += wt[p, j] * y
    return out


def _under(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items()
            if k.startswith(prefix)}


def forward(cfg, weights, tokens, dtype=torch.float64):
    """Logits [tokens, vocab] of one sequence, and the residual stream after
    every layer [layers, tokens, width]."""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.as_tensor(tokens)
    x = W["embed"][ids] + W["pos"][torch.arange(len(ids))]
    trail = []
    for n, layer in enumerate(cfg["layers"]):
        p = f"l{layer.get('weights_of', n)}."
        mix = {"attention": attention, "mlstm": mlstm}[layer["type"]]
        x = x + zero_centred_norm(
            mix(x, _under(W, p + "mix."), layer["mixer"], eps),
            W[p + "norm1"], eps)
        ml = layer["mlp"]
        if ml is not None:
            ff = {"dense": dense_ff, "moe": moe}[ml["kind"]]
            x = x + zero_centred_norm(ff(x, _under(W, p + "mlp."), ml),
                                      W[p + "norm2"], eps)
        trail.append(x)
    x = zero_centred_norm(x, W["final.norm"], eps)
    return x @ W["embed"].T, torch.stack(trail)


def random_weights(cfg, seed=0, dtype=torch.bfloat16):
    """Random weights with every tensor that `cfg` asks for."""
    g = torch.Generator().manual_seed(seed)

    def r(*shape, std=None):
        std = shape[-1] ** -0.5 if std is None else std
        return (torch.randn(*shape, generator=g) * std).to(dtype)

    wd = cfg["width"]
    W = {"embed": r(cfg["vocab"], wd, std=1.0),
         "pos": r(cfg["max_positions"], wd, std=0.3),
         "final.norm": r(wd, std=0.2)}
    for n, layer in enumerate(cfg["layers"]):
        if "weights_of" in layer:
            continue
        p, c = f"l{n}.", layer["mixer"]
        H, d, dv = c["heads"], c["dim"], c["vdim"]
        W[p + "norm1"] = r(wd, std=0.2)
        kv = c.get("kv_heads", H)
        W[p + "mix.q"] = r(H * d, wd)
        W[p + "mix.k"] = r(kv * d, wd)
        W[p + "mix.v"] = r(kv * dv, wd)
        W[p + "mix.o"] = r(wd, H * dv)
        if layer["type"] == "attention":
            W[p + "mix.sink"] = r(H, std=1.0)
            W[p + "mix.g"] = r(H, wd)
        else:
            W[p + "mix.g"] = r(H * dv, wd)
            W[p + "mix.norm"] = (1 + 0.2 * torch.randn(
                H * dv, generator=g)).to(dtype)
            W[p + "mix.i"] = r(H, wd)
            W[p + "mix.i.b"] = r(H, std=1.0)
            W[p + "mix.f"] = r(H, wd)
            W[p + "mix.f.b"] = (3 + torch.randn(H, generator=g)).to(dtype)
        ml = layer["mlp"]
        if ml is None:
            continue
        W[p + "norm2"] = r(wd, std=0.2)
        if ml["kind"] == "dense":
            W[p + "mlp.gate"] = r(ml["ff"], wd)
            W[p + "mlp.up"] = r(ml["ff"], wd)
            W[p + "mlp.down"] = r(wd, ml["ff"])
        else:
            W[p + "mlp.router"] = r(ml["router"]["experts"], wd, std=0.3)
            for e in range(ml["router"]["experts"]):
                W[f"{p}mlp.e{e}.up"] = r(ml["expert"]["ff"], wd)
                W[f"{p}mlp.e{e}.down"] = r(wd, ml["expert"]["ff"])
    return W
