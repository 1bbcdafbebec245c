"""Plain, slow Pemolorn: one function per mechanism, straight from the equations, in torch on the CPU.

Written for comparison only: it shares no code with the package, keeps no cache and no state (a sequence is
always recomputed whole) and loops over tokens, heads and experts where that is clearest.  All functions work in
the dtype of their inputs (float32 or float64).
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square, eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def scalar_norm(x, g, eps):
    """One gain for all coordinates."""
    return rms(x, eps) * g


def short_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the first token."""
    T, taps = u.shape[0], w.shape[1]
    ext = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return sum(w[:, j] * ext[j:j + T] for j in range(taps))


def rotate(x, positions, base, dims):
    """x [T, heads, D]: neighbours (2i, 2i + 1) of the first ``dims`` dimensions turned by position * base^(-2i / dims)."""
    out = x.clone()
    i = torch.arange(dims // 2, dtype=torch.float64)
    a = positions.to(torch.float64)[:, None] * base ** (-2.0 * i / dims)
    c, s = a.cos().to(x.dtype)[:, None], a.sin().to(x.dtype)[:, None]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def window_mask(T, size, keep=0):
    """True where token i sees token j: its last ``size`` tokens and the first ``keep``."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    return (j <= i) & ((i - j < size) | (j < keep))


def pooled_mask(T, size, pool):
    """True where token i sees block b (tokens b pool .. b pool + pool - 1)."""
    i, last = torch.arange(T)[:, None], torch.arange(T // pool)[None] * pool + pool - 1
    return last <= i - size


def pooled(x, pool):
    """x [T, ...]: means of whole blocks."""
    n = x.shape[0] // pool
    return x[:n * pool].reshape(n, pool, *x.shape[1:]).mean(1)


def sink_softmax(scores, sink):
    """Row softmax whose denominator also holds exp(sink)."""
    z = torch.cat([scores, torch.zeros_like(scores[:, :1]) + sink], 1)
    return torch.softmax(z, 1)[:, :-1]


def attend(q, k, v, scale, mask, sink):
    """q [T, H, D], k [T, G, D], v [T, G, V]; mask: size with keep_first or pool.  Heads side by side [T, H V]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    see = window_mask(T, mask["size"], mask.get("keep_first", 0))
    pool, out = mask.get("pool"), []
    if pool:
        k, v = torch.cat([k, pooled(k, pool)]), torch.cat([v, pooled(v, pool)])
        see = torch.cat([see, pooled_mask(T, mask["size"], pool)], 1)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T * scale).masked_fill(~see, -math.inf)
        out.append(sink_softmax(s, sink[h]) @ v[:, g])
    return torch.cat(out, 1)


def attention(h, p, m, eps, kv=None):
    """Window attention with kept first tokens; per-head norms.  ``kv``: another layer's (keys, values).  Returns the
    output and this layer's keys and values."""
    T = h.shape[0]
    q = rms((h @ p["q"].T).view(T, m["heads"], m["dim"]), eps) * p["q.norm"]
    if kv is None:
        k = rms((h @ p["k"].T).view(T, m["kv_heads"], m["dim"]), eps) * p["k.norm"]
        kv = k, (h @ p["v"].T).view(T, m["kv_heads"], m["vdim"])
    return attend(q, *kv, m["scale"], m["mask"], p["sink"]) @ p["o"].T, kv


def pooled_attention(h, p, m, eps):
    """Convolved projections, norms over whole projections, rotation, window and pooled blocks."""
    T, pos = h.shape[0], torch.arange(h.shape[0])

    def proj(name):
        return short_conv(h @ p[name].T, p[name + ".conv"])
    q = (rms(proj("q"), eps) * p["q.norm"]).view(T, m["heads"], m["dim"])
    k = (rms(proj("k"), eps) * p["k.norm"]).view(T, m["kv_heads"], m["dim"])
    v = proj("v").view(T, m["kv_heads"], m["vdim"])
    q, k = (rotate(x, pos, m["rot"]["base"], m["rot"]["dims"]) for x in (q, k))
    return attend(q, k, v, m["scale"], m["mask"], p["sink"]) @ p["o"].T


def min_gru(z, u):
    """Pre-activations of the gate and the candidate [T, C]: the states S_t [T, C], from zero."""
    S, out = torch.zeros_like(z[0]), []
    for t in range(z.shape[0]):
        g = torch.sigmoid(z[t])
        c = torch.where(u[t] >= 0, u[t] + 0.5, torch.sigmoid(u[t]))
        S = (1 - g) * S + g * c
        out.append(S)
    return torch.stack(out)


def recurrence(h, p):
    S = min_gru(h @ p["z"].T + p["z.b"], h @ p["x"].T + p["x.b"])
    gate = h @ p["g"].T
    return (S * gate * torch.sigmoid(gate)) @ p["o"].T


def parallel(h, p, m, eps):
    left = pooled_attention(h, section(p, "left."), m["left"], eps)
    right = recurrence(h, section(p, "right."))
    return (rms(left, eps) * p["left.out"] + rms(right, eps) * p["right.out"]) / 2


def relu_squared(h, p):
    return torch.clamp(h @ p["up"].T, min=0.0) ** 2 @ p["down"].T


def expert(h, p, name, limit):
    g = torch.clamp(h @ p[name + ".gate"].T, max=limit)
    u = torch.clamp(h @ p[name + ".up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ p[name + ".down"].T


def route(h, p, top):
    """Per token the chosen outputs of the router and their weights: two lists of lists."""
    score = torch.softmax(h @ p["router"].T, -1)
    choice = score + p["correction"]
    ids, weights = [], []
    for t in range(h.shape[0]):
        c = choice[t].tolist()
        best = sorted(range(len(c)), key=lambda e: -c[e])[:top]
        ids.append(best)
        weights.append([score[t, e] for e in best])
    return ids, weights


def experts(h, p, f):
    n = f["router"]["experts"]
    ids, weights = route(h, p, f["router"]["top"])
    return torch.stack([sum(w * (expert(h[t], p, f"e{e}", f["expert"]["limit"]) if e < n else h[t])
                            for e, w in zip(ids[t], weights[t])) for t in range(h.shape[0])])


def section(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def forward(cfg, w, tokens, dtype=torch.float32):
    """cfg: the parsed config.json; w: name -> tensor.  Returns (logits [T, vocab], stream after every layer)."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps, after, kvs = cfg["norm"]["eps"], [], {}
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = section(w, f"l{i}."), layer["mixer"], layer["mlp"]
        mix, h = section(p, "mix."), scalar_norm(x, p["norm1"], eps)
        if layer["type"] == "parallel":
            y = parallel(h, mix, m, eps)
        else:
            y, kvs[i] = attention(h, mix, m, eps, kvs.get(m.get("kv_from")))
        x = x + scalar_norm(y, p["norm1b"], eps)
        if f is not None:
            h, ffw = scalar_norm(x, p["norm2"], eps), section(p, "mlp.")
            y = relu_squared(h, ffw) if f["kind"] == "dense" else experts(h, ffw, f)
            x = x + scalar_norm(y, p["norm2b"], eps)
        after.append(x)
    return scalar_norm(x, w["final.norm"], eps) @ w["head"].T, torch.stack(after)
