"""Plain, slow Zisapel: one function per mechanism, straight from the equations, in torch on the CPU.

Written for comparison only: it shares no code with the package, keeps no cache and no state (a
sequence is always recomputed whole) and loops over tokens, heads and experts where that is clearest.
All functions work in the dtype of their inputs (float32 or float64).
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square, eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def before(h):
    """Row t holds h of token t - 1; zeros for the first."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def mix(h, mu):
    return h + (before(h) - h) * mu


def gated(y, h, w, b):
    return y * torch.sigmoid(h @ w.T + b)


def yarn_angles(T, rot, dtype):
    """(cos, sin) [T, dims / 2] with the length scaling's magnitude in both."""
    n, base = rot["dims"], rot["base"]
    i = torch.arange(n // 2, dtype=torch.float64)
    f, mag = base ** (-2.0 * i / n), 1.0
    s = rot.get("scaling")
    if s:
        def dim(t):
            return n * math.log(s["original"] / (2 * math.pi * t)) / (2 * math.log(base))
        lo, hi = max(math.floor(dim(s["fast"])), 0), min(math.ceil(dim(s["slow"])), n - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        f = f / s["factor"] * ramp + f * (1 - ramp)
        mag = 0.1 * math.log(s["factor"]) + 1.0
    a = torch.arange(T, dtype=torch.float64)[:, None] * f
    return (a.cos() * mag).to(dtype), (a.sin() * mag).to(dtype)


def rotate_pairs(x, cos, sin):
    """x [T, ..., dims]: neighbours (2i, 2i + 1) rotated."""
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (-1,)
    c, s = cos.view(shape), sin.view(shape)
    u, v = x[..., 0::2], x[..., 1::2]
    out = torch.empty_like(x)
    out[..., 0::2] = u * c - v * s
    out[..., 1::2] = v * c + u * s
    return out


def window_mask(T, size):
    """True where query i sees key j."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None]
    return (d >= 0) & (d < size)


def softmax_with_sink(scores, sink):
    """Row softmax whose denominator also holds exp(sink)."""
    z = torch.cat([scores, torch.full_like(scores[:, :1], 0.0) + sink], 1)
    return torch.softmax(z, 1)[:, :-1]


def latent_attention(h, p, m, eps):
    """m: heads, dim, rot_dim, vdim, kv_rank, scale, rot, mask; p: q, dkv, dkv.norm, uk, uv, sink, g, o."""
    T, H, D, R, V = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = (h @ p["q"].T).view(T, H, D + R)
    down = h @ p["dkv"].T
    c = rms(down[:, :m["kv_rank"]], eps) * p["dkv.norm"]
    cos, sin = yarn_angles(T, m["rot"], h.dtype)
    kr = rotate_pairs(down[:, m["kv_rank"]:], cos, sin)
    qr = rotate_pairs(q[:, :, D:], cos, sin)
    k = (c @ p["uk"].T).view(T, H, D)
    v = (c @ p["uv"].T).view(T, H, V)
    see = window_mask(T, m["mask"]["size"])
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for n in range(H):
        s = (q[:, n, :D] @ k[:, n].T + qr[:, n] @ kr.T) * m["scale"]
        out[:, n] = softmax_with_sink(s.masked_fill(~see, -math.inf), p["sink"][n]) @ v[:, n]
    return (out.reshape(T, H * V) * torch.sigmoid(h @ p["g"].T)) @ p["o"].T


def wkv_decay(hw, p):
    return torch.exp(-torch.exp(torch.tanh(hw @ p["w1"].T) @ p["w2"].T + p["w0"]))


def wkv_recurrence(r, k, v, w, u):
    """r, k, v, w [T, H, D], u [H, D]: outputs [T, H, D], token by token."""
    T, H, D = r.shape
    S = torch.zeros(H, D, D, dtype=r.dtype)          # [key channel, value channel]
    out = torch.zeros_like(v)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hij,hi->hj", S + u[:, :, None] * kv, r[t])
        S = w[t][:, :, None] * S + kv
    return out


def wkv(h, p, m, eps):
    T, H, D = h.shape[0], m["heads"], m["dim"]

    def heads(x):
        return x.view(T, H, D)
    r, k, v = (heads(mix(h, p["mu." + s]) @ p[s].T) for s in "rkv")
    z = mix(h, p["mu.g"]) @ p["g"].T
    gate = z * torch.sigmoid(z)
    w = heads(wkv_decay(mix(h, p["mu.w"]), p))
    o = rms(wkv_recurrence(r, k, v, w, p["u"]), eps).reshape(T, H * D)
    return (o * p["norm"] * gate) @ p["o"].T


def clamped_glu(h, p, limit):
    g = torch.clamp(h @ p["gate"].T, max=limit)
    u = torch.clamp(h @ p["up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ p["down"].T


def expert(h, p, name):
    z = h @ p[name + ".gate"].T
    return (z * torch.sigmoid(z) * (h @ p[name + ".up"].T)) @ p[name + ".down"].T


def route(h, p, r):
    """Per token the chosen experts and their weights: two lists of lists."""
    E, n, keep, top = r["experts"], r["groups"]["count"], r["groups"]["keep"], r["top"]
    score = torch.sigmoid(h @ p["router"].T)
    choice = score + p["correction"]
    size, ids, weights = E // n, [], []
    for t in range(h.shape[0]):
        c = choice[t].tolist()
        group = [sum(sorted(c[g * size:(g + 1) * size])[-2:]) for g in range(n)]
        kept = sorted(range(n), key=lambda g: -group[g])[:keep]
        can = [e for e in range(E) if e // size in kept]
        best = sorted(can, key=lambda e: -c[e])[:top]
        s = score[t, best]
        ids.append(best)
        weights.append(s / (s.sum() + 1e-20) * r["scale"])
    return ids, weights


def experts(h, p, f):
    ids, weights = route(h, p, f["router"])
    out = torch.stack([sum(w * expert(h[t], p, f"e{e}") for e, w in zip(ids[t], weights[t])) for t in range(h.shape[0])])
    return out + expert(h, p, "shared") if f.get("shared") else out


def section(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def forward(cfg, w, tokens, dtype=torch.float32):
    """cfg: the parsed config.json; w: name -> tensor.  Returns (logits [T, vocab], stream after every layer)."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps, after = cfg["norm"]["eps"], []
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p, f = section(w, f"l{i}."), layer["mlp"]
        mixer = {"wkv": wkv, "latent_attention": latent_attention}[layer["type"]]
        y = mixer(mix(x, p["shift"]), section(p, "mix."), layer["mixer"], eps)
        x = x + layer_norm(gated(y, x, p["rg1"], p["rg1.b"]), p["norm1"], eps)
        if f is not None:
            ffw = section(p, "mlp.")
            y = clamped_glu(x, ffw, f["limit"]) if f["kind"] == "dense" else experts(x, ffw, f)
            x = x + layer_norm(gated(y, x, p["rg2"], p["rg2.b"]), p["norm2"], eps)
        after.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"], torch.stack(after)
