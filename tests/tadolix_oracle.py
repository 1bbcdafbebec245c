"""Plain, slow Tadolix: one function per mechanism, straight from the equations, in torch on the CPU.

Written for comparison only: it shares no code with the package, keeps no cache and no state (a sequence is
always recomputed whole) and loops over tokens, heads and streams where that is clearest.  All functions work in
the dtype of their inputs (float32 or float64).
"""
from __future__ import annotations

import functools
import math
from fractions import Fraction

import torch


def rms(x, eps):
    """x over its root mean square, eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    """The weight counts from zero."""
    return rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def embedding(table, tokens, scale):
    """Scaled token rows plus the sinusoids of the positions: even entries sines, odd ones cosines."""
    x = table[tokens] * scale
    T, W = x.shape
    e = torch.arange(W)
    angle = torch.arange(T, dtype=torch.float64)[:, None] * 10000.0 ** (-2.0 * (e // 2).double() / W)
    return x + torch.where(e % 2 == 0, angle.sin(), angle.cos()).to(x.dtype)


def short_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the first token."""
    T, taps = u.shape[0], w.shape[1]
    ext = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return sum(w[:, j] * ext[j:j + T] for j in range(taps))


def input_conv(h, w):
    return h + short_conv(h, w)


def read_streams(xs, weights):
    return sum(a * x for a, x in zip(weights, xs))


def write_streams(xs, y, mix, out):
    """Stream t from all old ones (mix[from, to]) and the sublayer's result."""
    return [sum(mix[s, t] * xs[s] for s in range(len(xs))) + out[t] * y for t in range(len(xs))]


@functools.cache
def bucket(n, rows, far):
    """The table's row for a distance of n tokens: its own below half the rows, from there on logarithmically up to the
    last at ``far`` (compared exactly, in integers: the k-th step starts at half (far / half)^(k / steps))."""
    half = rows // 2
    if n < half:
        return n
    steps, k = rows - half, 0
    while k < steps - 1 and Fraction(n, half) ** steps >= Fraction(far) ** (k + 1) / Fraction(half) ** (k + 1):
        k += 1
    return half + k


def chunk_mask(T, size):
    """True where token i sees token j: not ahead of it and in the same run of ``size`` positions (0: all before it)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    return (j <= i) & (i // size == j // size if size else torch.ones(T, T, dtype=torch.bool))


def attend(q, k, v, scale, cap, rel, far, size):
    """q [T, H, D], k [T, G, D], v [T, G, V], rel [rows, H].  Heads side by side [T, H V]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    see = chunk_mask(T, size)
    rows = torch.tensor([bucket(n, rel.shape[0], far) for n in range(T)])
    back = (torch.arange(T)[:, None] - torch.arange(T)[None]).clamp(min=0)
    out = []
    for h in range(H):
        g = h // (H // G)
        s = q[:, h] @ k[:, g].T * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        s = (s + rel[rows[back], h]).masked_fill(~see, -math.inf)
        out.append(torch.softmax(s, 1) @ v[:, g])
    return torch.cat(out, 1)


def attention(h, p, m, eps):
    T = h.shape[0]
    q = rms((h @ p["q"].T).view(T, m["heads"], m["dim"]), eps)
    k = rms((h @ p["k"].T).view(T, m["kv_heads"], m["dim"]), eps)
    v = (h @ p["v"].T).view(T, m["kv_heads"], m["vdim"])
    o = attend(q, k, v, m["scale"], m["softcap"], p["rel"], m["bias_max"], m["mask"]["size"])
    return (o * torch.sigmoid(h @ p["g"].T)) @ p["o"].T


def min_gru(z, u):
    """Pre-activations of the gate and the candidate [T, C]: the states S_t [T, C], from zero."""
    S, out = torch.zeros_like(z[0]), []
    for t in range(z.shape[0]):
        g = torch.sigmoid(z[t])
        c = torch.where(u[t] >= 0, u[t] + 0.5, torch.sigmoid(u[t]))
        S = (1 - g) * S + g * c
        out.append(S)
    return torch.stack(out)


def gated_recurrence(h, p):
    S = min_gru(h @ p["z"].T + p["z.b"], h @ p["x"].T + p["x.b"])
    gate = h @ p["g"].T
    return (S * gate * torch.sigmoid(gate)) @ p["o"].T


def parallel(h, p, m, eps):
    return m["left_scale"] * attention(h, section(p, "left."), m["left"], eps) + \
        m["right_scale"] * gated_recurrence(h, section(p, "right."))


def block_gate(u, w, b):
    """u [T, C] in equal parts, w [parts, out, in]: the sigmoid of each part's own product."""
    parts = u.view(u.shape[0], w.shape[0], -1)
    return torch.sigmoid(torch.stack([parts[:, k] @ w[k].T + b[k] for k in range(w.shape[0])], 1)).flatten(1)


def rglru(u, r, i, lam):
    """The states S_t [T, C] of the real-gated recurrence over u, from zero."""
    S, out = torch.zeros_like(u[0]), []
    rate = torch.log1p(torch.exp(-lam.abs())) + lam.clamp(min=0.0)            # log(1 + e^lam)
    for t in range(u.shape[0]):
        a = torch.exp(-8.0 * r[t] * rate)
        S = a * S + torch.sqrt(1.0 - a * a) * i[t] * u[t]
        out.append(S)
    return torch.stack(out)


def recurrent_block(h, p):
    y = gelu_tanh(h @ p["y"].T + p["y.b"])
    u = short_conv(h @ p["x"].T + p["x.b"], p["conv"]) + p["conv.b"]
    S = rglru(u, block_gate(u, p["ra"], p["ra.b"]), block_gate(u, p["ri"], p["ri.b"]), p["lam"])
    return (S * y) @ p["o"].T


def feed_forward(h, p):
    return (gelu_tanh(h @ p["gate"].T) * (h @ p["up"].T)) @ p["down"].T


def section(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def layer_runs(cfg):
    """Layer indices in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(cfg, w, tokens, dtype=torch.float32):
    """cfg: the parsed config.json; w: name -> tensor.  Returns (logits [T, vocab], sum of the streams after every layer
    run)."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps, after = cfg["norm"]["eps"], []
    e = embedding(w["embed"], torch.as_tensor(tokens, dtype=torch.long), cfg["embedding"]["scale"])
    xs = [e] * cfg["streams"]
    for i in layer_runs(cfg):
        layer, p = cfg["layers"][i], section(w, f"l{i}.")
        m, mix = layer["mixer"], section(p, "mix.")
        h = input_conv(norm(read_streams(xs, p["hc1.in"]), p["norm1"], eps), p["canon1"])
        y = parallel(h, mix, m, eps) if layer["type"] == "parallel" else recurrent_block(h, mix)
        xs = write_streams(xs, y, p["hc1.mix"], p["hc1.out"])
        if layer["mlp"] is not None:
            y = feed_forward(norm(read_streams(xs, p["hc2.in"]), p["norm2"], eps), section(p, "mlp."))
            xs = write_streams(xs, y, p["hc2.mix"], p["hc2.out"])
        after.append(sum(xs))
    return norm(sum(xs), w["final.norm"], eps) @ w["head"].T, torch.stack(after)
