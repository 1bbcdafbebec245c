"""Plain, slow Vofosun: one function per mechanism, straight from the equations, in torch on the CPU.

Written for comparison only: it shares no code with the package, keeps no cache and no state (a
sequence is always recomputed whole) and loops over heads and positions where that is clearest.
All functions work in the dtype of their inputs (float32 or float64).
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square, eps under the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centred_norm(x, w, eps):
    """RMS norm whose weight is stored as the distance from one."""
    return rms(x, eps) * (1.0 + w)


def causal_conv(h, w):
    """h [T, W]; w [W, taps].  out_t = sum_j w[:, j] h_(t - taps + 1 + j); nothing before position 0."""
    T, taps = h.shape[0], w.shape[1]
    out = torch.zeros_like(h)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


def input_convolution(h, w):
    return h + causal_conv(h, w)


def depth_average(xs, weights):
    """sum_j weights[j] xs[j]: xs = [embedding output, result of layer 0, ..., result of this layer]."""
    assert len(xs) == len(weights)
    out = torch.zeros_like(xs[0])
    for a, x in zip(weights, xs):
        out = out + a * x
    return out


def latent_attention(h, p, heads, dim, vdim, scale, eps):
    """p: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, o.  Scores per head over every key j <= i."""
    T = h.shape[0]
    cq = rms(h @ p["dq"].T, eps) * p["dq.norm"]
    q = (cq @ p["uq"].T).view(T, heads, dim)
    c = rms(h @ p["dkv"].T, eps) * p["dkv.norm"]
    k = (c @ p["uk"].T).view(T, heads, dim)
    v = (c @ p["uv"].T).view(T, heads, vdim)
    out = torch.zeros(T, heads, vdim, dtype=h.dtype)
    future = torch.triu(torch.ones(T, T, dtype=torch.bool), 1)
    for n in range(heads):
        s = (q[:, n] @ k[:, n].T) * scale
        s = s.masked_fill(future, -math.inf)
        out[:, n] = torch.softmax(s, -1) @ v[:, n]
    return out.reshape(T, heads * vdim) @ p["o"].T


def clamped_glu(h, p, limit):
    """p: gate, gate.b, up, up.b, down, down.b."""
    g = torch.clamp(h @ p["gate"].T + p["gate.b"], max=limit)
    u = torch.clamp(h @ p["up"].T + p["up.b"], min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ p["down"].T + p["down.b"]


def softcap(logits, cap):
    return cap * torch.tanh(logits / cap)


def section(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def forward(cfg, w, tokens, dtype=torch.float32):
    """cfg: the parsed config.json; w: name -> tensor.  Returns (logits [T, vocab], stream after every layer)."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    xs, after = [x], []
    for i, layer in enumerate(cfg["layers"]):
        mx, ff = layer["mixer"], layer["mlp"]
        assert layer["type"] == "latent_attention"
        h = centred_norm(x, w[f"l{i}.norm1"], eps)
        y = latent_attention(input_convolution(h, w[f"l{i}.canon1"]), section(w, f"l{i}.mix."), mx["heads"],
                             mx["dim"], mx["vdim"], mx["scale"], eps)
        if ff is not None:
            y = y + clamped_glu(input_convolution(h, w[f"l{i}.canon2"]), section(w, f"l{i}.mlp."), ff["limit"])
        xs.append(x + y)
        x = depth_average(xs, w[f"l{i}.dwa"])
        after.append(x)
    logits = centred_norm(x, w["final.norm"], eps) @ w["head"].T
    return softcap(logits, cfg["logit_softcap"]), torch.stack(after)
