"""Plain-PyTorch fp32 reference implementations of every native op.

They define the exact semantics (including the paged KV-cache layouts) that the HIP kernels in
``csrc/kernels`` must reproduce; the numerics tests compare the two, and CPU-only runs (CI,
BASELINE config 1) execute these.  Inputs/outputs use the same dtypes as the kernels (bf16
activations), the math runs in fp32.

These define the semantics the HIP kernels are tested against -- the attention/sampling the
reference's engines run behind local_llm_summarizer.py:107 and llamacpp_summarizer.py:108-113.
"""
from __future__ import annotations

import math

import numpy as np
import torch

KV_BLOCK = 32


def v_slot_perm(device=None) -> torch.Tensor:
    """slot index (0..31) of every key inside a KV block in the transposed V cache."""
    k = torch.arange(KV_BLOCK, device=device)
    hi, g, j = k >> 4, (k >> 2) & 3, (k & 3) + 4 * (k >> 4)
    del hi
    return 8 * g + j


def v_groups(v_cache: torch.Tensor) -> torch.Tensor:
    """View of a V cache [nblk, Hkv, D, 32] as its storage order [nblk, Hkv, 4, D, 8]: slot position
    p of row d lives at [..., p // 8, d, p % 8] (common.h kv_v_off) -- the 8 positions of one P.V
    fragment stay 16 contiguous bytes, and one token's column spans 16 cache lines instead of 64."""
    nb, h, d, s = v_cache.shape
    return v_cache.view(nb, h, s // 8, d, 8)


def rmsnorm(x, w, eps, residual=None):
    """Returns (out, new_residual).  With residual: residual <- x + residual; out = norm(residual)."""
    if residual is not None:
        r = (x.float() + residual.float()).to(x.dtype)
        base = r
    else:
        r = None
        base = x
    xf = base.float()
    out = xf * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps) * w.float()
    return out.to(x.dtype), r


def layernorm(x, gamma, beta, eps, bias=None, residual=None):
    xf = x.float()
    if bias is not None:
        xf = xf + bias.float()
    if residual is not None:
        xf = xf + residual.float()
    out = torch.nn.functional.layer_norm(xf, (xf.shape[-1],), gamma.float(), beta.float(), eps)
    return out.to(x.dtype)


def embed_layernorm(ids, positions, word_emb, pos_emb, type_emb, gamma, beta, eps):
    x = word_emb[ids.long()].float() + pos_emb[positions.long()].float() + type_emb[0].float()
    return torch.nn.functional.layer_norm(x, (x.shape[-1],), gamma.float(), beta.float(), eps).to(word_emb.dtype)


def rope_cos_sin(max_pos: int, head_dim: int, theta: float, device=None, llama3_scaling=None) -> torch.Tensor:
    """[max_pos, D/2, 2] fp32 table of (cos, sin) for rotate-half RoPE.

    ``llama3_scaling`` = (factor, low_freq_factor, high_freq_factor, original_max_positions): the
    Llama-3.1 frequency rescaling (long wavelengths divided by ``factor``, short ones kept, a
    smooth blend in between)."""
    inv = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float64) / head_dim))
    if llama3_scaling is not None:
        factor, low, high, orig = llama3_scaling
        wavelen = 2 * math.pi / inv
        scaled = torch.where(wavelen > orig / low, inv / factor, inv)
        smooth = (orig / wavelen - low) / (high - low)
        blend = (1 - smooth) * scaled / factor + smooth * scaled
        medium = ~(wavelen < orig / high) & ~(wavelen > orig / low)
        inv = torch.where(medium, blend, scaled)
    t = torch.arange(max_pos, dtype=torch.float64)
    ang = torch.outer(t, inv)
    return torch.stack([ang.cos(), ang.sin()], -1).float().to(device)


def _to_cache(x, cache, scale):
    """Value as stored in a cache of ``cache.dtype`` (fp8 e4m3fn caches hold x / scale, clamped)."""
    if cache.dtype == torch.float8_e4m3fn:
        return (x.float() / scale).clamp(-448.0, 448.0).to(torch.float8_e4m3fn)
    return x.to(cache.dtype)


def rope_kv_write(qkv, positions, slots, cos_sin, k_cache, v_cache, Hq, Hkv, D, k_scale=1.0, v_scale=1.0):
    """Apply RoPE to q/k of the fused projection, write k/v into the paged cache. Returns q."""
    T = qkv.shape[0]
    x = qkv.float().view(T, Hq + 2 * Hkv, D)
    cs = cos_sin[positions.long()]  # [T, D/2, 2]
    cos, sin = cs[..., 0][:, None, :], cs[..., 1][:, None, :]
    half = D // 2

    def rot(t):
        a, b = t[..., :half], t[..., half:]
        return torch.cat([a * cos - b * sin, b * cos + a * sin], -1)

    q = rot(x[:, :Hq]).to(qkv.dtype)
    k = rot(x[:, Hq:Hq + Hkv]).to(qkv.dtype)
    v = x[:, Hq + Hkv:].to(qkv.dtype)
    perm = v_slot_perm(qkv.device)
    for t in range(T):
        s = int(slots[t])
        if s < 0:
            continue
        blk, off = divmod(s, KV_BLOCK)
        k_cache[blk, :, off, :] = _to_cache(k[t], k_cache, k_scale)
        p = int(perm[off])
        v_groups(v_cache)[blk, :, p >> 3, :, p & 7] = _to_cache(v[t], v_cache, v_scale)
    return q


def gather_kv(k_cache, v_cache, block_table, n, k_scale=1.0, v_scale=1.0):
    """Contiguous K, V [n, Hkv, D] of one sequence from the paged caches (fp8 caches dequantized
    to fp32 with their scales)."""
    perm = v_slot_perm(k_cache.device)
    nb = (n + KV_BLOCK - 1) // KV_BLOCK
    blocks = block_table[:nb].long()
    k = k_cache[blocks].permute(0, 2, 1, 3).reshape(nb * KV_BLOCK, k_cache.shape[1], k_cache.shape[3])
    vt = v_groups(v_cache)[blocks].permute(0, 1, 3, 2, 4).reshape(nb, v_cache.shape[1], v_cache.shape[2], KV_BLOCK)
    v = vt[..., perm].permute(0, 3, 1, 2).reshape(nb * KV_BLOCK, v_cache.shape[1], v_cache.shape[2])
    if k_cache.dtype == torch.float8_e4m3fn:
        k, v = k.float() * k_scale, v.float() * v_scale
    return k[:n], v[:n]


def _attend(q, k, v, scale, causal_offset=None, window=0):
    """q [m, Hq, D], k/v [n, Hkv, D] -> [m, Hq, D] fp32 (GQA).  ``window`` > 0: sliding-window
    attention as HF Mistral masks it -- a query at position p sees keys k with p - window < k <= p."""
    Hq, Hkv = q.shape[1], k.shape[1]
    G = Hq // Hkv
    kk = k.float().repeat_interleave(G, 1)
    vv = v.float().repeat_interleave(G, 1)
    s = torch.einsum("mhd,nhd->hmn", q.float(), kk) * scale
    m, n = q.shape[0], k.shape[0]
    if causal_offset is not None or window:
        off = causal_offset if causal_offset is not None else n - m
        pos = torch.arange(m, device=q.device)[:, None] + off
        keys = torch.arange(n, device=q.device)[None, :]
        mask = keys > pos
        if window:
            mask = mask | (keys <= pos - window)
        s = s.masked_fill(mask[None], float("-inf"))
    p = torch.softmax(s, -1)
    return torch.einsum("hmn,nhd->mhd", p, vv)


def paged_decode_attention(q, k_cache, v_cache, block_tables, ctx_lens, scale, window=0, k_scale=1.0, v_scale=1.0):
    out = torch.empty_like(q)
    for b in range(q.shape[0]):
        n = int(ctx_lens[b])
        k, v = gather_kv(k_cache, v_cache, block_tables[b], n, k_scale, v_scale)
        out[b] = _attend(q[b:b + 1], k, v, scale, window=window)[0].to(q.dtype)
    return out


def prefill_attention(q, k_cache, v_cache, block_tables, cu_q, ctx_lens, scale, window=0, k_scale=1.0, v_scale=1.0):
    out = torch.empty_like(q)
    for s in range(len(cu_q) - 1):
        a, b = int(cu_q[s]), int(cu_q[s + 1])
        if b == a:
            continue
        n = int(ctx_lens[s])
        k, v = gather_kv(k_cache, v_cache, block_tables[s], n, k_scale, v_scale)
        out[a:b] = _attend(q[a:b], k, v, scale, causal_offset=n - (b - a), window=window).to(q.dtype)
    return out


def encoder_attention(qkv, cu_seqlens, H, D, scale):
    T = qkv.shape[0]
    x = qkv.view(T, 3, H, D)
    out = torch.empty(T, H, D, dtype=qkv.dtype, device=qkv.device)
    for s in range(len(cu_seqlens) - 1):
        a, b = int(cu_seqlens[s]), int(cu_seqlens[s + 1])
        if b == a:
            continue
        out[a:b] = _attend(x[a:b, 0], x[a:b, 1], x[a:b, 2], scale).to(qkv.dtype)
    return out


def silu_mul(gu):
    F = gu.shape[-1] // 2
    g, u = gu[..., :F].float(), gu[..., F:].float()
    return (torch.nn.functional.silu(g) * u).to(gu.dtype)


# gate/up rows of the fused MLP projection are stored interleaved in groups of GU_GROUP rows, so a
# 16-row MFMA n-tile of the decode GEMM holds 8 gate rows and the 8 matching up rows
# (csrc/kernels/dgemm.hip SwiGLU epilogue; the prefill silu_mul and the GEMV read the same layout)
GU_GROUP = 8


def interleave_gate_up(gu_w: torch.Tensor) -> torch.Tensor:
    """[gate; up] rows (2F, H) -> 8-row groups [gate 8t..8t+7; up 8t..8t+7] (F % 8 == 0)."""
    F, G = gu_w.shape[0] // 2, GU_GROUP
    g, u = gu_w[:F].reshape(F // G, G, -1), gu_w[F:].reshape(F // G, G, -1)
    return torch.stack([g, u], 1).reshape(2 * F, -1).contiguous()


def deinterleave_gate_up(w: torch.Tensor) -> torch.Tensor:
    F, G = w.shape[0] // 2, GU_GROUP
    v = w.reshape(F // G, 2, G, -1)
    return torch.cat([v[:, 0].reshape(F, -1), v[:, 1].reshape(F, -1)]).contiguous()


def pack_dgemm_weight(w: torch.Tensor, bn: int) -> torch.Tensor:
    """Row-major W[N, K] -> the decode GEMM's fragment-packed layout for bn-row workgroups,
    [N/bn, K/32, bn/16, 64, 8]: packed[t, kg, w, 16 q + r, j] = W[bn t + 16 w + r, 32 kg + 8 q + j]
    (lane 16q + r of a 16x16x32 MFMA holds B[k = 8q + j][n = r]; one workgroup's slice is contiguous)."""
    N, K = w.shape
    v = w.reshape(N // bn, bn // 16, 16, K // 32, 4, 8)          # t, w, r, kg, q, j
    return v.permute(0, 3, 1, 4, 2, 5).reshape(N // bn, K // 32, bn // 16, 64, 8).contiguous()


def unpack_dgemm_weight(p: torch.Tensor) -> torch.Tensor:
    T, G, NW = p.shape[0], p.shape[1], p.shape[2]
    v = p.reshape(T, G, NW, 4, 16, 8)                              # t, kg, w, q, r, j
    return v.permute(0, 2, 4, 1, 3, 5).reshape(T * NW * 16, G * 32).contiguous()


def silu_mul_interleaved(gu):
    F, G = gu.shape[-1] // 2, GU_GROUP
    v = gu.reshape(*gu.shape[:-1], F // G, 2, G).float()
    return (torch.nn.functional.silu(v[..., 0, :]) * v[..., 1, :]).reshape(*gu.shape[:-1], F).to(gu.dtype)


def bias_gelu(x, bias):
    xf = x.float() + (bias.float() if bias is not None else 0.0)
    return torch.nn.functional.gelu(xf).to(x.dtype)


def sample_greedy(logits):
    """argmax, NaN ranked as -inf (as the HIP sampler): an all-NaN row gives token 0."""
    x = logits.float()
    return torch.argmax(torch.nan_to_num(x, nan=-math.inf, posinf=math.inf, neginf=-math.inf), -1).to(torch.int32)


def truncation_keep(sorted_logits: torch.Tensor, top_p: float, min_p: float) -> int:
    """How many of the (descending) top-k logits survive top-p then min-p (at least one)."""
    v = sorted_logits.float()
    p = torch.softmax(v, -1)
    minp_logit = float(v[0]) + math.log(min_p) if min_p > 0 else -math.inf
    cum, keep = 0.0, 0
    while keep < v.numel():
        if keep > 0 and float(v[keep]) < minp_logit:
            break
        cum += float(p[keep])
        keep += 1
        if cum >= top_p:
            break
    return max(1, keep)


def sample_truncated(logits, temperature, top_k, top_p, min_p, generator=None, cap: int = 256):
    """top-k -> top-p -> min-p -> temperature -> draw (ties ordered by index), one id per row."""
    out = []
    for row in logits.float():
        row = torch.nan_to_num(row, nan=-math.inf, posinf=math.inf, neginf=-math.inf)
        k = min(top_k if top_k > 0 else cap, cap, row.numel())
        vals, idx = torch.sort(row, descending=True, stable=True)
        vals, idx = vals[:k], idx[:k]
        keep = truncation_keep(vals, top_p, min_p)
        if temperature <= 0:
            out.append(int(idx[0]))
            continue
        p = torch.softmax(vals[:keep] / temperature, -1)
        out.append(int(idx[torch.multinomial(p, 1, generator=generator)[0]]))
    return torch.tensor(out, dtype=torch.int32)


def knn_scores(X, Q, xnorm2=None, qnorm2=None):
    dots = Q.float() @ X.float().T
    if xnorm2 is None:
        return dots
    return -(xnorm2.float()[None, :] + qnorm2.float()[:, None] - 2 * dots)


def l2_normalize(x):
    xf = x.float()
    n2 = xf.pow(2).sum(-1)
    inv = torch.where(n2 > 0, torch.rsqrt(n2), torch.zeros_like(n2))
    return (xf * inv[:, None]).to(x.dtype), n2


def pool(hidden, cu_seqlens, mode="mean", normalize=True):
    outs = []
    for s in range(len(cu_seqlens) - 1):
        a, b = int(cu_seqlens[s]), int(cu_seqlens[s + 1])
        h = hidden[a:b].float()
        if b == a:
            v = torch.zeros(hidden.shape[-1], device=hidden.device)
        elif mode == "cls":
            v = h[0]
        else:
            v = h.mean(0)
        if normalize:
            n = v.norm()
            v = v / n if n > 0 else v
        outs.append(v)
    return torch.stack(outs) if outs else torch.empty(0, hidden.shape[-1])


def softmax_scale(head_dim: int) -> float:
    return 1.0 / math.sqrt(head_dim)


def quant_fp8_rows(x: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """fp32 reference of the per-row FP8 quantisation kernel."""
    xf = x.float()
    amax = xf.abs().amax(1, keepdim=True)
    s = torch.where(amax > 0, amax / 448.0, torch.ones_like(amax))
    return (xf / s).clamp(-448.0, 448.0).to(torch.float8_e4m3fn), s


# ----------------------------------------------------- 32-bit residual stream (stream.hip)
def tail_slots(taps: int) -> int:
    """Convolution inputs a cache block keeps per layer: the taps - 1 live ones and two spare rows (a
    position that is run again must not overwrite what it reads), never more than the block's positions."""
    return 0 if taps <= 1 else min(taps + 1, KV_BLOCK)


def sinusoids(positions, turns, width):
    """[T, width]: sine and cosine of positions * turns[i] turns at entries 2i and 2i + 1."""
    a = positions.to(torch.float64)[:, None] * turns * (2.0 * math.pi)
    return torch.stack([a.sin(), a.cos()], -1).flatten(1)[:, :width].to(torch.float32)


def depth_norm(x, hist, part, bias, dwa, n, eps, pre=None, j0=0):
    """X_n = x + sum of part slabs + bias into hist[n]; returns (sum_j dwa[j] X_j, 1 / rms of it); ``pre``
    is the sum of the first j0 terms."""
    if part is not None:
        new = x + part.sum(0) + (bias if bias is not None else 0.0)
        hist[n].copy_(new)
        j0 = j0 if pre is not None else 0
        x = torch.einsum("j,jtw->tw", dwa[j0:n + 1].float(), hist[j0:n + 1])
        x = x if pre is None else x + pre
    return x, 1.0 / torch.sqrt((x * x).mean(-1) + eps)


def input_conv(h, portions, block_tables, tail, weights):
    """h [T, W] fp32 convolution inputs of packed portions [(first row, rows, first position, sequence)];
    tail [blocks, slots, W] read for positions before a portion and updated (``block_tables`` [sequences]: one row of
    slots per sequence).  weights: per sublayer [taps, W].  Returns one h + conv(h) per sublayer."""
    outs = [h.clone() for _ in weights]
    taps = weights[0].shape[0]

    def block(seq, q):
        return int(block_tables[seq, q // KV_BLOCK] if block_tables.dim() == 2 else block_tables[seq])
    for row0, n, pos0, seq in portions:
        past = []
        for q in range(pos0 - taps + 1, pos0):
            if q < 0:
                past.append(torch.zeros_like(h[0]))
            else:
                past.append(tail[block(seq, q), q % tail.shape[1]])
        ext = torch.cat([torch.stack(past), h[row0:row0 + n]]) if past else h[row0:row0 + n]
        for o, w in zip(outs, weights):
            for j in range(taps):
                o[row0:row0 + n] += w[j] * ext[j:j + n]
        for r in range(n):
            q = pos0 + r
            # the last inputs of the portion and of every block it crosses
            if taps > 1 and (r >= n - (taps - 1) or KV_BLOCK - q % KV_BLOCK <= taps - 1):
                tail[block(seq, q), q % tail.shape[1]] = h[row0 + r]
    return outs


def clamped_glu(g, u, limit, alpha, beta, cubic=0.0):
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(alpha * g * (1.0 + cubic * g * g)) * (u + beta)


# ----------------------------------------------------- latent attention (latent.hip)
def latent_norm(part, nq, wq, wc, eps):
    """(normed query latent, normed cached latent) of the joint down projection's fp32 slabs."""
    y = part.sum(0)
    q, c = y[:, :nq], y[:, nq:]
    q = q / torch.sqrt((q * q).mean(-1, keepdim=True) + eps) * wq
    c = c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * wc
    return q, c


def latent_attention(q, cache, block_tables, cu_q, ctx_lens, scale, window=0, sink=None, vcols=None):
    """q [T, H, RS]; cache [blocks, 32, RS]: softmax over the sequence's cached rows, per row causal and at most
    ``window`` keys back (0: all), exp(sink[h]) added to the denominator; the value is a row's first ``vcols``
    columns."""
    vcols = vcols or q.shape[2]
    out = torch.empty(*q.shape[:2], vcols, dtype=q.dtype)
    for s in range(len(ctx_lens)):
        a, b, ctx = int(cu_q[s]), int(cu_q[s + 1]), int(ctx_lens[s])
        nb = -(-ctx // KV_BLOCK)
        c = cache[block_tables[s, :nb].long()].reshape(nb * KV_BLOCK, -1)[:ctx].float()
        sc = torch.matmul(q[a:b].float(), c.t()) * scale                        # [n, H, ctx]
        back = torch.arange(ctx - (b - a), ctx)[:, None] - torch.arange(ctx)[None]
        hidden = (back < 0) | (back >= window) if window else back < 0
        sc.masked_fill_(hidden[:, None], float("-inf"))
        if sink is not None:
            sc = torch.cat([sc, sink.float().view(1, -1, 1).expand(b - a, -1, 1)], -1)
        p = torch.softmax(sc, -1)[..., :ctx]
        out[a:b] = torch.matmul(p, c[:, :vcols]).to(q.dtype)
    return out


# ----------------------------------------------------- rotary tables
def rotate_pairs(x, positions, freq, mag):
    """Neighbouring dimensions (2i, 2i + 1) of x [T, ..., 2n] rotated by positions * freq[i], scaled by mag."""
    a = positions.to(torch.float32)[:, None] * freq
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (-1,)
    c, s = (a.cos() * mag).view(shape), (a.sin() * mag).view(shape)
    u, v = x[..., 0::2].float(), x[..., 1::2].float()
    return torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)


# ----------------------------------------------------- gated, post-normed branches (gated.hip)
META_TAIL, META_SLOT = 4, 3        # row word: rows before it in its portion (0, 1, 2 = more) | last two rows | slot << 3


def row_meta(portions) -> np.ndarray:
    """Row words of packed portions [(rows, state slot)]."""
    out = []
    for n, slot in portions:
        r = np.arange(n)
        out.append(np.minimum(r, 2) | np.where(r >= n - 2, META_TAIL, 0) | (slot << META_SLOT))
    return np.concatenate(out).astype(np.int32)


def layernorm_rows(y, w, eps):
    d = y - y.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def before_rows(x, meta, positions, prev):
    """(x of the token before, x of the one before that) per row; prev [slots, 2, W] holds the rows of positions
    before a portion at position % 2; zeros before the first token."""
    xp, xpp = torch.zeros_like(x), torch.zeros_like(x)
    for t, (m, p) in enumerate(zip(meta.tolist(), positions.tolist())):
        lead, slot = m & 3, m >> META_SLOT
        if p >= 1:
            xp[t] = x[t - 1] if lead >= 1 else prev[slot, (p - 1) % 2]
        if p >= 2:
            xpp[t] = x[t - 2] if lead >= 2 else prev[slot, p % 2]
    return xp, xpp


def shift_mix(x, xp, xpp, positions, shift, mus):
    """Token shift of x, then (``mus`` [n, W]) each mix of the shifted row with the one before it."""
    h = x + (xp - x) * shift
    if mus is None:
        return [h]
    hp = (xp + (xpp - xp) * shift) * (positions >= 1).to(x.dtype)[:, None]
    return [h + (hp - h) * mu for mu in mus]


# ----------------------------------------------------- per-channel decay recurrence (wkv.hip)
LOG_DECAY_MIN = -104.0             # exp(-104) is 0 in fp32


def wkv(r, k, v, w, u, S):
    """r, k, v, w [T, H, D] fp32, u [H, D], S [H, D, D] (updated): o_t = (S + u k v^T)^T r, S = w S + k v^T."""
    out = torch.empty_like(v)
    for t in range(r.shape[0]):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hij,hi->hj", S + u[:, :, None] * kv, r[t])
        S.mul_(w[t][:, :, None]).add_(kv)
    return out


def wkv_decay(w1, w2, w0):
    """w1 [T, R]: exp(-exp(tanh(w1) w2^T + w0))."""
    return torch.exp(torch.clamp(-torch.exp(torch.tanh(w1) @ w2.float().t() + w0), min=LOG_DECAY_MIN))


def wkv_out(o, norm, gate, eps):
    """o [T, H, D] over its root mean square per head, times norm and silu(gate) [T, H D]."""
    o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps)
    return o.flatten(1) * norm * (gate * torch.sigmoid(gate))


# ----------------------------------------------------- routed experts (moe.hip)
def route(logits, correction, groups, keep, top, scale, softmax=False, renorm=True):
    """logits [T, E] fp32: (ids [T, top], weights [T, top]).  Sigmoid (or softmax) scores; the choice adds
    ``correction``; a group counts by its two largest choice scores and only the best ``keep`` groups take part.  The
    weights are the chosen scores, over their sum with ``renorm``."""
    s = torch.softmax(logits, -1) if softmax else torch.sigmoid(logits)
    c = s + correction
    T, E = c.shape
    g = c.view(T, groups, E // groups)
    best = g.topk(min(2, E // groups), -1).values.sum(-1)
    kept = torch.zeros_like(best, dtype=torch.bool).scatter_(1, best.topk(keep, -1).indices, True)
    c = c.masked_fill(~kept.repeat_interleave(E // groups, 1), float("-inf"))
    ids = c.topk(top, -1).indices
    w = s.gather(1, ids)
    return ids.to(torch.int32), (w / (w.sum(-1, keepdim=True) + 1e-20) if renorm else w) * scale


def moe_rows(ids, experts, tile):
    """Rows of (token, choice) pairs sorted by expert, every expert's rows padded to whole tiles: (token per row
    [M], row per pair [T, top], expert per tile [M / tile]), pad rows token 0, tiles past the last -1.  Choices past the
    last expert take no row (their row per pair is 0)."""
    T, top = ids.shape
    n_tiles = moe_max_tiles(T * top, experts, tile)
    rows, pos, te = np.zeros(n_tiles * tile, np.int32), np.zeros((T, top), np.int32), np.full(n_tiles, -1, np.int32)
    at = 0
    for e in range(experts):
        pairs = (ids == e).nonzero().tolist()
        for i, (t, c) in enumerate(pairs):
            rows[at + i], pos[t, c] = t, at + i
        m = -(-len(pairs) // tile)
        te[at // tile:at // tile + m] = e
        at += m * tile
    return rows, pos, te


def moe_max_tiles(pairs: int, experts: int, tile: int) -> int:
    """Most tiles that ``pairs`` rows over ``experts`` experts can take."""
    return min(pairs, pairs // tile + min(experts, pairs))


# ----------------------------------------------------- branches between two norms (branch.hip)
def rms_rows(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def relu_sq(x):
    return torch.clamp(x, min=0.0).square()


# ----------------------------------------------------- minimal gated recurrence (gru.hip)
def min_gru(z, u, S):
    """Pre-activations of gate and candidate [T, C], S [C] (updated): the states S_t [T, C]."""
    g, c = torch.sigmoid(z), torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    a, out = torch.sigmoid(-z), torch.empty_like(z)
    for t in range(z.shape[0]):
        S.mul_(a[t]).add_(g[t] * c[t])
        out[t] = S
    return out


# ----------------------------------------------------- hyper-connections (hyper.hip)
def hyper_update(x, y, mix, out):
    """x [T, S, W]: x_t <- sum_s mix[s, t] x_s + out[t] y."""
    return torch.einsum("tsw,sq->tqw", x, mix) + out[:, None] * y[:, None]


# ----------------------------------------------------- real-gated recurrence behind a short convolution (rglru.hip)
def gelu_tanh(z):
    return z * torch.sigmoid(2.0 * math.sqrt(2.0 / math.pi) * z * (1.0 + 0.044715 * z * z))


def rglru(u, pr, pi, rate, S):
    """u and the gates' pre-activations [T, C], S [C] (updated): the states S_t [T, C]."""
    la, out = rate * torch.sigmoid(pr), torch.empty_like(u)
    a, b = torch.exp(la), torch.sqrt(-torch.expm1(2.0 * la)) * torch.sigmoid(pi) * u
    for t in range(u.shape[0]):
        S.mul_(a[t]).add_(b[t])
        out[t] = S
    return out


# ----------------------------------------------------- grouped attention over two key ranges (qkv.hip, gqa.hip)
def conv_over_time(u, w, lead, positions, slots, tail):
    """u [T, C] fp32, w [taps, C]: y_t = sum_d w[taps - 1 - d] u_(t - d) inside each sequence.  ``lead`` rows of the same
    portion lie before a row; older inputs from ``tail`` [slots, taps - 1, C] (position p at row p % (taps - 1))."""
    taps, y = w.shape[0], u * w[-1]
    for t, (n, p) in enumerate(zip(lead.tolist(), positions.tolist())):
        for d in range(1, min(taps - 1, p) + 1):
            y[t] += w[taps - 1 - d] * (u[t - d] if d <= n else tail[int(slots[t]), (p - d) % (taps - 1)])
    return y


def head_norm(x, w, eps, per_head, heads):
    """RMS norm of x [T, heads * dim] over all of it, or per head (``w`` [dim])."""
    if not per_head:
        return rms_rows(x, eps) * w
    return (rms_rows(x.view(x.shape[0], heads, -1), eps) * w).flatten(1)


def rotate_heads(x, positions, freq):
    """The first 2 len(freq) dimensions of x [T, heads, dim] turned in neighbouring pairs."""
    n = 2 * freq.numel()
    return torch.cat([rotate_pairs(x[..., :n], positions, freq, 1.0), x[..., n:]], -1)


def paged_rows(cache, table, n):
    """The first n rows [n, G, D] of a sequence in a cache [blocks, G, entries, D]."""
    e = cache.shape[2]
    return cache[table[:-(-n // e)].long()].transpose(1, 2).reshape(-1, cache.shape[1], cache.shape[3])[:n]


def grouped_attention(q, k, v, pooled, block_tables, cu_q, ctx_lens, size, keep, pool, sink, vdim, chunked=False, softcap=0.0,
                      bias=None):
    """q [T, H, D] scaled by log2(e) (with a softcap: by 2 log2(e) / softcap); k, v [blocks, G, 32, D], ``pooled`` their block
    means [blocks, G, E, D] (pool > 0).  A row sees its last ``size`` keys (0: all; ``chunked``: those of its own run of
    ``size`` positions), the first ``keep``, and the means of blocks of ``pool`` keys wholly ahead of the window; ``bias``
    [H, n] by distance joins the scores, exp(sink) the denominator.  fp32."""
    T, H, D = q.shape
    out = torch.empty(T, H * vdim, dtype=torch.float32)
    for s in range(len(ctx_lens)):
        a, b, ctx = int(cu_q[s]), int(cu_q[s + 1]), int(ctx_lens[s])
        K, V = (paged_rows(c, block_tables[s], ctx).float() for c in (k, v))
        pos, j = torch.arange(ctx - (b - a), ctx)[:, None], torch.arange(ctx)[None]
        near = pos // size == j // size if chunked else pos - j < size
        see = (j <= pos) & (near | (j < keep)) if size else j <= pos
        n = max(ctx - size, 0) // pool if pool else 0
        if n:
            PK, PV = (paged_rows(c, block_tables[s], n).float() for c in pooled)
            K, V = torch.cat([K, PK]), torch.cat([V, PV])
            see = torch.cat([see, torch.arange(n)[None] < (pos - size + 1).clamp(min=0) // pool], 1)
        for h in range(H):
            g = h * K.shape[1] // H
            sc = q[a:b, h].float() @ K[:, g].t()
            sc = softcap * torch.tanh(sc * (0.5 * math.log(2.0))) if softcap else sc * math.log(2.0)
            if bias is not None:
                sc = sc + bias[h][(pos - j).clamp(0, bias.shape[1] - 1)]
            sc = sc.masked_fill(~see, float("-inf"))
            if sink is not None:
                sc = torch.cat([sc, sink[h].expand(b - a, 1)], 1)
            p = torch.softmax(sc, -1)[:, :K.shape[0]]
            out[a:b, h * vdim:(h + 1) * vdim] = p @ V[:, g, :vdim]
    return out
