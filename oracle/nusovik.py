"""Oracle: the Nusovik decoder, plain and slow, on the CPU (TEST INFRASTRUCTURE ONLY).

One function per mechanism, written from the design's equations over whole sequences: no cache, no pages, no state slots, no
batches.  The framework's answer for a token must equal ``logits(...)[position]`` however the sequence was cut, batched and placed.

Notation: x [T, D] residual stream; N(y) = y / sqrt(mean y^2 + eps) * w.
  x_0       = s E[t] + P(position)
  layer     x <- x + N1(mixer(x));  x <- x + N2(ff(x))
  logits    = a W_head N_f(x)

``rounding`` selects the arithmetic: ``None`` = everything in ``dtype`` (fp32 or fp64); ``"bf16"`` = bf16 at every matrix-product
input, in what the cache keeps of a token and behind the short convolutions, everything else in ``dtype``.
"""

from __future__ import annotations

import math

import torch

__all__ = ["sinusoid", "rms", "bucket", "chunk_attention", "chunk_mixer", "short_conv", "softplus", "scan1", "mamba1_mixer", "scan2", "gated_norm",
           "mamba2_mixer", "parallel_mixer", "dense_ff", "residuals_and_logits", "logits"]


def _rounder(rounding):
    if rounding is None:
        return lambda t: t
    assert rounding == "bf16"
    return lambda t: t.to(torch.bfloat16).to(t.dtype)


def sinusoid(T, width, dtype, first=0):
    """[T, width]: element 2 i is sin(p 10000^(-2 i / width)), element 2 i + 1 the cosine of the same."""
    p = torch.arange(first, first + T, dtype=torch.float64)[:, None]
    e = torch.arange(width)
    a = p * 10000.0 ** (-2.0 * (e // 2).double() / width)
    return torch.where(e % 2 == 0, torch.sin(a), torch.cos(a)).to(dtype)


def rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def bucket(n, rows, far):
    """Row of the distance table: distances below half the rows have one each, from there on they are spaced by logarithm up to `far`."""
    half = rows // 2
    if n < half:
        return n
    if half == 0:
        return 0
    step = math.log(n / half) / math.log(far / half) * (rows - half)
    return min(rows - 1, half + math.floor(step + 1e-9))


def chunk_attention(q, k, v, scale, rel, far, size, sink, r=lambda t: t):
    """q [T, H, d], k [T, G, d], v [T, G, dv], rel [rows, H], sink [H] -> [T, H, dv].  A query sees the keys of its own chunk of `size`
    positions that are not behind it; the denominator holds exp(sink) besides."""
    T, H = q.shape[:2]
    of = H // k.shape[1]
    i = torch.arange(T)
    dist = (i[:, None] - i[None, :])
    seen = (dist >= 0) & (i[:, None] // size == i[None, :] // size)
    rows = torch.tensor([bucket(n, rel.shape[0], far) for n in range(min(T, size))])[dist.clamp(0, min(T, size) - 1)]
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h // of].t()) * scale + rel[:, h][rows]
        s = s.masked_fill(~seen, float("-inf"))
        m = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        e = torch.exp(s - m)
        out[:, h] = r(e) @ v[:, h // of] / (e.sum(-1, keepdim=True) + torch.exp(sink[h] - m))
    return out


def chunk_mixer(x, m, w, p, eps, r=lambda t: t):
    """The attention half: `m` its sizes, w[p + name] its tensors -> the gated heads [T, H dv] (ahead of the output projection)."""
    T, H, G, d = x.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (x @ w[p + "q"].t() + w[p + "q.b"]).view(T, H, d)
    k = (x @ w[p + "k"].t() + w[p + "k.b"]).view(T, G, d)
    o = chunk_attention(r(rms(q, eps) * w[p + "q.norm"]), r(rms(k, eps) * w[p + "k.norm"]), r(k), m["scale"], w[p + "rel"], m["bias_max"],
                        m["mask"]["size"], w[p + "sink"], r)
    return (o * torch.sigmoid(x @ w[p + "g"].t())[:, :, None]).reshape(T, -1)


def short_conv(x, w, b):
    """y_t = silu(b + sum_j w[:, j] x_(t - taps + 1 + j)), zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x) + b
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * x[:T - back]
    return y * torch.sigmoid(y)


def softplus(z):
    return z.clamp(min=0) + torch.log1p(torch.exp(-z.abs()))


def scan1(x, dt, a_log, b, c, d, state=None):
    """x, dt [T, C], a_log [C, N], b, c [T, N], d [C] -> (y [T, C], the state [C, N] behind the last token)."""
    S = torch.zeros_like(a_log) if state is None else state.clone()
    A = -torch.exp(a_log)
    y = torch.empty_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * b[t][None, :]
        y[t] = (S * c[t][None, :]).sum(1) + d * x[t]
    return y, S


def mamba1_mixer(h, m, w, p, r=lambda t: t):
    inner, N, R = m["inner"], m["state"], m["dt_rank"]
    xz = h @ w[p + "in"].t()
    x = r(short_conv(xz[:, :inner], w[p + "conv"], w[p + "conv.b"]))
    low = x @ w[p + "x"].t()
    dt = softplus(r(low[:, :R]) @ w[p + "dt"].t() + w[p + "dt.b"])
    y, _ = scan1(x, dt, w[p + "A_log"], low[:, R:R + N], low[:, R + N:], w[p + "D"])
    z = xz[:, inner:]
    return r(y * z * torch.sigmoid(z)) @ w[p + "o"].t()


def scan2(x, dt, a_log, b, c, d, state=None):
    """x [T, H, P], dt [T, H], a_log [H], b, c [T, G, N], d [H] -> (y [T, H, P], the state [H, N, P] behind the last token)."""
    T, H, P = x.shape
    of = torch.arange(H) // (H // b.shape[1])
    S = torch.zeros(H, b.shape[2], P, dtype=x.dtype) if state is None else state.clone()
    A = -torch.exp(a_log)
    y = torch.empty_like(x)
    for t in range(T):
        S = torch.exp(dt[t] * A)[:, None, None] * S + dt[t][:, None, None] * b[t][of][:, :, None] * x[t][:, None, :]
        y[t] = (S * c[t][of][:, :, None]).sum(1) + d[:, None] * x[t]
    return y, S


def gated_norm(y, z, w, parts, eps):
    """y silu(z), every one of the equal parts over its own root mean square, times w."""
    y = (y * z * torch.sigmoid(z)).view(y.shape[0], parts, -1)
    return rms(y, eps).reshape(y.shape[0], -1) * w


def mamba2_mixer(h, m, w, p, eps, r=lambda t: t):
    """The state-space half -> the normed heads [T, H P] (ahead of the output projection)."""
    T, H, P, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = (h @ w[p + "in"].t()).split([inner, inner + 2 * G * N, H], -1)
    xbc = r(short_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, b, c = xbc.split([inner, G * N, G * N], -1)
    y, _ = scan2(x.reshape(T, H, P), softplus(dt + w[p + "dt_bias"]), w[p + "A_log"], b.reshape(T, G, N), c.reshape(T, G, N), w[p + "D"])
    return gated_norm(y.reshape(T, inner), z, w[p + "norm"], m["norm_groups"], eps)


def parallel_mixer(h, m, w, p, eps, r=lambda t: t):
    left = r(m["left_scale"] * chunk_mixer(h, m["left"], w, p + "left.", eps, r))
    right = r(m["right_scale"] * mamba2_mixer(h, m["right"], w, p + "right.", eps, r))
    return left @ w[p + "left.o"].t() + right @ w[p + "right.o"].t()


def dense_ff(h, w, p, r=lambda t: t):
    return r((h @ w[p + "up"].t()).clamp(min=0).pow(2)) @ w[p + "down"].t()


@torch.no_grad()
def residuals_and_logits(cfg, weights, tokens, dtype=torch.float32, rounding=None):
    """-> ([layers, T, D] residual stream behind every layer, [T, V] logits)."""
    r = _rounder(rounding)
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"] + sinusoid(len(tokens), cfg["width"], dtype)
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        y = mamba1_mixer(r(x), m, w, p + "mix.", r) if layer["type"] == "mamba1" else parallel_mixer(r(x), m, w, p + "mix.", eps, r)
        x = x + rms(y, eps) * w[p + "norm1"]
        if layer.get("mlp") is not None:
            x = x + rms(dense_ff(r(x), w, p + "mlp.", r), eps) * w[p + "norm2"]
        after.append(x)
    return torch.stack(after), cfg["logit_scale"] * (r(rms(x, eps) * w["final.norm"]) @ w["head"].t())


def logits(cfg, weights, tokens, dtype=torch.float32, rounding=None):
    return residuals_and_logits(cfg, weights, tokens, dtype, rounding)[1]
