"""Oracle: the Vimesun decoder, plain and slow, on the CPU (TEST INFRASTRUCTURE ONLY).

One function per mechanism, written from the design's equations over whole sequences: no cache, no
pages, no batches.  The framework's answer for a token must equal ``logits(...)[position]`` however
the sequence was cut, batched and placed in the pool.

Notation: x [T, D] residual stream (fp32), e = embedding output, m = residual multiplier.
  e_p       = E[t_p] + P[p]
  layer     x <- x + m (attention(ln1(x)) + ff(ln2(x)))           both branches read the same x
  loop      before the first layer of every pass: x <- W_in [x ; e]
  logits    = W_head ln_f(x)

``rounding`` selects the arithmetic: ``None`` = everything in ``dtype`` (fp32 or fp64);
``"bf16"`` = the rounding points of the device path (bf16 at every matrix-product input, in q / k
after their unit norm, in v), everything else in ``dtype``.
"""

from __future__ import annotations

import torch

__all__ = ["layer_norm", "unit_rms", "slopes", "window_attention", "squared_relu_ff", "embedding", "loop_input",
           "layer", "residuals_and_logits", "logits"]


def _rounder(rounding):
    if rounding is None:
        return lambda t: t
    assert rounding == "bf16"
    return lambda t: t.to(torch.bfloat16).to(t.dtype)


def layer_norm(x, w, b, eps):
    """(x - mean) / sqrt(mean squared deviation + eps) * w + b over the last dimension."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt(d.pow(2).mean(-1, keepdim=True) + eps) * w + b


def unit_rms(x, eps):
    """x over its root mean square (no weight), eps inside the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def slopes(heads, dtype=torch.float32):
    """Per-head distance slopes 2^(-8 (h + 1) / H)."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=dtype)


def window_attention(q, k, v, scale, window, slope=None, sink=True):
    """q [T, H, dk], k [T, G, dk], v [T, G, dv] of ONE whole sequence -> [T, H, dv].

    s_ij = scale q_i.k_j - slope_h (i - j) for 0 <= i - j < window;  p_ij = exp(s_ij) / ([sink] + sum_j exp(s_ij)):
    the sink is one more score of 0 in the denominator that carries no value."""
    T, H, _ = q.shape
    G, dv = v.shape[1], v.shape[2]
    out = torch.empty(T, H, dv, dtype=q.dtype)
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    seen = (dist >= 0) & (dist < window)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].t()) * scale
        if slope is not None:
            s = s - slope[h] * dist.to(s.dtype)
        s = s.masked_fill(~seen, float("-inf"))
        top = s.amax(-1, keepdim=True)
        if sink:
            top = top.clamp(min=0.0)
        p = torch.exp(s - top)
        den = p.sum(-1, keepdim=True)
        if sink:
            den = den + torch.exp(-top)
        out[:, h] = (p / den) @ v[:, g]
    return out


def squared_relu_ff(x, up, down, r=lambda t: t):
    """down relu(up x)^2"""
    return r(torch.relu(x @ up.t()).pow(2)) @ down.t()


def embedding(tokens, table, positions):
    return table[tokens] + positions[:tokens.shape[0]]


def loop_input(x, e, w_in, r=lambda t: t):
    """W_in [x ; e], the state first."""
    return r(torch.cat([x, e], -1)) @ w_in.t()


def layer(x, i, cfg, w, r):
    spec, eps = cfg["layers"][i], cfg["norm"]["eps"]
    mix, p = spec["mixer"], f"l{i}."
    T = x.shape[0]
    a = r(layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps))
    q = r(unit_rms((a @ w[p + "mix.q"].t()).view(T, mix["heads"], mix["dim"]), eps))
    k = r(unit_rms((a @ w[p + "mix.k"].t()).view(T, mix["kv_heads"], mix["dim"]), eps))
    v = r((a @ w[p + "mix.v"].t()).view(T, mix["kv_heads"], mix["vdim"]))
    o = window_attention(q, k, v, mix["scale"], mix["mask"]["size"], slopes(mix["heads"], x.dtype))
    y = r(o.reshape(T, -1)) @ w[p + "mix.o"].t()
    if spec.get("mlp") is not None:
        b = r(layer_norm(x, w[p + "norm2"], w[p + "norm2.b"], eps))
        y = y + squared_relu_ff(b, w[p + "mlp.up"], w[p + "mlp.down"], r)
    return x + cfg["residual_mult"] * y


def layer_runs(cfg):
    """Order in which the layers run: (layer, first of a loop pass)."""
    loop = cfg.get("loop")
    n = len(cfg["layers"])
    if loop is None:
        return [(i, False) for i in range(n)]
    lo, hi = loop["start"], loop["stop"]
    return ([(i, False) for i in range(lo)] + [(i, i == lo) for _ in range(loop["times"]) for i in range(lo, hi)]
            + [(i, False) for i in range(hi, n)])


@torch.no_grad()
def residuals_and_logits(cfg, weights, tokens, dtype=torch.float32, rounding=None):
    """-> ([layer runs, T, D] residual stream behind every layer run, [T, V] logits)."""
    r = _rounder(rounding)
    w = {n: t.to(dtype) for n, t in weights.items()}
    x = e = embedding(torch.as_tensor(tokens), w["embed"], w["pos"])
    after = []
    for i, first in layer_runs(cfg):
        if first:
            x = loop_input(x, e, w["loop.in"], r)
        x = layer(x, i, cfg, w, r)
        after.append(x)
    y = r(layer_norm(x, w["final.norm"], w["final.norm.b"], cfg["norm"]["eps"])) @ w["head"].t()
    return torch.stack(after), y


def logits(cfg, weights, tokens, dtype=torch.float32, rounding=None):
    return residuals_and_logits(cfg, weights, tokens, dtype, rounding)[1]
