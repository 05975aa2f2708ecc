"""Oracle: the Rapodra decoder, plain and slow, on the CPU (TEST INFRASTRUCTURE ONLY).

One function per mechanism, written from the design's equations over whole sequences: no cache, no pages, no batches.
The framework's answer for a token must equal ``logits(...)[position]`` however the sequence was cut, batched and placed
in the pool.

Notation: x [T, D] residual stream (fp32); N(.) grouped RMS norm; C(h) = h + causal convolution of h over time.
  x_0       = E[t]
  layer     x <- x + N1b(mixer(C1(N1(x))));   x <- x + N2b(ff(C2(N2(x))))      (the second half only where there is an ff)
  logits    = s tanh(W_head N_f(x) / s)

``rounding`` selects the arithmetic: ``None`` = everything in ``dtype`` (fp32 or fp64); ``"bf16"`` = the rounding points of
the device path (bf16 at every matrix-product input, in the convolution's inputs, in the cached latents), everything else
in ``dtype``.
"""

from __future__ import annotations

import torch

__all__ = ["group_rms", "causal_conv", "latent_attention", "clipped_glu_ff", "silu_glu", "route", "expert_ff", "softcap",
           "residuals_and_logits", "logits"]


def _rounder(rounding):
    if rounding is None:
        return lambda t: t
    assert rounding == "bf16"
    return lambda t: t.to(torch.bfloat16).to(t.dtype)


def group_rms(x, w, groups, eps):
    """Every one of `groups` equal consecutive parts over its own sqrt(mean square + eps); the whole times w."""
    p = x.unflatten(-1, (groups, -1))
    return (p / torch.sqrt(p.pow(2).mean(-1, keepdim=True) + eps)).flatten(-2) * w


def causal_conv(h, w):
    """y_t = sum_j w[:, j] h_(t - taps + 1 + j): the last column of w meets the token itself, zeros before the start."""
    T, taps = h.shape[0], w.shape[1]
    y = torch.zeros_like(h)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * h[:T - back]
    return y


def latent_attention(q, c, w_uk, w_uv, scale, window, r=lambda t: t):
    """q [T, H, dk], latents c [T, R], w_uk [H dk, R], w_uv [H dv, R] of ONE sequence -> [T, H, dv].

    k = W_uk c, v = W_uv c per head; softmax of scale q.k over the keys with 0 <= i - j < window."""
    T, H, dk = q.shape
    i = torch.arange(T)
    back = i[:, None] - i[None, :]
    seen = (back >= 0) & (back < window)
    dv = w_uv.shape[0] // H
    k, v = (c @ w_uk.t()).view(T, H, dk), (c @ w_uv.t()).view(T, H, dv)
    out = torch.empty(T, H, dv, dtype=q.dtype)
    for h in range(H):
        s = (r(q[:, h]) @ r(k[:, h]).t()) * scale
        p = torch.softmax(s.masked_fill(~seen, float("-inf")), -1)
        out[:, h] = r(p) @ r(v[:, h])
    return out


def clipped_glu_ff(h, gate, up, down, limit, r=lambda t: t):
    """g = min(W_gate h, limit), u = W_up h clamped to +-limit; W_down (g sigmoid(1.702 g) (u + 1))"""
    g = (h @ gate.t()).clamp(max=limit)
    u = (h @ up.t()).clamp(-limit, limit)
    return r(g * torch.sigmoid(1.702 * g) * (u + 1)) @ down.t()


def silu_glu(h, gate, up, down, r=lambda t: t):
    """W_down (silu(W_gate h) * (W_up h))"""
    g = h @ gate.t()
    return r(g * torch.sigmoid(g) * (h @ up.t())) @ down.t()


def route(h, w, b, top):
    """-> (chosen experts [T, top], their softmax weights over the chosen logits)."""
    z = h @ w.t() + b
    val, idx = z.topk(top, -1)
    return idx, torch.softmax(val, -1)


def expert_ff(h, weights, prefix, experts, top, r=lambda t: t):
    idx, p = route(h, weights[prefix + "router"], weights[prefix + "router.b"], top)
    y = torch.zeros_like(h)
    for e in range(experts):
        rows, place = (idx == e).nonzero(as_tuple=True)
        if rows.numel():
            n = f"{prefix}e{e}."
            y[rows] += p[rows, place, None] * silu_glu(h[rows], weights[n + "gate"], weights[n + "up"], weights[n + "down"], r)
    return y


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


@torch.no_grad()
def residuals_and_logits(cfg, weights, tokens, dtype=torch.float32, rounding=None):
    """-> ([layers, T, D] residual stream behind every layer, [T, V] logits)."""
    r = _rounder(rounding)
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]

    def norm(x, name):
        return group_rms(x, w[name], groups, eps)

    def mixed(x, norm_name, conv_name):
        h = r(norm(x, norm_name))
        return r(h + causal_conv(h, w[conv_name]))
    x = w["embed"][torch.as_tensor(tokens)]
    T, after, latents = x.shape[0], [], {}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        h = mixed(x, p + "norm1", p + "canon1")
        if m.get("kv_from") is None:
            latents[i] = r(group_rms(h @ w[p + "mix.dkv"].t(), w[p + "mix.dkv.norm"], 1, eps))
        c = latents[i if m.get("kv_from") is None else m["kv_from"]]
        q = (h @ w[p + "mix.q"].t()).view(T, m["heads"], m["dim"])
        o = latent_attention(q, c, w[p + "mix.uk"], w[p + "mix.uv"], m["scale"], m["mask"]["size"], r)
        x = x + norm(r(o.reshape(T, -1)) @ w[p + "mix.o"].t(), p + "norm1b")
        f = spec.get("mlp")
        if f is not None:
            h = mixed(x, p + "norm2", p + "canon2")
            if f["kind"] == "dense":
                y = clipped_glu_ff(h, w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"], f["limit"], r)
            else:
                y = expert_ff(h, w, p + "mlp.", f["router"]["experts"], f["router"]["top"], r)
            x = x + norm(y, p + "norm2b")
        after.append(x)
    z = r(norm(x, "final.norm")) @ w["head"].t()
    return torch.stack(after), softcap(z, cfg["logit_softcap"])


def logits(cfg, weights, tokens, dtype=torch.float32, rounding=None):
    return residuals_and_logits(cfg, weights, tokens, dtype, rounding)[1]
