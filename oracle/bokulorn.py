"""Oracle: the Bokulorn decoder, plain and slow, on the CPU (TEST INFRASTRUCTURE ONLY).

One function per mechanism, written from the design's equations over whole sequences: no cache, no pages, no state slots, no
batches.  The framework's answer for a token must equal ``logits(...)[position]`` however the sequence was cut, batched and placed.

Notation: x [T, D] residual stream (fp32); N(x) = x / sqrt(mean x^2 + eps) * (1 + w).
  x_0       = s E[t]
  layer     h = N1(x);  x <- x + (mixer(h) + experts(h))
  logits    = W_head N_f(x)

``rounding`` selects the arithmetic: ``None`` = everything in ``dtype`` (fp32 or fp64); ``"bf16"`` = bf16 at every matrix-product
input and in what the cache keeps of a token, everything else in ``dtype``.
"""

from __future__ import annotations

import torch

__all__ = ["rms", "rotate", "latent_kv", "latent_attention", "short_conv", "unit", "decays", "delta_rule", "delta_heads", "delta_mixer", "pick",
           "expert_ff", "resolve", "residuals_and_logits", "logits"]


def _rounder(rounding):
    if rounding is None:
        return lambda t: t
    assert rounding == "bf16"
    return lambda t: t.to(torch.bfloat16).to(t.dtype)


def rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def rotate(x, base, dims, first=0):
    """x [T, ..., n]: the pairs (i, i + dims / 2) of the first `dims` elements turned by position * base^(-2 i / dims)."""
    half = dims // 2
    p = torch.arange(first, first + x.shape[0], dtype=torch.float64)
    f = torch.tensor(float(base), dtype=torch.float64) ** (-2.0 * torch.arange(half, dtype=torch.float64) / dims)
    a = (p[:, None] * f[None, :]).view(x.shape[0], *([1] * (x.dim() - 2)), half)
    c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def latent_kv(h, w_dkv, w_norm, rank, eps, rot=None, r=lambda t: t):
    """What a token leaves behind: the normed latent [T, rank] and the shared rotated key part [T, rot_dim] (or None)."""
    y = h @ w_dkv.t()
    c = r(rms(y[:, :rank], eps) * w_norm)
    return c, (r(rotate(y[:, rank:], rot["base"], rot["dims"])) if rot is not None else None)


def latent_attention(q, c, k_rot, w_uk, w_uv, scale, r=lambda t: t):
    """q [T, H, dim + rot] (rotated already), latents c [T, R], k_rot [T, rot] or None -> [T, H, dv]; causal, plain softmax."""
    T, H, dq = q.shape
    dk, dv = w_uk.shape[0] // H, w_uv.shape[0] // H
    k, v = (c @ w_uk.t()).view(T, H, dk), (c @ w_uv.t()).view(T, H, dv)
    ahead = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = torch.empty(T, H, dv, dtype=q.dtype)
    for i in range(H):
        s = r(q[:, i, :dk]) @ r(k[:, i]).t()
        if k_rot is not None:
            s = s + r(q[:, i, dk:]) @ k_rot.t()
        p = torch.softmax((s * scale).masked_fill(ahead, float("-inf")), -1)
        out[:, i] = r(p) @ r(v[:, i])
    return out


def latent_mixer(h, m, w, p, eps, per_head, r=lambda t: t):
    """`m` = the layer's mixer entry; w[p + name] its tensors.  The gate has one row per head, or one per element of the heads."""
    T, H, rot = h.shape[0], m["heads"], m.get("rot")
    nr = m.get("rot_dim", 0)
    c_q = r(rms(h @ w[p + "dq"].t(), eps) * w[p + "dq.norm"])
    q = (c_q @ w[p + "uq"].t()).view(T, H, m["dim"] + nr)
    if nr:
        q = torch.cat([q[..., :m["dim"]], rotate(q[..., m["dim"]:], rot["base"], rot["dims"])], -1)
    c, k_rot = latent_kv(h, w[p + "dkv"], w[p + "dkv.norm"], m["kv_rank"], eps, rot if nr else None, r)
    o = latent_attention(q, c, k_rot, w[p + "uk"], w[p + "uv"], m["scale"], r)
    g = torch.sigmoid(h @ w[p + "g"].t())
    o = o * g.view(T, H, 1 if per_head else m["vdim"])
    return r(o.reshape(T, -1)) @ w[p + "o"].t()


def short_conv(x, w):
    """y_t = silu(sum_j w[:, j] x_(t - taps + 1 + j)), zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * x[:T - back]
    return y * torch.sigmoid(y)


def unit(x):
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def decays(z, a_log, dt_bias):
    """z [T, H, d] -> log decay per head and key channel: -exp(A_h) softplus(z + dt_bias)."""
    H = a_log.shape[0]
    t = z + dt_bias.view(H, -1)
    return -torch.exp(a_log).view(H, 1) * (t.clamp(min=0) + torch.log1p(torch.exp(-t.abs())))


def delta_rule(q, k, v, log_g, beta, state=None):
    """q, k [T, H, d], v [T, H, dv], log_g [T, H, d], beta [T, H] -> (o [T, H, dv], the state [H, d, dv] behind the last token).

    S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q"""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = torch.exp(log_g[t])[:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def delta_heads(q, k, v, b, z, gate, conv, a_log, dt_bias, w_norm, eps):
    """From the projections of a whole sequence to the heads' outputs: q, k [T, G d], v [T, H dv], b [T, H], z [T, H d], gate [T, H dv],
    conv = the three convolutions' weights -> [T, H dv], and the state behind the last token."""
    T, H = b.shape
    d, dv = z.shape[1] // H, v.shape[1] // H
    G = q.shape[1] // d
    of = torch.arange(H) // (H // G)
    q, k, v = (short_conv(x, w) for x, w in zip((q, k, v), conv))
    q, k = unit(q.view(T, G, d))[:, of] * d ** -0.5, unit(k.view(T, G, d))[:, of]
    o, S = delta_rule(q, k, v.view(T, H, dv), decays(z.view(T, H, d), a_log, dt_bias), torch.sigmoid(b))
    return (rms(o, eps) * w_norm * torch.sigmoid(gate).view(T, H, dv)).reshape(T, H * dv), S


def delta_mixer(h, m, w, p, eps, r=lambda t: t):
    z = r(h @ w[p + "a1"].t()) @ w[p + "a2"].t()
    gate = r(h @ w[p + "g1"].t()) @ w[p + "g2"].t()
    y, _ = delta_heads(*(h @ w[p + n].t() for n in "qkvb"), z, gate, [w[p + n + ".conv"] for n in "qkv"], w[p + "A_log"], w[p + "dt_bias"],
                       w[p + "norm"], eps)
    return r(y) @ w[p + "o"].t()


def pick(z, correction, top, groups, keep):
    """Router logits z [T, E] -> (chosen experts [T, top], their weights)."""
    T, E = z.shape
    s = torch.sigmoid(z)
    choice = s + correction
    if groups > 1 or keep < groups:
        g = choice.view(T, groups, E // groups)
        score = g.topk(min(2, E // groups), -1).values.sum(-1)
        best = score.topk(keep, -1).indices
        ok = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, best, True)
        choice = g.masked_fill(~ok[:, :, None], float("-inf")).reshape(T, E)
    idx = choice.topk(top, -1).indices
    w = s.gather(1, idx)
    return idx, w / (w.sum(-1, keepdim=True) + 1e-20)


def expert_ff(h, f, w, p, r=lambda t: t):
    rt = f["router"]
    idx, share = pick(h @ w[p + "router"].t(), w[p + "correction"], rt["top"], rt["groups"]["count"], rt["groups"]["keep"])
    y = torch.zeros_like(h)
    for e in range(rt["experts"]):
        rows, place = (idx == e).nonzero(as_tuple=True)
        if rows.numel():
            a = (h[rows] @ w[f"{p}e{e}.up"].t()).clamp(min=0).pow(2)
            y[rows] += share[rows, place, None] * (r(a) @ w[f"{p}e{e}.down"].t())
    return y


def resolve(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


@torch.no_grad()
def residuals_and_logits(cfg, weights, tokens, dtype=torch.float32, rounding=None):
    """-> ([layers, T, D] residual stream behind every layer, [T, V] logits)."""
    r = _rounder(rounding)
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps = cfg["norm"]["eps"]

    def norm(x, name):
        return r(rms(x, eps) * (1 + w[name]))
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    after = []
    for i in range(len(cfg["layers"])):
        j = resolve(cfg["layers"], i)
        spec, p = cfg["layers"][j], f"l{j}."
        h = norm(x, p + "norm1")
        if spec["type"] == "channel_delta":
            y = delta_mixer(h, spec["mixer"], w, p + "mix.", eps, r)
        else:
            y = latent_mixer(h, spec["mixer"], w, p + "mix.", eps, spec["type"] == "latent_attention", r)
        if spec.get("mlp") is not None:
            y = y + expert_ff(h, spec["mlp"], w, p + "mlp.", r)
        x = x + y
        after.append(x)
    return torch.stack(after), norm(x, "final.norm") @ w["head"].t()


def logits(cfg, weights, tokens, dtype=torch.float32, rounding=None):
    return residuals_and_logits(cfg, weights, tokens, dtype, rounding)[1]
