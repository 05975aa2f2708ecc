"""Small Bokulorn configurations and weights for the tests (made here, from a seed)."""

import math

import torch

from oracle import bokulorn as R


def latent(heads, dim, vdim, rank, q_rank, rot_dim, dims=None, base=500.0, mlp=None, scale=None):
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "rot_dim": rot_dim,
        "rot": {"base": base, "dims": rot_dim if dims is None else dims}, "scale": scale or 1.6 / math.sqrt(dim + rot_dim)}}


def latent2(heads, dim, vdim, rank, q_rank, mlp=None, scale=None):
    return {"type": "latent_attention_2", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "scale": scale or 1.6 / math.sqrt(dim)}}


def delta(heads, kv_heads, dim, vdim, conv, mlp=None):
    return {"type": "channel_delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def moe(experts, top, ff, count=1, keep=1):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}}}


def again(layers, j):
    return dict(layers[j], weights_of=j)


def config(width, vocab, layers, scale=2.0, eps=1e-4):
    return {"architecture": "Bokulorn", "width": width, "vocab": vocab, "layers": layers, "embedding": {"scale": scale}, "norm": {"eps": eps}}


def _uneven():
    own = [delta(6, 2, 20, 13, 3, moe(9, 3, 22, 3, 2)), latent(3, 20, 26, 36, 28, 12, 8, mlp=moe(5, 1, 40)), latent2(5, 12, 9, 50, 22, None)]
    return config(120, 203, own + [again(own, 0), again(own, 1), again(own, 2)], scale=3.0, eps=1e-2)


def _wide():
    own = [latent(18, 64, 64, 160, 96, 64, base=3000.0, mlp=moe(8, 2, 64, 2, 1)), latent2(34, 16, 24, 64, 128, moe(6, 6, 32)), delta(4, 4, 128, 160, 4, None)]
    return config(320, 336, own + [again(own, 2)], scale=1.0, eps=1e-5)


def _taps():
    # one tap beside seven; shared key heads; a layer that runs a later layer's tensors; a rank above 256
    own = [delta(2, 1, 192, 48, 1, moe(12, 5, 48, 4, 2)), delta(3, 3, 24, 64, 7, None), latent(4, 32, 32, 272, 40, 20, 4, mlp=None)]
    own[1:1] = [{**own[2], "weights_of": 3}]
    return config(128, 256, own, scale=4.0, eps=1e-3)


def _plain():
    # beyond the matrix-core attention (rank above 512, heads above 256, a rotated part above 64), heads that are no multiple of
    # 4: the plain kernels in bf16 too; the largest state
    return config(64, 128, [latent(2, 22, 264, 520, 30, 96, 90), latent(1, 250, 32, 64, 70, 10, 10, mlp=moe(4, 2, 16, 2, 2)),
                            delta(1, 1, 256, 256, 16), latent2(3, 7, 5, 33, 9)], scale=2.5, eps=0.05)


CASES = {"uneven": _uneven, "wide": _wide, "taps": _taps, "plain": _plain}


def weights(cfg, seed, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    D, w = cfg["width"], {}

    def mat(name, n, k, gain=1.0):
        w[name] = (torch.randn(n, k, generator=g) * gain / math.sqrt(k)).to(dtype)

    def vec(name, n, mean=0.0, spread=0.3):
        w[name] = (mean + spread * torch.randn(n, generator=g)).to(dtype)
    mat("embed", cfg["vocab"], D, math.sqrt(D))
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        m, f, p = layer["mixer"], layer["mlp"], f"l{i}.mix."
        vec(f"l{i}.norm1", D)
        H, dv = m["heads"], m["vdim"]
        if layer["type"] == "channel_delta":
            G, d, taps, rank = m["kv_heads"], m["dim"], m["conv"], 10 + 3 * i
            for n, c in (("q", G * d), ("k", G * d), ("v", H * dv)):
                mat(p + n, c, D)
                w[p + n + ".conv"] = (torch.randn(c, taps, generator=g) * 1.2 / math.sqrt(taps)).to(dtype)
            mat(p + "b", H, D, 1.5)
            w[p + "A_log"] = (torch.rand(H, generator=g) * 4 - 3).to(dtype)      # memories of a few to a few hundred tokens
            vec(p + "dt_bias", H * d, -2.0, 1.0)
            mat(p + "a1", rank, D)
            mat(p + "a2", H * d, rank)
            mat(p + "g1", rank + 5, D)
            mat(p + "g2", H * dv, rank + 5, 1.5)
            vec(p + "norm", dv, 1.0)
        else:
            nr = m.get("rot_dim", 0)
            mat(p + "dq", m["q_rank"], D)
            vec(p + "dq.norm", m["q_rank"], 1.0)
            mat(p + "uq", H * (m["dim"] + nr), m["q_rank"])
            mat(p + "dkv", m["kv_rank"] + nr, D)
            vec(p + "dkv.norm", m["kv_rank"], 1.0)
            mat(p + "uk", H * m["dim"], m["kv_rank"])
            mat(p + "uv", H * dv, m["kv_rank"])
            mat(p + "g", H if nr else H * dv, D, 1.5)
        mat(p + "o", D, H * dv, 2.0 if layer["type"] == "channel_delta" else 5.0)
        if f is None:
            continue
        E, ff, p = f["router"]["experts"], f["expert"]["ff"], f"l{i}.mlp."
        mat(p + "router", E, D, 1.5)
        vec(p + "correction", E, 0.0, 0.4)
        for e in range(E):
            mat(f"{p}e{e}.up", ff, D, 1.5)
            mat(f"{p}e{e}.down", D, ff)
    vec("final.norm", D)
    mat("head", cfg["vocab"], D, 2.0)
    return w


_tokens = {}


def close_calls(z, correction, top, groups, keep):
    """How near the choice of experts is to another one, per row: the last chosen against the first refused expert of the eligible
    groups, the last kept against the first refused group."""
    T, E = z.shape
    c = torch.sigmoid(z) + correction
    gap = torch.full((T,), float("inf"), dtype=z.dtype)
    if keep < groups:
        g = c.view(T, groups, -1)
        v, best = g.topk(min(2, E // groups), -1).values.sum(-1).topk(keep + 1, -1)
        gap = v[:, -2] - v[:, -1]
        ok = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, best[:, :keep], True)
        c = g.masked_fill(~ok[:, :, None], float("-inf")).reshape(T, E)
    if top < E // groups * keep:
        v = c.topk(top + 1, -1).values
        gap = torch.minimum(gap, v[:, -2] - v[:, -1])
    return gap


def tokens(cfg, w, n, seed, margin=0.02):
    """Random tokens without a close call of any router (with the device's rounding it may fall either way)."""
    key = (id(w), n, seed)
    if key in _tokens:
        return _tokens[key][1]
    g = torch.Generator().manual_seed(seed)
    t = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    real = R.pick
    while any(x["mlp"] for x in cfg["layers"]):
        gap = torch.full((n,), float("inf"))

        def spy(z, *rule):
            gap.copy_(torch.minimum(gap, close_calls(z, *rule).float()))
            return real(z, *rule)
        R.pick = spy
        try:
            R.logits(cfg, w, t, torch.float32, "bf16")
        finally:
            R.pick = real
        bad = (gap < margin).nonzero().flatten().tolist()
        if not bad:
            break
        # (a replaced token changes everything behind it: keep to the first few)
        for i in bad[:max(1, len(bad) // 3)]:
            t[i] = int(torch.randint(0, cfg["vocab"], (1,), generator=g))
    _tokens[key] = (w, t)          # (w is kept alive: its id is the key)
    return t


def error(got, ref):
    """Root mean square of the difference (mean taken off) per row over the reference's overall scale."""
    d = got.double() - ref.double()
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / ref.double().std()).max().item()
