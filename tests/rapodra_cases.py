"""Small Rapodra configurations and weights for the tests (made here, from a seed)."""

import math

import torch

from oracle import rapodra as R


def latent(heads, dim, vdim, rank, window, mlp=None, kv_from=None, scale=None):
    mix = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "mask": {"size": window},
           "scale": scale if scale is not None else 1.6 / math.sqrt(dim)}
    if kv_from is not None:
        mix["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mix, "mlp": mlp}


def dense(ff, limit=1.1):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def config(width, vocab, layers, groups=1, taps=4, cap=9.0, eps=1e-4):
    return {"architecture": "Rapodra", "width": width, "vocab": vocab, "layers": layers, "canon": {"taps": taps},
            "norm": {"eps": eps, "groups": groups}, "logit_softcap": cap}


CASES = {
    # sizes that are no multiple of anything, latents read by a later layer, a layer without feed-forward, a large eps
    "uneven": lambda: config(120, 203, [latent(3, 20, 26, 36, 37, dense(90, 0.8)), latent(5, 12, 9, 36, 11, None, kv_from=0),
                                        latent(2, 33, 48, 50, 200, moe(7, 3, 22)), latent(6, 17, 31, 50, 23, moe(5, 1, 40), kv_from=2)],
                             groups=3, taps=3, cap=5.0, eps=1e-2),
    # more than one group of sixteen heads, all experts chosen, convolutions of one tap (no state), window 1 beside a window
    # longer than any sequence
    "wide": lambda: config(320, 336, [latent(18, 64, 64, 160, 5000, moe(20, 2, 64)), latent(34, 16, 24, 64, 1, dense(200, 3.0)),
                                      latent(2, 128, 160, 160, 96, moe(4, 4, 32), kv_from=0)], groups=1, taps=1, cap=30.0),
    # a long convolution, parts of eight elements, a rank above 256
    "taps": lambda: config(128, 256, [latent(4, 48, 32, 272, 64, dense(128, 0.5)), latent(4, 64, 48, 32, 33, moe(12, 5, 48))],
                           groups=16, taps=7, cap=12.0, eps=1e-5),
    # sizes beyond the matrix-core attention (rank above 512, heads above 256): the plain kernel in bf16 too; as many taps as a
    # page has tokens
    "plain": lambda: config(64, 128, [latent(2, 24, 264, 520, 20, dense(64)), latent(1, 288, 32, 64, 40, moe(3, 2, 16)),
                                      latent(3, 16, 16, 520, 64, None, kv_from=0)], groups=4, taps=16, cap=4.0, eps=0.05),
}


def weights(cfg, seed, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    D, taps = cfg["width"], cfg["canon"]["taps"]
    w = {}

    def mat(name, n, k, gain=1.0):
        w[name] = (torch.randn(n, k, generator=g) * gain / math.sqrt(k)).to(dtype)

    def norm(name, n=D, level=1.0):
        w[name] = (level * (1 + 0.3 * torch.randn(n, generator=g))).to(dtype)
    w["embed"] = torch.randn(cfg["vocab"], D, generator=g).to(dtype)
    for i, layer in enumerate(cfg["layers"]):
        m, f, p = layer["mixer"], layer["mlp"], f"l{i}."
        norm(p + "norm1")
        norm(p + "norm1b", level=0.8)
        w[p + "canon1"] = (torch.randn(D, taps, generator=g) * 0.5 / math.sqrt(taps)).to(dtype)
        mat(p + "mix.q", m["heads"] * m["dim"], D)
        if m.get("kv_from") is None:
            mat(p + "mix.dkv", m["kv_rank"], D)
            norm(p + "mix.dkv.norm", m["kv_rank"])
        mat(p + "mix.uk", m["heads"] * m["dim"], m["kv_rank"])
        mat(p + "mix.uv", m["heads"] * m["vdim"], m["kv_rank"])
        mat(p + "mix.o", D, m["heads"] * m["vdim"])
        if f is None:
            continue
        norm(p + "norm2")
        norm(p + "norm2b", level=0.8)
        w[p + "canon2"] = (torch.randn(D, taps, generator=g) * 0.5 / math.sqrt(taps)).to(dtype)
        if f["kind"] == "dense":
            mat(p + "mlp.gate", f["ff"], D)
            mat(p + "mlp.up", f["ff"], D)
            mat(p + "mlp.down", D, f["ff"])
        else:
            E, ff = f["router"]["experts"], f["expert"]["ff"]
            mat(p + "mlp.router", E, D, 1.5)
            w[p + "mlp.router.b"] = (torch.randn(E, generator=g)).to(dtype)
            for e in range(E):
                mat(f"{p}mlp.e{e}.gate", ff, D, 1.5)
                mat(f"{p}mlp.e{e}.up", ff, D)
                mat(f"{p}mlp.e{e}.down", D, ff)
    norm("final.norm")
    mat("head", cfg["vocab"], D, 2.0)
    return w


_tokens = {}


def tokens(cfg, w, n, seed, margin=0.06):
    """Random tokens without a close call of any router: the last chosen and the first refused expert's logits differ by
    `margin` of the logits' spread at every position (with the device's rounding, a closer pair may fall either way)."""
    key = (id(w), n, seed)
    if key in _tokens:
        return _tokens[key][1]
    g = torch.Generator().manual_seed(seed)
    t = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    real = R.route
    while any(x["mlp"] and x["mlp"]["kind"] == "moe" for x in cfg["layers"]):
        gap = torch.full((n,), float("inf"))

        def spy(h, rw, b, top):
            z = h @ rw.t() + b
            if top < z.shape[1]:
                v = z.topk(top + 1, -1).values
                gap.copy_(torch.minimum(gap, ((v[:, -2] - v[:, -1]) / z.std()).float()))
            return real(h, rw, b, top)
        R.route = spy
        try:
            R.logits(cfg, w, t, torch.float32, "bf16")
        finally:
            R.route = real
        bad = (gap < margin).nonzero().flatten().tolist()
        if not bad:
            break
        # (a replaced token changes what follows through the convolutions and the attention: keep to the first few)
        for i in bad[:max(1, len(bad) // 3)]:
            t[i] = int(torch.randint(0, cfg["vocab"], (1,), generator=g))
    _tokens[key] = (w, t)          # (w is kept alive: its id is the key)
    return t


def error(got, ref):
    """Root mean square of the difference (mean taken off) per row over the reference's overall scale."""
    d = got.double() - ref.double()
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / ref.double().std()).max().item()
