"""Small Vimesun configurations and weights for the tests (made here, from a seed)."""

import math

import torch


def att(heads, kv, dim, vdim, window, ff=None, scale=None):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "mask": {"size": window},
                      "scale": scale if scale is not None else 1.7 / math.sqrt(dim)},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, loop=None, mult=0.6, eps=1e-4, max_positions=640):
    out = {"architecture": "Vimesun", "width": width, "vocab": vocab, "layers": layers, "residual_mult": mult,
           "norm": {"eps": eps}, "max_positions": max_positions}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CASES = {
    # sizes that are no multiple of anything, a layer without feed-forward, three heads per kv head, a loop in the middle
    "uneven": lambda: config(100, 203, [att(6, 2, 20, 26, 37, 90), att(3, 1, 33, 13, 5), att(4, 4, 48, 80, 200, 52)],
                             loop=(1, 3, 3), mult=0.45, eps=1e-2),
    # one head per kv head, 128-wide heads, window 1 beside a window longer than any sequence, no loop
    "plain": lambda: config(192, 336, [att(4, 4, 128, 64, 1, 256), att(6, 3, 64, 128, 5000, 320), att(8, 1, 96, 96, 16, 64)],
                            mult=1.0, eps=1e-6),
    # heads wider than 128, many heads on one kv head, a loop of one pass over everything
    "wide": lambda: config(320, 512, [att(2, 1, 160, 200, 65, 384), att(24, 1, 32, 16, 100, 128)], loop=(0, 2, 1), mult=0.8),
    # a single layer that runs four times, then nothing
    "looped": lambda: config(64, 128, [att(2, 2, 16, 16, 64, 48)], loop=(0, 1, 4), mult=0.3, eps=1e-5),
}


def weights(cfg, seed, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    D = cfg["width"]
    w = {}

    def mat(name, n, k, gain=1.0):
        w[name] = (torch.randn(n, k, generator=g) * gain / math.sqrt(k)).to(dtype)

    def norm(name):
        w[name] = (1 + 0.3 * torch.randn(D, generator=g)).to(dtype)
        w[name + ".b"] = (0.3 * torch.randn(D, generator=g)).to(dtype)
    # (an offset: a norm that forgets the mean shows)
    w["embed"] = (torch.randn(cfg["vocab"], D, generator=g) + 0.4).to(dtype)
    w["pos"] = (0.5 * torch.randn(cfg["max_positions"], D, generator=g)).to(dtype)
    if cfg.get("loop"):
        mat("loop.in", D, 2 * D)
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        norm(p + "norm1")
        mat(p + "mix.q", m["heads"] * m["dim"], D)
        mat(p + "mix.k", m["kv_heads"] * m["dim"], D)
        mat(p + "mix.v", m["kv_heads"] * m["vdim"], D)
        mat(p + "mix.o", D, m["heads"] * m["vdim"], 2.0)
        if layer["mlp"] is not None:
            norm(p + "norm2")
            mat(p + "mlp.up", layer["mlp"]["ff"], D)
            mat(p + "mlp.down", D, layer["mlp"]["ff"])
    norm("final.norm")
    mat("head", cfg["vocab"], D)
    return w


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def error(got, ref):
    """Root mean square of the difference (mean taken off) per row over the reference's overall scale."""
    d = got.double() - ref.double()
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / ref.double().std()).max().item()
