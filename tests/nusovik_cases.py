"""Small Nusovik configurations and weights for the tests (made here, from a seed)."""

import math

import torch


def mamba1(inner, state, rank, conv, ff=None):
    return {"type": "mamba1", "mlp": dense(ff), "mixer": {"inner": inner, "state": state, "dt_rank": rank, "conv": conv}}


def dense(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def left(heads, kv_heads, dim, chunk, far, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale or 1.6 / math.sqrt(dim), "bias_max": far, "mask": {"size": chunk}}


def right(heads, vdim, state, groups, parts, conv):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": parts, "conv": conv}


def parallel(a, b, ff=None, scales=(0.8, 1.3)):
    return {"type": "parallel", "mlp": dense(ff), "mixer": {"left": a, "right": b, "left_scale": scales[0], "right_scale": scales[1]}}


def config(width, vocab, layers, scale=2.0, eps=1e-4, logit_scale=0.7):
    return {"architecture": "Nusovik", "width": width, "vocab": vocab, "layers": layers, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "logit_scale": logit_scale}


# rows of every layer's distance table (config.json does not give them)
ROWS = {"uneven": (9, 6), "wide": (32, 16), "taps": (2, 5, 1), "plain": (24, 12)}


def _uneven():
    return config(122, 203, [mamba1(50, 10, 7, 3, 90), parallel(left(6, 2, 20, 37, 30), right(4, 13, 20, 2, 4, 5)), mamba1(68, 3, 20, 4),
                             parallel(left(3, 3, 34, 50, 11), right(6, 10, 33, 3, 2, 2), 41, (1.7, 0.6))], scale=3.0, eps=0.15)


def _wide():
    return config(256, 336, [parallel(left(8, 2, 64, 128, 100), right(8, 64, 128, 1, 1, 4), 384, (1.0, 1.0)), mamba1(512, 16, 24, 4),
                             parallel(left(16, 1, 128, 64, 64), right(4, 128, 64, 4, 8, 4), None, (0.5, 2.0)), mamba1(256, 64, 40, 4, 192)],
                  scale=3.0, eps=1e-5, logit_scale=1.0)


def _taps():
    # one tap beside seven and two; a chunk of a page; tables of one, two and five rows; heads wider than 128; one state
    return config(96, 131, [parallel(left(2, 1, 200, 16, 2), right(3, 48, 5, 3, 2, 1)), mamba1(90, 1, 3, 1, 64), mamba1(130, 30, 33, 7),
                            parallel(left(4, 4, 8, 90, 40), right(2, 20, 2, 1, 2, 7), 70), mamba1(48, 100, 1, 2),
                            parallel(left(1, 1, 48, 1, 9), right(1, 64, 16, 1, 1, 2))], scale=3.0, eps=0.1, logit_scale=2.5)


def _plain():
    # beyond the matrix-core attention (heads above 256, more than 64 query heads per kv head); the largest states
    return config(64, 128, [parallel(left(2, 2, 264, 70, 60), right(1, 256, 256, 1, 4, 16), 30), mamba1(36, 200, 9, 16),
                            parallel(left(70, 1, 8, 33, 20), right(2, 130, 144, 2, 1, 3))], scale=2.5, eps=0.05)


CASES = {"uneven": _uneven, "wide": _wide, "taps": _taps, "plain": _plain}


def weights(cfg, seed, rows=(8,), dtype=torch.bfloat16):
    """rows: of the distance tables, in the order of the layers that have one (the last one for the rest)"""
    g = torch.Generator().manual_seed(seed)
    D, w, rows = cfg["width"], {}, list(rows)

    def mat(name, n, k, gain=1.0):
        w[name] = (torch.randn(n, k, generator=g) * gain / math.sqrt(k)).to(dtype)

    def vec(name, n, mean=0.0, spread=0.3):
        w[name] = (mean + spread * torch.randn(n, generator=g)).to(dtype)

    def conv(p, c, taps):
        w[p + "conv"] = (torch.randn(c, taps, generator=g) * 1.2 / math.sqrt(taps)).to(dtype)
        vec(p + "conv.b", c)

    def logs(name, *shape):                              # memories of a few to a few hundred tokens
        w[name] = (torch.rand(*shape, generator=g) * 4 - 3).to(dtype)
    mat("embed", cfg["vocab"], D, math.sqrt(D))
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        vec(f"l{i}.norm1", D, 1.0)
        if layer["type"] == "mamba1":
            C, N, R = m["inner"], m["state"], m["dt_rank"]
            mat(p + "in", 2 * C, D)
            conv(p, C, m["conv"])
            mat(p + "x", R + 2 * N, C, 0.6)
            mat(p + "dt", C, R, 1.0)
            vec(p + "dt.b", C, -1.5, 1.0)
            logs(p + "A_log", C, N)
            vec(p + "D", C, 1.0, 0.5)
            mat(p + "o", D, C)
        else:
            a, b = m["left"], m["right"]
            H, G, d, n = a["heads"], a["kv_heads"], a["dim"], p + "left."
            mat(n + "q", H * d, D)
            vec(n + "q.b", H * d, 0.0, 0.5)
            mat(n + "k", G * d, D)
            vec(n + "k.b", G * d, 0.0, 0.5)
            vec(n + "q.norm", d, 1.0)
            vec(n + "k.norm", d, 1.0)
            r = rows.pop(0) if len(rows) > 1 else rows[0]
            w[n + "rel"] = (torch.randn(r, H, generator=g) * 1.5).to(dtype)
            vec(n + "sink", H, 1.5, 1.0)
            mat(n + "g", H, D, 1.5)
            mat(n + "o", D, H * d)
            H, P, N, G, n = b["heads"], b["vdim"], b["state"], b["groups"], p + "right."
            C = H * P + 2 * G * N
            mat(n + "in", H * P + C + H, D)
            conv(n, C, b["conv"])
            vec(n + "dt_bias", H, -1.5, 1.0)
            logs(n + "A_log", H)
            vec(n + "D", H, 0.5, 0.5)
            vec(n + "norm", H * P, 1.0)
            mat(n + "o", D, H * P)
        if layer["mlp"] is not None:
            vec(f"l{i}.norm2", D, 1.0)
            mat(f"l{i}.mlp.up", layer["mlp"]["ff"], D, 1.5)
            mat(f"l{i}.mlp.down", D, layer["mlp"]["ff"])
    vec("final.norm", D, 1.0)
    mat("head", cfg["vocab"], D, 2.0)
    return w


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def error(got, ref):
    """Root mean square of the difference (mean taken off) per row over the reference's overall scale."""
    d = got.double() - ref.double()
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / ref.double().std()).max().item()
