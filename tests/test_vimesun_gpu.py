"""Vimesun on the MI355X: every kernel of the layer stack against the oracle's mechanism of the same name, and the model
through the framework's engine against the oracle's whole-sequence logits -- prompts whole, in portions and token by token,
in mixed batches, over a KV pool small enough that pages and slots are used again."""

import json
import math

import pytest
import torch

from oracle import vimesun as V
from tests.vimesun_cases import CASES, att, config, error, tokens, weights

pytestmark = pytest.mark.gpu

# fp32: rounding only.  bf16: against the oracle with the device's rounding points (what is left is summation order and
# the rounding flips it causes).
LIMIT = {"float32": 2e-5, "bfloat16": 2.5e-2}


@pytest.fixture(scope="module")
def lib():
    from vllm_neuron_amd import _native
    return _native


def dev(t):
    return t.to("cuda").contiguous()


def pad16(n):
    return (n + 15) // 16 * 16


# ---- kernels -----------------------------------------------------------------------------------------
@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("T,D", [(1, 64), (3, 100), (17, 2050), (5, 8192)])
def test_layernorm_two_outputs(lib, T, D, f32):
    torch.manual_seed(D)
    ld, ldy = pad16(D), (D + 63) // 64 * 64
    x = torch.zeros(T, ld)
    x[:, :D] = torch.randn(T, D) * torch.linspace(1, 30, T)[:, None] + 5.0
    wb = [torch.zeros(ld) for _ in range(4)]
    for t in wb:
        t[:D] = torch.randn(D)
    d = [dev(t) for t in wb]
    dt = torch.float32 if f32 else torch.bfloat16
    ys = [torch.zeros(T, ldy, dtype=dt, device="cuda") for _ in range(2)]
    xd = dev(x)
    lib.check(lib.load_library().mi_op_layernorm2(xd.data_ptr(), T, D, ld, 1e-3, d[0].data_ptr(), d[1].data_ptr(), ys[0].data_ptr(),
                                                  d[2].data_ptr(), d[3].data_ptr(), ys[1].data_ptr(), ldy, f32, None))
    torch.cuda.synchronize()
    for y, (w, b) in zip(ys, ((wb[0], wb[1]), (wb[2], wb[3]))):
        ref = V.layer_norm(x[:, :D].double(), w[:D].double(), b[:D].double(), 1e-3)
        got = y.cpu().double()
        assert (got[:, D:] == 0).all()
        tol = 1e-5 if f32 else 1e-2
        assert ((got[:, :D] - ref).abs() <= tol * (1 + ref.abs())).all()


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("D", [64, 99])
def test_embedding_with_learned_positions(lib, D, f32):
    torch.manual_seed(1)
    dt = torch.float32 if f32 else torch.bfloat16
    tab, ptab = torch.randn(50, D).to(dt), torch.randn(40, D).to(dt)
    ids, pos = torch.tensor([3, 49, 0, 3], dtype=torch.int32), torch.tensor([0, 39, 7, 1], dtype=torch.int32)
    ld = pad16(D)
    out, x0 = (torch.full((4, ld), 9.0, device="cuda") for _ in range(2))
    a = [dev(t) for t in (ids, pos, tab, ptab)]
    lib.check(lib.load_library().mi_op_embed_pos(*(t.data_ptr() for t in a), 4, D, ld, out.data_ptr(), x0.data_ptr(), f32, None))
    torch.cuda.synchronize()
    ref = tab.float()[ids.long()] + ptab.float()[pos.long()]
    assert torch.equal(out.cpu()[:, :D], ref) and (out.cpu()[:, D:] == 0).all() and torch.equal(out, x0)


def spec_of(lib, H, G, dk, dv, window, scale, bias=1, sink=1, unit=1):
    return lib.layer_spec(dict(num_heads=H, num_kv_heads=G, qk_dim=dk, v_dim=dv, window=window, scale=scale, qk_unit_norm=unit,
                               distance_bias=bias, softmax_sink=sink, ff_kind=0, ff_size=0))


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("unit", [0, 1])
@pytest.mark.parametrize("H,G,dk,dv", [(8, 2, 64, 80), (3, 1, 20, 13), (4, 4, 33, 128), (2, 1, 200, 160)])
def test_unit_norm_and_kv_scatter(lib, H, G, dk, dv, unit, f32):
    torch.manual_seed(2)
    T, bs, nb = 9, 16, 5
    n = (H + G) * dk + G * dv
    ldq = pad16(n)
    qkv = torch.randn(T, ldq) * 3
    slots = torch.tensor([17, 40, -1, 79, 16, 63, 64, 1, 30], dtype=torch.int32)
    dt = torch.float32 if f32 else torch.bfloat16
    q = torch.full((T, H, pad16(dk)), 7.0, dtype=dt, device="cuda")
    kp = torch.full((nb, G, bs, pad16(dk)), 7.0, dtype=dt, device="cuda")
    vp = torch.full((nb, G, bs, pad16(dv)), 7.0, dtype=dt, device="cuda")
    spec = spec_of(lib, H, G, dk, dv, 8, 1.0, unit=unit)
    a, b = dev(qkv), dev(slots)
    lib.check(lib.load_library().mi_op_qkv_scatter(a.data_ptr(), ldq, T, spec, 1e-3, b.data_ptr(), bs, q.data_ptr(), kp.data_ptr(),
                                                   vp.data_ptr(), f32, None))
    torch.cuda.synchronize()
    f = (lambda t: V.unit_rms(t, 1e-3)) if unit else (lambda t: t)
    qr = f(qkv[:, :H * dk].reshape(T, H, dk).double())
    kr = f(qkv[:, H * dk:(H + G) * dk].reshape(T, G, dk).double())
    vr = qkv[:, (H + G) * dk:n].reshape(T, G, dv).double()
    tol = 1e-5 if f32 else 1.2e-2

    def close(got, ref, d):
        got = got.cpu().double()
        assert (got[..., d:] == 0).all() and ((got[..., :d] - ref).abs() <= tol * (1 + ref.abs())).all()
    close(q, qr, dk)
    kp, vp = kp.cpu(), vp.cpu()
    written = torch.zeros(nb, bs, dtype=torch.bool)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            close(kp[s // bs, :, s % bs], kr[t], dk)
            close(vp[s // bs, :, s % bs], vr[t], dv)
            written[s // bs, s % bs] = True
    assert (kp.permute(0, 2, 1, 3)[~written] == 7.0).all() and (vp.permute(0, 2, 1, 3)[~written] == 7.0).all()


class Paged:
    """One random sequence per request, its K / V scattered over shuffled pool blocks, and a ragged set of queries."""

    def __init__(self, H, G, dk, dv, segs, bs, seed, q_gain=1.0):
        g = torch.Generator().manual_seed(seed)
        self.H, self.G, self.dk, self.dv, self.bs = H, G, dk, dv, bs
        self.segs, row = [], 0
        for i, (pos0, n) in enumerate(segs):
            self.segs.append((row, n, pos0, i))
            row += n
        self.T, self.max_ctx = row, max(p + n for p, n in segs)
        self.MB = -(-self.max_ctx // bs) + 1
        nb = 1 + sum(-(-(p + n) // bs) for p, n in segs) + 3
        perm = (torch.randperm(nb - 1, generator=g) + 1).tolist()
        self.bt = torch.zeros(len(segs), self.MB, dtype=torch.int32)
        self.q = [V.unit_rms(torch.randn(p + n, H, dk, generator=g), 1e-6) * q_gain for p, n in segs]
        self.k = [V.unit_rms(torch.randn(p + n, G, dk, generator=g), 1e-6) for p, n in segs]
        self.v = [torch.randn(p + n, G, dv, generator=g) for p, n in segs]
        for i, (p, n) in enumerate(segs):
            for b in range(-(-(p + n) // bs)):
                self.bt[i, b] = perm.pop()
        self.nb = nb

    def run(self, lib, spec, slopes, f32, path):
        dt = torch.float32 if f32 else torch.bfloat16
        r = (lambda t: t) if f32 else (lambda t: t.to(torch.bfloat16).float())
        # rows nobody wrote hold something large but finite: reading one shows
        kp = torch.full((self.nb, self.G, self.bs, pad16(self.dk)), 50.0)
        vp = torch.full((self.nb, self.G, self.bs, pad16(self.dv)), 50.0)
        kp[..., self.dk:] = 0
        vp[..., self.dv:] = 0
        q = torch.zeros(self.T, self.H, pad16(self.dk))
        pos = torch.zeros(self.T, dtype=torch.int32)
        ctx = torch.tensor([p + n for _, n, p, _ in self.segs], dtype=torch.int32)
        ref = torch.zeros(self.T, self.H * self.dv, dtype=torch.float64)
        for row, n, p, i in self.segs:
            q[row:row + n, :, :self.dk] = self.q[i][p:]
            pos[row:row + n] = torch.arange(p, p + n)
            for t in range(p + n):
                b = int(self.bt[i, t // self.bs])
                kp[b, :, t % self.bs, :self.dk] = self.k[i][t]
                vp[b, :, t % self.bs, :self.dv] = self.v[i][t]
            o = V.window_attention(r(self.q[i]).double(), r(self.k[i]).double(), r(self.v[i]).double(), spec.scale,
                                   spec.window if spec.window else 1 << 30, slopes.double() if spec.distance_bias else None,
                                   bool(spec.softmax_sink))
            ref[row:row + n] = o[p:].reshape(n, -1)
        ldo = (self.H * self.dv + 63) // 64 * 64
        out = torch.zeros(self.T, ldo, dtype=dt, device="cuda")
        a = [dev(x) for x in (slopes.float(), q.to(dt), kp.to(dt), vp.to(dt), self.bt, pos, ctx)]
        segs = torch.tensor(self.segs, dtype=torch.int32).contiguous()
        lib.check(lib.load_library().mi_op_window_attn(
            spec, a[0].data_ptr(), a[1].data_ptr(), a[2].data_ptr(), a[3].data_ptr(), self.bs, a[4].data_ptr(), self.MB,
            a[5].data_ptr(), a[6].data_ptr(), segs.data_ptr(), len(self.segs), self.T, self.max_ctx, out.data_ptr(), ldo,
            int(f32), path, None))
        torch.cuda.synchronize()
        got = out.cpu().double()
        assert (got[:, self.H * self.dv:] == 0).all()
        return got[:, :self.H * self.dv], ref


PATHS = [(1, 1), (0, 1), (0, 0)]      # (fp32?, path): plain fp32, plain bf16, MFMA
SEGS = [(0, 70), (45, 1), (31, 2), (0, 1), (100, 130), (299, 1), (0, 3), (64, 65)]


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("H,G,dk,dv,window,bs", [
    (8, 2, 64, 80, 96, 16), (6, 2, 20, 13, 37, 32), (4, 4, 128, 128, 0, 48), (24, 1, 32, 16, 5, 16), (2, 1, 160, 256, 129, 32),
    (8, 1, 100, 64, 1, 16), (5, 5, 64, 64, 64, 16)])
def test_window_attention(lib, H, G, dk, dv, window, bs, f32, path):
    spec = spec_of(lib, H, G, dk, dv, window, 2.5 / math.sqrt(dk))
    got, ref = Paged(H, G, dk, dv, SEGS, bs, seed=H + window).run(lib, spec, V.slopes(H), f32, path)
    assert ((got - ref).abs() <= (2e-5 if f32 else 1.5e-2) * (1 + ref.abs())).all(), (got - ref).abs().max()


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("bias,sink", [(0, 0), (1, 0), (0, 1)])
def test_bias_and_sink_are_options(lib, bias, sink, f32, path):
    spec = spec_of(lib, 6, 3, 48, 32, 50, 0.3, bias=bias, sink=sink, unit=bias)     # unit = 0: the running-maximum softmax
    got, ref = Paged(6, 3, 48, 32, SEGS, 16, seed=5).run(lib, spec, V.slopes(6), f32, path)
    assert ((got - ref).abs() <= (2e-5 if f32 else 1.5e-2) * (1 + ref.abs())).all()


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("top,unit", [(40.0, 1), (90.0, 1), (700.0, 1), (60.0, 0)])
def test_large_scores(lib, top, unit, f32, path):
    """Scores up to `top` and down to -top: within and beyond what a fixed softmax reference can span; unit = 0 says nothing
    about the heads' size, so q may be anything."""
    p = Paged(4, 2, 64, 64, SEGS, 16, seed=16, q_gain=1.0 if unit else 3.0)
    for i in range(len(p.k)):
        for t in range(0, p.k[i].shape[0], 3):             # exact matches and exact opposites among the random keys
            p.k[i][t] = V.unit_rms(p.q[i][t, ::2], 1e-6) * (1 if t % 2 else -1)
    spec = spec_of(lib, 4, 2, 64, 64, 90, top / 64, unit=unit)
    got, ref = p.run(lib, spec, V.slopes(4), f32, path)
    # (the error of a score grows with its size)
    assert ((got - ref).abs() <= (1e-3 if f32 else 3e-2) * (1 + ref.abs())).all(), (got - ref).abs().max()


@pytest.mark.parametrize("f32,path", PATHS)
def test_sink_with_every_score_far_below_zero(lib, f32, path):
    p = Paged(4, 2, 64, 64, SEGS, 16, seed=6)
    for i in range(len(p.k)):       # every key points away from every query of its group: scores around -20
        d = V.unit_rms(torch.randn(64, generator=torch.Generator().manual_seed(i)), 1e-6)
        p.q[i] = d.expand_as(p.q[i]) + 0.05 * p.q[i]
        p.k[i] = -d.expand_as(p.k[i]) + 0.05 * p.k[i]
    spec = spec_of(lib, 4, 2, 64, 64, 90, 8.0 / 64)
    got, ref = p.run(lib, spec, V.slopes(4), f32, path)
    assert 0 < ref.abs().max() < 0.1                       # the sink holds nearly all of the weight
    assert ((got - ref).abs() <= 1e-6 + (1e-4 if f32 else 2e-2) * ref.abs().max()).all()


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("window,bs", [(96, 16), (33, 32), (64, 16), (128, 32), (16, 16), (1, 16), (200, 48)])
def test_window_edge_key_stands_out(lib, window, bs, f32, path):
    """One key per query direction with a score far above the rest, placed at every distance around the edge: just inside it
    takes the row, one further out it must have no influence at all -- in prompts, at page borders and in decoding."""
    H, G, dk, dv = 4, 2, 64, 48
    segs = [(260, 1), (259, 2), (191, 80), (0, 240), (256, 1), (255, 3)]
    for off in (-1, 0, 1, -bs):                            # distance window - 1 (inside), window, ... of the segment's last row
        p = Paged(H, G, dk, dv, segs, bs, seed=window + 7)
        for i, (pos0, n) in enumerate(segs):
            last = pos0 + n - 1
            j = last - (window - 1) - off
            if 0 <= j <= last:
                u = V.unit_rms(torch.randn(G, dk, generator=torch.Generator().manual_seed(i)), 1e-6)
                p.k[i][j] = u
                for h in range(H):
                    p.q[i][last, h] = u[h // (H // G)]
                p.v[i][j] = 30.0
        spec = spec_of(lib, H, G, dk, dv, window, 30.0 / dk)
        got, ref = p.run(lib, spec, V.slopes(H) * 0.01, f32, path)
        assert ((got - ref).abs() <= (5e-5 if f32 else 2e-2) * (1 + ref.abs())).all(), (off, (got - ref).abs().max())


@pytest.mark.parametrize("f32,path", PATHS)
def test_far_key_of_a_long_context(lib, f32, path):
    """A key more than two thousand tokens back that holds a decoded token's attention (context split over work-groups)."""
    H, G, dk, dv = 4, 1, 64, 64
    p = Paged(H, G, dk, dv, [(2300, 1), (2250, 40)], 32, seed=9)
    key = 32 * 3 + 31
    for i, n in enumerate((2301, 2290)):
        u = V.unit_rms(torch.randn(dk, generator=torch.Generator().manual_seed(50 + i)), 1e-6)
        p.k[i][key] = u
        p.q[i][n - 1, :] = u
        p.v[i][key] = 9.0
    for window in (0, 2400, 2301 - key, 2300 - key, 2290 - key, 2289 - key):
        spec = spec_of(lib, H, G, dk, dv, window, 20.0 / dk)
        got, ref = p.run(lib, spec, V.slopes(H) * 1e-3, f32, path)
        assert (ref[0].abs().max() > 5) == (window in (0, 2400, 2301 - key))
        assert (ref[-1].abs().max() > 5) == (window != 2289 - key)
        assert ((got - ref).abs() <= (5e-5 if f32 else 2e-2) * (1 + ref.abs())).all()


# ---- model ---------------------------------------------------------------------------------------------
def replay(cfg, w, dtype, max_tokens=768, max_live=4, block_size=16, **override):
    from vllm_neuron_amd.models import config_from_dict
    from vllm_neuron_amd.replay import TraceReplay
    return TraceReplay.from_config(config_from_dict(cfg), dtype, max_tokens, max_live, block_size,
                                   override={"state_dict": w, **override})


_refs = {}


def reference(name, cfg, w, toks, dtype):
    """Oracle logits of a whole sequence (shared between the tests of a case)."""
    key = (name, tuple(toks), dtype)
    if key not in _refs:
        _refs[key] = V.logits(cfg, w, toks, torch.float64 if dtype == "float32" else torch.float32,
                              None if dtype == "float32" else "bf16")
    return _refs[key]


@pytest.fixture(scope="module", params=[(n, d) for n in CASES for d in LIMIT], ids=lambda p: f"{p[0]}-{p[1]}")
def served(request):
    name, dtype = request.param
    cfg = CASES[name]()
    w = weights(cfg, 11)
    r = replay(cfg, w, dtype)
    yield name, dtype, cfg, w, r
    r.engine.close()


_uid = [0]


def uid():
    _uid[0] += 1
    return f"r{_uid[0]}"


def score(r, toks, cuts):
    """One request alone, cut into portions; -> logits at every position."""
    rid, out, at = uid(), [], 0
    for i, n in enumerate(cuts):
        part = toks[at:at + n]
        at += n
        out.append(r.step([{"id": rid, "tokens": part, "want": list(range(len(part)))}], [rid] if at >= len(toks) else [])[0])
    assert at >= len(toks)
    return torch.cat(out)


def test_whole_prompts(served):
    name, dtype, cfg, w, r = served
    for n in (1, 2, 15, 16, 17, 130, 333):
        toks = tokens(cfg, n, n)
        assert error(score(r, toks, [n]), reference(name, cfg, w, toks, dtype)) <= LIMIT[dtype], n


def test_token_by_token_equals_the_prompt(served):
    name, dtype, cfg, w, r = served
    toks = tokens(cfg, 130, 130)
    ref = reference(name, cfg, w, toks, dtype)
    assert error(score(r, toks, [1] * 130), ref) <= LIMIT[dtype]
    assert error(score(r, toks, [60] + [1] * 70), ref) <= LIMIT[dtype]


@pytest.mark.parametrize("cuts", [[2] * 65, [3] * 44, [5] * 26, [16] * 9, [17] * 8, [33] * 4, [100, 2, 28],
                                  [2, 1, 5, 1, 40, 2, 2, 1, 64, 12]])
def test_portions(served, cuts):
    name, dtype, cfg, w, r = served
    toks = tokens(cfg, 130, 130)
    assert error(score(r, toks, cuts), reference(name, cfg, w, toks, dtype)) <= LIMIT[dtype]


def test_mixed_batches_over_reused_pages(served):
    """Up to four live requests, portions beside single tokens, requests left out of steps and ended; the pool holds far
    fewer tokens than the requests together."""
    name, dtype, cfg, w, r = served
    g = torch.Generator().manual_seed(3)

    def rnd(a, b):
        return int(torch.randint(a, b, (1,), generator=g))
    todo = [tokens(cfg, n, 1000 + i) for i, n in enumerate([150, 9, 70, 1, 120, 47, 64, 33, 90, 16, 2, 81])]
    total, pool = sum(map(len, todo)), 768 // 16
    assert total < 768 and r.engine.scheduler.block_pool.num_free() == pool
    live, worst, seen, steps, used = {}, 0.0, 0, 0, 0
    while todo or live:
        while todo and len(live) < 4:
            live[uid()] = [todo.pop(0), 0]
        entries, end = [], []
        for rid, st in live.items():
            if len(live) > 1 and rnd(0, 5) == 0:
                continue                                    # left out of this step
            n = min(1 if rnd(0, 2) else rnd(1, 50), len(st[0]) - st[1])
            entries.append({"id": rid, "tokens": st[0][st[1]:st[1] + n], "want": sorted({0, n // 2, n - 1})})
        if not entries:
            continue
        for e in entries:
            st = live[e["id"]]
            e["at"], st[1] = st[1], st[1] + len(e["tokens"])
            if st[1] == len(st[0]):
                end.append(e["id"])
        outs = r.step(entries, end)
        used += sum(len(e["tokens"]) for e in entries)
        for e, o in zip(entries, outs):
            ref = reference(name, cfg, w, live[e["id"]][0], dtype)
            worst = max(worst, error(o, ref[[e["at"] + x for x in e["want"]]]))
            seen += len(e["want"])
        for rid in end:
            del live[rid]
        steps += 1
    assert worst <= LIMIT[dtype] * 1.5, worst
    assert used == total and steps > 20 and seen > 100
    r.engine.scheduler.schedule()
    assert r.engine.scheduler.block_pool.num_free() == pool         # everything came back


def test_batch_does_not_change_a_request(served):
    """The same request alone and beside others: the same logits beyond rounding (here: to the bf16 / fp32 limit's tenth)."""
    name, dtype, cfg, w, r = served
    toks, other = tokens(cfg, 90, 90), [tokens(cfg, n, 400 + n) for n in (33, 2, 71)]
    alone = score(r, toks, [90])
    rid, ids = uid(), [uid() for _ in other]
    outs = r.step([{"id": ids[0], "tokens": other[0], "want": []}, {"id": rid, "tokens": toks[:50], "want": list(range(50))},
                   {"id": ids[1], "tokens": other[1], "want": []}, {"id": ids[2], "tokens": other[2], "want": [3]}], [])
    outs2 = r.step([{"id": ids[1], "tokens": [1], "want": [0]}, {"id": rid, "tokens": toks[50:], "want": list(range(40))}],
                   [rid] + ids)
    both = torch.cat([outs[1], outs2[1]])
    assert error(both, alone) <= LIMIT[dtype]


@pytest.mark.parametrize("dtype", list(LIMIT))
def test_long_decoding_and_pages_of_ended_requests(dtype):
    """A pool of exactly one long request: every sequence runs over the pages of the one before, decoding far past the
    windows, across page borders, with graph replays."""
    name = "uneven"
    cfg = CASES[name]()
    w = weights(cfg, 11)
    r = replay(cfg, w, dtype, max_tokens=304)
    for seed in (21, 22):
        toks = tokens(cfg, 300, seed)
        assert error(score(r, toks, [40] + [1] * 260), reference(name, cfg, w, toks, dtype)) <= LIMIT[dtype]
    r.engine.close()


def test_a_full_pool_is_reported():
    cfg = CASES["looped"]()
    r = replay(cfg, weights(cfg, 1), "bfloat16", max_tokens=64)
    r.step([{"id": "a", "tokens": tokens(cfg, 60, 1), "want": []}], [])
    with pytest.raises(RuntimeError, match="scheduled"):
        r.step([{"id": "b", "tokens": tokens(cfg, 20, 1), "want": []}], [])
    r.engine.close()


def test_layer_by_layer(served):
    """The residual stream behind every layer run (a looped layer counts once per pass)."""
    name, dtype, cfg, w, r = served
    native = r.engine.worker.model_runner.model.model
    toks = tokens(cfg, 45, 8)
    res, _ = V.residuals_and_logits(cfg, w, toks, torch.float64 if dtype == "float32" else torch.float32,
                                    None if dtype == "float32" else "bf16")
    native.keep_layer_residuals(True)
    score(r, toks, [45])
    got = native.layer_residuals(45)
    native.keep_layer_residuals(False)
    assert got.shape == res.shape == (len(V.layer_runs(cfg)), 45, cfg["width"])
    for i in range(got.shape[0]):
        scale = res[i].std()
        assert ((got[i].double() - res[i].double()).pow(2).mean().sqrt() / scale) <= LIMIT[dtype], i


# ---- generation through the engine ------------------------------------------------------------------------
def greedy(cfg, w, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(V.logits(cfg, w, seq, torch.float64)[-1].argmax()))
    return seq[len(prompt):]


@pytest.mark.parametrize("chunked", [False, True])
@pytest.mark.parametrize("device_sampling", [False, True])
def test_greedy_generation(chunked, device_sampling):
    """MI355XEngine.generate, both schedulers: fp32 text equals the oracle's.  The prompts share a prefix, so the
    prefix-caching scheduler serves the second one from cached pages."""
    from vllm_neuron_amd._vllm_compat import SamplingParams
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg = CASES["uneven"]()
    w = weights(cfg, 11)
    base = tokens(cfg, 70, 5)
    prompts = [base, base[:64] + tokens(cfg, 11, 6), tokens(cfg, 1, 7), tokens(cfg, 21, 8), tokens(cfg, 33, 9)]
    override = {"state_dict": w}
    if chunked:
        override.update(is_block_kv_layout=True, chunked_prefill_config={"max_num_seqs": 3})
    if device_sampling:
        override["on_device_sampling_config"] = {"dynamic": True}
    eng = MI355XEngine(config_from_dict(cfg), dtype="float32", max_model_len=256, max_num_seqs=3, block_size=16,
                       enable_prefix_caching=not chunked, enable_chunked_prefill=chunked,
                       max_num_batched_tokens=48 if chunked else None, override_mi355x_config=override)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10))
    assert [o.token_ids for o in outs] == [greedy(cfg, w, p, 10) for p in prompts]
    assert (max(o.num_cached_tokens for o in outs) >= 64) == (not chunked)
    eng.close()


def test_batch_line_kv_layout():
    """Without prefix caching the custom scheduler keeps one block per sequence ("batch line")."""
    from vllm_neuron_amd._vllm_compat import SamplingParams
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg = CASES["looped"]()
    w = weights(cfg, 2)
    eng = MI355XEngine(config_from_dict(cfg), dtype="float32", max_model_len=128, max_num_seqs=2, enable_prefix_caching=False,
                       override_mi355x_config={"state_dict": w})
    prompts = [tokens(cfg, n, n) for n in (30, 7, 19)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=8))
    assert [o.token_ids for o in outs] == [greedy(cfg, w, p, 8) for p in prompts]
    eng.close()


def test_speculation_yields_the_greedy_text():
    from types import SimpleNamespace

    from vllm_neuron_amd._vllm_compat import SamplingParams, SimpleSpeculativeConfig
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg, small = CASES["uneven"](), config(64, 203, [att(2, 1, 32, 32, 24, 64)])
    w = weights(cfg, 11)
    spec = SimpleSpeculativeConfig(num_speculative_tokens=3, draft_model_config=SimpleNamespace(
        model="", hf_config=config_from_dict(small)))
    eng = MI355XEngine(config_from_dict(cfg), dtype="float32", max_model_len=128, max_num_seqs=2, block_size=16,
                       speculative_config=spec, override_mi355x_config={"state_dict": w, "draft_state_dict": weights(small, 4)})
    prompts = [tokens(cfg, n, 60 + n) for n in (30, 12)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10))
    assert [o.token_ids for o in outs] == [greedy(cfg, w, p, 10) for p in prompts]
    eng.close()


# ---- loading and the command line ----------------------------------------------------------------------------
def write_model(path, cfg, w):
    from safetensors.torch import save_file
    path.mkdir(exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(path / "model.safetensors"))


@pytest.mark.parametrize("dtype", list(LIMIT))
def test_trace_run_command(tmp_path, monkeypatch, capsys, dtype):
    import io

    import numpy as np

    from vllm_neuron_amd import replay as cmd
    cfg = CASES["wide"]()
    w = weights(cfg, 5)
    write_model(tmp_path / "m", cfg, w)
    a, b = tokens(cfg, 50, 1), tokens(cfg, 20, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [29, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:19], "want": []}], "end": []},
             {"step": 7, "entries": [{"id": "b", "tokens": b[19:], "want": [0]}, {"id": "a", "tokens": a[30:], "want": [0, 19]}],
              "end": ["a", "b"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps)) + "\n"))
    assert cmd.main(["--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "128"]) == 0
    assert [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 7"]
    assert not (tmp_path / "1.f32").exists() and sorted(p.name for p in (tmp_path / "m").iterdir()) == ["config.json", "model.safetensors"]
    ra, rb = reference("wide5", cfg, w, a, dtype), reference("wide5", cfg, w, b, dtype)

    def read(n):
        return torch.from_numpy(np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, cfg["vocab"]))
    assert error(read(0), ra[[29, 3]]) <= LIMIT[dtype]
    assert error(read(7), torch.stack([rb[19], ra[30], ra[49]])) <= LIMIT[dtype]


@pytest.mark.parametrize("chunk", [0, 24])
def test_generate_command(tmp_path, capsys, chunk):
    from vllm_neuron_amd.generate import main
    cfg = CASES["looped"]()
    w = weights(cfg, 5)
    write_model(tmp_path / "m", cfg, w)
    prompts = [tokens(cfg, 40, 1), tokens(cfg, 3, 2)]
    argv = ["--model", str(tmp_path / "m"), "--dtype", "float32", "--max-tokens", "6", "--block-size", "16", "--chunked-prefill", str(chunk)]
    for p in prompts:
        argv += ["--prompt", ",".join(map(str, p))]
    assert main(argv) == 0
    lines = [json.loads(x) for x in capsys.readouterr().out.splitlines() if x.startswith("{")]
    assert [x["tokens"] for x in lines] == [greedy(cfg, w, p, 6) for p in prompts]


def test_weight_artifacts_round_trip(tmp_path):
    """A served checkpoint folder keeps its device images; the second start loads them and answers the same."""
    from vllm_neuron_amd._vllm_compat import SamplingParams
    from vllm_neuron_amd.engine import MI355XEngine
    cfg = CASES["uneven"]()
    write_model(tmp_path / "m", cfg, weights(cfg, 6))
    texts = []
    for start in range(2):
        eng = MI355XEngine(None, str(tmp_path / "m"), max_model_len=128, max_num_seqs=2, block_size=16)
        assert eng.worker.model_runner.model.loaded_from_artifacts == (start == 1)
        texts.append(eng.generate([tokens(cfg, 20, 1)], SamplingParams(temperature=0.0, max_tokens=12))[0].token_ids)
        eng.close()
    assert texts[0] == texts[1] and len(texts[0]) == 12


def test_loading_refuses_what_does_not_fit():
    cfg = CASES["looped"]()
    w = weights(cfg, 1)
    short = {k: v for k, v in w.items() if k != "l0.norm2.b"}
    with pytest.raises(RuntimeError, match="l0.norm2.b"):
        r = replay(cfg, short, "bfloat16")
        r.engine.worker.model_runner.initialize_kv_cache(None)
    with pytest.raises(ValueError, match="shape"):
        replay(cfg, {**w, "l0.mix.o": w["l0.mix.o"][:, :8].contiguous()}, "bfloat16")
    with pytest.raises(ValueError, match="not part"):
        replay(cfg, {**w, "l7.mix.o": w["l0.mix.o"]}, "bfloat16")
    with pytest.raises(NotImplementedError):
        replay(cfg, w, "bfloat16", quantized=True)
    with pytest.raises(ValueError, match="float16"):
        replay(cfg, w, "float16")
