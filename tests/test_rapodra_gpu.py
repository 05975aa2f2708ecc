"""Rapodra on the MI355X: every kernel of the sandwich block against the oracle's mechanism of the same name, and the model
through the framework's engine against the oracle's whole-sequence logits -- prompts whole, in portions and token by token,
in mixed batches, over a KV pool small enough that pages (and the convolution state in them) are used again."""

import json
import math

import pytest
import torch

from oracle import rapodra as R
from tests.rapodra_cases import CASES, config, dense, error, latent, moe, tokens, weights

pytestmark = pytest.mark.gpu

# fp32: rounding only.  bf16: against the oracle with the rounding points of the device path (latent-space scores, summation
# order and the flips they cause are what is left).
LIMIT = {"float32": 3e-5, "bfloat16": 4e-2}


@pytest.fixture(scope="module")
def lib():
    from vllm_neuron_amd import _native
    return _native


def dev(t):
    return t.to("cuda").contiguous()


def pad(n, m):
    return (n + m - 1) // m * m


def ptr(t):
    return None if t is None else t.data_ptr()


# ---- rows: post-norm, residual sum, pre-norm, convolution ---------------------------------------------------------------
def sandwich(lib, x, T, D, groups, eps, f32, y=None, pair_w=None, w_post=None, w_pre=None, conv=None):
    """-> (residual [T, D], output [T, D]); conv: dict(w [D, taps], ring, keep, bs, bt, pos, slots, segs)"""
    ld, ldy = pad(D, 16), pad(D, 64)
    dt = torch.float32 if f32 else torch.bfloat16

    def wide(t, rows):
        out = torch.zeros(rows, ld)
        out[:, :D] = t
        return dev(out)
    keep = [wide(x, T), torch.full((T, ld), 7.0, device="cuda"), None if y is None else wide(y, y.shape[0]),
            None if pair_w is None else dev(pair_w.float()), None if w_post is None else wide(w_post, 1), None if w_pre is None else wide(w_pre, 1)]
    out = torch.zeros(T, ldy, dtype=dt, device="cuda")
    c = [None] * 5
    taps = kept = bs = MB = nseg = 0
    segs = None
    if conv is not None:
        taps = conv["w"].shape[1]
        cw = torch.zeros(taps, ld)
        cw[:, :D] = conv["w"].t()
        c = [dev(cw), conv["ring"], dev(conv["bt"]), dev(conv["pos"]), dev(conv["slots"])]
        kept, bs, MB = conv["keep"], conv["bs"], conv["bt"].shape[1]
        if conv.get("segs") is not None:
            segs = torch.tensor(conv["segs"], dtype=torch.int32).contiguous()
            nseg = segs.shape[0]
    lib.check(lib.load_library().mi_op_sandwich_rows(
        ptr(keep[0]), ptr(keep[1]), ptr(keep[2]), ptr(keep[3]), 0 if pair_w is None else pair_w.shape[1], ptr(keep[4]), ptr(keep[5]), T, D, ld,
        groups, eps, ptr(c[0]), taps, ptr(c[1]), kept, bs, ptr(c[2]), MB, ptr(c[3]), ptr(c[4]), ptr(segs), nseg, ptr(out), ldy, f32, None))
    torch.cuda.synchronize()
    assert (out[:, D:] == 0).all()
    return keep[1].cpu()[:, :D], out.cpu().float()[:, :D]


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("T,D,groups", [(1, 64, 1), (3, 120, 3), (40, 120, 120), (5, 2050, 25), (33, 4096, 8), (2, 8192, 2)])
def test_norms_around_the_residual_sum(lib, T, D, groups, f32):
    torch.manual_seed(D)
    x, y = torch.randn(T, D) * 3 + 1, torch.randn(T, D) * torch.linspace(0.01, 20, T)[:, None]
    wp, wn = torch.randn(D), torch.randn(D)
    got_x, got = sandwich(lib, x, T, D, groups, 1e-2, f32, y=y, w_post=wp, w_pre=wn)
    ref_x = x.double() + R.group_rms(y.double(), wp.double(), groups, 1e-2)
    assert ((got_x - ref_x).abs() <= 2e-5 * (1 + ref_x.abs())).all()
    ref = R.group_rms(ref_x, wn.double(), groups, 1e-2)
    assert ((got - ref).abs() <= (2e-5 if f32 else 1e-2) * (1 + ref.abs())).all()
    none_x, only = sandwich(lib, x, T, D, groups, 1e-2, f32, w_pre=wn)           # nothing to add: the residual is left alone
    assert (none_x == 7.0).all()
    ref = R.group_rms(x.double(), wn.double(), groups, 1e-2)
    assert ((only - ref).abs() <= (2e-5 if f32 else 1e-2) * (1 + ref.abs())).all()


def test_experts_are_summed_with_their_weights(lib):
    torch.manual_seed(3)
    T, D, top = 9, 100, 5
    x, y, p = torch.randn(T, D), torch.randn(T * top, D), torch.softmax(torch.randn(T, top), -1)
    got, _ = sandwich(lib, x, T, D, 4, 1e-3, 1, y=y, pair_w=p, w_post=torch.ones(D))
    ref = x.double() + R.group_rms((p[:, :, None] * y.view(T, top, D)).sum(1).double(), 1.0, 4, 1e-3)
    assert ((got - ref).abs() <= 2e-5 * (1 + ref.abs())).all()


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("D,taps,bs", [(100, 4, 16), (64, 2, 32), (1030, 16, 16), (72, 1, 16), (64, 9, 16)])
def test_convolution_over_portions_pages_and_sequences(lib, D, taps, bs, f32):
    """Sequences cut at every kind of place (inside a page, at its edge, single tokens, portions of two), several in a batch,
    their pages shuffled; every output equals the whole sequence's."""
    g = torch.Generator().manual_seed(D + taps)
    n_seq, L = 3, 75
    w_pre = torch.ones(D)
    cw = torch.randn(D, taps, generator=g) / taps
    xs = [torch.randn(L, D, generator=g) for _ in range(n_seq)]
    rnd = (lambda t: t) if f32 else (lambda t: t.to(torch.bfloat16).float())
    hs = [rnd(R.group_rms(x, w_pre, 2, 1e-5)) for x in xs]
    refs = [h.double() + R.causal_conv(h.double(), cw.double()) for h in hs]
    keep = min(bs, taps - 1)
    MB = -(-L // bs)
    perm = (torch.randperm(n_seq * MB, generator=g) + 1).to(torch.int32)
    tables = perm.view(n_seq, MB)
    # rows nobody wrote hold something large: reading one shows
    ring = torch.full((n_seq * MB + 1, max(keep, 1), pad(D, 64)), 1e4, dtype=torch.float32 if f32 else torch.bfloat16, device="cuda")
    at = [0] * n_seq
    plan = [[5, 1, 2], [1, 1, 1], [10, 16, 33], [2, 2, 2], [1, 0, 1], [17, 15, 1], [1, 1, 1], [3, 1, 1], [16, 20, 0], [1, 1, 1], [18, 17, 32], [0, 1, 0]]
    for step in plan:
        live = [(i, min(n, L - at[i])) for i, n in enumerate(step) if min(n, L - at[i]) > 0]
        if not live:
            continue
        T = sum(n for _, n in live)
        pos = torch.cat([torch.arange(at[i], at[i] + n) for i, n in live]).to(torch.int32)
        bt = torch.stack([tables[i] for i, _ in live])
        slots = torch.cat([tables[i][torch.arange(at[i], at[i] + n) // bs] * bs + torch.arange(at[i], at[i] + n) % bs for i, n in live]).to(torch.int32)
        segs, row = [], 0
        for j, (i, n) in enumerate(live):
            segs.append((row, n, at[i], j))
            row += n
        single = all(n == 1 for _, n in live)
        x = torch.cat([xs[i][at[i]:at[i] + n] for i, n in live])
        _, got = sandwich(lib, x, T, D, 2, 1e-5, f32, w_pre=w_pre, conv=dict(w=cw, ring=ring, keep=keep, bs=bs, bt=bt, pos=pos, slots=slots,
                                                                            segs=None if single else segs))
        ref = torch.cat([refs[i][at[i]:at[i] + n] for i, n in live])
        assert ((got - ref).abs() <= (2e-5 if f32 else 2e-2) * (1 + ref.abs())).all(), (step, at, (got - ref).abs().max())
        for i, n in live:
            at[i] += n
    assert at == [74, 75, 74] or min(at) > 60


# ---- latent attention --------------------------------------------------------------------------------------------------
def spec_of(lib, H, dk, dv, rank, window, scale):
    return lib.layer_spec(dict(mixer_kind=1, num_heads=H, num_kv_heads=1, qk_dim=dk, v_dim=dv, kv_rank=rank, kv_from=-1, window=window,
                               scale=scale))


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("H,dk,rank", [(3, 20, 36), (18, 64, 160), (2, 33, 520)])
def test_latent_norm_and_scatter(lib, H, dk, rank, f32):
    torch.manual_seed(rank)
    T, bs, nb = 9, 16, 5
    ldq = pad(H * dk + rank, 16)
    qd, cn = torch.randn(T, ldq) * 3, torch.randn(rank)
    slots = torch.tensor([17, 40, -1, 79, 16, 63, 64, 1, 30], dtype=torch.int32)
    dt = torch.float32 if f32 else torch.bfloat16
    q = torch.full((T, H, pad(dk, 32)), 7.0, dtype=dt, device="cuda")
    pool = torch.full((nb * bs, pad(rank, 32)), 7.0, dtype=dt, device="cuda")
    a = [dev(t) for t in (qd, cn, slots)]
    lib.check(lib.load_library().mi_op_latent_scatter(ptr(a[0]), ldq, T, spec_of(lib, H, dk, 8, rank, 4, 1.0), None, None, ptr(a[1]), 1e-3, ptr(a[2]), bs,
                                                      ptr(q), ptr(pool), f32, None))
    torch.cuda.synchronize()
    tol = 1e-5 if f32 else 1.2e-2
    q, pool = q.cpu().double(), pool.cpu().double()
    ref_q = qd[:, :H * dk].reshape(T, H, dk).double()
    assert (q[..., dk:] == 0).all() and ((q[..., :dk] - ref_q).abs() <= tol * (1 + ref_q.abs())).all()
    ref = R.group_rms(qd[:, H * dk:H * dk + rank].double(), cn.double(), 1, 1e-3)
    free = torch.ones(nb * bs, dtype=torch.bool)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            assert (pool[s, rank:] == 0).all() and ((pool[s, :rank] - ref[t]).abs() <= tol * (1 + ref[t].abs())).all()
            free[s] = False
    assert (pool[free] == 7.0).all()


class Paged:
    """One random sequence per request, its latents scattered over shuffled pool blocks, and a ragged set of queries."""

    def __init__(self, H, dk, dv, rank, segs, bs, seed):
        g = torch.Generator().manual_seed(seed)
        self.H, self.dk, self.dv, self.rank, self.bs = H, dk, dv, rank, bs
        self.segs, row = [], 0
        for i, (pos0, n) in enumerate(segs):
            self.segs.append((row, n, pos0, i))
            row += n
        self.T, self.max_ctx = row, max(p + n for p, n in segs)
        self.MB = -(-self.max_ctx // bs) + 1
        self.nb = 1 + sum(-(-(p + n) // bs) for p, n in segs) + 3
        perm = (torch.randperm(self.nb - 1, generator=g) + 1).tolist()
        self.bt = torch.zeros(len(segs), self.MB, dtype=torch.int32)
        self.uk = (torch.randn(H * dk, rank, generator=g) / math.sqrt(rank)).to(torch.bfloat16).float()
        self.uv = (torch.randn(H * dv, rank, generator=g) / math.sqrt(rank)).to(torch.bfloat16).float()
        self.q = [torch.randn(p + n, H, dk, generator=g) for p, n in segs]
        self.c = [torch.randn(p + n, rank, generator=g) for p, n in segs]
        for i, (p, n) in enumerate(segs):
            for b in range(-(-(p + n) // bs)):
                self.bt[i, b] = perm.pop()

    def run(self, lib, window, scale, f32, path):
        dt = torch.float32 if f32 else torch.bfloat16
        r = (lambda t: t) if f32 else (lambda t: t.to(torch.bfloat16).float())
        rp, dkp = pad(self.rank, 32), pad(self.dk, 32)
        pool = torch.full((self.nb, self.bs, rp), 30.0)              # rows nobody wrote: large but finite
        pool[..., self.rank:] = 0
        q = torch.zeros(self.T, self.H, dkp)
        pos = torch.zeros(self.T, dtype=torch.int32)
        ref = torch.zeros(self.T, self.H * self.dv, dtype=torch.float64)
        for row, n, p, i in self.segs:
            q[row:row + n, :, :self.dk] = self.q[i][p:]
            pos[row:row + n] = torch.arange(p, p + n)
            at = torch.arange(p + n)
            pool[self.bt[i, at // self.bs].long(), at % self.bs, :self.rank] = self.c[i]
            o = R.latent_attention(r(self.q[i]).double(), r(self.c[i]).double(), self.uk.double(), self.uv.double(), scale,
                                   window if window else 1 << 30)
            ref[row:row + n] = o[p:].reshape(n, -1)
        ldo = pad(self.H * self.dv, 64)
        out = torch.zeros(self.T, ldo, dtype=dt, device="cuda")
        a = [dev(x) for x in (self.uk, self.uv, q.to(dt), pool.to(dt), self.bt, pos)]
        segs = torch.tensor(self.segs, dtype=torch.int32).contiguous()
        spec = spec_of(lib, self.H, self.dk, self.dv, self.rank, window, scale)
        lib.check(lib.load_library().mi_op_latent_attn(spec, ptr(a[0]), ptr(a[1]), ptr(a[2]), ptr(a[3]), self.bs, ptr(a[4]), self.MB,
                                                       ptr(a[5]), ptr(segs), len(self.segs), self.T, self.max_ctx, ptr(out), ldo, f32, path, None))
        torch.cuda.synchronize()
        got = out.cpu().double()
        assert (got[:, self.H * self.dv:] == 0).all()
        got = got[:, :self.H * self.dv]
        if path == 3:                        # written-out keys: segments of two rows and more
            rows = torch.cat([torch.arange(row, row + n) for row, n, _, _ in self.segs if n > 1])
            got, ref = got[rows], ref[rows]
        return got, ref


PATHS = [(1, 1), (0, 1), (0, 2), (0, 3)]      # (fp32?, path): plain fp32, plain bf16, rows in the latent space, written-out keys
SEGS = [(0, 70), (45, 1), (31, 2), (0, 1), (100, 130), (299, 1), (0, 3), (64, 65), (190, 17)]


def close(got, ref, f32, tol=2e-2):
    assert ((got - ref).abs() <= (3e-5 if f32 else tol) * (1 + ref.abs())).all(), (got - ref).abs().max()


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("H,dk,dv,rank,window,bs", [
    (4, 64, 40, 96, 96, 16), (3, 20, 13, 36, 37, 32), (18, 32, 32, 160, 0, 48), (34, 16, 24, 64, 5, 16), (2, 160, 200, 288, 129, 32),
    (70, 8, 8, 32, 1, 16), (5, 128, 128, 512, 64, 16)])
def test_latent_attention(lib, H, dk, dv, rank, window, bs, f32, path):
    got, ref = Paged(H, dk, dv, rank, SEGS, bs, seed=H + window).run(lib, window, 1.5 / math.sqrt(dk), f32, path)
    close(got, ref, f32)


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("n_seq", [40, 300])
def test_many_decoding_rows(lib, n_seq, f32, path):
    """Rows of many sequences: one context split per row, head groups that share a tile."""
    if path == 3:
        pytest.skip("single tokens")
    g = torch.Generator().manual_seed(1)
    segs = [(int(torch.randint(0, 150, (1,), generator=g)), 1) for _ in range(n_seq)]
    got, ref = Paged(40, 16, 16, 64, segs, 16, seed=2).run(lib, 70, 0.4, f32, path)
    close(got, ref, f32)


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("window,bs", [(96, 16), (33, 32), (64, 16), (128, 32), (16, 16), (1, 16), (200, 48)])
def test_window_edge_key_stands_out(lib, window, bs, f32, path):
    """One key per row with a score far above the rest, placed at every distance around the edge: just inside it takes the row,
    one further out it must have no influence at all -- in prompts, at page borders and in decoding."""
    H, dk, dv, rank = 4, 32, 48, 64
    segs = [(260, 1), (259, 2), (191, 80), (0, 240), (256, 1), (255, 3)]
    for off in (-1, 0, 1, -bs):                            # distance window - 1 (inside), window, ... of the segment's last row
        p = Paged(H, dk, dv, rank, segs, bs, seed=window + 7)
        hit = []
        for i, (pos0, n) in enumerate(segs):
            last = pos0 + n - 1
            j = last - (window - 1) - off
            if 0 <= j <= last:
                k = (p.uk @ p.c[i][j].to(torch.bfloat16).float()).view(H, dk)
                p.q[i][last] = 18.0 * math.sqrt(dk) * k / k.pow(2).sum(-1, keepdim=True)
                hit.append((i, last, j))
        got, ref = p.run(lib, window, 1 / math.sqrt(dk), f32, path)
        close(got, ref, f32, 3e-2)
        for i, last, j in hit:                             # (the case does what it says)
            row = p.segs[i][0] + p.segs[i][1] - 1
            if path == 3:
                continue
            v = (p.uv @ p.c[i][j]).double()
            assert (torch.cosine_similarity(ref[row], v, 0) > 0.8) == (last - j < window)


@pytest.mark.parametrize("f32,path", PATHS)
def test_far_key_of_a_long_context(lib, f32, path):
    """A key more than two thousand tokens back that holds a decoded token's attention (context split over work-groups)."""
    H, dk, dv, rank = 4, 32, 32, 128
    key = 32 * 3 + 31
    segs = [(2300, 1), (2250, 40)]
    p = Paged(H, dk, dv, rank, segs, 32, seed=9)
    for i, n in enumerate((2301, 2290)):
        k = (p.uk @ p.c[i][key].to(torch.bfloat16).float()).view(H, dk)
        p.q[i][n - 1] = 25.0 * math.sqrt(dk) * k / k.pow(2).sum(-1, keepdim=True)
    for window in (0, 2400, 2301 - key, 2300 - key, 2290 - key, 2289 - key):
        got, ref = p.run(lib, window, 1 / math.sqrt(dk), f32, path)
        close(got, ref, f32, 3e-2)
        v = (p.uv @ p.c[1][key]).double()
        assert (torch.cosine_similarity(ref[-1], v, 0) > 0.8) == (window != 2289 - key)


# ---- router and experts ----------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("f32,path", [(1, 1), (0, 1), (0, 2)])
@pytest.mark.parametrize("T,D,E,top,ff", [(1, 64, 4, 1, 16), (5, 120, 7, 3, 22), (32, 320, 64, 8, 40), (3, 1024, 300, 5, 64), (150, 192, 6, 6, 72),
                                          (700, 128, 12, 2, 130)])
def test_router_and_experts(lib, T, D, E, top, ff, f32, path):
    g = torch.Generator().manual_seed(T + E)
    b16 = lambda t: t.to(torch.bfloat16).float()
    w, b = b16(torch.randn(E, D, generator=g) / math.sqrt(D)), torch.randn(E, generator=g)
    gate, up = (b16(torch.randn(E, ff, D, generator=g) / math.sqrt(D)) for _ in range(2))
    down = b16(torch.randn(E, D, ff, generator=g) / math.sqrt(ff))
    x = b16(torch.randn(T, D, generator=g))
    z = x.double() @ w.double().t() + b.double()
    if top < E:                               # no close calls
        for _ in range(50):
            v = z.topk(top + 1, -1).values
            bad = (v[:, -2] - v[:, -1]) < 1e-3
            if not bad.any():
                break
            x[bad] = b16(torch.randn(int(bad.sum()), D, generator=g))
            z = x.double() @ w.double().t() + b.double()
    Kd, ldy = pad(D, 64), pad(D, 16)
    xd = torch.zeros(T, Kd)
    xd[:, :D] = x
    a = [dev(t) for t in (xd.to(torch.float32 if f32 else torch.bfloat16), w, b, gate, up, down)]
    ids = torch.full((T, top), -1, dtype=torch.int32, device="cuda")
    p = torch.zeros(T, top, device="cuda")
    y = torch.zeros(T * top, ldy, device="cuda")
    for _ in range(2):                        # (the second call finds what the first left behind, as a layer's next step does)
        lib.check(lib.load_library().mi_op_experts(ptr(a[0]), Kd, T, D, E, top, ff, ptr(a[1]), ptr(a[2]), ptr(a[3]), ptr(a[4]), ptr(a[5]),
                                                   ptr(ids), ptr(p), ptr(y), ldy, 0, 0, f32, path, None))
    torch.cuda.synchronize()
    ref_ids, ref_p = R.route(x.double(), w.double(), b.double(), top)
    assert torch.equal(ids.cpu().long(), ref_ids)
    assert (p.cpu() - ref_p).abs().max() < (1e-6 if f32 else 1e-5)
    y = y.cpu().double().view(T, top, ldy)[:, :, :D]
    r = (lambda t: t) if f32 else (lambda t: b16(t.float()).double())
    for e in range(E):
        rows, place = (ref_ids == e).nonzero(as_tuple=True)
        if rows.numel():
            ref = R.silu_glu(x[rows].double(), gate[e].double(), up[e].double(), down[e].double(), r)
            assert ((y[rows, place] - ref).abs() <= (2e-5 if f32 else 1.5e-2) * (1 + ref.abs())).all()


def test_router_prefers_the_lower_of_equal_experts(lib):
    T, D, E = 3, 64, 70
    a = [dev(t) for t in (torch.ones(T, D).to(torch.bfloat16), torch.zeros(E, D), torch.zeros(E), torch.zeros(E, 16, D), torch.zeros(E, 16, D),
                          torch.zeros(E, D, 16))]
    for path in (1, 2):
        ids, p = torch.full((T, 4), -1, dtype=torch.int32, device="cuda"), torch.zeros(T, 4, device="cuda")
        y = torch.zeros(T * 4, D, device="cuda")
        lib.check(lib.load_library().mi_op_experts(ptr(a[0]), 64, T, D, E, 4, 16, ptr(a[1]), ptr(a[2]), ptr(a[3]), ptr(a[4]), ptr(a[5]), ptr(ids),
                                                   ptr(p), ptr(y), D, 0, 0, 0, path, None))
        torch.cuda.synchronize()
        assert ids.cpu().tolist() == [[0, 1, 2, 3]] * T and torch.allclose(p.cpu(), torch.full((T, 4), 0.25))


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
        _refs[key] = R.logits(cfg, w, toks, torch.float64 if dtype == "float32" else torch.float32,
                              None if dtype == "float32" else "bf16")
    return _refs[key]


_cases = {}


def case(name):
    if name not in _cases:
        cfg = CASES[name]()
        _cases[name] = (cfg, weights(cfg, 11))
    return _cases[name]


@pytest.fixture(scope="module", params=[(n, d) for n in CASES for d in LIMIT], ids=lambda p: f"{p[0]}-{p[1]}")
def served(request):
    name, dtype = request.param
    cfg, w = case(name)
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
    for n in cuts:
        part = toks[at:at + n]
        at += n
        out.append(r.step([{"id": rid, "tokens": part, "want": list(range(len(part)))}], [rid] if at >= len(toks) else [])[0])
    assert at >= len(toks)
    return torch.cat(out)


def test_whole_prompts(served):
    name, dtype, cfg, w, r = served
    for n in (1, 2, 15, 16, 17, 130, 300):
        toks = tokens(cfg, w, n, n)
        assert error(score(r, toks, [n]), reference(name, cfg, w, toks, dtype)) <= LIMIT[dtype], n


def test_token_by_token_equals_the_prompt(served):
    name, dtype, cfg, w, r = served
    toks = tokens(cfg, w, 130, 130)
    ref = reference(name, cfg, w, toks, dtype)
    assert error(score(r, toks, [1] * 130), ref) <= LIMIT[dtype]
    assert error(score(r, toks, [70] + [1] * 60), ref) <= LIMIT[dtype]


@pytest.mark.parametrize("cuts", [[2] * 65, [3] * 44, [5] * 26, [16] * 9, [17] * 8, [33] * 4, [64, 66], [65, 65], [100, 2, 28], [30, 100],
                                  [2, 1, 5, 1, 40, 2, 2, 1, 64, 12]])
def test_portions(served, cuts):
    name, dtype, cfg, w, r = served
    toks = tokens(cfg, w, 130, 130)
    assert error(score(r, toks, cuts), reference(name, cfg, w, toks, dtype)) <= LIMIT[dtype]


def test_mixed_batches_over_reused_pages(served):
    """Up to four live requests, portions beside single tokens, requests left out of steps and ended; the pool holds far
    fewer tokens than the requests together."""
    name, dtype, cfg, w, r = served
    g = torch.Generator().manual_seed(3)

    def rnd(a, b):
        return int(torch.randint(a, b, (1,), generator=g))
    pool = 768 // 16
    todo = [tokens(cfg, w, n, 1000 + i) for i, n in enumerate([150, 9, 90, 1, 160, 47, 130, 33, 130, 16, 2, 121])]
    total = sum(map(len, todo))
    assert total > 768 and r.engine.scheduler.block_pool.num_free() == pool
    live, worst, seen, steps, used = {}, 0.0, 0, 0, 0
    while todo or live:
        while todo and len(live) < 4:
            live[uid()] = [todo.pop(0), 0]
        entries, end = [], []
        for rid, st in live.items():
            if len(live) > 1 and rnd(0, 5) == 0:
                continue                                    # left out of this step
            n = min(1 if rnd(0, 2) else rnd(1, 80), len(st[0]) - st[1])
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
    assert used == total and steps > 15 and seen > 60
    r.engine.scheduler.schedule()
    assert r.engine.scheduler.block_pool.num_free() == pool         # everything came back


def test_batch_does_not_change_a_request(served):
    name, dtype, cfg, w, r = served
    toks, other = tokens(cfg, w, 90, 90), [tokens(cfg, w, n, 400 + n) for n in (33, 2, 71)]
    alone = score(r, toks, [90])
    rid, ids = uid(), [uid() for _ in other]
    outs = r.step([{"id": ids[0], "tokens": other[0], "want": []}, {"id": rid, "tokens": toks[:50], "want": list(range(50))},
                   {"id": ids[1], "tokens": other[1], "want": []}, {"id": ids[2], "tokens": other[2], "want": [3]}], [])
    outs2 = r.step([{"id": ids[1], "tokens": [1], "want": [0]}, {"id": rid, "tokens": toks[50:], "want": list(range(40))}],
                   [rid] + ids)
    assert error(torch.cat([outs[1], outs2[1]]), alone) <= LIMIT[dtype]


@pytest.mark.parametrize("dtype", list(LIMIT))
def test_long_decoding_and_pages_of_ended_requests(dtype):
    """A pool of exactly one long request: every sequence runs over the pages of the one before, decoding far past the
    windows, across page borders, with graph replays."""
    cfg, w = case("uneven")
    r = replay(cfg, w, dtype, max_tokens=304)
    for seed in (21, 22):
        toks = tokens(cfg, w, 300, seed)
        assert error(score(r, toks, [40] + [1] * 260), reference("uneven", cfg, w, toks, dtype)) <= LIMIT[dtype]
    r.engine.close()


def test_layer_by_layer(served):
    name, dtype, cfg, w, r = served
    native = r.engine.worker.model_runner.model.model
    toks = tokens(cfg, w, 45, 8)
    res, _ = R.residuals_and_logits(cfg, w, toks, torch.float64 if dtype == "float32" else torch.float32,
                                    None if dtype == "float32" else "bf16")
    score(r, toks[:1], [1])
    native.keep_layer_residuals(True)
    score(r, toks, [45])
    got = native.layer_residuals(45)
    native.keep_layer_residuals(False)
    assert got.shape == res.shape == (len(cfg["layers"]), 45, cfg["width"])
    for i in range(got.shape[0]):
        assert ((got[i].double() - res[i].double()).pow(2).mean().sqrt() / res[i].std()) <= LIMIT[dtype], i


def test_a_wide_row_and_a_large_batch():
    """Hidden rows beyond one work-group's first pass, 40 requests decoding at once (the grouped experts and the GEMMs)."""
    cfg = config(2112, 160, [latent(3, 32, 32, 64, 24, moe(6, 2, 48)), latent(3, 32, 32, 64, 48, dense(192), kv_from=0)], groups=2, taps=4)
    w = weights(cfg, 9)
    r = replay(cfg, w, "bfloat16", max_tokens=40 * 48, max_live=40)
    seqs = [tokens(cfg, w, n, 7000 + n % 3) for n in (30, 31, 32)]
    ids = [uid() for _ in range(40)]
    worst = 0.0
    r.step([{"id": rid, "tokens": seqs[i % 3][:20], "want": []} for i, rid in enumerate(ids)], [])
    for p in range(20, 28):
        outs = r.step([{"id": rid, "tokens": [seqs[i % 3][p]], "want": [0]} for i, rid in enumerate(ids)], ids if p == 27 else [])
        for i, o in enumerate(outs):
            worst = max(worst, error(o, reference(f"wide{i % 3}", cfg, w, seqs[i % 3], "bfloat16")[p:p + 1]))
    assert worst <= LIMIT["bfloat16"], worst
    r.engine.close()


# ---- generation through the engine ------------------------------------------------------------------------
def greedy(cfg, w, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(R.logits(cfg, w, seq, torch.float64)[-1].argmax()))
    return seq[len(prompt):]


@pytest.mark.parametrize("chunked", [False, True])
@pytest.mark.parametrize("device_sampling", [False, True])
def test_greedy_generation(chunked, device_sampling):
    """MI355XEngine.generate, both schedulers: fp32 text equals the oracle's.  The prompts share a prefix, so the
    prefix-caching scheduler serves the second one from cached pages -- latents and convolution state."""
    from vllm_neuron_amd._vllm_compat import SamplingParams
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg, w = case("uneven")

    def rnd(n, seed):
        return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
    base = rnd(70, 5)
    prompts = [base, base[:64] + rnd(11, 6), rnd(1, 7), rnd(21, 8), rnd(33, 9)]
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
    cfg, w = case("taps")
    eng = MI355XEngine(config_from_dict(cfg), dtype="float32", max_model_len=128, max_num_seqs=2, enable_prefix_caching=False,
                       override_mi355x_config={"state_dict": w})
    prompts = [torch.randint(0, 256, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in (30, 7, 19)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=8))
    assert [o.token_ids for o in outs] == [greedy(cfg, w, p, 8) for p in prompts]
    eng.close()


@pytest.mark.parametrize("k,max_len", [(3, 128), (5, 48)])
def test_speculation_yields_the_greedy_text(k, max_len):
    """Candidates of a step are segments of k tokens: rejected ones leave latents and convolution inputs behind that the next
    step must not see.  The draft is the target without the convolutions' past, right about half of the time.  max_len 48:
    sequences end at the model length, inside a speculation window."""
    import copy
    from types import SimpleNamespace

    from vllm_neuron_amd._vllm_compat import SamplingParams, SimpleSpeculativeConfig
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg, w = case("uneven")
    w = dict(w)
    for name in w:
        if "canon" in name:
            w[name] = torch.cat([w[name][:, :-1] * 0.35, w[name][:, -1:]], 1)
    small = copy.deepcopy(cfg)
    small["canon"]["taps"] = 1
    wd = {n: (t[:, -1:].contiguous() if "canon" in n else t) for n, t in w.items()}
    spec = SimpleSpeculativeConfig(num_speculative_tokens=k, draft_model_config=SimpleNamespace(model="", hf_config=config_from_dict(small)))
    eng = MI355XEngine(config_from_dict(cfg), dtype="float32", max_model_len=max_len, max_num_seqs=2, block_size=16, speculative_config=spec,
                       override_mi355x_config={"state_dict": w, "draft_state_dict": wd})
    prompts = [torch.randint(0, 203, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in (30, 12)]
    ids = [eng.add_request(p, SamplingParams(temperature=0.0, max_tokens=30)) for p in prompts]
    steps = 0
    while eng.has_unfinished_requests():
        eng.step()
        steps += 1
    texts = [eng.outputs[i].token_ids for i in ids]
    assert texts == [greedy(cfg, w, p, min(30, max_len - len(p))) for p in prompts]
    assert steps < 0.85 * max(map(len, texts)) + 2, steps           # some candidates were accepted ...
    assert steps > max(map(len, texts)) / k + 2, steps               # ... and some were not
    eng.close()


def test_speculation_with_an_accepting_draft():
    """A model without state (one tap) as its own draft: every candidate is accepted."""
    from types import SimpleNamespace

    from vllm_neuron_amd._vllm_compat import SamplingParams, SimpleSpeculativeConfig
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg, w = case("wide")
    spec = SimpleSpeculativeConfig(num_speculative_tokens=4, draft_model_config=SimpleNamespace(model="", hf_config=config_from_dict(cfg)))
    eng = MI355XEngine(config_from_dict(cfg), dtype="float32", max_model_len=128, max_num_seqs=2, block_size=16, speculative_config=spec,
                       override_mi355x_config={"state_dict": w, "draft_state_dict": w})
    prompts = [torch.randint(0, 336, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in (20, 9)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12))
    assert [o.token_ids for o in outs] == [greedy(cfg, w, p, 12) for p in prompts]
    eng.close()


def test_a_draft_with_convolution_state_is_refused():
    from types import SimpleNamespace

    from vllm_neuron_amd._vllm_compat import SimpleSpeculativeConfig
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg, w = case("uneven")
    spec = SimpleSpeculativeConfig(num_speculative_tokens=3, draft_model_config=SimpleNamespace(model="", hf_config=config_from_dict(cfg)))
    with pytest.raises(NotImplementedError, match="convolution"):
        MI355XEngine(config_from_dict(cfg), max_model_len=128, max_num_seqs=2, block_size=16, speculative_config=spec,
                     override_mi355x_config={"state_dict": w, "draft_state_dict": w})


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
    cfg, w = case("wide")
    write_model(tmp_path / "m", cfg, w)
    a, b = tokens(cfg, w, 90, 1), tokens(cfg, w, 20, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:70], "want": [69, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:19], "want": []}], "end": []},
             {"step": 7, "entries": [{"id": "b", "tokens": b[19:], "want": [0]}, {"id": "a", "tokens": a[70:], "want": [0, 19]}],
              "end": ["a", "b"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps)) + "\n"))
    assert cmd.main(["--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "128"]) == 0
    assert [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 7"]
    assert not (tmp_path / "1.f32").exists() and sorted(p.name for p in (tmp_path / "m").iterdir()) == ["config.json", "model.safetensors"]
    ra, rb = reference("wide", cfg, w, a, dtype), reference("wide", cfg, w, b, dtype)

    def read(n):
        return torch.from_numpy(np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, cfg["vocab"]))
    assert error(read(0), ra[[69, 3]]) <= LIMIT[dtype]
    assert error(read(7), torch.stack([rb[19], ra[70], ra[89]])) <= LIMIT[dtype]


@pytest.mark.parametrize("chunk", [0, 24])
def test_generate_command(tmp_path, capsys, chunk):
    from vllm_neuron_amd.generate import main
    cfg, w = case("uneven")
    write_model(tmp_path / "m", cfg, w)
    prompts = [torch.randint(0, 203, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in (40, 3)]
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
    cfg, w = case("uneven")
    write_model(tmp_path / "m", cfg, w)
    texts = []
    for start in range(2):
        eng = MI355XEngine(None, str(tmp_path / "m"), max_model_len=128, max_num_seqs=2, block_size=16)
        assert eng.worker.model_runner.model.loaded_from_artifacts == (start == 1)
        texts.append(eng.generate([list(range(20))], SamplingParams(temperature=0.0, max_tokens=12))[0].token_ids)
        eng.close()
    assert texts[0] == texts[1] and len(texts[0]) == 12


def test_loading_refuses_what_does_not_fit():
    cfg, w = case("uneven")
    short = {k: v for k, v in w.items() if k != "l2.mlp.e4.down"}
    with pytest.raises(RuntimeError, match="l2.mlp.e4.down"):
        r = replay(cfg, short, "bfloat16")
        r.engine.worker.model_runner.initialize_kv_cache(None)
    with pytest.raises(ValueError, match="shape"):
        replay(cfg, {**w, "l0.canon1": w["l0.canon1"][:, :2].contiguous()}, "bfloat16")
    for name in ("l1.mix.dkv", "l1.norm2", "l2.mlp.e7.up", "final.norm.b", "pos"):        # another layer's latents; no ff; 7 experts; ...
        with pytest.raises(ValueError, match="not part"):
            replay(cfg, {**w, name: w["l0.norm1"]}, "bfloat16")
    with pytest.raises(NotImplementedError):
        replay(cfg, w, "bfloat16", quantized=True)


def test_synthetic_weights_run():
    """Random weights made on the device (benchmarks) fill every tensor of the configuration."""
    cfg = CASES["uneven"]()
    from vllm_neuron_amd.models import config_from_dict
    from vllm_neuron_amd.replay import TraceReplay
    r = TraceReplay.from_config(config_from_dict(cfg), "bfloat16", 128, override={"synthetic_weights": {"seed": 3, "std": 0.1}})
    out = score(r, list(range(40)), [30] + [1] * 10)
    assert torch.isfinite(out).all() and out.std() > 0.01
    r.engine.close()
