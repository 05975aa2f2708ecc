"""Nusovik on the MI355X: chunked attention with distance tables, learned sinks and gates, the short convolution, both recurrences and
the gated norm against the oracle's mechanisms of the same names, and the model through the framework's engine against the oracle's
whole-sequence logits -- prompts whole, in portions and token by token, in mixed batches, over a KV pool and state slots that are
used again."""

import json
import math

import pytest
import torch

from oracle import nusovik as R
from tests.nusovik_cases import CASES, ROWS, config, error, left, mamba1, parallel, right, tokens, weights

pytestmark = pytest.mark.gpu

# fp32: rounding only.  bf16: against the oracle with the rounding points of the device path (summation order and the flips it causes
# are what is left).
LIMIT = {"float32": 3e-5, "bfloat16": 2.5e-2}


def check(got, ref, dtype, what=""):
    """fp32: every row within the limit.  bf16: nearly every row (a normed sublayer whose output nearly cancels blows its rounding up; which
    rows those are is the weights' doing, and fp32 is held to every row)."""
    d = got.double() - ref.double()
    d = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / ref.double().std()
    if dtype == "float32":
        assert d.max() <= LIMIT[dtype], (what, d.max())
    else:
        assert (d > LIMIT[dtype]).sum() <= max(1, d.numel() // 50) and d.max() <= 8 * LIMIT[dtype], (what, d.max(), (d > LIMIT[dtype]).sum())


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


def b16(t):
    return t.to(torch.bfloat16).float()


def dtype_of(f32):
    return torch.float32 if f32 else torch.bfloat16


def close(got, ref, tol):
    assert ((got - ref).abs() <= tol * (1 + ref.abs())).all(), (got - ref).abs().max()


# ---- rows --------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("f32", [1, 0])
@pytest.mark.parametrize("D", [64, 99, 122, 2048])
def test_embedding_with_sinusoidal_positions(lib, D, f32):
    g = torch.Generator().manual_seed(D)
    table, ids = torch.randn(50, D, generator=g).to(dtype_of(f32)), torch.tensor([3, 0, 49, 7, 7, 21], dtype=torch.int32)
    pos = torch.tensor([0, 1, 2, 1000, 65537, 1000003], dtype=torch.int32)
    ld, ldy = pad(D, 16), pad(D, 64)
    resid, out = torch.full((6, ld), 7.0, device="cuda"), torch.zeros(6, ldy, dtype=dtype_of(f32), device="cuda")
    a = [dev(t) for t in (ids, pos, table)]
    lib.check(lib.load_library().mi_op_embed_sinusoid(ptr(a[0]), ptr(a[1]), ptr(a[2]), 2.5, 1e4, 6, D, ld, ptr(resid), ptr(out), ldy, f32, None))
    torch.cuda.synchronize()
    ref = torch.stack([2.5 * table[int(i)].double() + R.sinusoid(1, D, torch.float64, int(p))[0] for i, p in zip(ids, pos)])
    got = resid.cpu().double()
    assert (got[:, D:] == 0).all() and (got[:, :D] - ref).abs().max() < 2e-6
    close(out.cpu().double()[:, :D], ref, 2e-6 if f32 else 5e-3)


@pytest.mark.parametrize("f32", [1, 0])
@pytest.mark.parametrize("norm,bias,shared", [(1, 1, 1), (1, 0, 0), (0, 1, 1), (1, 1, 0)])
@pytest.mark.parametrize("H,G,d", [(8, 2, 64), (6, 2, 20), (3, 3, 33), (2, 1, 200)])
def test_query_key_norms_biases_and_keys_as_values(lib, H, G, d, norm, bias, shared, f32):
    g = torch.Generator().manual_seed(H + d)
    T, bs, nb = 9, 16, 6
    n = (H + G) * d + (0 if shared else G * d)
    ldq = pad(n, 16) + 16
    qkv, b, wq, wk = torch.randn(T, ldq, generator=g) * 3, torch.randn((H + G) * d, generator=g), torch.randn(d, generator=g), torch.randn(d, generator=g)
    slots = torch.tensor([17, 40, -1, 79, 16, 63, 64, 1, 30], dtype=torch.int32)
    dp, dt = pad(d, 16), dtype_of(f32)
    q, kp, vp = (torch.full(s, 7.0, dtype=dt, device="cuda") for s in ((T, H, dp), (nb, G, bs, dp), (nb, G, bs, dp)))
    spec = lib.layer_spec(dict(num_heads=H, num_kv_heads=G, qk_dim=d, v_dim=d, qk_norm=norm, keys_as_values=shared))
    a = [dev(t) for t in (qkv, b, wq, wk, slots)]
    lib.check(lib.load_library().mi_op_head_scatter(ptr(a[0]), ldq, T, spec, ptr(a[1]) if bias else None, ptr(a[2]) if norm else None, ptr(a[3]) if norm else None,
                                                    1e-3, ptr(a[4]), bs, ptr(q), ptr(kp), ptr(vp), f32, None))
    torch.cuda.synchronize()
    x = qkv.double()
    heads = x[:, :(H + G) * d] + (b.double() if bias else 0)
    raw_q, raw_k = heads[:, :H * d].view(T, H, d), heads[:, H * d:].reshape(T, G, d)
    f = (lambda t, w: R.rms(t, 1e-3) * w.double()) if norm else (lambda t, w: t)
    rv = raw_k if shared else x[:, (H + G) * d:n].reshape(T, G, d)
    tol = 1e-5 if f32 else 1e-2

    def same(got, ref):
        got = got.cpu().double()
        assert (got[..., d:] == 0).all()
        close(got[..., :d], ref, tol)
    same(q, f(raw_q, wq))
    written = torch.zeros(nb, bs, dtype=torch.bool)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            same(kp[s // bs, :, s % bs], f(raw_k, wk)[t])
            same(vp[s // bs, :, s % bs], rv[t])
            written[s // bs, s % bs] = True
    assert (kp.cpu().permute(0, 2, 1, 3)[~written] == 7.0).all() and (vp.cpu().permute(0, 2, 1, 3)[~written] == 7.0).all()


@pytest.mark.parametrize("f32", [1, 0])
@pytest.mark.parametrize("T,n,parts", [(3, 52, 4), (1, 512, 1), (40, 120, 120), (33, 2048, 8), (2, 60, 3), (5, 8192, 2), (2, 57, 19)])
def test_gated_norm(lib, T, n, parts, f32):
    g = torch.Generator().manual_seed(n)
    ldy, ldz, ldo = pad(n, 16), pad(n, 16) + 32, pad(n, 64)
    y, z, w = torch.randn(T, ldy, generator=g) * 3, torch.randn(T, ldz, generator=g) * 2, torch.randn(n, generator=g)
    out = torch.full((T, ldo), 7.0, dtype=dtype_of(f32), device="cuda")
    a = [dev(t) for t in (y, z, w)]
    lib.check(lib.load_library().mi_op_gated_norm(ptr(a[0]), ldy, ptr(a[1]), ldz, ptr(a[2]), n, parts, 1e-2, T, ptr(out), ldo, f32, None))
    torch.cuda.synchronize()
    got = out.cpu().double()
    assert (got[:, n:] == 7.0).all()
    close(got[:, :n], R.gated_norm(y[:, :n].double(), z[:, :n].double(), w.double(), parts, 1e-2), 2e-5 if f32 else 1e-2)


# ---- attention -----------------------------------------------------------------------------------------------------------
class Paged:
    """One random sequence per request, its K / V scattered over shuffled pool blocks, and a ragged set of queries."""

    def __init__(self, H, G, d, segs, bs, chunk, rows, far, seed, scale):
        g = torch.Generator().manual_seed(seed)
        self.H, self.G, self.d, self.bs, self.chunk, self.far, self.scale = H, G, d, bs, chunk, far, scale
        self.segs, row = [], 0
        for i, (pos0, n) in enumerate(segs):
            self.segs.append((row, n, pos0, i))
            row += n
        self.T, self.max_ctx = row, max(p + n for p, n in segs)
        self.MB = -(-self.max_ctx // bs) + 1
        self.nb = 4 + sum(-(-(p + n) // bs) for p, n in segs)
        perm = (torch.randperm(self.nb - 1, generator=g) + 1).tolist()
        self.bt = torch.zeros(len(segs), self.MB, dtype=torch.int32)
        for i, (p, n) in enumerate(segs):
            for b in range(-(-(p + n) // bs)):
                self.bt[i, b] = perm.pop()
        self.q, self.k, self.v = ([torch.randn(p + n, heads, d, generator=g) for p, n in segs] for heads in (H, G, G))
        self.rel, self.sink = torch.randn(rows, H, generator=g) * 2, torch.randn(H, generator=g) + 1
        self.gate = torch.randn(self.T, H + 5, generator=g)

    def run(self, lib, f32, path, mult=0.7):
        H, G, d, bs, dp = self.H, self.G, self.d, self.bs, pad(self.d, 16)
        dt, r = dtype_of(f32), (lambda t: t) if f32 else b16
        # rows nobody wrote hold something large but finite: reading one shows
        kp, vp = torch.full((self.nb, G, bs, dp), 50.0), torch.full((self.nb, G, bs, dp), 50.0)
        kp[..., d:] = 0
        vp[..., d:] = 0
        q, pos = torch.zeros(self.T, H, dp), torch.zeros(self.T, dtype=torch.int32)
        ctx = torch.tensor([p + n for _, n, p, _ in self.segs], dtype=torch.int32)
        ref = torch.zeros(self.T, H, d, dtype=torch.float64)
        for row, n, p, i in self.segs:
            q[row:row + n, :, :d] = self.q[i][p:]
            pos[row:row + n] = torch.arange(p, p + n)
            at = torch.arange(p + n)
            blk, off = self.bt[i, at // bs].long(), at % bs
            kp[blk, :, off, :d] = self.k[i]
            vp[blk, :, off, :d] = self.v[i]
            o = R.chunk_attention(r(self.q[i]).double(), r(self.k[i]).double(), r(self.v[i]).double(), self.scale, self.rel.double(), self.far, self.chunk,
                                  self.sink.double())
            ref[row:row + n] = o[p:]
        ref = (ref * mult * torch.sigmoid(self.gate[:, :H].double())[:, :, None]).reshape(self.T, -1)
        ldo = pad(H * d, 64)
        out = torch.zeros(self.T, ldo, dtype=dt, device="cuda")
        spec = lib.layer_spec(dict(num_heads=H, num_kv_heads=G, qk_dim=d, v_dim=d, chunk=self.chunk, scale=self.scale, rel_rows=self.rel.shape[0], rel_far=self.far,
                                   softmax_sink=2))
        a = [dev(x) for x in (self.sink, self.rel, self.gate, q.to(dt), kp.to(dt), vp.to(dt), self.bt, pos, ctx)]
        segs = torch.tensor(self.segs, dtype=torch.int32).contiguous()
        lib.check(lib.load_library().mi_op_chunk_attn(
            spec, ptr(a[0]), ptr(a[1]), ptr(a[2]), self.gate.shape[1], mult, ptr(a[3]), ptr(a[4]), ptr(a[5]), bs, ptr(a[6]), self.MB, ptr(a[7]), ptr(a[8]), ptr(segs),
            len(self.segs), self.T, self.max_ctx, ptr(out), ldo, int(f32), path, None))
        torch.cuda.synchronize()
        got = out.cpu().double()
        assert (got[:, H * d:] == 0).all()
        return got[:, :H * d], ref


PATHS = [(1, 1), (0, 1), (0, 0)]      # (fp32?, path): plain fp32, plain bf16, MFMA
SEGS = [(0, 70), (45, 1), (31, 2), (0, 1), (100, 130), (299, 1), (0, 3), (64, 65), (190, 17), (255, 1), (256, 1)]


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("H,G,d,chunk,rows,far,bs", [
    (8, 2, 64, 96, 12, 90, 16), (6, 2, 20, 37, 9, 30, 32), (4, 4, 128, 1000, 32, 128, 48), (24, 1, 32, 5, 2, 2, 16), (2, 1, 200, 129, 16, 300, 32),
    (64, 1, 8, 64, 7, 20, 16), (3, 3, 96, 1, 4, 5, 16), (70, 1, 8, 50, 5, 20, 16), (4, 2, 64, 256, 1, 3, 16)])
def test_chunked_attention(lib, H, G, d, chunk, rows, far, bs, f32, path):
    got, ref = Paged(H, G, d, SEGS, bs, chunk, rows, far, H + chunk, 1.6 / math.sqrt(d)).run(lib, f32, path)
    close(got, ref, 2e-5 if f32 else 1.5e-2)


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("chunk,bs", [(96, 16), (33, 32), (64, 16), (16, 16), (200, 48), (1, 16), (257, 32)])
def test_chunk_edge_key_stands_out(lib, chunk, bs, f32, path):
    """A key whose score is far above the rest at the first position of the query's chunk, then at the last one of the chunk before: the
    first takes the row, the second must have no influence at all -- in prompts, at page borders and in decoding."""
    H, G, d = 4, 2, 64
    segs = [(260, 1), (259, 2), (191, 80), (0, 240), (256, 1), (255, 3), (2 * chunk, 1), (2 * chunk - 1, 1), (chunk, 40)]
    for off in (0, -1, 1):
        p = Paged(H, G, d, segs, bs, chunk, 6, 40, chunk + 7, 0.2)
        hit = 0
        for i, (pos0, n) in enumerate(segs):
            last = pos0 + n - 1
            j = last // chunk * chunk + off
            if not 0 <= j <= last:
                continue
            u = torch.nn.functional.normalize(torch.randn(G, d, generator=torch.Generator().manual_seed(i)), dim=-1)
            p.k[i][j] = 14 * u
            p.q[i][last] = 14 * u.repeat_interleave(H // G, 0)
            p.v[i][j] = 30.0
            row = sum(x[1] for x in segs[:i]) + n - 1
            p.gate[row, :H] = 9.0
            hit += 1
        got, ref = p.run(lib, f32, path)
        rows = [sum(x[1] for x in segs[:i]) + n - 1 for i, (_, n) in enumerate(segs)]
        assert (ref[rows].abs().max() > 15) == (off >= 0 and hit > 0)
        assert off or hit == len(segs)
        close(got, ref, 5e-5 if f32 else 2e-2)


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("rows,far,chunk", [(16, 128, 400), (16, 128, 90), (9, 30, 400), (4, 300, 301), (64, 40, 400)])
def test_every_distance_has_its_own_bias(lib, rows, far, chunk, f32, path):
    """Equal keys, a table whose rows differ by far more than the tolerance: a bucket that starts one distance off, a distance counted
    from the wrong end or a saturated tail shows in the weights of the values.  128 / 8 is a power of two: every second bucket
    starts where the logarithms' quotient is a whole number."""
    H, G, d = 4, 1, 32
    segs = [(0, 320), (300, 1), (130, 70), (17, 1), (380, 2), (388, 1)]
    p = Paged(H, G, d, segs, 16, chunk, rows, far, 3, 0.1)
    for k in p.k:
        k[:] = 0.0
    p.rel = torch.tensor([[math.log(1 + (7 * b + 3 * h) % 11) for h in range(H)] for b in range(rows)])
    p.sink[:] = -3.0
    got, ref = p.run(lib, f32, path)
    close(got, ref, 2e-5 if f32 else 1e-2)
    for b in range(rows):                                   # one row alone holds the weight: its distances are the sum's terms
        p.rel = torch.full((rows, H), -30.0)
        p.rel[b] = 4.0
        if b in (0, 1, rows // 2, rows - 2, rows - 1):
            got, ref = p.run(lib, f32, path)
            close(got, ref, 5e-5 if f32 else 1.2e-2)


@pytest.mark.parametrize("f32,path", PATHS)
@pytest.mark.parametrize("sink", [-40.0, 0.0, 6.0, 30.0])
def test_sinks_of_any_size(lib, sink, f32, path):
    p = Paged(4, 2, 64, SEGS, 16, 90, 8, 60, 6, 0.2)
    p.sink = torch.tensor([sink, 0.0, -sink, sink / 2])
    got, ref = p.run(lib, f32, path)
    close(got, ref, 3e-5 if f32 else 1.5e-2)
    if sink == 30.0:
        assert ref[:, :64].abs().max() < 1e-3
        assert ((got - ref)[:, :64].abs() <= 1e-9 + (1e-4 if f32 else 2e-2) * ref[:, :64].abs().max()).all()


@pytest.mark.parametrize("f32,path", PATHS)
def test_far_key_of_a_long_chunk(lib, f32, path):
    """A key more than two thousand tokens back that holds a decoded token's attention (context split over work-groups), and the same
    one position ahead of the chunk."""
    H, G, d, key = 4, 1, 64, 127
    for chunk, seen in ((4000, True), (128, False), (127, True)):
        p = Paged(H, G, d, [(2300, 1), (2250, 40)] if chunk == 4000 else [(chunk + 126, 1), (130, 70)], 32, chunk, 16, 900, 9, 0.2)
        n = [a + b for _, b, a, _ in p.segs]
        for i in range(2):
            at = key if chunk != 127 else (n[i] - 1) // 127 * 127
            u = torch.nn.functional.normalize(torch.randn(d, generator=torch.Generator().manual_seed(50 + i)), dim=0)
            p.k[i][at] = 12 * u
            p.q[i][-1, :] = 12 * u
            p.v[i][at] = 9.0
        p.gate[:] = 9.0
        got, ref = p.run(lib, f32, path)
        assert (ref[0].abs().max() > 5) == seen
        close(got, ref, 5e-5 if f32 else 2e-2)


# ---- short convolution and recurrences --------------------------------------------------------------------------------------
class Steps:
    """Sequences that a recurrent kernel meets in portions: rows, positions, slots."""

    def __init__(self, lengths, slots=None):
        self.lengths, self.at = lengths, [0] * len(lengths)
        self.slots = slots or list(range(len(lengths)))
        self.n_slots = max(self.slots) + 1

    def step(self, live, *rows):
        """live: (sequence, tokens); rows: per quantity a list of [length, ...] tensors -> concatenated rows, segments, positions, slots"""
        segs, pos, out, row = [], [], [[] for _ in rows], 0
        for j, (i, n) in enumerate(live):
            p = self.at[i]
            assert p + n <= self.lengths[i]
            segs.append((row, n, p, j))
            pos += range(p, p + n)
            for o, r in zip(out, rows):
                o.append(r[i][p:p + n])
            self.at[i] += n
            row += n
        i32 = dict(dtype=torch.int32)
        return [torch.cat(o) for o in out], torch.tensor(segs, **i32).contiguous(), torch.tensor(pos, **i32), torch.tensor([self.slots[i] for i, _ in live], **i32), row


# portions of three sequences (lengths 70, 150, 33): several in a step, down to one token, sequences left out
PLANS = [[[(0, 70), (1, 150), (2, 33)]], [[(0, 2), (1, 64), (2, 1)], [(0, 17), (1, 1)], [(2, 2), (1, 65), (0, 1)], [(0, 50)], [(1, 20), (2, 30)]],
         [[(1, 149), (0, 1)], [(1, 1), (0, 1)], [(0, 3), (2, 31)], [(2, 2), (0, 65)]]]
LENGTHS = [70, 150, 33]


def single(plan):                                     # token generation: one row per sequence, no segments
    return all(n == 1 for _, n in plan)


@pytest.mark.parametrize("f32", [1, 0])
@pytest.mark.parametrize("C,taps", [(50, 3), (320, 4), (7, 1), (600, 2), (33, 7), (64, 16)])
def test_short_convolution(lib, C, taps, f32):
    g = torch.Generator().manual_seed(C)
    w, b = torch.randn(taps, C, generator=g) / math.sqrt(taps), torch.randn(C, generator=g)
    ldx, ldy = pad(C, 16) + 16, pad(C, 64)
    x = [torch.randn(n, ldx, generator=g) * 2 for n in LENGTHS]
    ref = [R.short_conv(t[:, :C].double(), w.t().double(), b.double()) for t in x]
    a = [dev(w), dev(b)]
    for plan in PLANS + [[[(i, 1) for i in range(3)]] * 20]:
        st = Steps(LENGTHS, [3, 0, 2])
        ring = torch.full((st.n_slots, taps, C), 1e4, device="cuda")
        for live in plan:
            at = [st.at[i] for i, _ in live]
            (rows,), segs, pos, slots, T = st.step(live, x)
            xd, y = dev(rows), torch.full((T, ldy), 7.0, dtype=dtype_of(f32), device="cuda")
            n = 0 if single(live) else len(live)
            lib.check(lib.load_library().mi_op_short_conv(ptr(xd), ldx, ptr(a[0]), ptr(a[1]), C, taps, ptr(ring), st.n_slots, ptr(slots), ptr(pos), ptr(segs), n, T,
                                                          ptr(y), ldy, f32, None))
            torch.cuda.synchronize()
            got = y.cpu().double()
            assert (got[:, C:] == 0).all()
            close(got[:, :C], torch.cat([ref[i][p:p + n] for (i, n), p in zip(live, at)]), 1e-5 if f32 else 1e-2)
        assert (ring[1] == 1e4).all()                   # nobody's slot


class Scan:
    def __init__(self, lib, C, N, rank, seed, lengths=LENGTHS, slots=None, strong=False):
        g = torch.Generator().manual_seed(seed)
        self.lib, self.C, self.N, self.rank, self.lengths = lib, C, N, rank, lengths
        self.st = Steps(lengths, slots)
        self.b, self.c = pad(rank, 16), pad(rank, 16) + pad(N, 16)
        self.ldl, self.ld = self.c + pad(N, 16), pad(C, 64)
        r = b16                                          # (inputs of the low-rank product, and x, as the bf16 model rounds them)
        self.x = [r(torch.randn(n, self.ld, generator=g)) for n in lengths]
        self.low = [r(torch.randn(n, self.ldl, generator=g)) for n in lengths]
        self.z = [torch.randn(n, self.ld, generator=g) for n in lengths]
        self.w_dt = r(torch.randn(C, rank, generator=g) / math.sqrt(rank))
        self.bias, self.d = torch.randn(C, generator=g) + (2 if strong else -1.5), torch.randn(C, generator=g)
        self.a_log = torch.rand(C, N, generator=g) * 4 - (0.5 if strong else 3)
        self.ref, self.final = [], []
        for x, lo, z in zip(self.x, self.low, self.z):
            x, lo, z = x[:, :C].double(), lo.double(), z[:, :C].double()
            dt = R.softplus(lo[:, :rank] @ self.w_dt.double().t() + self.bias.double())
            y, S = R.scan1(x, dt, self.a_log.double(), lo[:, self.b:self.b + N], lo[:, self.c:self.c + N], self.d.double())
            self.ref.append(y * z * torch.sigmoid(z))
            self.final.append(S)
        self.np = lib.load_library().mi_op_scan_state(N)
        self.state = torch.full((self.st.n_slots, C, self.np), 1e4, device="cuda")
        self.fixed = [dev(t) for t in (self.w_dt, self.bias, self.a_log, self.d)]
        self.spec = lib.layer_spec(dict(mixer_kind=3, ssm_inner=C, ssm_state=N, dt_rank=rank))

    def step(self, live, f32=1):
        at = [self.st.at[i] for i, _ in live]
        (x, lo, z), segs, pos, slots, T = self.st.step(live, self.x, self.low, self.z)
        xd, ld, zd = dev(x.to(dtype_of(f32))), dev(lo), dev(z)
        y = torch.full((T, self.ld), 7.0, dtype=dtype_of(f32), device="cuda")
        w, b, a, d = self.fixed
        self.lib.check(self.lib.load_library().mi_op_scan(
            self.spec, ptr(xd), self.ld, ptr(ld), self.ldl, self.b, self.c, ptr(w), ptr(b), ptr(a), ptr(d), ptr(zd), self.ld, ptr(self.state), self.st.n_slots, ptr(slots),
            ptr(pos), ptr(segs), 0 if single(live) else len(live), T, ptr(y), self.ld, f32, None))
        torch.cuda.synchronize()
        got = y.cpu().double()
        assert (got[:, self.C:] == 7.0).all()
        return got[:, :self.C], torch.cat([self.ref[i][p:p + n] for (i, n), p in zip(live, at)])

    def check_state(self, i, tol=3e-5):
        s = self.state[self.st.slots[i]].cpu().double()
        close(s[:, :self.N], self.final[i], tol)
        assert (s[:, self.N:] == 0).all()


@pytest.mark.parametrize("f32", [1, 0])
@pytest.mark.parametrize("C,N,rank", [(50, 10, 7), (384, 16, 24), (20, 1, 1), (37, 33, 5), (64, 64, 70), (24, 100, 8), (18, 200, 3), (16, 256, 16), (9000, 16, 9)])
def test_selective_scan(lib, C, N, rank, f32):
    """(9000 channels: two states per lane)"""
    for plan in PLANS[:1 if C == 9000 else 3]:
        s = Scan(lib, C, N, rank, C + N, slots=[3, 0, 2])
        for live in plan:
            got, ref = s.step(live, f32)
            close(got, ref, 5e-5 if f32 else 1.2e-2)
        for i in range(3):
            if s.st.at[i] == LENGTHS[i]:
                s.check_state(i)
        assert (s.state[1] == 1e4).all()


@pytest.mark.parametrize("strong", [False, True])
def test_selective_scan_token_by_token_and_slots_used_again(lib, strong):
    s = Scan(lib, 70, 12, 6, 5, lengths=[70, 40, 70], slots=[0, 1, 0], strong=strong)
    for _ in range(70):
        close(*s.step([(0, 1)]), 5e-5)
    close(*s.step([(1, 2)]), 5e-5)
    s.check_state(0)
    close(*s.step([(2, 30), (1, 1)]), 5e-5)            # the slot of the first sequence, from zeros by position
    for _ in range(37):
        close(*s.step([(1, 1), (2, 1)]), 5e-5)
    close(*s.step([(2, 3)]), 5e-5)
    s.check_state(1)
    s.check_state(2)


class Ssd:
    def __init__(self, lib, H, P, N, G, seed, lengths=LENGTHS, slots=None, strong=False):
        g = torch.Generator().manual_seed(seed)
        self.lib, self.H, self.P, self.N, self.G, self.lengths = lib, H, P, N, G, lengths
        self.st, self.C = Steps(lengths, slots), H * P + 2 * G * N
        self.ldx, self.ldt, self.ldy = pad(self.C, 16), pad(H, 16), pad(H * P, 16)
        self.x = [b16(torch.randn(n, self.ldx, generator=g)) for n in lengths]
        self.dt = [torch.randn(n, self.ldt, generator=g) for n in lengths]
        if strong:                                       # steps that wipe the state beside steps that keep it, within a chunk
            for t in self.dt:
                t += torch.where(torch.rand(t.shape[0], 1, generator=g) < 0.3, 60.0, -6.0)
        self.bias, self.d, self.a_log = torch.randn(H, generator=g) - 1.5, torch.randn(H, generator=g), torch.rand(H, generator=g) * 4 - (1 if strong else 3)
        self.ref, self.final = [], []
        for x, dt in zip(self.x, self.dt):
            T = x.shape[0]
            x, b, c = x[:, :self.C].double().split([H * P, G * N, G * N], -1)
            y, S = R.scan2(x.reshape(T, H, P), R.softplus(dt[:, :H].double() + self.bias.double()), self.a_log.double(), b.reshape(T, G, N), c.reshape(T, G, N),
                           self.d.double())
            self.ref.append(y.reshape(T, -1))
            self.final.append(S)
        self.state = torch.full((self.st.n_slots, H, pad(N, 16), pad(P, 16)), 1e4, device="cuda")
        self.fixed = [dev(t) for t in (self.bias, self.a_log, self.d)]
        self.spec = lib.layer_spec(dict(beside_kind=4, ssm_heads=H, ssm_dim=P, ssm_state=N, ssm_groups=G))

    def step(self, live, f32=1, chunks=64):
        at = [self.st.at[i] for i, _ in live]
        (x, dt), segs, pos, slots, T = self.st.step(live, self.x, self.dt)
        xd, dd = dev(x.to(dtype_of(f32))), dev(dt)
        y = torch.full((T, self.ldy), 7.0, device="cuda")
        b, a, d = self.fixed
        self.lib.check(self.lib.load_library().mi_op_ssd(
            self.spec, ptr(xd), self.ldx, ptr(dd), self.ldt, ptr(b), ptr(a), ptr(d), ptr(self.state), self.st.n_slots, ptr(slots), ptr(pos), ptr(segs),
            0 if single(live) else len(live), T, chunks, ptr(y), self.ldy, f32, None))
        torch.cuda.synchronize()
        got = y.cpu().double()
        assert (got[:, self.H * self.P:] == 7.0).all()
        return got[:, :self.H * self.P], torch.cat([self.ref[i][p:p + n] for (i, n), p in zip(live, at)])

    def check_state(self, i, tol=3e-5):
        s = self.state[self.st.slots[i]].cpu().double()
        close(s[:, :self.N, :self.P], self.final[i], tol)
        assert (s[:, self.N:] == 0).all() and (s[:, :, self.P:] == 0).all()


SSD_SHAPES = [(4, 13, 20, 2), (8, 64, 128, 1), (6, 10, 33, 3), (3, 48, 5, 3), (1, 256, 256, 1), (2, 20, 1, 1), (2, 130, 144, 2), (5, 16, 16, 5), (12, 32, 64, 4), (1, 1, 200, 1)]


@pytest.mark.parametrize("f32", [1, 0])
@pytest.mark.parametrize("H,P,N,G", SSD_SHAPES)
def test_state_space_duality(lib, H, P, N, G, f32):
    for k, plan in enumerate(PLANS):
        s = Ssd(lib, H, P, N, G, H + P + N, slots=[3, 0, 2])
        for live in plan:
            got, ref = s.step(live, f32, chunks=(64, 2, 1)[k])       # (few chunks in memory: the state goes on through its slot)
            close(got, ref, 5e-5)
        for i in range(3):
            if s.st.at[i] == LENGTHS[i]:
                s.check_state(i)
        assert (s.state[1] == 1e4).all()


@pytest.mark.parametrize("strong", [False, True])
def test_state_space_duality_token_by_token_and_slots_used_again(lib, strong):
    s = Ssd(lib, 4, 24, 40, 2, 5, lengths=[70, 40, 200], slots=[0, 1, 0], strong=strong)
    for _ in range(70):
        close(*s.step([(0, 1)]), 5e-5)
    close(*s.step([(1, 2)]), 5e-5)
    s.check_state(0)
    close(*s.step([(2, 130), (1, 1)]), 5e-5)
    for _ in range(37):
        close(*s.step([(1, 1), (2, 1)]), 5e-5)
    close(*s.step([(2, 33)]), 5e-5)
    s.check_state(1)
    s.check_state(2)


def test_a_strong_decay_leaves_the_following_steps_exact(lib):
    """Half a chunk of steps whose decays' logarithms sum to thousands, then steps that decay by next to nothing: a difference of running
    sums in fp32 would lose three digits of those."""
    s = Ssd(lib, 2, 16, 16, 1, 8, lengths=[64])
    s.dt[0][:32], s.dt[0][32:] = 90.0, -9.0
    s.a_log[:] = 1.5
    x, b, c = s.x[0][:, :s.C].double().split([32, 16, 16], -1)
    y, S = R.scan2(x.reshape(64, 2, 16), R.softplus(s.dt[0][:, :2].double() + s.bias.double()), s.a_log.double(), b.reshape(64, 1, 16), c.reshape(64, 1, 16), s.d.double())
    s.ref, s.final, s.fixed[1] = [y.reshape(64, -1)], [S], dev(s.a_log)
    got, ref = s.step([(0, 64)])
    assert ((got - ref).abs() <= 2e-6 * (1 + ref.abs().max())).all()
    s.check_state(0, 2e-6)


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
        _cases[name] = (cfg, weights(cfg, 11, ROWS[name]))
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
    for n in (1, 2, 15, 16, 17, 65, 130, 300):
        toks = tokens(cfg, n, n)
        check(score(r, toks, [n]), reference(name, cfg, w, toks, dtype), dtype, n)


def test_token_by_token_equals_the_prompt(served):
    name, dtype, cfg, w, r = served
    toks = tokens(cfg, 130, 130)
    ref = reference(name, cfg, w, toks, dtype)
    check(score(r, toks, [1] * 130), ref, dtype)
    check(score(r, toks, [70] + [1] * 60), ref, dtype)


@pytest.mark.parametrize("cuts", [[2] * 65, [3] * 44, [5] * 26, [16] * 9, [17] * 8, [33] * 4, [37, 93], [64, 66], [65, 65], [100, 2, 28], [30, 100],
                                  [2, 1, 5, 1, 40, 2, 2, 1, 64, 12]])
def test_portions(served, cuts):
    name, dtype, cfg, w, r = served
    toks = tokens(cfg, 130, 130)
    check(score(r, toks, cuts), reference(name, cfg, w, toks, dtype), dtype)


def test_mixed_batches_over_reused_pages_and_slots(served):
    """Up to four live requests, portions beside single tokens, requests left out of steps and ended; the pool holds far
    fewer tokens than the requests together, and there are four state slots."""
    name, dtype, cfg, w, r = served
    g = torch.Generator().manual_seed(3)

    def rnd(a, b):
        return int(torch.randint(a, b, (1,), generator=g))
    pool = 768 // 16
    todo = [tokens(cfg, n, 1000 + i) for i, n in enumerate([150, 9, 90, 1, 160, 47, 130, 33, 130, 16, 2, 121])]
    total = sum(map(len, todo))
    assert total > 768 and r.engine.scheduler.block_pool.num_free() == pool
    live, got, want, steps, used = {}, [], [], 0, 0
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
            got.append(o)
            want.append(ref[[e["at"] + x for x in e["want"]]])
        for rid in end:
            del live[rid]
        steps += 1
    check(torch.cat(got), torch.cat(want), dtype)
    assert used == total and steps > 15 and sum(map(len, got)) > 60
    r.engine.scheduler.schedule()
    assert r.engine.scheduler.block_pool.num_free() == pool         # everything came back


def test_batch_does_not_change_a_request(served):
    name, dtype, cfg, w, r = served
    toks, other = tokens(cfg, 90, 90), [tokens(cfg, n, 400 + n) for n in (33, 2, 71)]
    alone = score(r, toks, [90])
    rid, ids = uid(), [uid() for _ in other]
    outs = r.step([{"id": ids[0], "tokens": other[0], "want": []}, {"id": rid, "tokens": toks[:50], "want": list(range(50))},
                   {"id": ids[1], "tokens": other[1], "want": []}, {"id": ids[2], "tokens": other[2], "want": [3]}], [])
    outs2 = r.step([{"id": ids[1], "tokens": [1], "want": [0]}, {"id": rid, "tokens": toks[50:], "want": list(range(40))}],
                   [rid] + ids)
    check(torch.cat([outs[1], outs2[1]]), alone, dtype)


def test_layer_by_layer(served):
    name, dtype, cfg, w, r = served
    native = r.engine.worker.model_runner.model.model
    toks = tokens(cfg, 45, 8)
    res, _ = R.residuals_and_logits(cfg, w, toks, torch.float64 if dtype == "float32" else torch.float32, None if dtype == "float32" else "bf16")
    score(r, toks[:1], [1])
    native.keep_layer_residuals(True)
    score(r, toks, [45])
    got = native.layer_residuals(45)
    native.keep_layer_residuals(False)
    assert got.shape == res.shape == (len(cfg["layers"]), 45, cfg["width"])
    for i in range(got.shape[0]):
        assert ((got[i].double() - res[i].double()).pow(2).mean().sqrt() / res[i].std()) <= LIMIT[dtype], i


@pytest.mark.parametrize("dtype", list(LIMIT))
def test_long_decoding_and_pages_of_ended_requests(dtype):
    """A pool of exactly one long request: every sequence runs over the pages (and the state slot) of the one before, decoding
    across page and chunk borders, with graph replays."""
    cfg, w = case("uneven")
    r = replay(cfg, w, dtype, max_tokens=304, max_live=1)
    for seed in (21, 22):
        toks = tokens(cfg, 300, seed)
        check(score(r, toks, [40] + [1] * 260), reference("uneven", cfg, w, toks, dtype), dtype)
    r.engine.close()


def test_a_wide_row_and_a_large_batch():
    """Hidden rows beyond one work-group's first pass, 40 requests decoding at once (the GEMMs), a prompt whose output projections
    leave a K-split's sum to the next norm."""
    cfg = config(2112, 160, [mamba1(256, 8, 16, 4, 128), parallel(left(4, 2, 32, 48, 30), right(4, 32, 32, 2, 1, 4), 96), mamba1(96, 20, 8, 3)])
    w = weights(cfg, 9)
    r = replay(cfg, w, "bfloat16", max_tokens=40 * 48, max_live=40)
    seqs = [tokens(cfg, n, 7000 + n % 3) for n in (30, 31, 32)]
    ids = [uid() for _ in range(40)]
    got, want = [], []
    r.step([{"id": rid, "tokens": seqs[i % 3][:20], "want": []} for i, rid in enumerate(ids)], [])
    for p in range(20, 28):
        outs = r.step([{"id": rid, "tokens": [seqs[i % 3][p]], "want": [0]} for i, rid in enumerate(ids)], ids if p == 27 else [])
        for i, o in enumerate(outs):
            got.append(o)
            want.append(reference(f"wide{i % 3}", cfg, w, seqs[i % 3], "bfloat16")[p:p + 1])
    check(torch.cat(got), torch.cat(want), "bfloat16")
    toks = tokens(cfg, 700, 5)
    check(score(r, toks, [640, 60]), reference("wide row", cfg, w, toks, "bfloat16"), "bfloat16")
    r.engine.close()


def test_state_over_thousands_of_tokens():
    """Channels that hardly decay: what the first tokens left in the state is still there thousands of tokens on, in one portion and cut."""
    cfg = config(64, 96, [mamba1(32, 4, 4, 4), parallel(left(2, 1, 16, 100, 50), right(2, 16, 16, 1, 1, 2))])
    w = weights(cfg, 4)
    for n in w:
        if n.endswith("A_log"):
            w[n] = w[n] - 5
    toks = tokens(cfg, 3000, 1)
    changed = [(toks[0] + 1) % 96] + toks[1:]
    want = [10, 1023, 2047, 2048, 2999]
    ref, other = (R.logits(cfg, w, t, torch.float64)[want] for t in (toks, changed))
    assert error(ref[1:], other[1:]) > 1e-3               # the first token still shows
    r = replay(cfg, w, "float32", max_tokens=3008, max_live=1)
    rid = uid()
    check(r.step([{"id": rid, "tokens": toks, "want": want}], [rid])[0], ref, "float32")
    rid, got, at = uid(), [], 0
    for n in (1000, 1, 777, 2, 1220):
        got += r.step([{"id": rid, "tokens": toks[at:at + n], "want": [x - at for x in want if at <= x < at + n]}], [rid] if at + n == 3000 else [])
        at += n
    check(torch.cat(got), ref, "float32")
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
    """MI355XEngine.generate, both schedulers, more requests than state slots: fp32 text equals the oracle's.  Prompts share a
    prefix, which is computed again: prefix caching, asked for, is off with recurrent state."""
    from vllm_neuron_amd._vllm_compat import SamplingParams
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg, w = case("uneven")
    base = tokens(cfg, 70, 5)
    prompts = [base, base[:64] + tokens(cfg, 11, 6), tokens(cfg, 1, 7), tokens(cfg, 21, 8), tokens(cfg, 33, 9)]
    override = {"state_dict": w}
    if chunked:
        override.update(is_block_kv_layout=True, chunked_prefill_config={"max_num_seqs": 3})
    if device_sampling:
        override["on_device_sampling_config"] = {"dynamic": True}
    eng = MI355XEngine(config_from_dict(cfg), dtype="float32", max_model_len=256, max_num_seqs=3, block_size=16,
                       enable_prefix_caching=True, enable_chunked_prefill=chunked,
                       max_num_batched_tokens=48 if chunked else None, override_mi355x_config=override)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10))
    assert [o.token_ids for o in outs] == [greedy(cfg, w, p, 10) for p in prompts]
    assert max(o.num_cached_tokens for o in outs) == 0
    eng.close()


def test_graph_replays_equal_eager_steps():
    """Every replay of a captured token-generation step, with eager work of other requests in between, against the same steps
    without graphs."""
    cfg, w = case("wide")
    toks, other = tokens(cfg, 60, 3), tokens(cfg, 40, 4)
    outs = []
    for graphs in (1, 0):
        r = replay(cfg, w, "bfloat16", use_graphs=graphs)
        a, got = uid(), []
        r.step([{"id": a, "tokens": toks[:40], "want": []}], [])
        for i in range(40, 60):
            got.append(r.step([{"id": a, "tokens": [toks[i]], "want": [0]}], [])[0])
            if i % 5 == 0:
                b = uid()
                got.append(r.step([{"id": b, "tokens": other[:i - 20], "want": [0]}], [b])[0])
        outs.append(torch.cat(got))
        r.engine.close()
    assert torch.equal(outs[0], outs[1])


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
    a, b = tokens(cfg, 90, 1), tokens(cfg, 20, 2)
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
    check(read(0), ra[[69, 3]], dtype)
    check(read(7), torch.stack([rb[19], ra[70], ra[89]]), dtype)


@pytest.mark.parametrize("chunk", [0, 24])
def test_generate_command(tmp_path, capsys, chunk):
    from vllm_neuron_amd.generate import main
    cfg, w = case("uneven")
    write_model(tmp_path / "m", cfg, w)
    prompts = [tokens(cfg, n, n) for n in (40, 3)]
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
        texts.append(eng.generate([list(range(60))], SamplingParams(temperature=0.0, max_tokens=12))[0].token_ids)
        eng.close()
    assert texts[0] == texts[1] and len(texts[0]) == 12


def test_loading_refuses_what_does_not_fit():
    cfg, w = case("uneven")
    short = {k: v for k, v in w.items() if k != "l1.mix.left.sink"}
    with pytest.raises(RuntimeError, match="l1.mix.left.sink"):
        r = replay(cfg, short, "bfloat16")
        r.engine.worker.model_runner.initialize_kv_cache(None)
    with pytest.raises(ValueError, match="shape"):
        replay(cfg, {**w, "l0.mix.conv": w["l0.mix.conv"][:, :2].contiguous()}, "bfloat16")
    for name in ("l4.norm1", "l2.norm2", "l1.mix.left.v", "l1.mix.q", "l1.mix.right.dt", "l0.mix.left.q", "l2.mlp.up", "final.norm.b", "pos"):
        with pytest.raises(ValueError, match="not part"):
            replay(cfg, {**w, name: w["l0.norm1"]}, "bfloat16")
    with pytest.raises(NotImplementedError):
        replay(cfg, w, "bfloat16", quantized=True)


def test_layers_without_attention_alone():
    """No KV pool at all: every layer keeps its state in the slots."""
    cfg = config(96, 150, [mamba1(64, 8, 6, 4, 40), mamba1(48, 16, 4, 2)])
    w = weights(cfg, 2)
    r = replay(cfg, w, "float32")
    toks = tokens(cfg, 130, 1)
    check(score(r, toks, [50, 2] + [1] * 78), R.logits(cfg, w, toks, torch.float64), "float32")
    r.engine.close()


def test_synthetic_weights_run():
    """Random weights made on the device (benchmarks) fill every tensor of the configuration."""
    from vllm_neuron_amd.models import config_from_dict, fill_sizes
    from vllm_neuron_amd.replay import TraceReplay
    c = config_from_dict(CASES["uneven"]())
    fill_sizes(c, lambda name: (16, 1))
    r = TraceReplay.from_config(c, "bfloat16", 128, override={"synthetic_weights": {"seed": 3, "std": 0.1}})
    out = score(r, list(range(40)), [30] + [1] * 10)
    assert torch.isfinite(out).all() and out.std() > 0.01
    r.engine.close()
