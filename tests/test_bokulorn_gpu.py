"""Bokulorn on the MI355X: the delta rule, the rotated latent attention and the grouped sigmoid router against the oracle's mechanisms of
the same names, and the model through the framework's engine against the oracle's whole-sequence logits -- prompts whole, in
portions and token by token, in mixed batches, over a KV pool and state slots that are used again."""

import json
import math

import pytest
import torch

from oracle import bokulorn as R
from tests.bokulorn_cases import CASES, close_calls, config, delta, error, latent, latent2, moe, tokens, weights

pytestmark = pytest.mark.gpu

# fp32: rounding only.  bf16: against the oracle with the rounding points of the device path (latent-space scores, summation
# order and the flips they cause are what is left).
LIMIT = {"float32": 3e-5, "bfloat16": 2e-2}


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


# ---- the delta rule ----------------------------------------------------------------------------------------------------
class Delta:
    """Sequences of one layer: projections, the oracle's outputs, and the device's state slots and rings (filled with something large:
    a slot read without having been written shows)."""

    def __init__(self, lib, H, G, d, dv, taps, lengths, seed, slots=None, strong=False):
        g = torch.Generator().manual_seed(seed)
        self.lib, self.H, self.G, self.d, self.dv, self.taps, self.lengths = lib, H, G, d, dv, taps, lengths
        self.C = 2 * G * d + H * dv
        self.beta = pad(self.C, 16) + 16
        self.ldp, self.gate = self.beta + pad(H, 16), pad(H * d, 16)
        self.ldz = self.gate + pad(H * dv, 16)
        self.conv = torch.randn(taps, self.C, generator=g) * 1.2 / math.sqrt(taps)
        self.a_log = torch.rand(H, generator=g) * 4 - (0.5 if strong else 3)
        self.dt = torch.randn(H * d, generator=g) + (2 if strong else -2)
        self.norm, self.eps = 1 + 0.3 * torch.randn(dv, generator=g), 1e-3
        self.proj = [torch.full((n, self.ldp), 1e3) for n in lengths]
        self.z = [torch.randn(n, self.ldz, generator=g) * 1.5 for n in lengths]
        self.ref, self.final = [], []
        cw = self.conv.t().double()
        qk = G * d
        for n, p, z in zip(lengths, self.proj, self.z):
            p[:, :self.C] = torch.randn(n, self.C, generator=g)
            p[:, self.beta:self.beta + H] = torch.randn(n, H, generator=g) * 2
            x = p.double()
            o, S = R.delta_heads(x[:, :qk], x[:, qk:2 * qk], x[:, 2 * qk:self.C], x[:, self.beta:self.beta + H], z[:, :H * d].double(),
                                 z[:, self.gate:self.gate + H * dv].double(), (cw[:qk], cw[qk:2 * qk], cw[2 * qk:]), self.a_log.double(),
                                 self.dt.double(), self.norm.double(), self.eps)
            self.ref.append(o)
            self.final.append(S)
        self.slots = slots or list(range(len(lengths)))
        n = max(self.slots) + 1
        self.state = torch.full((n, H, pad(d, 16), pad(dv, 16)), 1e4, device="cuda")
        self.ring = torch.full((n, taps, self.C), 1e4, device="cuda")
        self.fixed = [dev(t) for t in (self.conv, self.a_log, self.dt, self.norm)]
        self.at = [0] * len(lengths)
        self.spec = lib.layer_spec(dict(mixer_kind=2, num_heads=H, num_kv_heads=G, qk_dim=d, v_dim=dv, conv_taps=taps))

    def step(self, live, f32=1, chunks=64, single=False):
        """live: (sequence, tokens); -> (got, reference) rows"""
        segs, rows, pos, ref, row = [], [], [], [], 0
        for j, (i, n) in enumerate(live):
            p = self.at[i]
            segs.append((row, n, p, j))
            rows.append((self.proj[i][p:p + n], self.z[i][p:p + n]))
            pos += range(p, p + n)
            ref.append(self.ref[i][p:p + n])
            self.at[i] += n
            row += n
        proj, z = dev(torch.cat([a for a, _ in rows])), dev(torch.cat([b for _, b in rows]))
        ldo = pad(self.H * self.dv, 64)
        out = torch.full((row, ldo), 7.0, dtype=torch.float32 if f32 else torch.bfloat16, device="cuda")
        slots = torch.tensor([self.slots[i] for i, _ in live], dtype=torch.int32)
        pos, segs = torch.tensor(pos, dtype=torch.int32), torch.tensor(segs, dtype=torch.int32).contiguous()
        c, a, dt, nm = self.fixed
        self.lib.check(self.lib.load_library().mi_op_delta_rule(
            self.spec, ptr(proj), self.ldp, self.beta, ptr(z), self.ldz, self.gate, ptr(c), ptr(a), ptr(dt), ptr(nm), self.eps, ptr(self.state), ptr(self.ring),
            self.state.shape[0], ptr(slots), ptr(pos), None if single else ptr(segs), 0 if single else len(live), row, chunks, ptr(out), ldo, f32, None))
        torch.cuda.synchronize()
        got = out.cpu()
        assert (got[:, self.H * self.dv:] == 7.0).all()
        return got[:, :self.H * self.dv].double(), torch.cat(ref)

    def check_state(self, i, tol=3e-5):
        s = self.state[self.slots[i]].cpu().double()
        assert ((s[:, :self.d, :self.dv] - self.final[i]).abs() <= tol * (1 + self.final[i].abs())).all()
        assert (s[:, self.d:] == 0).all() and (s[:, :, self.dv:] == 0).all()


def close(got, ref, f32, tol=1.2e-2):
    assert ((got - ref).abs() <= (5e-5 if f32 else tol) * (1 + ref.abs())).all(), (got - ref).abs().max()


SHAPES = [(6, 2, 20, 13, 3), (2, 2, 128, 128, 4), (8, 8, 64, 64, 4), (3, 1, 192, 48, 1), (1, 1, 256, 256, 16), (4, 4, 16, 200, 2), (5, 5, 7, 3, 7), (16, 4, 96, 80, 4)]


@pytest.mark.parametrize("f32", [1, 0])
@pytest.mark.parametrize("shape", SHAPES)
def test_delta_prompt(lib, shape, f32):
    x = Delta(lib, *shape, [77, 2, 16, 33], seed=sum(shape))
    close(*x.step([(0, 77), (1, 2), (2, 16), (3, 33)], f32), f32)
    for i in range(4):
        x.check_state(i)


@pytest.mark.parametrize("single", [True, False])
@pytest.mark.parametrize("shape", SHAPES)
def test_delta_token_by_token(lib, shape, single):
    x = Delta(lib, *shape, [24, 24, 24], seed=sum(shape), slots=[2, 0, 1])
    for _ in range(24):
        close(*x.step([(2, 1), (0, 1), (1, 1)], single=single), 1)
    for i in range(3):
        x.check_state(i)


@pytest.mark.parametrize("strong", [False, True])
@pytest.mark.parametrize("shape", SHAPES[:4])
def test_delta_portions_beside_tokens(lib, shape, strong):
    """Cuts inside and at the edges of chunks and of the convolution's reach, sequences left out of steps, factors of a few chunks at a
    time; strong: decays down to exp(-100) a token."""
    x = Delta(lib, *shape, [150, 150, 150], seed=3 + sum(shape), slots=[1, 3, 0], strong=strong)
    plan = [[5, 1, 2], [1, 1, 1], [10, 16, 33], [2, 2, 2], [1, 0, 1], [17, 15, 1], [1, 1, 1], [3, 1, 1], [16, 48, 0], [1, 1, 1], [49, 17, 32], [0, 1, 0],
            [44, 46, 75]]
    for step in plan:
        close(*x.step([(i, n) for i, n in enumerate(step) if n], chunks=3), 1)
    assert x.at == [150, 150, 150]
    for i in range(3):
        x.check_state(i)


def test_delta_slots_are_used_again(lib):
    """A slot holds the former sequence's state and convolution inputs when the next one starts in it: a prompt, or a single token."""
    x = Delta(lib, 4, 2, 32, 32, 4, [40, 21, 30], seed=5, slots=[0, 0, 0])
    close(*x.step([(0, 40)]), 1)
    close(*x.step([(1, 1)], single=True), 1)
    close(*x.step([(1, 20)]), 1)
    close(*x.step([(2, 30)]), 1)
    x.check_state(2)


def test_delta_long_memory(lib):
    """Without decay a write of the first token is read out hundreds of tokens later."""
    x = Delta(lib, 2, 1, 64, 32, 4, [400], seed=8)
    for t in (x.a_log, x.fixed[1]):
        t.fill_(-20.0)
    qk = x.G * x.d
    p, cw = x.proj[0].double(), x.conv.t().double()
    x.ref[0], x.final[0] = R.delta_heads(p[:, :qk], p[:, qk:2 * qk], p[:, 2 * qk:x.C], p[:, x.beta:x.beta + 2], x.z[0][:, :2 * x.d].double(),
                                         x.z[0][:, x.gate:x.gate + 2 * x.dv].double(), (cw[:qk], cw[qk:2 * qk], cw[2 * qk:]), x.a_log.double(), x.dt.double(),
                                         x.norm.double(), x.eps)
    close(*x.step([(0, 333)]), 1)
    for _ in range(67):
        close(*x.step([(0, 1)], single=True), 1)
    x.check_state(0)


def test_delta_refuses_what_it_is_not_built_for(lib):
    with pytest.raises(ValueError, match="sizes"):
        Delta(lib, 2, 2, 264, 16, 4, [3], seed=1).step([(0, 3)])
    x = Delta(lib, 2, 2, 16, 16, 4, [3], seed=1)
    x.slots = [5]
    with pytest.raises(ValueError, match="slot"):
        x.step([(0, 3)])


# ---- latent attention with a rotated part ------------------------------------------------------------------------------
def latent_spec(lib, H, dk, dv, rank, nr, dims, scale):
    return lib.layer_spec(dict(mixer_kind=1, num_heads=H, num_kv_heads=1, qk_dim=dk, v_dim=dv, kv_rank=rank, kv_from=-1, window=0, scale=scale, rot_dim=nr,
                               rot_dims=dims, rot_base=100.0))


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("H,dk,rank,nr,dims", [(3, 20, 36, 12, 8), (18, 64, 160, 64, 64), (2, 33, 520, 6, 6), (5, 7, 64, 96, 0), (4, 32, 64, 32, 2)])
def test_rotation_and_scatter(lib, H, dk, rank, nr, dims, f32):
    g = torch.Generator().manual_seed(H + dk)
    bs, nb, base = 16, 6, 100.0
    pos = torch.tensor([0, 1, 2, 15, 16, 77, 3, 40, 1000], dtype=torch.int32)
    T = pos.numel()
    dq = dk + nr
    ldq = pad(H * dq + rank + nr, 16)
    qd, cn = torch.randn(T, ldq, generator=g) * 2, 1 + 0.3 * torch.randn(rank, generator=g)
    slots = torch.tensor([17, 40, -1, 79, 16, 63, 64, 1, 30], dtype=torch.int32)
    dt = torch.float32 if f32 else torch.bfloat16
    a = torch.arange(1001, dtype=torch.float64)[:, None] * base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / max(dims, 1))
    table = torch.stack([a.cos(), a.sin()], -1).float()
    if dims == 0:
        table = torch.zeros(4)
    rp, nrp = pad(rank, 32), pad(nr, 32)
    q = torch.full((T, H, pad(dq, 32)), 7.0, dtype=dt, device="cuda")
    pool = torch.full((nb * bs, rp + nrp), 7.0, dtype=dt, device="cuda")
    x = [dev(t) for t in (qd, table, pos, cn, slots)]
    lib.check(lib.load_library().mi_op_latent_scatter(ptr(x[0]), ldq, T, latent_spec(lib, H, dk, 8, rank, nr, dims, 1.0), ptr(x[1]), ptr(x[2]), ptr(x[3]), 1e-3,
                                                      ptr(x[4]), bs, ptr(q), ptr(pool), f32, None))
    torch.cuda.synchronize()
    tol = 1e-5 if f32 else 1.2e-2
    q, pool = q.cpu().double(), pool.cpu().double()

    def turned(v, i):
        return R.rotate(v[None].double(), base, dims, first=int(pos[i]))[0] if dims else v.double()
    for i in range(T):
        heads = qd[i, :H * dq].view(H, dq)
        ref = torch.cat([heads[:, :dk].double(), turned(heads[:, dk:], i)], -1)
        assert ((q[i, :, :dq] - ref).abs() <= tol * (1 + ref.abs())).all() and (q[i, :, dq:] == 0).all()
        if slots[i] < 0:
            continue
        row = pool[slots[i]]
        c = R.rms(qd[i, H * dq:H * dq + rank].double(), 1e-3) * cn.double()
        k = turned(qd[i, H * dq + rank:H * dq + rank + nr], i)
        assert ((row[:rank] - c).abs() <= tol * (1 + c.abs())).all() and (row[rank:rp] == 0).all()
        assert ((row[rp:rp + nr] - k).abs() <= tol * (1 + k.abs())).all() and (row[rp + nr:] == 0).all()
    untouched = sorted(set(range(nb * bs)) - set(slots.tolist()))
    assert (pool[untouched] == 7.0).all()


SEGS = [(0, 70), (45, 1), (31, 2), (0, 1), (100, 130), (299, 1), (0, 3), (64, 65), (190, 17)]


@pytest.mark.parametrize("f32,path", [(1, 1), (0, 1), (0, 2), (0, 3)])      # plain fp32, plain bf16, rows in the latent space, written-out keys
@pytest.mark.parametrize("H,dk,dv,rank,nr,bs", [(4, 64, 40, 96, 32, 16), (3, 20, 13, 36, 12, 32), (18, 32, 32, 160, 64, 48), (2, 128, 128, 512, 64, 32),
                                                (34, 16, 24, 64, 33, 16), (70, 8, 8, 250, 8, 16)])
def test_latent_attention_with_a_rotated_part(lib, H, dk, dv, rank, nr, bs, f32, path):
    """A key whose two parts both matter: the score of one far key stands out through the rotated part, of another through the latent."""
    g = torch.Generator().manual_seed(H + rank)
    scale, n_seq = 1.5 / math.sqrt(dk + nr), len(SEGS)
    r = (lambda t: t) if f32 else b16
    rp, cp, dq, dkp = pad(rank, 32), pad(rank, 32) + pad(nr, 32), dk + nr, pad(dk + nr, 32)
    uk, uv = b16(torch.randn(H * dk, rank, generator=g) / math.sqrt(rank)), b16(torch.randn(H * dv, rank, generator=g) / math.sqrt(rank))
    max_ctx = max(p + n for p, n in SEGS)
    MB = -(-max_ctx // bs)
    bt = (torch.randperm(n_seq * MB, generator=g) + 1).to(torch.int32).view(n_seq, MB)
    pool = torch.full((n_seq * MB + 1, bs, cp), 30.0)                        # rows nobody wrote: large but finite
    pool[..., rank:rp] = 0
    pool[..., rp + nr:] = 0
    T = sum(n for _, n in SEGS)
    q, pos, ref = torch.zeros(T, H, dkp), torch.zeros(T, dtype=torch.int32), torch.zeros(T, H * dv, dtype=torch.float64)
    segs, row = [], 0
    for i, (p, n) in enumerate(SEGS):
        c, kr, qi = torch.randn(p + n, rank, generator=g), torch.randn(p + n, nr, generator=g), torch.randn(p + n, H, dq, generator=g)
        if p + n > 20:                                                       # the last row asks for two far keys
            kr[3] = 6 * qi[-1, 0, dk:] / qi[-1, 0, dk:].norm()
            c[9] = 6 * torch.nn.functional.normalize(uk[:dk].t() @ qi[-1, 0, :dk], dim=0)
        at = torch.arange(p + n)
        pool[bt[i, at // bs].long(), at % bs, :rank] = c
        pool[bt[i, at // bs].long(), at % bs, rp:rp + nr] = kr
        q[row:row + n, :, :dq] = qi[p:]
        pos[row:row + n] = torch.arange(p, p + n)
        o = R.latent_attention(r(qi).double(), r(c).double(), r(kr).double(), uk.double(), uv.double(), scale)
        ref[row:row + n] = o[p:].reshape(n, -1)
        segs.append((row, n, p, i))
        row += n
    ldo = pad(H * dv, 64)
    dt = torch.float32 if f32 else torch.bfloat16
    out = torch.zeros(T, ldo, dtype=dt, device="cuda")
    a = [dev(x) for x in (uk, uv, q.to(dt), pool.to(dt), bt, pos)]
    sg = torch.tensor(segs, dtype=torch.int32).contiguous()
    lib.check(lib.load_library().mi_op_latent_attn(latent_spec(lib, H, dk, dv, rank, nr, 0, scale), ptr(a[0]), ptr(a[1]), ptr(a[2]), ptr(a[3]), bs, ptr(a[4]), MB,
                                                   ptr(a[5]), ptr(sg), n_seq, T, max_ctx, ptr(out), ldo, f32, path, None))
    torch.cuda.synchronize()
    got = out.cpu().double()
    assert (got[:, H * dv:] == 0).all()
    got = got[:, :H * dv]
    if path == 3:                        # written-out keys: segments of two rows and more
        rows = torch.cat([torch.arange(r0, r0 + n) for r0, n, _, _ in segs if n > 1])
        got, ref = got[rows], ref[rows]
    assert ((got - ref).abs() <= (3e-5 if f32 else 2.5e-2) * (1 + ref.abs())).all(), (got - ref).abs().max()


# ---- router and experts --------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("f32,path", [(1, 1), (0, 1), (0, 2)])
@pytest.mark.parametrize("T,D,E,top,ff,groups,keep", [(1, 64, 8, 3, 96, 2, 1), (5, 120, 9, 3, 22, 3, 2), (33, 100, 64, 8, 40, 8, 4), (70, 256, 12, 5, 48, 4, 2),
                                                      (9, 64, 5, 1, 40, 1, 1), (20, 64, 6, 6, 16, 1, 1), (40, 64, 7, 2, 16, 7, 3), (12, 64, 320, 6, 16, 10, 3)])
def test_grouped_sigmoid_router_and_squared_relu_experts(lib, T, D, E, top, ff, groups, keep, f32, path):
    g = torch.Generator().manual_seed(E + T)
    w, corr = b16(torch.randn(E, D, generator=g) * 1.5 / math.sqrt(D)), b16(0.4 * torch.randn(E, generator=g) - (1.0 if E == 9 else 0.0))
    up, down = b16(torch.randn(E, ff, D, generator=g) / math.sqrt(D)), b16(torch.randn(E, D, ff, generator=g) / math.sqrt(ff))
    x = b16(torch.randn(T, D, generator=g))
    rule = (corr.double(), top, groups, keep)
    for _ in range(200):                      # no close calls
        bad = close_calls(x.double() @ w.double().t(), *rule) < 1e-5
        if not bad.any():
            break
        x[bad] = b16(torch.randn(int(bad.sum()), D, generator=g))
    Kd, ldy = pad(D, 64), pad(D, 16)
    xd = torch.zeros(T, Kd)
    xd[:, :D] = x
    a = [dev(t) for t in (xd.to(torch.float32 if f32 else torch.bfloat16), w, corr, up, down)]
    ids, p = torch.full((T, top), -1, dtype=torch.int32, device="cuda"), torch.zeros(T, top, device="cuda")
    y = torch.zeros(T * top, ldy, device="cuda")
    for _ in range(2):                        # (the second call finds what the first left behind, as a layer's next step does)
        lib.check(lib.load_library().mi_op_experts(ptr(a[0]), Kd, T, D, E, top, ff, ptr(a[1]), ptr(a[2]), None, ptr(a[3]), ptr(a[4]), ptr(ids), ptr(p), ptr(y), ldy,
                                                   groups, keep, f32, path, None))
    torch.cuda.synchronize()
    ref_ids, ref_p = R.pick(x.double() @ w.double().t(), *rule)
    assert torch.equal(ids.cpu().long(), ref_ids)
    assert (p.cpu() - ref_p).abs().max() < 1e-5
    y = y.cpu().double().view(T, top, ldy)[:, :, :D]
    for e in range(E):
        rows, place = (ref_ids == e).nonzero(as_tuple=True)
        if rows.numel():
            h = (x[rows].double() @ up[e].double().t()).clamp(min=0).pow(2)
            ref = (h if f32 else b16(h.float()).double()) @ down[e].double().t()
            assert ((y[rows, place] - ref).abs() <= (2e-5 if f32 else 1.5e-2) * (1 + ref.abs())).all()


def test_router_prefers_the_lower_of_equal_groups_and_experts(lib):
    T, D, E = 3, 64, 72
    a = [dev(t) for t in (torch.ones(T, D).to(torch.bfloat16), torch.zeros(E, D), torch.zeros(E), torch.zeros(E, 16, D), torch.zeros(E, D, 16))]
    for path in (1, 2):
        ids, p = torch.full((T, 5), -1, dtype=torch.int32, device="cuda"), torch.zeros(T, 5, device="cuda")
        y = torch.zeros(T * 5, D, device="cuda")
        lib.check(lib.load_library().mi_op_experts(ptr(a[0]), 64, T, D, E, 5, 16, ptr(a[1]), ptr(a[2]), None, ptr(a[3]), ptr(a[4]), ptr(ids), ptr(p), ptr(y), D,
                                                   18, 2, 0, path, None))
        torch.cuda.synchronize()
        assert ids.cpu().tolist() == [[0, 1, 2, 3, 4]] * T and torch.allclose(p.cpu(), torch.full((T, 5), 0.2))


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("T,D", [(3, 512), (40, 120), (5, 2050), (2, 8192)])
def test_rows_without_a_post_norm(lib, T, D, f32):
    """x += sum of the experts' outputs; norm."""
    torch.manual_seed(D)
    top, ld, ldy = 3, pad(D, 16), pad(D, 64)
    x, y, p, w = torch.randn(T, D), torch.randn(T * top, D), torch.rand(T, top), torch.randn(D)

    def wide(t):
        out = torch.zeros(t.shape[0], ld)
        out[:, :D] = t
        return dev(out)
    a = [wide(x), torch.zeros(T, ld, device="cuda"), wide(y), dev(p), wide(w[None])]
    out = torch.zeros(T, ldy, dtype=torch.float32 if f32 else torch.bfloat16, device="cuda")
    lib.check(lib.load_library().mi_op_sandwich_rows(ptr(a[0]), ptr(a[1]), ptr(a[2]), ptr(a[3]), top, None, ptr(a[4]), T, D, ld, 1, 1e-3, None, 0, None, 0, 16,
                                                     None, 1, None, None, None, 0, ptr(out), ldy, f32, None))
    torch.cuda.synchronize()
    ref_x = x.double() + (p[:, :, None] * y.view(T, top, D)).sum(1).double()
    assert ((a[1].cpu()[:, :D] - ref_x).abs() <= 1e-5 * (1 + ref_x.abs())).all()
    ref = R.rms(ref_x, 1e-3) * w.double()
    assert ((out.cpu().double()[:, :D] - ref).abs() <= (2e-5 if f32 else 1e-2) * (1 + ref.abs())).all()


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
    for n in (1, 2, 15, 16, 17, 130, 300, 420):
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


def test_mixed_batches_over_reused_pages_and_slots(served):
    """Up to four live requests, portions beside single tokens, requests left out of steps and ended; the pool holds far
    fewer tokens than the requests together, and there are four state slots."""
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
    """A pool of exactly one long request: every sequence runs over the pages (and the state slot) of the one before, decoding
    across page borders, with graph replays."""
    cfg, w = case("uneven")
    r = replay(cfg, w, dtype, max_tokens=304, max_live=1)
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
    """Hidden rows beyond one work-group's first pass, 40 requests decoding at once (the grouped experts and the GEMMs), a prompt
    whose output projection leaves a K-split's sum to the next norm."""
    own = [delta(4, 2, 32, 32, 4, moe(6, 2, 48, 2, 1)), latent(3, 32, 32, 64, 48, 32, mlp=moe(4, 1, 32)), latent2(3, 32, 32, 64, 64)]
    cfg = config(2112, 160, own + [dict(own[0], weights_of=0)])
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
    toks = tokens(cfg, w, 700, 5)
    assert error(score(r, toks, [640, 60]), reference("wide", cfg, w, toks, "bfloat16")) <= LIMIT["bfloat16"]
    r.engine.close()


def test_prompts_longer_than_the_factors_memory():
    """More chunks than are kept at a time (512): the scan goes on from the state in its slot."""
    cfg = config(64, 96, [delta(2, 1, 16, 16, 4, moe(4, 2, 16)), delta(2, 2, 16, 32, 2)])
    w = weights(cfg, 4)
    r = replay(cfg, w, "float32", max_tokens=9600, max_live=1)
    toks = tokens(cfg, w, 9000, 1, margin=1e-4)
    rid = uid()
    out = r.step([{"id": rid, "tokens": toks, "want": [10, 8190, 8191, 8192, 8193, 8999]}], [rid])[0]
    ref = R.logits(cfg, w, toks, torch.float64)
    assert error(out, ref[[10, 8190, 8191, 8192, 8193, 8999]]) <= LIMIT["float32"]
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
                       enable_prefix_caching=True, enable_chunked_prefill=chunked,
                       max_num_batched_tokens=48 if chunked else None, override_mi355x_config=override)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10))
    assert [o.token_ids for o in outs] == [greedy(cfg, w, p, 10) for p in prompts]
    assert max(o.num_cached_tokens for o in outs) == 0
    eng.close()


def test_prefix_caching_without_recurrent_layers():
    from vllm_neuron_amd._vllm_compat import SamplingParams
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg = config(96, 150, [latent(3, 16, 16, 40, 24, 8, mlp=moe(4, 2, 24, 2, 1)), latent2(2, 16, 24, 32, 40)])
    w = weights(cfg, 2)
    base = torch.randint(0, 150, (70,), generator=torch.Generator().manual_seed(1)).tolist()
    prompts = [base, base[:64] + [3, 5, 7]]
    eng = MI355XEngine(config_from_dict(cfg), dtype="float32", max_model_len=128, max_num_seqs=2, block_size=16, override_mi355x_config={"state_dict": w})
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=8))
    assert [o.token_ids for o in outs] == [greedy(cfg, w, p, 8) for p in prompts] and outs[1].num_cached_tokens == 64
    eng.close()


def test_graph_replays_equal_eager_steps():
    """Every replay of a captured token-generation step, with eager work of other requests in between, against the same steps
    without graphs."""
    cfg, w = case("wide")
    toks, other = tokens(cfg, w, 60, 3), tokens(cfg, w, 40, 4)
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


def test_speculation_with_recurrent_state_is_refused():
    from types import SimpleNamespace

    from vllm_neuron_amd._vllm_compat import SimpleSpeculativeConfig
    from vllm_neuron_amd.engine import MI355XEngine
    from vllm_neuron_amd.models import config_from_dict
    cfg, w = case("uneven")
    spec = SimpleSpeculativeConfig(num_speculative_tokens=3, draft_model_config=SimpleNamespace(model="", hf_config=config_from_dict(cfg)))
    with pytest.raises(NotImplementedError, match="recurrent state|block KV layout"):
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
    short = {k: v for k, v in w.items() if k != "l0.mlp.e4.down"}
    with pytest.raises(RuntimeError, match="l0.mlp.e4.down"):
        r = replay(cfg, short, "bfloat16")
        r.engine.worker.model_runner.initialize_kv_cache(None)
    with pytest.raises(ValueError, match="shape"):
        replay(cfg, {**w, "l0.mix.q.conv": w["l0.mix.q.conv"][:, :2].contiguous()}, "bfloat16")
    for name in ("l3.norm1", "l2.mlp.router", "l0.mlp.e9.up", "l0.mlp.e1.gate", "l2.mix.a1", "final.norm.b", "pos"):   # a shared layer's; no ff; 9 experts; ...
        with pytest.raises(ValueError, match="not part"):
            replay(cfg, {**w, name: w["l0.norm1"]}, "bfloat16")
    with pytest.raises(NotImplementedError):
        replay(cfg, w, "bfloat16", quantized=True)


def test_state_slots_are_checked():
    """The library refuses a step without state slots, with a slot twice or out of range."""
    cfg, w = case("uneven")
    r = replay(cfg, w, "float32")
    r.step([{"id": "a", "tokens": [1], "want": []}], ["a"])
    native = r.engine.worker.model_runner.model.model
    i = torch.arange(2)
    for seq in (None, [1, 1], [0, 4], [-1, 0]):
        with pytest.raises(ValueError, match="slot"):
            native.forward_rows(i, i * 0, 16 + 16 * i, torch.tensor([[1], [2]]), torch.ones(2), torch.zeros(2), [0],
                                seq_ids=None if seq is None else torch.tensor(seq))
    r.engine.close()


def test_synthetic_weights_run():
    """Random weights made on the device (benchmarks) fill every tensor of the configuration."""
    from vllm_neuron_amd.models import config_from_dict
    from vllm_neuron_amd.replay import TraceReplay
    c = config_from_dict(CASES["uneven"]())
    for layer in c.stack["layers"]:
        if layer["mixer_kind"] == 2:
            layer["decay_rank"] = layer["gate_rank"] = 16
    r = TraceReplay.from_config(c, "bfloat16", 128, override={"synthetic_weights": {"seed": 3, "std": 0.1}})
    out = score(r, list(range(40)), [30] + [1] * 10)
    assert torch.isfinite(out).all() and out.std() > 0.01
    r.engine.close()
