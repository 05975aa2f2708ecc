"""Nusovik on the CPU: configuration reader and registry, the oracle's own mechanisms against hand computations, mistakes planted in
the oracle (to show that the GPU tests' cases would catch them)."""

import json
import math

import pytest
import torch

from oracle import nusovik as R
from tests.nusovik_cases import CASES, ROWS, config, error, left, mamba1, parallel, right, tokens, weights
from vllm_neuron_amd.models import SUPPORTED_ARCHITECTURES, config_from_dict, fill_sizes, has_recurrent_state, load_config, stack_of


def test_config_reader_takes_every_size_from_the_file():
    raw = CASES["uneven"]()
    c = config_from_dict(raw)
    s = stack_of(c)
    assert c.architectures == ["Nusovik"] and "Nusovik" in SUPPORTED_ARCHITECTURES
    assert (s["width"], s["vocab_size"], s["max_positions"], s["norm_eps"], s["embed_scale"], s["logit_scale"], s["pos_base"]) == (122, 203, 0, 0.15, 3.0, 0.7, 1e4)
    m, p, m2, p2 = s["layers"]
    assert (m["ssm_inner"], m["ssm_state"], m["dt_rank"], m["conv_taps"], m["ff_kind"], m["ff_size"]) == (50, 10, 7, 3, 1, 90)
    assert (p["num_heads"], p["num_kv_heads"], p["qk_dim"], p["v_dim"], p["chunk"], p["rel_far"]) == (6, 2, 20, 20, 37, 30.0)
    assert p["scale"] == raw["layers"][1]["mixer"]["left"]["scale"] and (p["mix_mult"], p["beside_mult"]) == (0.8, 1.3)
    assert (p["ssm_heads"], p["ssm_dim"], p["ssm_state"], p["ssm_groups"], p["ssm_parts"], p["conv_taps"]) == (4, 13, 20, 2, 4, 5)
    assert (p["ff_kind"], m2["ff_kind"], p2["ff_size"], m2["ssm_inner"]) == (0, 0, 41, 68)
    assert c.num_hidden_layers == 4 and c.head_dim == 34 and has_recurrent_state(c)


def test_a_model_of_scans_alone():
    c = config_from_dict(config(64, 64, [mamba1(32, 4, 3, 2)]))
    assert has_recurrent_state(c) and c.sizes_from == {} and c.num_key_value_heads == 1 and c.head_dim >= 1


@pytest.mark.parametrize("change", [
    lambda r: r["layers"][0].update(type="mamba2"), lambda r: r["layers"][0]["mixer"].update(conv=0), lambda r: r["layers"][0]["mlp"].update(kind="moe"),
    lambda r: r["layers"][1]["mixer"]["left"].update(kv_heads=4), lambda r: r["layers"][1]["mixer"]["left"].update(vdim=24),
    lambda r: r["layers"][1]["mixer"]["left"]["mask"].update(size=0), lambda r: r["layers"][1]["mixer"]["right"].update(groups=3),
    lambda r: r["layers"][1]["mixer"]["right"].update(norm_groups=5), lambda r: r["layers"][1]["mixer"]["right"].update(conv=0), lambda r: r.update(layers=[])])
def test_config_reader_refuses_what_does_not_fit(change):
    raw = json.loads(json.dumps(CASES["uneven"]()))
    change(raw)
    with pytest.raises(ValueError):
        config_from_dict(raw)


def test_sizes_the_checkpoint_gives(tmp_path):
    from safetensors.torch import save_file

    from vllm_neuron_amd.worker.mi355x_model_loader import _checkpoint_shapes
    cfg = CASES["uneven"]()
    w = weights(cfg, 1, ROWS["uneven"])
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    for source in ({}, {"state_dict": w}):
        c = load_config(str(tmp_path))
        fill_sizes(c, _checkpoint_shapes(str(tmp_path), source))
        assert [x.get("rel_rows") for x in stack_of(c)["layers"]] == [None, 9, None, 6]
    with pytest.raises(ValueError, match="l1.mix.left.rel"):
        fill_sizes(config_from_dict(cfg), {}.get)


def test_native_structs_follow_the_config():
    from vllm_neuron_amd._native import stack_config
    c = config_from_dict(CASES["uneven"]())
    fill_sizes(c, lambda n: (9, 6))
    st = stack_config(dict(stack_of(c), compute_dtype=1))
    assert st.num_layers == 4 and st.block_kind == 3 and st.norm_groups == 1 and st.norm_offset == 0.0 and st.embed_scale == 3.0
    assert st.pos_base == 1e4 and abs(st.logit_scale - 0.7) < 1e-6 and st.layers[1].rel_rows == 9 and st.layers[1].beside_kind == 4
    assert st.layers[0].mixer_kind == 3 and st.layers[0].weights_of == -1 and st.layers[3].keys_as_values == 1 and st.layers[3].softmax_sink == 2


def test_prefix_caching_and_drafts():
    from vllm_neuron_amd._vllm_compat import (SimpleCacheConfig, SimpleDeviceConfig, SimpleModelConfig, SimpleParallelConfig, SimpleSchedulerConfig,
                                              SimpleVllmConfig)
    from vllm_neuron_amd.platform import MI355XPlatform
    from vllm_neuron_amd.worker.mi355x_model_loader import check_draft
    c = config_from_dict(CASES["taps"]())
    cfg = SimpleVllmConfig(model_config=SimpleModelConfig(model="", hf_config=c, max_model_len=128),
                           cache_config=SimpleCacheConfig(block_size=16, enable_prefix_caching=True), parallel_config=SimpleParallelConfig(),
                           scheduler_config=SimpleSchedulerConfig(max_num_seqs=2, max_model_len=128), device_config=SimpleDeviceConfig("cpu"))
    MI355XPlatform.check_and_update_config(cfg)
    assert not cfg.cache_config.enable_prefix_caching
    with pytest.raises(NotImplementedError, match="state"):
        check_draft(stack_of(c))


# ---- the oracle's mechanisms ---------------------------------------------------------------------
def test_sinusoid_by_hand():
    s = R.sinusoid(4, 5, torch.float64)
    for p in range(4):
        want = [f(p * 10000.0 ** (-2 * i / 5)) for i in range(3) for f in (math.sin, math.cos)][:5]
        assert s[p].tolist() == pytest.approx(want)


def test_buckets_by_hand():
    assert [R.bucket(n, 8, 64) for n in (0, 1, 3, 4, 7, 8, 15, 16, 31, 32, 63, 64, 999)] == [0, 1, 3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]
    assert [R.bucket(n, 16, 128) for n in (7, 8, 11, 12, 16, 22, 23, 32, 64, 90, 91)] == [7, 8, 8, 9, 10, 10, 11, 12, 14, 14, 15]
    assert [R.bucket(n, 5, 40) for n in (0, 1, 2, 5, 6, 14, 15, 39, 40)] == [0, 1, 2, 2, 3, 3, 4, 4, 4]
    assert [R.bucket(n, 1, 9) for n in (0, 5, 50)] == [0, 0, 0] and [R.bucket(n, 2, 4) for n in (0, 1, 9)] == [0, 1, 1]


def test_chunk_attention_by_hand():
    """Three chunks of two positions; the bias counts from the distance, the sink once and without a value."""
    k = torch.tensor([1.0, -1.0, 0.5, 2.0, 0.0], dtype=torch.float64).view(5, 1, 1)
    q, v = torch.ones(5, 1, 1, dtype=torch.float64), torch.arange(1.0, 6.0, dtype=torch.float64).view(5, 1, 1)
    rel, sink = torch.tensor([[0.25], [-0.5]], dtype=torch.float64), torch.tensor([0.75], dtype=torch.float64)
    o = R.chunk_attention(q, k, v, 0.5, rel, 2, 2, sink)
    for i in range(5):
        js = range(i // 2 * 2, i + 1)
        e = [math.exp(0.5 * k[j].item() + rel[min(i - j, 1)].item()) for j in js]
        assert o[i].item() == pytest.approx(sum(x * (j + 1) for x, j in zip(e, js)) / (sum(e) + math.exp(0.75)))


def test_short_convolution_by_hand():
    y = R.short_conv(torch.tensor([[1.0], [10.0], [100.0], [1000.0]], dtype=torch.float64), torch.tensor([[4.0, 3.0, 2.0]], dtype=torch.float64),
                     torch.tensor([0.5], dtype=torch.float64))
    z = torch.tensor([2.5, 23.5, 234.5, 2340.5], dtype=torch.float64)
    assert torch.allclose(y.flatten(), z / (1 + torch.exp(-z)))


def test_scans_by_hand():
    x, dt = torch.tensor([[2.0], [3.0]], dtype=torch.float64), torch.tensor([[0.5], [0.25]], dtype=torch.float64)
    b, c = torch.tensor([[1.0, 2.0], [0.5, -1.0]], dtype=torch.float64), torch.tensor([[1.0, 1.0], [2.0, 3.0]], dtype=torch.float64)
    a = torch.tensor([[math.log(2.0), 0.0]], dtype=torch.float64)
    y, S = R.scan1(x, dt, a, b, c, torch.tensor([10.0], dtype=torch.float64))
    s = [1.0, 2.0]
    assert y[0].item() == pytest.approx(3.0 + 20.0)
    s = [s[0] * math.exp(-0.5) + 0.75 * 0.5, s[1] * math.exp(-0.25) - 0.75]
    assert y[1].item() == pytest.approx(2 * s[0] + 3 * s[1] + 30.0) and S.flatten().tolist() == pytest.approx(s)
    y2, S2 = R.scan2(x.view(2, 1, 1), dt, a[0, :1], b.view(2, 1, 2), c.view(2, 1, 2), torch.tensor([10.0], dtype=torch.float64))
    s = [math.exp(-0.5) + 0.375, 2 * math.exp(-0.5) - 0.75]
    assert y2.flatten().tolist() == pytest.approx([23.0, 2 * s[0] + 3 * s[1] + 30.0]) and S2.flatten().tolist() == pytest.approx(s)


def test_gated_norm_by_hand():
    y = R.gated_norm(torch.tensor([[1.0, 2.0, 3.0, 4.0]], dtype=torch.float64), torch.full((1, 4), 50.0, dtype=torch.float64),
                     torch.tensor([1.0, 1.0, 1.0, 2.0], dtype=torch.float64), 2, 0.0)
    assert y.flatten().tolist() == pytest.approx([1 / math.sqrt(2.5), 2 / math.sqrt(2.5), 3 / math.sqrt(12.5), 8 / math.sqrt(12.5)])


@pytest.mark.parametrize("case", list(CASES))
def test_logits_of_a_prefix_do_not_depend_on_what_follows(case):
    cfg = CASES[case]()
    w = weights(cfg, 3, ROWS[case])
    t = tokens(cfg, 60, 1)
    a, b = R.logits(cfg, w, t, torch.float64), R.logits(cfg, w, t[:41], torch.float64)
    assert torch.allclose(a[:41], b, atol=1e-9)


# ---- the GPU tests' cases show a mistake in any mechanism (the mistakes are planted here, in the oracle) -------------
def _mistakes():
    def patch(**kw):
        def run(mp):
            for k, v in kw.items():
                mp.setattr(R, k, v)
        return run
    att, mix, conv, s1, s2, gn, rms, sin, bkt, sp, par = (R.chunk_attention, R.chunk_mixer, R.short_conv, R.scan1, R.scan2, R.gated_norm, R.rms, R.sinusoid, R.bucket,
                                                          R.softplus, R.parallel_mixer)

    def without(*names):                          # chunk_mixer with some tensors zero
        return lambda x, m, w, p, *a: mix(x, m, {**w, **{p + n: 0 * w[p + n] for n in names}}, p, *a)

    def split(f):                                 # the state is lost at 64 (the first six arguments are per token where they have its length)
        def run(*a):
            T = a[0].shape[0]
            parts = [f(*[t[s] if torch.is_tensor(t) and t.dim() > 1 and t.shape[0] == T else t for t in a]) for s in (slice(0, 64), slice(64, T))]
            return torch.cat([parts[0][0], parts[1][0]]), parts[1][1]
        return run

    def cut_conv(x, w, b):
        y = conv(x, w, b)
        y[64:] = conv(x[64:], w, b)
        return y

    def shifted(q, k, v, s, rel, far, size, sink, *a):                     # chunks counted one off
        z = [torch.cat([t[:1], t]) for t in (q, k, v)]
        return att(*z, s, rel, far, size, sink, *a)[1:]

    def normed_values(q, k, v, *a):
        return att(q, k, k, *a)

    def scaled_bias(q, k, v, s, rel, *a):
        return att(q, k, v, s, rel * s, *a)

    def scaled_sink(q, k, v, s, rel, far, size, sink, *a):
        return att(q, k, v, s, rel, far, size, sink * s, *a)

    def read_first(x, dt, a_log, b, c, d, state=None):                     # the write of a token is dt x B
        y, S = s1(x, dt, a_log, b, c, d)
        return y - dt * x * (b * c).sum(-1, keepdim=True), S
    return {
        "no positions": patch(sinusoid=lambda T, D, dt, first=0: torch.zeros(T, D, dtype=dt)), "positions start at one": patch(sinusoid=lambda T, D, dt, first=0: sin(T, D, dt, 1)),
        "sine and cosine in halves": patch(sinusoid=lambda T, D, dt, first=0: torch.cat([sin(T, D, dt)[:, ::2], sin(T, D, dt)[:, 1::2]], -1)),
        "no chunks": patch(chunk_attention=lambda q, k, v, s, rel, far, size, *a: att(q, k, v, s, rel, far, 10 ** 6, *a)),
        "chunks one larger": patch(chunk_attention=lambda q, k, v, s, rel, far, size, *a: att(q, k, v, s, rel, far, size + 1, *a)),
        "chunks one off": patch(chunk_attention=shifted), "values normed": patch(chunk_attention=normed_values), "scale on the bias": patch(chunk_attention=scaled_bias),
        "scale on the sink": patch(chunk_attention=scaled_sink), "scale left out": patch(chunk_attention=lambda q, k, v, s, *a: att(q, k, v, 1.0, *a)),
        "no sink": patch(chunk_attention=lambda q, k, v, s, rel, far, size, sink, *a: att(q, k, v, s, rel, far, size, sink - 50, *a)),
        "a sink of score zero": patch(chunk_attention=lambda q, k, v, s, rel, far, size, sink, *a: att(q, k, v, s, rel, far, size, 0 * sink, *a)),
        "no bias": patch(chunk_mixer=without("rel")), "buckets without a logarithm": patch(bucket=lambda n, rows, far: min(n, rows - 1)),
        "distances one off": patch(bucket=lambda n, rows, far: bkt(n + 1, rows, far)), "buckets reach twice as far": patch(bucket=lambda n, rows, far: bkt(n, rows, 2 * far)),
        "query bias left out": patch(chunk_mixer=without("q.b")), "key bias left out": patch(chunk_mixer=without("k.b")), "no output gate": patch(chunk_mixer=without("g")),
        "norm weights around zero": patch(chunk_mixer=lambda x, m, w, p, *a: mix(x, m, {**w, p + "q.norm": w[p + "q.norm"] + 1, p + "k.norm": w[p + "k.norm"] + 1}, p, *a)),
        "queries and keys not normed": patch(rms=lambda x, e: x if x.dim() == 3 and x.shape[-1] in (20, 34) else rms(x, e)),
        "key heads in the wrong order": patch(chunk_attention=lambda q, k, v, *a: att(q, k.flip(1), v.flip(1), *a)),
        "convolution reversed": patch(short_conv=lambda x, w, b: conv(x, w.flip(1), b)), "convolution bias left out": patch(short_conv=lambda x, w, b: conv(x, w, 0 * b)),
        "no activation behind the convolution": patch(short_conv=lambda x, w, b: _linear_conv(x, w, b)), "convolution state lost at 64": patch(short_conv=cut_conv),
        "step size without softplus": patch(softplus=lambda z: z.clamp(min=0)), "selective scan's state lost at 64": patch(scan1=split(s1)), "matrix state lost at 64": patch(scan2=split(s2)),
        "one decay per channel": patch(scan1=lambda x, dt, a, *r: s1(x, dt, a.mean(-1, keepdim=True).expand_as(a), *r)),
        "no decay": patch(scan1=lambda x, dt, a, *r: s1(x, dt, a - 50, *r)), "no decay of the matrices": patch(scan2=lambda x, dt, a, *r: s2(x, dt, a - 50, *r)),
        "input not scaled by the step": patch(scan1=lambda x, dt, a, b, c, d, s=None: s1(x, dt, a, b / dt.mean(-1, keepdim=True), c, d)),
        "read-out ahead of the write": patch(scan1=read_first), "skip left out": patch(scan1=lambda x, dt, a, b, c, d, s=None: s1(x, dt, a, b, c, 0 * d)),
        "skip of the matrices left out": patch(scan2=lambda x, dt, a, b, c, d, s=None: s2(x, dt, a, b, c, 0 * d)),
        "B and C exchanged": patch(scan1=lambda x, dt, a, b, c, d, s=None: s1(x, dt, a, c, b, d)), "B and C of the matrices exchanged": patch(scan2=lambda x, dt, a, b, c, d, s=None: s2(x, dt, a, c, b, d)),
        "groups in the wrong order": patch(scan2=lambda x, dt, a, b, c, d, s=None: s2(x, dt, a, b.flip(1), c.flip(1), d)),
        "gate behind the norm": patch(gated_norm=lambda y, z, w, parts, e: gn(y, 50 + 0 * z, w, parts, e) * z * torch.sigmoid(z)),
        "norm over the whole row": patch(gated_norm=lambda y, z, w, parts, e: gn(y, z, w, 1, e)), "no gate ahead of the norm": patch(gated_norm=lambda y, z, w, *a: gn(y, 50 + 0 * z, w, *a)),
        "eps left out": patch(rms=lambda x, e: rms(x, 1e-12)),
        "left scale left out": patch(parallel_mixer=lambda h, m, *a: par(h, {**m, "left_scale": 1.0}, *a)),
        "right scale left out": patch(parallel_mixer=lambda h, m, *a: par(h, {**m, "right_scale": 1.0}, *a)),
        "relu not squared": patch(dense_ff=lambda h, w, p, r=None: (h @ w[p + "up"].t()).clamp(min=0) @ w[p + "down"].t()),
    }


def _linear_conv(x, w, b):
    y = torch.zeros_like(x) + b
    for j in range(w.shape[1]):
        back = w.shape[1] - 1 - j
        y[back:] += w[:, j] * x[:x.shape[0] - back]
    return y


@pytest.fixture(scope="module")
def good():
    cfg = CASES["uneven"]()
    w = weights(cfg, 11, ROWS["uneven"])
    t = tokens(cfg, 130, 130)
    return cfg, w, t, R.logits(cfg, w, t)


@pytest.mark.parametrize("mistake", list(_mistakes()))
def test_cases_show_a_planted_mistake(mistake, monkeypatch, good):
    from tests.test_nusovik_gpu import LIMIT
    cfg, w, t, good = good
    _mistakes()[mistake](monkeypatch)
    assert error(R.logits(cfg, w, t), good) > 2 * LIMIT["bfloat16"]


@pytest.mark.parametrize("change", [lambda c, w: c["embedding"].update(scale=2.5), lambda c, w: w.update({"l0.norm1": w["l0.norm1"] + 1}), lambda c, w: c.update(logit_scale=0.8),
                                    lambda c, w: w.update({"l3.norm2": w["l3.norm2"] * 0 + 1}), lambda c, w: w.update({"final.norm": w["final.norm"] + 1})])
def test_cases_show_a_wrong_constant(change, good):
    from tests.test_nusovik_gpu import LIMIT
    cfg, w, t, good = good
    cfg, w = json.loads(json.dumps(cfg)), dict(w)
    change(cfg, w)
    assert error(R.logits(cfg, w, t), good) > 2 * LIMIT["bfloat16"]
