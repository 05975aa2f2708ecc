"""Vimesun on the CPU: configuration reader and registry, the oracle's own mechanisms against hand computations,
streaming input and request ends in the scheduler."""

import math

import pytest
import torch

from oracle import vimesun as V
from tests.vimesun_cases import CASES, att, config, error, tokens, weights
from vllm_neuron_amd.models import SUPPORTED_ARCHITECTURES, config_from_dict, load_config, stack_of


def test_config_reader_takes_every_size_from_the_file():
    raw = CASES["uneven"]()
    c = config_from_dict(raw)
    s = stack_of(c)
    assert c.architectures == ["Vimesun"] and "Vimesun" in SUPPORTED_ARCHITECTURES
    assert (s["width"], s["vocab_size"], s["max_positions"]) == (100, 203, 640)
    assert (s["loop_start"], s["loop_stop"], s["loop_times"]) == (1, 3, 3)
    assert s["residual_mult"] == 0.45 and s["norm_eps"] == 1e-2
    l0, l1 = s["layers"][0], s["layers"][1]
    assert (l0["num_heads"], l0["num_kv_heads"], l0["qk_dim"], l0["v_dim"], l0["window"], l0["ff_size"]) == (6, 2, 20, 26, 37, 90)
    assert l0["scale"] == raw["layers"][0]["mixer"]["scale"] and l0["ff_kind"] == 1
    assert l1["ff_kind"] == 0 and l1["ff_size"] == 0
    assert c.num_hidden_layers == 1 + 2 * 3 and c.vocab_size == 203


def test_config_reader_without_loop_and_from_a_folder(tmp_path):
    import json
    raw = CASES["plain"]()
    (tmp_path / "config.json").write_text(json.dumps(raw))
    c = load_config(str(tmp_path))
    assert stack_of(c)["loop_times"] == 0 and c.num_hidden_layers == 3
    raw["loop"] = None
    assert stack_of(config_from_dict(raw))["loop_times"] == 0


@pytest.mark.parametrize("change", [
    lambda r: r["layers"][0].update(type="recurrent"), lambda r: r["layers"][0]["mixer"].update(kv_heads=5),
    lambda r: r["layers"][0]["mlp"].update(kind="experts"), lambda r: r.update(loop={"start": 2, "stop": 9, "times": 2}),
    lambda r: r["layers"][0]["mixer"]["mask"].update(size=0), lambda r: r.update(architecture="Other")])
def test_config_reader_refuses_what_it_does_not_know(change):
    raw = CASES["uneven"]()
    change(raw)
    with pytest.raises(ValueError):
        config_from_dict(raw)


def test_llama_family_configs_have_no_stack():
    c = config_from_dict({"architectures": ["LlamaForCausalLM"], "vocab_size": 7})
    assert stack_of(c) is None and c.vocab_size == 7


def test_native_structs_follow_the_config():
    from vllm_neuron_amd._native import stack_config
    st = stack_config(dict(stack_of(config_from_dict(CASES["wide"]())), compute_dtype=1))
    assert st.num_layers == 2 and st.layers[1].num_heads == 24 and st.layers[1].window == 100 and st.compute_dtype == 1
    with pytest.raises(ValueError):
        stack_config({"layers": [{"heads": 1}]})


# ---- the oracle's mechanisms ---------------------------------------------------------------------
def test_layer_norm_takes_the_mean_off():
    x = torch.randn(5, 12, dtype=torch.float64) + 3
    w, b = torch.randn(12, dtype=torch.float64), torch.randn(12, dtype=torch.float64)
    ref = torch.nn.functional.layer_norm(x, (12,), w, b, 1e-3)
    assert torch.allclose(V.layer_norm(x, w, b, 1e-3), ref, atol=1e-12)


def test_slopes():
    assert V.slopes(4).tolist() == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]
    assert V.slopes(6)[0].item() == pytest.approx(2 ** (-8 / 6))


def test_window_edges_bias_and_sink_by_hand():
    T, W = 6, 3
    q = torch.zeros(T, 1, 2, dtype=torch.float64)
    k = torch.zeros(T, 1, 2, dtype=torch.float64)
    v = torch.eye(T, dtype=torch.float64)[:, None, :]
    slope = torch.tensor([0.25], dtype=torch.float64)
    o = V.window_attention(q, k, v, 1.0, W, slope)
    for i in range(T):
        e = {j: math.exp(-0.25 * (i - j)) for j in range(max(0, i - W + 1), i + 1)}
        den = 1 + sum(e.values())
        want = torch.tensor([e.get(j, 0.0) / den for j in range(T)], dtype=torch.float64)
        assert torch.allclose(o[i, 0], want, atol=1e-14)
    # without a sink the weights add up to one
    assert torch.allclose(V.window_attention(q, k, v, 1.0, W, slope, sink=False).sum(-1), torch.ones(T, 1, dtype=torch.float64))


def test_sink_holds_for_scores_far_below_zero():
    q = torch.full((1, 1, 1), 10.0)
    o = V.window_attention(q, -q, torch.ones(1, 1, 1), 1.0, 4)
    assert o.item() == pytest.approx(math.exp(-100), rel=1e-4)


def test_loop_order():
    cfg = config(8, 8, [att(1, 1, 4, 4, 4)] * 4, loop=(1, 3, 2))
    assert V.layer_runs(cfg) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    cfg["loop"]["times"] = 1
    assert [f for _, f in V.layer_runs(cfg)] == [False, True, False, False]


def test_logits_of_a_prefix_do_not_depend_on_what_follows():
    cfg = CASES["uneven"]()
    w, t = weights(cfg, 3), tokens(cfg, 60, 1)
    a, b = V.logits(cfg, w, t, torch.float64), V.logits(cfg, w, t[:41], torch.float64)
    assert torch.allclose(a[:41], b, atol=1e-10)


# ---- scheduler: streaming input, ends from outside ---------------------------------------------------
def _scheduler(num_blocks=9, block=16):
    from vllm_neuron_amd._vllm_compat import (KVCacheConfig, Scheduler, SimpleCacheConfig, SimpleSchedulerConfig,
                                              SimpleVllmConfig)
    cfg = SimpleVllmConfig(None, SimpleCacheConfig(block, None, False), scheduler_config=SimpleSchedulerConfig(
        4, 256, 128, chunked_prefill_enabled=True))
    return Scheduler(cfg, KVCacheConfig(num_blocks))


def test_streamed_request_is_scheduled_again_only_when_it_has_input():
    from vllm_neuron_amd._vllm_compat import ModelRunnerOutput, Request, SamplingParams
    s = _scheduler()
    s.add_request(Request("a", [1] * 20, SamplingParams()))

    def run(out):
        ids = list(out.num_scheduled_tokens)
        s.update_from_output(out, ModelRunnerOutput(ids, {r: i for i, r in enumerate(ids)}, [[] for _ in ids]))
        return out.num_scheduled_tokens
    assert run(s.schedule()) == {"a": 20}
    assert run(s.schedule()) == {}
    s.requests["a"].prompt_token_ids.extend([2] * 13)
    out = s.schedule()
    assert out.scheduled_cached_reqs.num_computed_tokens == [20] and out.scheduled_cached_reqs.new_block_ids[0] == ([3],)
    assert run(out) == {"a": 13}


def test_finish_requests_gives_the_blocks_back():
    from vllm_neuron_amd._vllm_compat import Request, SamplingParams
    s = _scheduler()
    free = s.block_pool.num_free()
    s.add_request(Request("a", [1] * 40, SamplingParams()))
    s.add_request(Request("b", [1] * 200, SamplingParams()))
    s.schedule()
    assert s.block_pool.num_free() < free
    s.finish_requests(["a", "b", "unknown"])
    assert s.block_pool.num_free() == free and not s.has_unfinished_requests()
    assert "a" in s.schedule().finished_req_ids


# ---- the GPU tests' cases show a mistake in any mechanism (the mistakes are planted here, in the oracle) -------------
def _mistakes():
    def patch(**kw):
        def run(mp):
            for k, v in kw.items():
                mp.setattr(V, k, v)
        return run
    attn, ff = V.window_attention, V.squared_relu_ff

    def window(d):
        return patch(window_attention=lambda q, k, v, sc, w, sl=None, sink=True: attn(q, k, v, sc, max(w + d, 1), sl, sink))
    return {
        "window one longer": window(1), "window one shorter": window(-1),
        "no window": patch(window_attention=lambda q, k, v, sc, w, sl=None, sink=True: attn(q, k, v, sc, 1 << 30, sl, sink)),
        "no sink": patch(window_attention=lambda q, k, v, sc, w, sl=None, sink=True: attn(q, k, v, sc, w, sl, False)),
        "no bias": patch(window_attention=lambda q, k, v, sc, w, sl=None, sink=True: attn(q, k, v, sc, w, None, sink)),
        "slopes from head 0": patch(slopes=lambda h, dt=torch.float32: torch.tensor([2.0 ** (-8.0 * i / h) for i in range(h)], dtype=dt)),
        "no unit norm": patch(unit_rms=lambda x, e: x),
        "norm without the mean": patch(layer_norm=lambda x, w, b, e: x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + e) * w + b),
        "norm without the bias": patch(layer_norm=lambda x, w, b, e, f=V.layer_norm: f(x, w, 0 * b, e)),
        "relu not squared": patch(squared_relu_ff=lambda x, u, d, r=None: torch.relu(x @ u.t()) @ d.t()),
        "positions off by one": patch(embedding=lambda t, e, p: e[t] + p[1:t.shape[0] + 1]),
        "loop input swapped": patch(loop_input=lambda x, e, w, r=None: torch.cat([e, x], -1) @ w.t()),
        "no loop": patch(layer_runs=lambda c: [(i, False) for i in range(len(c["layers"]))]),
        "feed-forward after the mixer": patch(layer=_sequential_layer),
        "residual multiplier left out": patch(layer=lambda x, i, c, w, r, f=V.layer: f(x, i, {**c, "residual_mult": 1.0}, w, r)),
    }


def _sequential_layer(x, i, cfg, w, r):
    import copy
    alone = copy.deepcopy(cfg)
    alone["layers"][i]["mlp"] = None
    y, full = V_layer(x, i, alone, w, r), cfg["layers"][i]["mlp"]
    if full is None:
        return y
    p = f"l{i}."
    b = V.layer_norm(y, w[p + "norm2"], w[p + "norm2.b"], cfg["norm"]["eps"])
    return y + cfg["residual_mult"] * V.squared_relu_ff(b, w[p + "mlp.up"], w[p + "mlp.down"], r)


V_layer = V.layer


@pytest.mark.parametrize("mistake", list(_mistakes()))
def test_cases_show_a_planted_mistake(mistake, monkeypatch):
    from tests.test_vimesun_gpu import LIMIT
    cfg = CASES["uneven"]()
    w, t = weights(cfg, 11), tokens(cfg, 130, 130)
    good = V.logits(cfg, w, t)
    _mistakes()[mistake](monkeypatch)
    assert error(V.logits(cfg, w, t), good) > 2 * LIMIT["bfloat16"]
