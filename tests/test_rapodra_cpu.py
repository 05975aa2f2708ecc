"""Rapodra on the CPU: configuration reader and registry, the oracle's own mechanisms against hand computations, mistakes
planted in the oracle (to show that the GPU tests' cases would catch them)."""

import math

import pytest
import torch

from oracle import rapodra as R
from tests.rapodra_cases import CASES, config, dense, error, latent, moe, tokens, weights
from vllm_neuron_amd.models import SUPPORTED_ARCHITECTURES, config_from_dict, load_config, stack_of


def test_config_reader_takes_every_size_from_the_file():
    raw = CASES["uneven"]()
    c = config_from_dict(raw)
    s = stack_of(c)
    assert c.architectures == ["Rapodra"] and "Rapodra" in SUPPORTED_ARCHITECTURES
    assert (s["width"], s["vocab_size"], s["max_positions"], s["norm_groups"], s["conv_taps"]) == (120, 203, 0, 3, 3)
    assert s["norm_eps"] == 1e-2 and s["logit_softcap"] == 5.0
    l0, l1, l2, l3 = s["layers"]
    assert (l0["num_heads"], l0["qk_dim"], l0["v_dim"], l0["kv_rank"], l0["window"], l0["ff_size"]) == (3, 20, 26, 36, 37, 90)
    assert l0["scale"] == raw["layers"][0]["mixer"]["scale"] and l0["ff_limit"] == 0.8 and l0["ff_alpha"] == 1.702
    assert l0["kv_from"] == -1 and l1["kv_from"] == 0 and l1["ff_kind"] == 0
    assert (l2["experts"], l2["experts_top"], l2["ff_size"]) == (7, 3, 22) and l3["kv_from"] == 2
    assert c.num_hidden_layers == 4 and c.vocab_size == 203


def test_config_from_a_folder(tmp_path):
    import json
    (tmp_path / "config.json").write_text(json.dumps(CASES["wide"]()))
    c = load_config(str(tmp_path))
    assert stack_of(c)["conv_taps"] == 1 and c.num_hidden_layers == 3 and c.max_position_embeddings >= 1 << 16


@pytest.mark.parametrize("change", [
    lambda r: r["layers"][0].update(type="attention"), lambda r: r["layers"][1]["mixer"].update(kv_from=1),
    lambda r: r["layers"][1]["mixer"].update(kv_from=3), lambda r: r["layers"][1]["mixer"].update(kv_rank=32),
    lambda r: r["layers"][3]["mixer"].update(kv_from=1, kv_rank=36), lambda r: r["layers"][0]["mlp"].update(kind="relu"),
    lambda r: r["layers"][2]["mlp"]["router"].update(top=8), lambda r: r["layers"][0]["mixer"]["mask"].update(size=0),
    lambda r: r["norm"].update(groups=7), lambda r: r["canon"].update(taps=0), lambda r: r.update(logit_softcap=0)])
def test_config_reader_refuses_what_does_not_fit(change):
    raw = CASES["uneven"]()
    change(raw)
    with pytest.raises(ValueError):
        config_from_dict(raw)


def test_native_structs_follow_the_config():
    from vllm_neuron_amd._native import stack_config
    st = stack_config(dict(stack_of(config_from_dict(CASES["uneven"]())), compute_dtype=1))
    assert st.num_layers == 4 and st.block_kind == 1 and st.norm_groups == 3 and st.conv_taps == 3
    assert st.layers[3].kv_from == 2 and st.layers[2].experts == 7 and st.layers[0].kv_from == -1


# ---- the oracle's mechanisms ---------------------------------------------------------------------
def test_group_rms_by_hand():
    x = torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=torch.float64)
    w = torch.tensor([1.0, 2.0, 1.0, 10.0], dtype=torch.float64)
    a, b = math.sqrt(12.5 + 0.5), math.sqrt(2 + 0.5)
    assert torch.allclose(R.group_rms(x, w, 2, 0.5), torch.tensor([[3 / a, 8 / a, 0, 20 / b]], dtype=torch.float64), atol=1e-14)


def test_causal_convolution_by_hand():
    h = torch.tensor([[1.0], [10.0], [100.0], [1000.0]])
    w = torch.tensor([[4.0, 3.0, 2.0]])            # the last column meets the token itself
    assert R.causal_conv(h, w).flatten().tolist() == [2.0, 23.0, 234.0, 2340.0]


def test_latent_attention_window_and_heads_by_hand():
    T, W = 6, 3
    c = torch.eye(T, dtype=torch.float64)
    q = torch.zeros(T, 2, 1, dtype=torch.float64)
    q[:, 1] = 1.0
    uk = torch.zeros(2, T, dtype=torch.float64)
    uk[1] = torch.arange(T)                           # head 1: the score of key j is j
    uv = torch.arange(2 * T, dtype=torch.float64).reshape(2, T)
    o = R.latent_attention(q, c, uk, uv, 1.0, W)
    for i in range(T):
        js = list(range(max(0, i - W + 1), i + 1))
        assert o[i, 0].item() == pytest.approx(sum(js) / len(js))
        z = sum(math.exp(j) for j in js)
        assert o[i, 1].item() == pytest.approx(sum(math.exp(j) * (T + j) for j in js) / z)


def test_clipped_gated_unit_by_hand():
    one = torch.ones(1, 1)
    for h, g, u in ((3.0, 1.5, 1.5), (-4.0, -4.0, -1.5), (0.5, 0.5, 0.5)):
        y = R.clipped_glu_ff(torch.tensor([[h]]), one, one, one, 1.5)
        assert y.item() == pytest.approx(g / (1 + math.exp(-1.702 * g)) * (u + 1), rel=1e-5)


def test_router_takes_the_largest_and_weighs_only_them():
    idx, p = R.route(torch.tensor([[1.0]]), torch.tensor([[1.0], [5.0], [2.0], [0.0]]), torch.tensor([0.0, -10.0, 0.0, 1.5]), 2)
    assert idx.tolist() == [[2, 3]]
    e = math.exp(1.5 - 2.0)
    assert p.flatten().tolist() == pytest.approx([1 / (1 + e), e / (1 + e)])


def test_softcap():
    assert R.softcap(torch.tensor([0.0, 100.0, -3.0]), 3.0).tolist() == pytest.approx([0.0, 3.0, -3 * math.tanh(1)])


@pytest.mark.parametrize("case", list(CASES))
def test_logits_of_a_prefix_do_not_depend_on_what_follows(case):
    cfg = CASES[case]()
    w = weights(cfg, 3)
    t = tokens(cfg, w, 60, 1)
    a, b = R.logits(cfg, w, t, torch.float64), R.logits(cfg, w, t[:41], torch.float64)
    assert torch.allclose(a[:41], b, atol=1e-9)


def test_a_draft_with_convolution_state_is_refused():
    from vllm_neuron_amd.worker.mi355x_model_loader import check_draft
    with pytest.raises(NotImplementedError, match="convolution"):
        check_draft(stack_of(config_from_dict(CASES["uneven"]())))
    check_draft(None)
    check_draft(stack_of(config_from_dict(CASES["wide"]())))      # one tap: no state


# ---- the GPU tests' cases show a mistake in any mechanism (the mistakes are planted here, in the oracle) -------------
def _mistakes():
    def patch(**kw):
        def run(mp):
            for k, v in kw.items():
                mp.setattr(R, k, v)
        return run
    attn, conv, rms, glu, route = R.latent_attention, R.causal_conv, R.group_rms, R.clipped_glu_ff, R.route

    def window(d):
        return patch(latent_attention=lambda q, c, k, v, s, w, r=None: attn(q, c, k, v, s, max(w + d, 1), r))

    def no_past(h, w, upto):                          # the inputs ahead of position `upto` are lost (a portion starts there)
        y = conv(h, w)
        y[upto:] = conv(h[upto:], w)
        return y
    return {
        "window one longer": window(1), "window one shorter": window(-1), "no window": window(1 << 30),
        "scale left out": patch(latent_attention=lambda q, c, k, v, s, w, r=None: attn(q, c, k, v, 1.0, w, r)),
        "latent not normed": patch(group_rms=lambda x, w, g, e: x * w if x.shape[-1] in (36, 50) else rms(x, w, g, e)),
        "norm over the whole row": patch(group_rms=lambda x, w, g, e: rms(x, w, 1, e)),
        "eps left out": patch(group_rms=lambda x, w, g, e: rms(x, w, g, 1e-12)),
        "no convolution": patch(causal_conv=lambda h, w: 0 * h),
        "convolution reversed": patch(causal_conv=lambda h, w: conv(h, w.flip(1))),
        "convolution state lost at 64": patch(causal_conv=lambda h, w: no_past(h, w, 64)),
        "convolution without the token itself": patch(causal_conv=lambda h, w: conv(h, torch.cat([w[:, :-1], 0 * w[:, -1:]], 1))),
        "gate not clipped": patch(clipped_glu_ff=lambda h, g, u, d, lim, r=None: _glu(h, g, u, d, 1e9, lim)),
        "up branch not clipped": patch(clipped_glu_ff=lambda h, g, u, d, lim, r=None: _glu(h, g, u, d, lim, 1e9)),
        "one not added": patch(clipped_glu_ff=lambda h, g, u, d, lim, r=None: _glu(h, g, u, d, lim, lim, 0.0)),
        "router bias left out": patch(route=lambda h, w, b, top: route(h, w, 0 * b, top)),
        "experts' weights squared": patch(route=_squared_weights),
        "no softcap": patch(softcap=lambda z, cap: z),
    }


def _glu(h, gate, up, down, lim_g, lim_u, one=1.0):
    g, u = (h @ gate.t()).clamp(max=lim_g), (h @ up.t()).clamp(-lim_u, lim_u)
    return (g * torch.sigmoid(1.702 * g) * (u + one)) @ down.t()


def _squared_weights(h, w, b, top):
    # (a factor common to a row's weights, as from a softmax over all experts, is taken out by the post-norm)
    val, idx = torch.softmax(h @ w.t() + b, -1).topk(top, -1)
    return idx, val.pow(2) / val.pow(2).sum(-1, keepdim=True)


@pytest.mark.parametrize("mistake", list(_mistakes()))
def test_cases_show_a_planted_mistake(mistake, monkeypatch):
    from tests.test_rapodra_gpu import LIMIT
    cfg = CASES["uneven"]()
    w = weights(cfg, 11)
    t = tokens(cfg, w, 130, 130)
    good = R.logits(cfg, w, t)
    _mistakes()[mistake](monkeypatch)
    assert error(R.logits(cfg, w, t), good) > 2 * LIMIT["bfloat16"]


@pytest.mark.parametrize("j", [0, 2])
def test_a_layer_reads_the_latents_it_names(j):
    """kv_from pointed at the other layer of the same rank changes the logits."""
    cfg = config(64, 64, [latent(2, 16, 16, 32, 40, dense(64)), latent(2, 16, 16, 32, 40, moe(4, 2, 16)), latent(2, 16, 16, 32, 40),
                          latent(2, 16, 16, 32, 40, dense(64), kv_from=1)], groups=2)
    w = weights(cfg, 5)
    t = tokens(cfg, w, 50, 1)
    good = R.logits(cfg, w, t)
    cfg["layers"][3]["mixer"]["kv_from"] = j
    assert error(R.logits(cfg, w, t), good) > 0.1
