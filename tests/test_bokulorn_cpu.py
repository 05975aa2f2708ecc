"""Bokulorn on the CPU: configuration reader and registry, state slots of the runner, the oracle's own mechanisms against hand
computations, mistakes planted in the oracle (to show that the GPU tests' cases would catch them)."""

import json
import math
from types import SimpleNamespace

import pytest
import torch

from oracle import bokulorn as R
from tests.bokulorn_cases import CASES, again, config, delta, error, latent, latent2, moe, tokens, weights
from vllm_neuron_amd.models import SUPPORTED_ARCHITECTURES, config_from_dict, fill_sizes, has_recurrent_state, load_config, stack_of


def test_config_reader_takes_every_size_from_the_file():
    raw = CASES["uneven"]()
    c = config_from_dict(raw)
    s = stack_of(c)
    assert c.architectures == ["Bokulorn"] and "Bokulorn" in SUPPORTED_ARCHITECTURES
    assert (s["width"], s["vocab_size"], s["max_positions"], s["norm_eps"], s["embed_scale"], s["norm_offset"]) == (120, 203, 0, 1e-2, 3.0, 1.0)
    d, a, b = s["layers"][:3]
    assert (d["num_heads"], d["num_kv_heads"], d["qk_dim"], d["v_dim"], d["conv_taps"]) == (6, 2, 20, 13, 3)
    assert (d["experts"], d["experts_top"], d["ff_size"], d["router_groups"], d["router_keep"]) == (9, 3, 22, 3, 2)
    assert (a["num_heads"], a["qk_dim"], a["v_dim"], a["kv_rank"], a["q_rank"], a["rot_dim"], a["rot_dims"], a["rot_base"]) == (3, 20, 26, 36, 28, 12, 8, 500.0)
    assert a["scale"] == raw["layers"][1]["mixer"]["scale"] and a["out_gate"] == 1 and b["out_gate"] == 2 and b.get("rot_dim", 0) == 0
    assert b["ff_kind"] == 0 and [x["weights_of"] for x in s["layers"]] == [-1, -1, -1, 0, 1, 2]
    assert c.num_hidden_layers == 6 and c.head_dim == 25 and has_recurrent_state(c)


def test_shared_layers_resolve_to_the_layer_with_tensors():
    own = [latent2(2, 8, 8, 32, 16, moe(4, 2, 16))]
    layers = own + [again(own, 0)]
    layers.append(dict(layers[1], weights_of=1))
    c = config_from_dict(config(64, 64, layers))
    assert [x["weights_of"] for x in stack_of(c)["layers"]] == [-1, 0, 0] and not has_recurrent_state(c)
    assert [x["weights_of"] for x in stack_of(config_from_dict(CASES["taps"]()))["layers"]] == [-1, 3, -1, -1]


@pytest.mark.parametrize("change", [
    lambda r: r["layers"][0].update(type="attention"), lambda r: r["layers"][0]["mixer"].update(kv_heads=4),
    lambda r: r["layers"][0]["mixer"].update(conv=0), lambda r: r["layers"][3].update(weights_of=3), lambda r: r["layers"][3].update(weights_of=6),
    lambda r: r["layers"][3].update(weights_of=1), lambda r: r["layers"][0].update(weights_of=3), lambda r: r["layers"][1]["mixer"]["rot"].update(dims=14),
    lambda r: r["layers"][1]["mixer"]["rot"].update(dims=7), lambda r: r["layers"][0]["mlp"].update(kind="dense"),
    lambda r: r["layers"][0]["mlp"]["router"].update(top=7), lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(count=4),
    lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(keep=4), lambda r: r["layers"][2]["mixer"].update(q_rank=0), lambda r: r.update(layers=[])])
def test_config_reader_refuses_what_does_not_fit(change):
    raw = json.loads(json.dumps(CASES["uneven"]()))
    change(raw)
    with pytest.raises(ValueError):
        config_from_dict(raw)


def test_sizes_the_checkpoint_gives(tmp_path):
    from safetensors.torch import save_file

    from vllm_neuron_amd.worker.mi355x_model_loader import _checkpoint_shapes
    cfg = CASES["uneven"]()
    w = weights(cfg, 1)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    for source in ({}, {"state_dict": w}):
        c = load_config(str(tmp_path))
        fill_sizes(c, _checkpoint_shapes(str(tmp_path), source))
        assert [(x.get("decay_rank"), x.get("gate_rank")) for x in stack_of(c)["layers"]] == [(10, 15), (None, None), (None, None), (10, 15), (None, None), (None, None)]
    with pytest.raises(ValueError, match="l0.mix.a1"):
        fill_sizes(config_from_dict(cfg), {}.get)


def test_native_structs_follow_the_config():
    from vllm_neuron_amd._native import stack_config
    c = config_from_dict(CASES["uneven"]())
    fill_sizes(c, lambda n: (11, 120))
    st = stack_config(dict(stack_of(c), compute_dtype=1))
    assert st.num_layers == 6 and st.block_kind == 2 and st.norm_groups == 1 and st.norm_offset == 1.0 and st.embed_scale == 3.0
    assert st.layers[3].weights_of == 0 and st.layers[0].decay_rank == 11 and st.layers[1].rot_dims == 8 and st.layers[0].router_keep == 2


def test_prefix_caching_is_switched_off_for_recurrent_models():
    from vllm_neuron_amd._vllm_compat import (SimpleCacheConfig, SimpleDeviceConfig, SimpleModelConfig, SimpleParallelConfig, SimpleSchedulerConfig,
                                              SimpleVllmConfig)
    from vllm_neuron_amd.platform import MI355XPlatform

    def after(raw):
        cfg = SimpleVllmConfig(model_config=SimpleModelConfig(model="", hf_config=config_from_dict(raw), max_model_len=128),
                               cache_config=SimpleCacheConfig(block_size=16, enable_prefix_caching=True), parallel_config=SimpleParallelConfig(),
                               scheduler_config=SimpleSchedulerConfig(max_num_seqs=2, max_model_len=128), device_config=SimpleDeviceConfig("cpu"))
        MI355XPlatform.check_and_update_config(cfg)
        return cfg.cache_config.enable_prefix_caching
    assert not after(CASES["uneven"]())
    assert after(config(64, 64, [latent2(2, 8, 8, 32, 16)]))


def test_speculation_with_recurrent_state_is_refused():
    from vllm_neuron_amd.worker.mi355x_model_loader import check_draft
    with pytest.raises(NotImplementedError, match="state"):
        check_draft(stack_of(config_from_dict(CASES["uneven"]())))
    check_draft(stack_of(config_from_dict(config(64, 64, [latent2(2, 8, 8, 32, 16)]))))


# ---- state slots -----------------------------------------------------------------------------------------------------------
def runner(slots):
    from vllm_neuron_amd.worker.mi355x_model_runner import MI355XModelRunner
    r = MI355XModelRunner.__new__(MI355XModelRunner)
    r.vllm_req_to_seq_id_mapping, r.free_seq_ids = {}, set(range(slots))
    return r


def test_state_slots_are_kept_given_back_and_used_again():
    r = runner(3)
    assert [r._state_slot(x, 0, {x}) for x in "abc"] == [0, 1, 2]
    assert r._state_slot("b", 40, {"b"}) == 1                          # left out of steps meanwhile: still its own
    r._release_state_slot("b")
    assert r._state_slot("d", 0, {"d"}) == 1 and not r.free_seq_ids
    with pytest.raises(RuntimeError, match="state"):
        r._state_slot("e", 5, {"e"})


def test_a_slot_of_a_request_that_starts_over_is_taken_last():
    """Four requests, three slots: one of the holders has been preempted (the scheduler runs at most three)."""
    r = runner(3)
    for x in "abc":
        r._state_slot(x, 0, {x})
    assert r._state_slot("d", 0, {"a", "b", "d"}) == 2                 # c is not in the step
    with pytest.raises(RuntimeError, match="c continues"):
        r._state_slot("c", 9, {"c"})
    with pytest.raises(RuntimeError, match="more requests"):
        r._state_slot("c", 0, {"a", "b", "c", "d"})
    r._release_state_slot("a")
    assert r._state_slot("c", 0, {"b", "c", "d"}) == 0                 # starts over


# ---- the oracle's mechanisms ---------------------------------------------------------------------
def test_rotation_by_hand():
    x = torch.tensor([[1.0, 2.0, 3.0, 4.0, 9.0]] * 3, dtype=torch.float64)
    y = R.rotate(x, 100.0, 4)
    assert torch.equal(y[0], x[0]) and (y[:, 4] == 9.0).all()
    for p in (1, 2):
        for i, a in ((0, p * 1.0), (1, p * 0.1)):
            u, v = x[p, i], x[p, i + 2]
            assert y[p, i].item() == pytest.approx(u * math.cos(a) - v * math.sin(a)) and y[p, i + 2].item() == pytest.approx(v * math.cos(a) + u * math.sin(a))


def test_latent_attention_by_hand():
    T = 5
    c, q = torch.eye(T, dtype=torch.float64), torch.ones(T, 1, 2, dtype=torch.float64)
    k_rot = torch.arange(T, dtype=torch.float64).view(T, 1)
    o = R.latent_attention(q, c, k_rot, 2 * torch.arange(T, dtype=torch.float64).view(1, T), torch.arange(T, dtype=torch.float64).view(1, T), 0.5)
    for i in range(T):
        e = [math.exp(0.5 * (2 * j + j)) for j in range(i + 1)]
        assert o[i, 0].item() == pytest.approx(sum(j * x for j, x in enumerate(e)) / sum(e))


def test_short_convolution_by_hand():
    y = R.short_conv(torch.tensor([[1.0], [10.0], [100.0], [1000.0]], dtype=torch.float64), torch.tensor([[4.0, 3.0, 2.0]], dtype=torch.float64))
    z = torch.tensor([2.0, 23.0, 234.0, 2340.0], dtype=torch.float64)
    assert torch.allclose(y.flatten(), z / (1 + torch.exp(-z)))


def test_delta_rule_by_hand():
    """One head of two key channels and one value: decay, then the write, then the read-out of the new state."""
    k = torch.tensor([[[1.0, 0.0]], [[0.6, 0.8]]], dtype=torch.float64)
    q = torch.tensor([[[1.0, 1.0]], [[2.0, -1.0]]], dtype=torch.float64)
    v = torch.tensor([[[3.0]], [[5.0]]], dtype=torch.float64)
    g = torch.log(torch.tensor([[[0.5, 0.25]], [[0.5, 0.1]]], dtype=torch.float64))
    o, S = R.delta_rule(q, k, v, g, torch.tensor([[0.5], [0.25]], dtype=torch.float64))
    assert o[0].item() == pytest.approx(1.5)                     # S = [1.5, 0]
    u = 0.25 * (5 - 0.75 * 0.6)                                   # S decays to [0.75, 0]
    s = [0.75 + 0.6 * u, 0.8 * u]
    assert o[1].item() == pytest.approx(2 * s[0] - s[1]) and S.flatten().tolist() == pytest.approx(s)


def test_decay_by_hand():
    z = torch.tensor([[[0.5, -30.0]]], dtype=torch.float64)
    g = R.decays(z, torch.tensor([math.log(2.0)], dtype=torch.float64), torch.tensor([0.5, 0.0], dtype=torch.float64))
    assert g.flatten().tolist() == pytest.approx([-2 * math.log(1 + math.e), -2 * math.exp(-30)])


def test_router_groups_and_correction_by_hand():
    logit = lambda s: math.log(s / (1 - s))                       # noqa: E731
    z = torch.tensor([[logit(0.9), logit(0.1), logit(0.6), logit(0.5), logit(0.2), logit(0.3)]], dtype=torch.float64)
    none = torch.zeros(6, dtype=torch.float64)
    idx, w = R.pick(z, none, 2, 3, 1)                             # groups: 1.0, 1.1, 0.5
    assert idx.tolist() == [[2, 3]] and w.flatten().tolist() == pytest.approx([6 / 11, 5 / 11])
    idx, w = R.pick(z, torch.tensor([0.0, 0.0, 0.0, -1.0, 0.0, 0.0], dtype=torch.float64), 2, 3, 2)      # groups: 1.0, 0.1, 0.5
    assert idx.tolist() == [[0, 5]] and w.flatten().tolist() == pytest.approx([0.75, 0.25])
    idx, w = R.pick(z, torch.full((6,), -2.0, dtype=torch.float64), 1, 1, 1)                             # negative choice scores
    assert idx.tolist() == [[0]] and w.item() == pytest.approx(1.0)


@pytest.mark.parametrize("case", list(CASES))
def test_logits_of_a_prefix_do_not_depend_on_what_follows(case):
    cfg = CASES[case]()
    w = weights(cfg, 3)
    t = tokens(cfg, w, 60, 1)
    a, b = R.logits(cfg, w, t, torch.float64), R.logits(cfg, w, t[:41], torch.float64)
    assert torch.allclose(a[:41], b, atol=1e-9)


# ---- the GPU tests' cases show a mistake in any mechanism (the mistakes are planted here, in the oracle) -------------
def _mistakes():
    def patch(**kw):
        def run(mp):
            for k, v in kw.items():
                mp.setattr(R, k, v)
        return run
    attn, conv, rms, rot, rule, pick, mixer, heads = (R.latent_attention, R.short_conv, R.rms, R.rotate, R.delta_rule, R.pick, R.latent_mixer, R.delta_heads)

    def cut(f, at):                               # what f carries along is lost ahead of position `at`
        def run(x, *a):
            y = f(x, *a)
            y[at:] = f(x[at:], *a)
            return y
        return run

    def lost_state(q, k, v, g, b, state=None):
        o, _ = rule(q[:64], k[:64], v[:64], g[:64], b[:64])
        o2, S = rule(q[64:], k[64:], v[64:], g[64:], b[64:])
        return torch.cat([o, o2]), S

    def read_first(q, k, v, g, b, state=None):
        o, S = rule(q, k, v, g, b)                # (the write of a token is about b v k^T)
        return o - (q * k).sum(-1, keepdim=True) * v * b[:, :, None], S
    return {
        "no rotation": patch(rotate=lambda x, *a: x), "positions start at one": patch(rotate=lambda x, b, d, first=0: rot(x, b, d, 1) if x.dim() == 3 else rot(x, b, d)),
        "neighbours paired": patch(rotate=lambda x, b, d, first=0: _neighbours(x, b, d)),
        "every element rotated": patch(rotate=lambda x, b, d, first=0: rot(x, b, x.shape[-1])),
        "rotated part left out": patch(latent_attention=lambda q, c, k, uk, uv, s, r=None: attn(q[..., :uk.shape[0] // q.shape[1]], c, None, uk, uv, s)),
        "scale left out": patch(latent_attention=lambda q, c, k, uk, uv, s, r=None: attn(q, c, k, uk, uv, 1.0)),
        "a far key lost": patch(latent_attention=lambda q, c, k, uk, uv, s, r=None: torch.cat([attn(q, c, k, uk, uv, s)[:100],
                                attn(q[16:], c[16:], None if k is None else k[16:], uk, uv, s)[84:]])),
        "query latent not normed": patch(rms=lambda x, e: x if x.shape[-1] in (28, 22) else rms(x, e)),
        "latent not normed": patch(rms=lambda x, e: x if x.shape[-1] in (36, 50) else rms(x, e)),
        "heads' output not normed": patch(rms=lambda x, e: x if x.shape[-1] == 13 else rms(x, e)),
        "eps left out": patch(rms=lambda x, e: rms(x, 1e-12)),
        "no output gate": patch(latent_mixer=lambda h, m, w, p, *a: mixer(h, m, {**w, p + "g": 0 * w[p + "g"]}, p, *a)),
        "no gate behind the recurrence": patch(delta_heads=lambda q, k, v, b, z, gate, *a: heads(q, k, v, b, z, 0 * gate, *a)),
        "convolution reversed": patch(short_conv=lambda x, w: conv(x, w.flip(1))), "convolution state lost at 64": patch(short_conv=cut(conv, 64)),
        "no convolution": patch(short_conv=lambda x, w: x * torch.sigmoid(x)),
        "no unit norm": patch(unit=lambda x: x), "key heads in the wrong order": patch(delta_heads=lambda q, k, v, b, *a: heads(_flipped(q, b, a), _flipped(k, b, a), v, b, *a)),
        "no decay": patch(decays=lambda z, a, d: 0 * z), "one decay per head": patch(decays=lambda z, a, d, f=R.decays: f(z, a, d).mean(-1, keepdim=True).expand_as(z)),
        "dt_bias left out": patch(decays=lambda z, a, d, f=R.decays: f(z, a, 0 * d)),
        "step size one": patch(delta_rule=lambda q, k, v, g, b, s=None: rule(q, k, v, g, torch.ones_like(b))),
        "decay after the write": patch(delta_rule=lambda q, k, v, g, b, s=None: rule(q, k, v, torch.cat([0 * g[:1], g[:-1]]), b)),
        "read-out ahead of the write": patch(delta_rule=read_first), "state lost at 64": patch(delta_rule=lost_state),
        "correction left out": patch(pick=lambda z, c, *a: pick(z, 0 * c, *a)), "groups left out": patch(pick=lambda z, c, top, n, k: pick(z, c, top, 1, 1)),
        "one score per group": patch(pick=_one_score), "correction in the weights": patch(pick=_corrected_weights),
        "weights not divided by their sum": patch(pick=_unscaled), "another layer's tensors shared": patch(resolve=lambda layers, i: i if i < 3 else (i + 1) % 3),
    }


def _neighbours(x, base, dims):
    order = torch.cat([torch.arange(0, dims, 2), torch.arange(1, dims, 2), torch.arange(dims, x.shape[-1])])
    y = torch.empty_like(x)
    y[..., order] = _rot(x[..., order], base, dims)
    return y


_rot, _pick = R.rotate, R.pick


def _flipped(x, b, a):                             # the key heads in reverse order
    d = a[0].shape[1] // b.shape[1]
    return x.view(x.shape[0], -1, d).flip(1).reshape(x.shape)


def _one_score(z, c, top, n, keep):
    if keep == n:
        return _pick(z, c, top, n, keep)
    s = (torch.sigmoid(z) + c).view(z.shape[0], n, -1)
    ok = torch.zeros(z.shape[0], n, dtype=torch.bool).scatter_(1, s.max(-1).values.topk(keep, -1).indices, True)
    s = s.masked_fill(~ok[:, :, None], float("-inf")).reshape(z.shape)
    idx = s.topk(top, -1).indices
    w = torch.sigmoid(z).gather(1, idx)
    return idx, w / w.sum(-1, keepdim=True)


def _corrected_weights(z, c, *a):
    idx, _ = _pick(z, c, *a)
    w = (torch.sigmoid(z) + c).gather(1, idx)
    return idx, w / w.sum(-1, keepdim=True)


def _unscaled(z, c, *a):
    idx, _ = _pick(z, c, *a)
    return idx, torch.sigmoid(z).gather(1, idx)


@pytest.fixture(scope="module")
def good():
    cfg = CASES["uneven"]()
    w = weights(cfg, 11)
    t = tokens(cfg, w, 130, 130)
    return cfg, w, t, R.logits(cfg, w, t)


@pytest.mark.parametrize("mistake", list(_mistakes()))
def test_cases_show_a_planted_mistake(mistake, monkeypatch, good):
    from tests.test_bokulorn_gpu import LIMIT
    cfg, w, t, good = good
    _mistakes()[mistake](monkeypatch)
    assert error(R.logits(cfg, w, t), good) > 2 * LIMIT["bfloat16"]


@pytest.mark.parametrize("change", [lambda c, w: c["embedding"].update(scale=2.5), lambda c, w: w.update({"l0.norm1": w["l0.norm1"] - 1}),
                                    lambda c, w: w.update({"final.norm": w["final.norm"] - 1})])
def test_cases_show_a_wrong_constant(change, good):
    from tests.test_bokulorn_gpu import LIMIT
    cfg, w, t, good = good
    cfg, w = json.loads(json.dumps(cfg)), dict(w)
    change(cfg, w)
    assert error(R.logits(cfg, w, t), good) > 2 * LIMIT["bfloat16"]
