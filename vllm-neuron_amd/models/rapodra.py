# SPDX-License-Identifier: Apache-2.0
"""Rapodra: configuration reader.  Everything that computes is the library's layer stack (csrc/stack.hip).

    x = embed[token]
    layer    x <- x + norm1b(attention(C1(norm1 x)));  x <- x + norm2b(ff(C2(norm2 x)))
    C(h)     h + a causal convolution of h over time, per channel; its last taps - 1 inputs are sequence state
    logits   softcap tanh(head final.norm(x) / softcap)

Attention works on a cached latent c per token (per head k = W_uk c, v = W_uv c; no positions) under a sliding window; a
layer may read the latents of an earlier layer.  The feed-forward is a gated unit with clipped branches, a mixture of
experts, or absent.  Norms are RMS norms over equal parts of the row.  Those mechanisms are the design's; every size and
constant below comes from config.json."""

from __future__ import annotations

from dataclasses import dataclass, field

from .._stack_enums import MI_ACT, MI_BLOCK, MI_FF, MI_MIX

SWISH_ALPHA = 1.702           # fixed by the design: the gate's slope in the clipped gated unit
UNBOUNDED_POSITIONS = 1 << 20  # no learned positions: a sequence may be as long as the cache allows


def _require(cond, what):
    if not cond:
        raise ValueError(f"Rapodra config.json: {what}")


def _layer(i: int, entry: dict, layers: list) -> dict:
    _require(entry.get("type") == "latent_attention", f"layer {i}: unknown layer type {entry.get('type')!r}")
    mix = entry["mixer"]
    window = int(mix["mask"]["size"])
    _require(window >= 1, f"layer {i}: mask.size must be at least 1")
    source = mix.get("kv_from")
    out = dict(mixer_kind=MI_MIX["latent"], num_heads=int(mix["heads"]), num_kv_heads=1, qk_dim=int(mix["dim"]), v_dim=int(mix["vdim"]),
               kv_rank=int(mix["kv_rank"]), kv_from=-1 if source is None else int(source), window=window, scale=float(mix["scale"]),
               ff_kind=MI_FF[None], ff_size=0)
    if source is not None:
        _require(0 <= int(source) < i and layers[int(source)]["kv_from"] < 0 and layers[int(source)]["kv_rank"] == out["kv_rank"],
                 f"layer {i}: kv_from must name an earlier layer with latents of its own and the same kv_rank")
    mlp = entry.get("mlp")
    if mlp is None:
        return out
    kind = mlp.get("kind")
    if kind == "dense":
        out.update(ff_kind=MI_FF["glu"], ff_size=int(mlp["ff"]), ff_act=MI_ACT["swish_clip"], ff_limit=float(mlp["limit"]),
                   ff_alpha=SWISH_ALPHA)
    elif kind == "moe":
        experts, top = int(mlp["router"]["experts"]), int(mlp["router"]["top"])
        _require(1 <= top <= experts, f"layer {i}: router.top must be 1 .. router.experts")
        out.update(ff_kind=MI_FF["moe"], ff_size=int(mlp["expert"]["ff"]), ff_act=MI_ACT["silu"], experts=experts, experts_top=top)
    else:
        raise ValueError(f"Rapodra config.json: layer {i}: unknown feed-forward {kind!r}")
    return out


@dataclass
class RapodraConfig:
    architecture = "Rapodra"
    stack: dict
    vocab_size: int
    hidden_size: int
    num_hidden_layers: int
    max_position_embeddings: int
    num_attention_heads: int
    num_key_value_heads: int        # one latent row per token
    head_dim: int                   # vLLM's single-layer cache spec counts K and V: half of the widest latent, rounded up
    architectures: list = field(default_factory=lambda: ["Rapodra"])
    model_type: str = "rapodra"
    tie_word_embeddings: bool = False

    @classmethod
    def from_dict(cls, raw: dict) -> "RapodraConfig":
        layers: list = []
        for i, entry in enumerate(raw["layers"]):
            layers.append(_layer(i, entry, layers))
        _require(layers, "no layers")
        width, groups, taps = int(raw["width"]), int(raw["norm"]["groups"]), int(raw["canon"]["taps"])
        _require(groups >= 1 and width % groups == 0, "norm.groups must divide width")
        _require(taps >= 1, "canon.taps must be at least 1")
        cap = float(raw["logit_softcap"])
        _require(cap > 0, "logit_softcap must be positive")
        stack = dict(layers=layers, width=width, vocab_size=int(raw["vocab"]), max_positions=0, norm_eps=float(raw["norm"]["eps"]),
                     residual_mult=1.0, block_kind=MI_BLOCK["sandwich"], norm_groups=groups, conv_taps=taps, logit_softcap=cap)
        return cls(stack=stack, vocab_size=stack["vocab_size"], hidden_size=width, num_hidden_layers=len(layers),
                   max_position_embeddings=UNBOUNDED_POSITIONS, num_attention_heads=max(x["num_heads"] for x in layers),
                   num_key_value_heads=1, head_dim=max((x["kv_rank"] + 1) // 2 for x in layers))
