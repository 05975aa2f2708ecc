# SPDX-License-Identifier: Apache-2.0
"""Nusovik: configuration reader.  Everything that computes is the library's layer stack (csrc/stack.hip).

    x = scale embed[token] + sinusoid(position)
    layer    x <- x + norm1 mixer(x);  x <- x + norm2 ff(x)       (RMS norms of the sublayers' outputs; they read x itself)
    logits   logit_scale head final.norm(x)

Mixers: 'parallel', attention beside a Mamba-2 mixer of the same x (grouped heads inside chunks of positions, weighted query / key
norms, values that are the projected keys, a bucketed distance bias, a learned softmax sink, a gate per head), and 'mamba1', a
selective scan.  Both recurrences keep their state and the last inputs of their convolutions per sequence.  Feed-forwards: squared
relu, or none.  Those mechanisms are the design's; every size and constant below comes from config.json, and the number of
distance buckets, which it does not give, from the checkpoint's table."""

from __future__ import annotations

from dataclasses import dataclass, field

from .._stack_enums import MI_BIAS, MI_BLOCK, MI_FF, MI_GATE, MI_MIX, MI_SINK

UNBOUNDED_POSITIONS = 1 << 20  # no learned positions: a sequence may be as long as the cache allows
POSITION_BASE = 10000.0


def _require(cond, what):
    if not cond:
        raise ValueError(f"Nusovik config.json: {what}")


def _taps(i: int, mix: dict) -> int:
    taps = int(mix["conv"])
    _require(taps >= 1, f"layer {i}: conv must be at least 1")
    return taps


def _parallel(i: int, mix: dict) -> dict:
    left, right = mix["left"], mix["right"]
    heads, kv, dim, vdim = (int(left[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    _require(kv > 0 and heads % kv == 0, f"layer {i}: heads must be a multiple of kv_heads")
    _require(dim == vdim, f"layer {i}: the values are the keys, vdim must be dim")
    chunk, far = int(left["mask"]["size"]), float(left["bias_max"])
    _require(chunk >= 1, f"layer {i}: mask.size must be at least 1")
    h2, p2, groups, parts = (int(right[k]) for k in ("heads", "vdim", "groups", "norm_groups"))
    _require(groups >= 1 and h2 % groups == 0, f"layer {i}: heads must be a multiple of groups")
    _require(parts >= 1 and h2 * p2 % parts == 0, f"layer {i}: norm_groups must divide the heads' columns")
    return dict(mixer_kind=MI_MIX["attention"], num_heads=heads, num_kv_heads=kv, qk_dim=dim, v_dim=vdim, kv_from=-1, window=0, chunk=chunk,
                scale=float(left["scale"]), qk_norm=1, qk_bias=1, keys_as_values=1, distance_bias=MI_BIAS["table"], rel_far=far,
                softmax_sink=MI_SINK["learned"], out_gate=MI_GATE["head"], mix_mult=float(mix["left_scale"]),
                beside_kind=MI_MIX["ssd"], beside_mult=float(mix["right_scale"]), ssm_heads=h2, ssm_dim=p2, ssm_state=int(right["state"]),
                ssm_groups=groups, ssm_parts=parts, conv_taps=_taps(i, right))


def _scan(i: int, mix: dict) -> dict:
    return dict(mixer_kind=MI_MIX["scan"], ssm_inner=int(mix["inner"]), ssm_state=int(mix["state"]), dt_rank=int(mix["dt_rank"]),
                conv_taps=_taps(i, mix), kv_from=-1)


def _layer(i: int, entry: dict) -> dict:
    kind = entry.get("type")
    if kind == "parallel":
        out = _parallel(i, entry["mixer"])
    elif kind == "mamba1":
        out = _scan(i, entry["mixer"])
    else:
        raise ValueError(f"Nusovik config.json: layer {i}: unknown layer type {kind!r}")
    mlp = entry.get("mlp")
    if mlp is None:
        out.update(ff_kind=MI_FF[None], ff_size=0)
    else:
        _require(mlp.get("kind") == "dense", f"layer {i}: unknown feed-forward {mlp.get('kind')!r}")
        out.update(ff_kind=MI_FF["relu2"], ff_size=int(mlp["ff"]))
    return out


@dataclass
class NusovikConfig:
    architecture = "Nusovik"
    stack: dict
    vocab_size: int
    hidden_size: int
    num_hidden_layers: int
    max_position_embeddings: int
    num_attention_heads: int
    num_key_value_heads: int
    head_dim: int                   # the widest head; the pools' own sizes are the library's
    sizes_from: dict                # (layer, field of mi_layer_spec) -> tensor whose rows give it
    architectures: list = field(default_factory=lambda: ["Nusovik"])
    model_type: str = "nusovik"
    tie_word_embeddings: bool = False

    @classmethod
    def from_dict(cls, raw: dict) -> "NusovikConfig":
        entries = raw["layers"]
        _require(entries, "no layers")
        layers = [_layer(i, e) for i, e in enumerate(entries)]
        attention = [x for x in layers if x["mixer_kind"] == MI_MIX["attention"]]
        width = int(raw["width"])
        stack = dict(layers=layers, width=width, vocab_size=int(raw["vocab"]), max_positions=0, norm_eps=float(raw["norm"]["eps"]),
                     residual_mult=1.0, block_kind=MI_BLOCK["post_norm"], norm_groups=1, embed_scale=float(raw["embedding"]["scale"]),
                     pos_base=POSITION_BASE, logit_scale=float(raw["logit_scale"]))
        return cls(stack=stack, vocab_size=stack["vocab_size"], hidden_size=width, num_hidden_layers=len(layers),
                   max_position_embeddings=UNBOUNDED_POSITIONS, num_attention_heads=max([x["num_heads"] for x in attention], default=1),
                   num_key_value_heads=max([x["num_kv_heads"] for x in attention], default=1),
                   head_dim=max([x["qk_dim"] for x in attention], default=1),
                   sizes_from={(i, "rel_rows"): f"l{i}.mix.left.rel" for i, x in enumerate(layers) if x["mixer_kind"] == MI_MIX["attention"]})
