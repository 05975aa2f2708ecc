# SPDX-License-Identifier: Apache-2.0
"""Vimesun: configuration reader.  Everything that computes is the library's layer stack (csrc/stack.hip).

    x = embed[token] + pos[position]
    layer    x <- x + residual_mult (attention(norm1 x) + down max(up norm2 x, 0)^2)
    loop     layers start .. stop - 1 run `times` times; x <- loop.in [x ; embedding output] ahead of every pass
    logits   head final.norm(x)

Attention: grouped heads with separate key and value sizes, unit-norm queries and keys, no rotation, a per-head linear
distance bias, a sliding window, and a softmax with one added to its denominator.  Norms are layer norms with bias.
Those mechanisms are the design's; every size and constant below comes from config.json."""

from __future__ import annotations

from dataclasses import dataclass, field

from .._stack_enums import MI_FF


def _require(cond, what):
    if not cond:
        raise ValueError(f"Vimesun config.json: {what}")


def _layer(i: int, entry: dict) -> dict:
    _require(entry.get("type") == "attention", f"layer {i}: unknown layer type {entry.get('type')!r}")
    mix = entry["mixer"]
    heads, kv = int(mix["heads"]), int(mix["kv_heads"])
    _require(kv > 0 and heads % kv == 0, f"layer {i}: heads must be a multiple of kv_heads")
    window = int(mix["mask"]["size"])
    _require(window >= 1, f"layer {i}: mask.size must be at least 1")
    out = dict(num_heads=heads, num_kv_heads=kv, qk_dim=int(mix["dim"]), v_dim=int(mix["vdim"]), window=window,
               scale=float(mix["scale"]), qk_unit_norm=1, distance_bias=1, softmax_sink=1, ff_kind=MI_FF[None], ff_size=0)
    mlp = entry.get("mlp")
    if mlp is not None:
        _require(mlp.get("kind") == "dense", f"layer {i}: unknown feed-forward {mlp.get('kind')!r}")
        out.update(ff_kind=MI_FF["relu2"], ff_size=int(mlp["ff"]))
    return out


@dataclass
class VimesunConfig:
    architecture = "Vimesun"
    stack: dict
    vocab_size: int
    hidden_size: int
    num_hidden_layers: int          # layer runs: a looped layer counts once per pass
    max_position_embeddings: int
    num_attention_heads: int
    num_key_value_heads: int        # per layer they may differ; vLLM's single-layer cache spec takes the largest
    head_dim: int
    architectures: list = field(default_factory=lambda: ["Vimesun"])
    model_type: str = "vimesun"
    tie_word_embeddings: bool = False

    @classmethod
    def from_dict(cls, raw: dict) -> "VimesunConfig":
        layers = [_layer(i, e) for i, e in enumerate(raw["layers"])]
        _require(layers, "no layers")
        loop = raw.get("loop") or {"start": 0, "stop": 0, "times": 0}
        start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
        _require(times == 0 or (times > 0 and 0 <= start < stop <= len(layers)), "loop: 0 <= start < stop <= layers, times >= 1")
        stack = dict(layers=layers, width=int(raw["width"]), vocab_size=int(raw["vocab"]),
                     max_positions=int(raw["max_positions"]), norm_eps=float(raw["norm"]["eps"]),
                     residual_mult=float(raw["residual_mult"]), loop_start=start, loop_stop=stop, loop_times=times)
        return cls(stack=stack, vocab_size=stack["vocab_size"], hidden_size=stack["width"],
                   num_hidden_layers=len(layers) + max(times - 1, 0) * (stop - start),
                   max_position_embeddings=stack["max_positions"],
                   num_attention_heads=max(x["num_heads"] for x in layers),
                   num_key_value_heads=max(x["num_kv_heads"] for x in layers),
                   head_dim=max(max(x["qk_dim"], x["v_dim"]) for x in layers))
