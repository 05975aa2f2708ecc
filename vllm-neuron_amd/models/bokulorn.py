# SPDX-License-Identifier: Apache-2.0
"""Bokulorn: configuration reader.  Everything that computes is the library's layer stack (csrc/stack.hip).

    x = scale embed[token]
    layer    h = norm1 x;  x <- x + mixer(h) + experts(h)       (RMS norms, weights stored around zero)
    logits   head final.norm(x)

Mixers: latent attention whose queries come from a latent too, with a rotated part beside the latent and a gate per head
('latent_attention') or without positions and a gate per element ('latent_attention_2'); a gated delta rule with one decay per
key channel ('channel_delta'), which keeps a matrix per head and the last inputs of its convolutions as sequence state.
Experts: squared relu, sigmoid router with a correction of the choice, chosen inside the best groups.  A layer may run another
layer's tensors.  Those mechanisms are the design's; every size and constant below comes from config.json, and the ranks
of two projections, which it does not give, from the checkpoint's tensors."""

from __future__ import annotations

from dataclasses import dataclass, field

from .._stack_enums import MI_ACT, MI_BLOCK, MI_FF, MI_GATE, MI_MIX, MI_ROUTE

UNBOUNDED_POSITIONS = 1 << 20  # no learned positions: a sequence may be as long as the cache allows
_GATES = {"latent_attention": "head", "latent_attention_2": "element"}


def _require(cond, what):
    if not cond:
        raise ValueError(f"Bokulorn config.json: {what}")


def _latent(i: int, kind: str, mix: dict) -> dict:
    out = dict(mixer_kind=MI_MIX["latent"], num_heads=int(mix["heads"]), num_kv_heads=1, qk_dim=int(mix["dim"]), v_dim=int(mix["vdim"]),
               kv_rank=int(mix["kv_rank"]), kv_from=-1, q_rank=int(mix["q_rank"]), window=0, scale=float(mix["scale"]),
               out_gate=MI_GATE[_GATES[kind]])
    _require(out["q_rank"] >= 1, f"layer {i}: q_rank must be at least 1")
    if kind == "latent_attention":
        out.update(rot_dim=int(mix["rot_dim"]), rot_dims=int(mix["rot"]["dims"]), rot_base=float(mix["rot"]["base"]))
        _require(out["rot_dim"] >= 1 and out["rot_dims"] % 2 == 0 and 0 <= out["rot_dims"] <= out["rot_dim"],
                 f"layer {i}: rot.dims must be even and at most rot_dim")
    return out


def _delta(i: int, mix: dict) -> dict:
    heads, kv = int(mix["heads"]), int(mix["kv_heads"])
    _require(kv > 0 and heads % kv == 0, f"layer {i}: heads must be a multiple of kv_heads")
    _require(int(mix["conv"]) >= 1, f"layer {i}: conv must be at least 1")
    return dict(mixer_kind=MI_MIX["delta"], num_heads=heads, num_kv_heads=kv, qk_dim=int(mix["dim"]), v_dim=int(mix["vdim"]),
                conv_taps=int(mix["conv"]), kv_from=-1, window=0, scale=1.0)


def _experts(i: int, mlp: dict | None) -> dict:
    if mlp is None:
        return dict(ff_kind=MI_FF[None], ff_size=0)
    _require(mlp.get("kind") == "moe", f"layer {i}: unknown feed-forward {mlp.get('kind')!r}")
    router = mlp["router"]
    experts, top, groups = int(router["experts"]), int(router["top"]), router.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(groups["count"]), int(groups["keep"])
    _require(count >= 1 and experts % count == 0 and 1 <= keep <= count, f"layer {i}: groups.count must divide the experts, 1 <= keep <= count")
    _require(1 <= top <= experts // count * keep, f"layer {i}: router.top must be 1 .. the experts of the kept groups")
    return dict(ff_kind=MI_FF["moe"], ff_size=int(mlp["expert"]["ff"]), ff_act=MI_ACT["relu2"], experts=experts, experts_top=top,
                router_score=MI_ROUTE["sigmoid"], router_groups=count, router_keep=keep)


def _layer(i: int, entry: dict) -> dict:
    kind = entry.get("type")
    if kind in _GATES:
        out = _latent(i, kind, entry["mixer"])
    elif kind == "channel_delta":
        out = _delta(i, entry["mixer"])
    else:
        raise ValueError(f"Bokulorn config.json: layer {i}: unknown layer type {kind!r}")
    out.update(_experts(i, entry.get("mlp")))
    return out


@dataclass
class BokulornConfig:
    architecture = "Bokulorn"
    stack: dict
    vocab_size: int
    hidden_size: int
    num_hidden_layers: int
    max_position_embeddings: int
    num_attention_heads: int
    num_key_value_heads: int        # one row per token
    head_dim: int                   # vLLM's single-layer cache spec counts K and V: half of the widest row, rounded up
    sizes_from: dict                # (layer, field of mi_layer_spec) -> tensor whose rows give it
    architectures: list = field(default_factory=lambda: ["Bokulorn"])
    model_type: str = "bokulorn"
    tie_word_embeddings: bool = False

    @classmethod
    def from_dict(cls, raw: dict) -> "BokulornConfig":
        entries = raw["layers"]
        _require(entries, "no layers")
        layers = [_layer(i, e) for i, e in enumerate(entries)]
        owner, sizes_from = [], {}
        for i, entry in enumerate(entries):
            j, seen = i, {i}
            while entries[j].get("weights_of") is not None:      # the layer that has the tensors
                j = int(entries[j]["weights_of"])
                _require(0 <= j < len(entries) and j not in seen, f"layer {i}: weights_of must lead to a layer with tensors of its own")
                seen.add(j)
            if j != i:
                _require(layers[i] == layers[j], f"layer {i}: weights_of names a layer with other sizes")
            owner.append(j)
            if layers[i]["mixer_kind"] == MI_MIX["delta"]:
                sizes_from[(i, "decay_rank")] = f"l{j}.mix.a1"
                sizes_from[(i, "gate_rank")] = f"l{j}.mix.g1"
        for i, j in enumerate(owner):
            layers[i]["weights_of"] = j if j != i else -1
        width = int(raw["width"])
        stack = dict(layers=layers, width=width, vocab_size=int(raw["vocab"]), max_positions=0, norm_eps=float(raw["norm"]["eps"]),
                     residual_mult=1.0, block_kind=MI_BLOCK["one_norm"], norm_groups=1, norm_offset=1.0,
                     embed_scale=float(raw["embedding"]["scale"]))
        row = max(x.get("kv_rank", 1) + x.get("rot_dim", 0) for x in layers)
        return cls(stack=stack, vocab_size=stack["vocab_size"], hidden_size=width, num_hidden_layers=len(layers),
                   max_position_embeddings=UNBOUNDED_POSITIONS, num_attention_heads=max(x["num_heads"] for x in layers),
                   num_key_value_heads=1, head_dim=(row + 1) // 2, sizes_from=sizes_from)
