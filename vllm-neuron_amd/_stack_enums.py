# SPDX-License-Identifier: Apache-2.0
"""Names of the layer-stack enumerations of include/mi355x_vllm.h (no torch, no library: the configuration readers use them)."""

MI_BLOCK = {"parallel": 0, "sandwich": 1, "one_norm": 2, "post_norm": 3}
MI_MIX = {"attention": 0, "latent": 1, "delta": 2, "scan": 3, "ssd": 4}
MI_BIAS = {None: 0, "slope": 1, "table": 2}
MI_SINK = {None: 0, "one": 1, "learned": 2}
MI_FF = {None: 0, "relu2": 1, "glu": 2, "moe": 3}
MI_ACT = {"silu": 0, "swish_clip": 1, "relu2": 2}
MI_GATE = {None: 0, "head": 1, "element": 2}
MI_ROUTE = {"softmax": 0, "sigmoid": 1}
