"""Helpers of the Tobilorn tests: small configurations, weights that make every mechanism loud, folders."""
from __future__ import annotations

import json
import math
import os

import torch


def attention(heads, kv_heads, dim, vdim, scale, diff, window=None, keep_first=0, base=1000.0, rot=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, diff=diff,
             rot={"base": base, "dims": dim - dim % 2 if rot is None else rot})
    if window is not None:
        m["mask"] = {"size": window, "keep_first": keep_first}
    return {"type": "attention", "mixer": m}


def moe(experts, top, ff, identity=0, shared=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top, "identity": identity}, "expert": {"ff": ff}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer: dict, mlp=None) -> dict:
    return dict(mixer, mlp=mlp)


def config(width, vocab, layers, loop=None, side=None, scale=1.0, logit_scale=1.0, eps=1e-5) -> dict:
    out = {"architecture": "Tobilorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "logit_scale": logit_scale, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side is not None:
        out["token_side"] = {"dim": side}
    return out


# Configurations that differ in every size and option: one to many heads a kv head, maps narrower and wider than half a
# value, partial, whole and no rotation, windows of one token, of a page, beside its border, of many pages and none, kept
# first tokens of none, one, within a page, beyond a page and beyond a step of 64 keys, more of them than the window holds,
# one to all experts chosen with and without identity experts, with and without a shared expert, layers without a
# feed-forward, loops over all, some and one of the layers, once and thrice, side vectors on and off borders of 8, sizes that
# are no multiples of 8.
# T_MIXED chooses all its experts, so no discrete choice can turn under bfloat16 rounding and long bfloat16 runs count
# to their end; fewer than all are chosen in T_WIDE, T_ODD, T_PLAIN and the expert layers alone.
T_MIXED = config(64, 211, [
    layer(attention(4, 2, 16, 24, 0.5, 0.2, window=20, keep_first=3), moe(3, 4, 40, identity=1, shared=48)),
    layer(attention(3, 1, 8, 16, 0.6, 0.5, window=33, keep_first=17, rot=4), None),
    layer(attention(2, 2, 24, 32, 0.4, -0.3), moe(3, 3, 24, shared=32)),
    layer(attention(6, 2, 16, 8, 0.5, 0.8, window=16, base=50.0), moe(2, 4, 16, identity=2)),
], loop=(1, 3, 3), side=16, scale=2.5, logit_scale=0.7)
T_WIDE = config(96, 333, [
    layer(attention(8, 2, 32, 48, 0.3, 0.4, window=100, keep_first=70, base=20000.0), moe(8, 2, 24, identity=2, shared=40)),
    layer(attention(5, 1, 40, 64, 0.25, 0.1, window=17, keep_first=4, rot=24), moe(6, 3, 32)),
    layer(attention(4, 4, 64, 128, 0.2, 0.6, window=64, keep_first=1), moe(5, 1, 40, identity=3, shared=24)),
], loop=(0, 3, 2), side=24, scale=8.0, logit_scale=0.25)
T_ODD = config(52, 97, [
    layer(attention(3, 1, 5, 7, 0.6, 0.3, window=9, keep_first=2), moe(6, 2, 12, identity=1, shared=20)),
    layer(attention(2, 2, 6, 11, 0.5, 0.25, window=1, keep_first=5, rot=2), None),
    layer(attention(4, 2, 12, 10, 0.5, 0.45, window=23, rot=0), moe(4, 2, 20, shared=9)),
    layer(attention(1, 1, 10, 6, 0.4, 0.15), moe(3, 2, 10, identity=2)),
], loop=(1, 2, 4), side=5, scale=1.5, logit_scale=1.3, eps=1e-2)
T_PLAIN = config(48, 101, [                 # no loop, no side vectors
    layer(attention(2, 1, 16, 32, 0.5, 0.35, window=32, keep_first=4), moe(4, 2, 24, identity=1, shared=24)),
    layer(attention(2, 1, 16, 32, 0.5, 0.35, window=32, keep_first=4), moe(4, 2, 24, identity=1, shared=24)),
])
ONLY = {
    "attention": config(48, 101, [layer(attention(4, 2, 16, 32, 0.6, 0.3))]),
    "attention_window": config(48, 101, [layer(attention(4, 1, 16, 24, 0.6, 0.3, window=40))]),
    "attention_keep": config(48, 101, [layer(attention(2, 2, 16, 16, 0.6, 0.4, window=40, keep_first=6))]),
    "attention_keep_many": config(48, 101, [layer(attention(4, 2, 32, 64, 0.4, 0.4, window=24, keep_first=90))]),
    "attention_many_heads": config(64, 101, [layer(attention(24, 1, 24, 40, 0.4, 0.3, window=50, keep_first=5))]),      # groups beyond sixteen columns
    "attention_widest": config(64, 101, [layer(attention(2, 1, 128, 256, 0.1, 0.3, window=70, keep_first=20))]),
    "attention_beyond": config(64, 101, [layer(attention(2, 1, 144, 40, 0.1, 0.3, window=70, keep_first=20))]),           # beyond the matrix-core kernels
    "moe": config(48, 101, [layer(attention(1, 1, 8, 8, 0.3, 0.1), moe(8, 2, 24, identity=3, shared=32))]),
    "moe_odd": config(44, 101, [layer(attention(1, 1, 8, 8, 0.3, 0.1), moe(6, 2, 20, identity=1, shared=10))]),
    "side": config(48, 101, [layer(attention(1, 1, 8, 8, 0.3, 0.1))] * 3, side=20, scale=3.0),
    "loop": config(48, 101, [layer(attention(1, 1, 8, 8, 0.3, 0.1))] * 3, loop=(1, 3, 3), scale=3.0),
    "loop_last": config(40, 101, [layer(attention(1, 1, 8, 8, 0.3, 0.1))] * 2, loop=(1, 2, 1), side=8),
}
CONFIGS = dict(mixed=T_MIXED, wide=T_WIDE, odd=T_ODD, plain=T_PLAIN, **{"only_" + k: v for k, v in ONLY.items()})


def make_weights(raw: dict, seed: int) -> dict:
    """bfloat16 tensors for a configuration, scaled so that every mechanism moves the logits: the second map takes a real
    share, biases and corrections are of the size of what they are added to, norms' weights spread around zero."""
    from tuff_amd.models.registry import build_model, config_from_dict
    g = torch.Generator().manual_seed(seed)
    model = build_model(config_from_dict(raw))
    out = {}
    for d in model.weight_decls():
        name, shape = d.name, tuple(d.shape)
        n = lambda std=1.0, mean=0.0: mean + std * torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if name in ("embed", "side.embed"):
            t = n(1.0)
        elif name == "head":
            t = n(1.0 / math.sqrt(shape[1]))
        elif name == "loop.in":
            t = n(0.8 / math.sqrt(shape[1] / 2))
        elif name == "loop.step":
            t = n(0.5)
        elif last in ("norm1", "norm1b", "norm2", "norm2b") or name == "final.norm":
            t = n(0.3)
        elif last == "norm":                              # the side path's plain weight
            t = n(0.3, 1.0)
        elif last == "b":
            t = n(0.5)
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            t = n(0.6 / math.sqrt(math.sqrt(shape[0])))
        elif last == "correction":
            t = n(0.1)
        elif name.endswith("side.gate"):                  # it reads the stream as it is: an activation in its curved part
            t = n(1.3 / math.sqrt(shape[1]) / max(1.0, raw["embedding"]["scale"]))
        elif last == "router":
            t = n(1.5 / math.sqrt(shape[1]))
        elif len(shape) == 2:
            t = n(1.3 / math.sqrt(shape[1]))
        else:
            t = n(0.5)
        out[name] = t.to(torch.bfloat16)
    return out


def write_folder(raw: dict, weights: dict, out_dir: str) -> str:
    from safetensors.torch import save_file
    os.makedirs(out_dir, exist_ok=True)
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(raw, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(out_dir, "model.safetensors"))
    return out_dir
