"""Helpers of the Kisutar tests: small configurations, weights that make every mechanism loud, folders."""
from __future__ import annotations

import json
import math
import os

import torch


def latent(heads, dim, rot, vdim, q_rank, kv_rank, scale, window=None, base=1000.0, kv_from=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale, rot={"base": base, "dims": rot})
    if window is not None:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer: dict, mlp=None) -> dict:
    return dict(mixer, mlp=mlp)


def config(width, vocab, layers, eps=1e-5) -> dict:
    return {"architecture": "Kisutar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# Configurations that differ in every size and option: one to many heads, plain parts wider and narrower than rotated
# ones, values of other widths than keys, latent rows and query rows on and off borders of 8, windows of one token, of a
# page, beside its border, of many pages and none, readers next to the layer they read and further up whose windows are
# narrower, wider and unbounded, one to all experts chosen, with and without a shared expert, layers without a
# feed-forward, sizes that are no multiples of 8.
# S_MIXED chooses all its experts, so no discrete choice can turn under bfloat16 rounding and long bfloat16 runs count
# to their end; fewer than all are chosen in S_WIDE, S_ODD, S_PLAIN and the expert layers alone.
S_MIXED = config(64, 211, [
    layer(latent(2, 16, 8, 24, 24, 32, 0.4, window=20), dense(40)),
    layer(latent(3, 8, 16, 16, 40, 24, 0.3), moe(4, 4, 40, 56)),
    layer(latent(4, 16, 16, 8, 16, 24, 0.35, window=33, kv_from=1), None),
    layer(latent(2, 24, 8, 16, 32, 32, 0.3, window=48, kv_from=0), moe(3, 3, 24)),
    layer(latent(1, 8, 8, 32, 8, 16, 0.5, window=16, base=50.0), dense(72)),
])
S_WIDE = config(96, 333, [
    layer(latent(5, 24, 16, 24, 48, 48, 0.2, window=17), moe(8, 2, 24, 40)),
    layer(latent(2, 32, 32, 8, 64, 48, 0.15, window=100, base=20000.0), dense(56)),
    layer(latent(6, 8, 32, 40, 24, 48, 0.25, kv_from=1, base=20000.0), moe(6, 3, 32)),
    layer(latent(3, 16, 32, 24, 40, 48, 0.2, window=15, kv_from=1, base=20000.0), moe(5, 1, 40, 24)),
    layer(latent(1, 40, 24, 40, 96, 40, 0.2, window=64), None),
    layer(latent(4, 16, 16, 16, 32, 48, 0.3, window=40, kv_from=0), dense(24)),
])
S_ODD = config(52, 97, [
    layer(latent(3, 5, 6, 7, 13, 20, 0.5, window=9), moe(6, 2, 12, 20)),
    layer(latent(1, 12, 2, 20, 20, 11, 0.4, window=1), dense(30)),
    layer(latent(3, 7, 2, 5, 9, 11, 0.4, window=23, kv_from=1), None),
    layer(latent(2, 10, 10, 6, 30, 22, 0.3), moe(4, 1, 20)),
], eps=1e-2)
S_PLAIN = config(48, 101, [
    layer(latent(2, 8, 8, 8, 16, 16, 0.4, window=32), moe(4, 2, 24, 24)),
    layer(latent(2, 8, 8, 8, 16, 16, 0.4, window=32, kv_from=0), dense(24)),
])
ONLY = {
    "latent": config(48, 101, [layer(latent(2, 16, 8, 24, 24, 32, 0.6))]),
    "latent_window": config(48, 101, [layer(latent(2, 16, 16, 24, 24, 32, 0.6, window=40))]),
    "latent_wide": config(64, 101, [layer(latent(3, 24, 16, 16, 40, 280, 0.3, window=70))]),       # a cache row beyond the matrix-core kernels
    "latent_many_heads": config(64, 101, [layer(latent(24, 16, 24, 8, 40, 128, 0.4, window=50))]),
    "latent_shared": config(48, 101, [layer(latent(2, 16, 8, 8, 24, 24, 0.5, window=24)), layer(latent(3, 8, 8, 16, 16, 24, 0.7, window=60, kv_from=0)),
                                      layer(latent(2, 8, 8, 16, 32, 24, 0.6, kv_from=0))]),
    "dense": config(40, 101, [layer(latent(1, 8, 4, 8, 8, 8, 0.3, window=4), dense(28))]),
    "moe": config(48, 101, [layer(latent(1, 8, 4, 8, 8, 8, 0.3), moe(8, 2, 24, 32))]),
    "moe_odd": config(44, 101, [layer(latent(1, 8, 4, 8, 8, 8, 0.3), moe(6, 2, 20, 10))]),
    "deep": config(32, 101, [layer(latent(1, 8, 8, 8, 8, 16, 0.4, window=6 + i)) for i in range(11)]),      # sums over twelve results
}
CONFIGS = dict(mixed=S_MIXED, wide=S_WIDE, odd=S_ODD, plain=S_PLAIN, **{"only_" + k: v for k, v in ONLY.items()})


def make_weights(raw: dict, seed: int) -> dict:
    """bfloat16 tensors for a configuration, scaled so that every mechanism moves the logits: mixers and feed-forwards
    add about the stream's own size, a row's share of the row before it spreads over (0, 1) and beyond, the sums over
    the layers take something of every result, sinks hold a share, the two numbers of the activation differ."""
    from tuff_amd.models.registry import build_model, config_from_dict
    g = torch.Generator().manual_seed(seed)
    model = build_model(config_from_dict(raw))
    out = {}
    for d in model.weight_decls():
        name, shape = d.name, tuple(d.shape)
        n = lambda std=1.0, mean=0.0: mean + std * torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if name == "embed":
            t = n(1.0)
        elif name == "head":
            t = n(1.0 / math.sqrt(shape[1]))
        elif last == "shift":
            t = n(0.4, 0.5)
        elif last == "dwa":
            t = n(0.35)
            t[-1] = t[-1] + 0.8
        elif last in ("norm1", "norm2", "norm"):
            t = n(0.2, 1.0)
        elif last == "sink":
            t = n(1.0, 0.5)
        elif last == "act":
            t = n(0.7)
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
