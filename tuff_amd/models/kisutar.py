"""The Kisutar decoder put together from parts.

x = embed[token].  Every layer is pre-norm with RMS norms; what its mixer reads is mixed with the row the token before
had there (token shift, x <- x + mixer(h + (h' - h) shift), h = norm1(x)), then x <- x + ff(norm2(x)); after the layer the
stream becomes a learned weighted sum of the embedding and the results of all layers so far (depth average).  The mixer
is latent attention whose queries go through a normed latent of their own, with a rotated key part shared by the heads
(halves of the rotated channels pair up), a sliding window and a sink per head; a layer with `kv_from` reads the latent
rows and rotated keys that an earlier layer keeps.  Feed-forwards: a dense layer with the xIELU activation, or experts
with the exact gelu behind a router whose weights are the chosen experts' shares of the softmax over all, plus a shared
expert.  Logits = head norm(x).

Tensors: 'embed', 'head', 'final.norm'; layer i: 'l<i>.norm1', 'l<i>.norm2', 'l<i>.shift', 'l<i>.dwa', 'l<i>.mix.*',
'l<i>.mlp.up|down|act' or 'l<i>.mlp.e<k>.up|down', 'l<i>.mlp.router', 'l<i>.mlp.shared.up|down'.
"""
from __future__ import annotations

from ..config.kisutar import KisutarConfig
from ..parts.base import WeightDecl
from ..parts.block import TokenShiftBlock
from ..parts.ffn import DenseMLP, MoE
from ..parts.latent import LatentAttentionMixer
from ..parts.norm import RMSNorm
from .decoder import DecoderModel, LayerRun


def _norm(cfg: KisutarConfig, name: str) -> RMSNorm:
    return RMSNorm(cfg.width, cfg.eps, name)


def _mixer(cfg: KisutarConfig, i: int) -> LatentAttentionMixer:
    m, p = cfg.layers[i]["mixer"], f"l{i}.mix."
    keys = ("dq", "dq.norm", "uq", "uk", "uv", "sink", "o") + (() if m.get("kv_from") is not None else ("dkv", "dkv.norm"))
    return LatentAttentionMixer(cfg.width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], norm_eps=cfg.eps,
                                scale=m["scale"], rot_base=m["rot"]["base"], rot_dims=m["rot"]["dims"], rot_halves=True,
                                window=(m.get("mask") or {}).get("size"), q_rank=m["q_rank"], exact_weights=True,
                                names={k: p + k for k in keys})


def _feed_forward(cfg: KisutarConfig, i: int):
    spec, d, p = cfg.layers[i].get("mlp"), cfg.width, f"l{i}.mlp."
    if spec is None:
        return None
    if spec["kind"] == "dense":
        return DenseMLP(d, spec["ff"], names={k: p + k for k in ("up", "down", "act")}, activation="xielu")
    r, shared = spec["router"], spec.get("shared")
    names = {"router": p + "router", "experts": [(f"{p}e{k}.up", f"{p}e{k}.down") for k in range(r["experts"])]}
    shared_ffn = None
    if shared is not None:
        shared_ffn = DenseMLP(d, shared["ff"], names={k: f"{p}shared.{k}" for k in ("up", "down")}, activation="gelu_erf")
    return MoE(d, r["experts"], r["top"], spec["expert"]["ff"], names=names, activation="gelu_erf", router_weights="softmax_all",
               scale_input=False, shared=shared_ffn)


def build_kisutar(cfg: KisutarConfig) -> DecoderModel:
    d = cfg.width
    blocks, runs = [], []
    for i, layer in enumerate(cfg.layers):
        ffn = _feed_forward(cfg, i)
        norm2 = _norm(cfg, f"l{i}.norm2") if ffn is not None else None
        blocks.append(TokenShiftBlock(_norm(cfg, f"l{i}.norm1"), _mixer(cfg, i), norm2, ffn, names={"shift": f"l{i}.shift"}))
        src = layer["mixer"].get("kv_from")
        # a layer's cache entry carries the layer's number; a reader runs on the entry of the layer it names
        runs.append(LayerRun(i, cache=i) if src is None else LayerRun(i, cache=src, writes=False))
    return DecoderModel(
        vocab_size=cfg.vocab, hidden_size=d, embedding=WeightDecl("embed", (cfg.vocab, d), "normal"),
        blocks=blocks, final_norm=_norm(cfg, "final.norm"), head=WeightDecl("head", (cfg.vocab, d), "normal"),
        schedule=runs, max_positions=cfg.max_positions, pad_hidden=True,
        depth_average=[WeightDecl(f"l{i}.dwa", (i + 2,), f"around:{1.0 / (i + 2)}") for i in range(len(cfg.layers))])
