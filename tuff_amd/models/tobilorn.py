"""The Tobilorn decoder put together from parts.

x = embed[token] * embedding.scale.  Every sublayer is normed before and after with RMS norms whose stored weight lies around
zero (x / rms * (1 + w)): x <- x + norm_b(sublayer(norm(x))).  The mixer is differential attention (two softmax maps a head
over the same values, the second taken off the first times one learned number a layer, each head normed) with biases, a
rotation of the first rot.dims channels of every map and a sliding window that keeps the sequence's first tokens visible.
The feed-forward is a mixture of silu-gated experts behind a softmax router: the choice runs on the scores plus a
correction, the weights are the chosen scores' shares of their sum, the last router.identity outputs are identity experts; a
shared expert is added.  After it a layer takes in the token's own vector, token_side.dim columns of one table, through a
narrow gated path with a norm.  Layers loop.start .. loop.stop - 1 run loop.times times in a row on the same tensors, each
pass with a cache of its own; every pass begins with a projection of the stream joined with the embedding, plus a vector of
the pass.  Logits = head norm(x) * logit_scale.

Tensors: 'embed', 'head', 'final.norm', 'side.embed', 'loop.in', 'loop.step'; layer i: 'l<i>.norm1', 'l<i>.norm1b',
'l<i>.norm2', 'l<i>.norm2b', 'l<i>.mix.q|k|v|o' with biases '.b', 'l<i>.mix.lq1|lk1|lq2|lk2', 'l<i>.mlp.e<k>.gate|up|down',
'l<i>.mlp.router', 'l<i>.mlp.correction', 'l<i>.mlp.shared.gate|up|down', 'l<i>.side.gate|proj|norm'.
"""
from __future__ import annotations

from ..config.tobilorn import TobilornConfig
from ..parts.attention import DifferentialAttentionMixer
from ..parts.base import WeightDecl
from ..parts.block import SandwichBlock
from ..parts.ffn import MoE, SwiGLU
from ..parts.loop import PassEntry
from ..parts.norm import RMSNorm
from ..parts.rope import Rotary
from ..parts.side import TokenSide
from .decoder import DecoderModel, LayerRun

ROTARY_TABLE_POSITIONS = 8192          # cosines and sines of this many positions are kept in a table


def _norm(cfg: TobilornConfig, name: str) -> RMSNorm:
    return RMSNorm(cfg.width, cfg.eps, name, offset=1.0)


def _mixer(cfg: TobilornConfig, i: int) -> DifferentialAttentionMixer:
    m, p = cfg.layers[i]["mixer"], f"l{i}.mix."
    rot, mask = m.get("rot"), m.get("mask") or {}
    position = None
    if rot and rot["dims"]:
        position = Rotary(m["dim"], rot["base"], rotary_dim=rot["dims"], table_positions=ROTARY_TABLE_POSITIONS)
    keys = ("q", "k", "v", "o", "q.b", "k.b", "v.b", "o.b", "lq1", "lk1", "lq2", "lk2")
    return DifferentialAttentionMixer(cfg.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], scale=m["scale"], diff=m["diff"],
                                      norm_eps=cfg.eps, position=position, window=mask.get("size"), keep_first=mask.get("keep_first", 0),
                                      names={k: p + k for k in keys})


def _feed_forward(cfg: TobilornConfig, i: int):
    spec, d, p = cfg.layers[i].get("mlp"), cfg.width, f"l{i}.mlp."
    if spec is None:
        return None
    r, shared = spec["router"], spec.get("shared")
    names = {"router": p + "router", "correction": p + "correction",
             "experts": [(f"{p}e{k}.gate", f"{p}e{k}.up", f"{p}e{k}.down") for k in range(r["experts"])]}
    shared_ffn = None
    if shared is not None:
        shared_ffn = SwiGLU(d, shared["ff"], names={k: f"{p}shared.{k}" for k in ("gate", "up", "down")})
    return MoE(d, r["experts"], r["top"], spec["expert"]["ff"], names=names, activation="silu", gated=True,
               router_weights="softmax_share", scale_input=False, shared=shared_ffn, identity=r.get("identity", 0))


def _side(cfg: TobilornConfig, i: int):
    if cfg.token_side is None:
        return None
    dim, p = cfg.token_side["dim"], f"l{i}.side."
    return TokenSide(cfg.width, dim, cfg.vocab, len(cfg.layers) * dim, i * dim, cfg.eps,
                     names={"table": "side.embed", "gate": p + "gate", "proj": p + "proj", "norm": p + "norm"})


def build_tobilorn(cfg: TobilornConfig) -> DecoderModel:
    d = cfg.width
    blocks = []
    for i in range(len(cfg.layers)):
        ffn = _feed_forward(cfg, i)
        before2 = _norm(cfg, f"l{i}.norm2") if ffn is not None else None
        after2 = _norm(cfg, f"l{i}.norm2b") if ffn is not None else None
        blocks.append(SandwichBlock(_norm(cfg, f"l{i}.norm1"), _mixer(cfg, i), _norm(cfg, f"l{i}.norm1b"), before2, ffn, after2,
                                    side=_side(cfg, i)))
    runs = [LayerRun(i, enter=begins) for i, begins in cfg.run_order()]        # every run has a cache of its own
    entry = PassEntry(d, cfg.loop["times"], names={"in": "loop.in", "step": "loop.step"}) if cfg.loop else None
    return DecoderModel(
        vocab_size=cfg.vocab, hidden_size=d, embedding=WeightDecl("embed", (cfg.vocab, d), "normal"),
        blocks=blocks, final_norm=_norm(cfg, "final.norm"), head=WeightDecl("head", (cfg.vocab, d), "normal"),
        schedule=runs, max_positions=cfg.max_positions, embedding_scale=float(cfg.embedding["scale"]),
        logit_scale=cfg.logit_scale, pad_hidden=True, entry=entry)
