"""Plain Kisutar decoder: whole sequences, no cache, one function per mechanism.

Pre-norm layers with RMS norms.  What a mixer reads is mixed channel by channel with the row the token before it
had there (token shift); after every layer the stream is replaced by a learned weighted sum of the embedding and
the results of all layers so far (depth average).  The mixer is latent attention: queries through a narrow normed
row, keys and values expanded from one narrow normed row a token, a rotated key part shared by the heads, a
sliding window and a sink per head; a layer may read the latent rows and rotated keys of an earlier layer.
Feed-forwards: a dense layer with the xIELU activation, or experts with the exact gelu behind a router whose
weights are the plain softmax over all experts, plus a shared expert.

Everything runs on the CPU in float64 from a configuration (the dict of config.json) and a dict of tensors
by checkpoint name.  Nothing of the product package is imported.

`rnd`: where given, applied to the activations that an engine with bfloat16 activations keeps in bfloat16
between two operations; norms, scores, routers, the shift and the residual stream stay exact.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def _same(t):
    return t


def bf16_round(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.float32).to(torch.bfloat16).to(t.dtype)


# ------------------------------------------------------------------------ small functions
def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def xielu(z, p, q):
    """z > 0: softplus(p) z^2 + z / 2;  z <= 0: (1/2 + softplus(q)) (e^z - 1 - z) + z / 2."""
    neg = torch.clamp(z, max=0.0)
    return torch.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (torch.expm1(neg) - neg)) + 0.5 * z


def token_shift(h, mix):
    """h[t] + (h[t - 1] - h[t]) * mix, zeros before the first token; h [T, d], mix [d]."""
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (prev - h) * mix


def depth_average(states, w):
    """sum_j w[j] states[j]: states are the embedding and the layers' results so far."""
    out = torch.zeros_like(states[0])
    for x, wj in zip(states, w):
        out = out + wj * x
    return out


def rotate_halves(x, base, dims, first=0):
    """x [T, ..., n]: channels i and i + dims / 2 (i < dims / 2) turn by (first + t) base^(-2 i / dims); the rest passes."""
    T = x.shape[0]
    half = dims // 2
    f = base ** (-2.0 * torch.arange(half, dtype=F64) / dims)
    a = torch.arange(first, first + T, dtype=F64)[:, None] * f
    a = a.view((T,) + (1,) * (x.dim() - 2) + (half,))
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a), x[..., dims:]], dim=-1)


# ----------------------------------------------------------------------- latent attention
def latent_rows(n, W, m, eps, rnd=_same):
    """What is kept of every token: the normed latent c [T, rank] and the rotated shared key part [T, rot]."""
    rank = m["kv_rank"]
    row = n @ W["dkv"].T
    c = rnd(rms_norm(row[:, :rank], W["dkv.norm"], eps))
    return c, rnd(rotate_halves(row[:, rank:], m["rot"]["base"], m["rot"]["dims"]))


def queries(n, W, m, eps, rnd=_same):
    """[T, heads, dim + rot]: through the narrow normed row, the last rot channels of a head rotated."""
    H, dk, dr = m["heads"], m["dim"], m["rot_dim"]
    cq = rnd(rms_norm(n @ W["dq"].T, W["dq.norm"], eps))
    q = rnd(cq @ W["uq"].T).view(-1, H, dk + dr)
    return torch.cat([q[..., :dk], rnd(rotate_halves(q[..., dk:], m["rot"]["base"], m["rot"]["dims"]))], dim=-1)


def latent_attention(n, rows, W, m, eps, rnd=_same, absorbed=False):
    """n [T, d], rows (this layer's or an earlier layer's) -> [T, d].  absorbed: with roundings, those of an engine
    that carries the queries into the latent space and sums latent rows (the same function without)."""
    T = n.shape[0]
    H, dk, dv, rank = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
    c, kr = rows
    q = queries(n, W, m, eps, rnd)
    uk, uv = W["uk"].view(H, dk, rank), W["uv"].view(H, dv, rank)
    if absorbed:
        ql = rnd(torch.einsum("ihd,hdr->ihr", q[..., :dk], uk))
        s = torch.einsum("ihr,jr->hij", ql, c)
    else:
        s = torch.einsum("ihd,jhd->hij", q[..., :dk], rnd(torch.einsum("jr,hdr->jhd", c, uk)))
    s = (s + torch.einsum("ihe,je->hij", q[..., dk:], kr)) * m["scale"]
    away = torch.arange(T)[:, None] - torch.arange(T)[None, :]                # i - j
    hidden = away < 0
    if m.get("mask"):
        hidden = hidden | (away >= m["mask"]["size"])
    s = s.masked_fill(hidden[None], -math.inf)
    top = torch.maximum(s.max(-1).values, W["sink"][:, None])                  # [H, T]
    e = torch.exp(s - top[..., None])
    p = e / (e.sum(-1) + torch.exp(W["sink"][:, None] - top))[..., None]
    if absorbed:
        o = torch.einsum("ihr,hdr->ihd", rnd(torch.einsum("hij,jr->ihr", p, c)), uv)
    else:
        o = torch.einsum("hij,jhd->ihd", p, rnd(torch.einsum("jr,hdr->jhd", c, uv)))
    return rnd(o.reshape(T, H * dv)) @ W["o"].T


# ------------------------------------------------------------------------ feed-forwards
def dense_ff(n, W, rnd=_same):
    return rnd(xielu(n @ W["up"].T, W["act"][0], W["act"][1])) @ W["down"].T


def route(n, W, spec, margins_out=None):
    """ids [T, top] and weights [T, top]: the largest logits (the lower index wins a tie) and their shares of the
    softmax over all experts.  margins_out: a list that receives, per token, the gap between the last chosen logit and
    the first left out as a share of the logits' spread (infinite where all are chosen)."""
    E, top = spec["router"]["experts"], spec["router"]["top"]
    z = n @ W["router"].T
    s = torch.exp(z - z.max(-1, keepdim=True).values)
    s = s / s.sum(-1, keepdim=True)
    T = n.shape[0]
    ids = torch.zeros(T, top, dtype=torch.long)
    margins = torch.full((T,), math.inf, dtype=F64)
    spread = (z - z.mean()).pow(2).mean().sqrt().clamp_min(1e-30)
    for t in range(T):
        order = sorted(range(E), key=lambda e: (-z[t, e].item(), e))
        ids[t] = torch.tensor(order[:top])
        if top < E:
            margins[t] = (z[t, order[top - 1]] - z[t, order[top]]) / spread
    if margins_out is not None:
        margins_out.append(margins)
    return ids, torch.gather(s, 1, ids)


def expert(n, up, down, rnd=_same):
    return rnd(gelu_erf(n @ up.T)) @ down.T


def moe_ff(n, W, spec, rnd=_same, margins_out=None):
    T, d = n.shape
    ids, wts = route(n, W, spec, margins_out)
    out = torch.zeros(T, d, dtype=F64)
    for t in range(T):
        for e, w in zip(ids[t].tolist(), wts[t]):
            out[t] = out[t] + w * expert(n[t], W[f"e{e}.up"], W[f"e{e}.down"], rnd)
    if spec.get("shared"):
        out = out + expert(n, W["shared.up"], W["shared.down"], rnd)
    return out


# ------------------------------------------------------------------------------- model
def _sub(weights, prefix):
    return {k[len(prefix):]: v.to(F64) for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg: dict, weights: dict, tokens, rnd=_same, on_layer=None, margins_out=None, absorbed=False) -> torch.Tensor:
    """Logits [T, vocab] of one sequence.  on_layer(i, x): called with the residual stream after every layer (after its
    depth average).  margins_out: see route()."""
    eps = cfg["norm"]["eps"]
    f64 = lambda name: weights[name].to(F64)
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x = f64("embed")[tokens]
    states, kept = [x], {}
    for i, layer in enumerate(cfg["layers"]):
        m, W = layer["mixer"], _sub(weights, f"l{i}.mix.")
        n = rnd(token_shift(rms_norm(x, f64(f"l{i}.norm1"), eps), f64(f"l{i}.shift")))
        src = m.get("kv_from")
        if src is None:
            kept[i] = latent_rows(n, W, m, eps, rnd)
            src = i
        x = x + latent_attention(n, kept[src], W, m, eps, rnd, absorbed)
        spec = layer.get("mlp")
        if spec is not None:
            n = rnd(rms_norm(x, f64(f"l{i}.norm2"), eps))
            Wf = _sub(weights, f"l{i}.mlp.")
            x = x + (dense_ff(n, Wf, rnd) if spec["kind"] == "dense" else moe_ff(n, Wf, spec, rnd, margins_out))
        states.append(x)
        x = depth_average(states, f64(f"l{i}.dwa"))
        if on_layer is not None:
            on_layer(i, x)
    return rnd(rms_norm(x, f64("final.norm"), eps)) @ f64("head").T
