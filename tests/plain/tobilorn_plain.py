"""Plain Tobilorn decoder: whole sequences, no cache, one function per mechanism.

Every sublayer is normed before and after (RMS norms, weights stored around zero); after the feed-forward a layer adds
what a narrow gated path makes of a vector looked up by the token's id.  The mixer is differential attention: two
softmax maps a head over the same values, the second taken off the first times one learned number a layer, the rest
normed per head; rotated halves, biases, a sliding window that keeps the first tokens visible.  The feed-forward is a
mixture of gated experts behind a softmax router with a correction of the choice and identity experts, plus a shared
expert.  A stretch of the layers runs several times; every pass begins with a projection of the stream joined with the
embedding and a vector of the pass's own.

Everything runs on the CPU in float64 from a configuration (the dict of config.json) and a dict of tensors
by checkpoint name.  Nothing of the product package is imported.

`rnd`: where given, applied to the activations that an engine with bfloat16 activations keeps in bfloat16
between two operations; norms, scores, softmax weights, routers and the residual stream stay exact.
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
def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def zero_centred_norm(x, w, eps):
    """The model's norm: its weight is stored around zero."""
    return unit_rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z / (1.0 + torch.exp(-z))


def rotate_halves(x, base, dims, first=0):
    """x [T, ..., n]: channels i and i + dims / 2 (i < dims / 2) turn by (first + t) base^(-2 i / dims); the rest passes."""
    T = x.shape[0]
    half = dims // 2
    f = base ** (-2.0 * torch.arange(half, dtype=F64) / dims)
    a = torch.arange(first, first + T, dtype=F64)[:, None] * f
    a = a.view((T,) + (1,) * (x.dim() - 2) + (half,))
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a), x[..., dims:]], dim=-1)


# ------------------------------------------------------------------ differential attention
def visible(T, mask):
    """[T, T] bool, i sees j: not after i, and within the window's last `size` or among the first `keep_first`."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    if mask:
        ok = ok & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    return ok


def softmax_map(q, k, scale, ok):
    """One map's weights [T, T] of one head: q, k [T, dim]."""
    s = ((q @ k.T) * scale).masked_fill(~ok, -math.inf)
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def map_weight(W, diff):
    """The number a layer's second map is taken off with."""
    return torch.exp((W["lq1"] * W["lk1"]).sum()) - torch.exp((W["lq2"] * W["lk2"]).sum()) + diff


def combine_maps(a1, a2, lam, diff, eps):
    """Outputs of a head's two maps [..., vdim] -> the head's output."""
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def attention(n, W, m, eps, rnd=_same):
    T = n.shape[0]
    H, G, D, Dv, diff = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["diff"]
    rot = m.get("rot") or {"base": 1.0, "dims": 0}
    q = (n @ W["q"].T + W["q.b"]).view(T, H, 2, D)
    k = (n @ W["k"].T + W["k.b"]).view(T, G, 2, D)
    v = rnd(n @ W["v"].T + W["v.b"]).view(T, G, Dv)
    q, k = rnd(rotate_halves(q, rot["base"], rot["dims"])), rnd(rotate_halves(k, rot["base"], rot["dims"]))
    ok = visible(T, m.get("mask"))
    lam = map_weight(W, diff)
    out = torch.zeros(T, H, Dv, dtype=F64)
    for h in range(H):
        g = h // (H // G)
        a1, a2 = (softmax_map(q[:, h, i], k[:, g, i], m["scale"], ok) @ v[:, g] for i in (0, 1))
        out[:, h] = combine_maps(a1, a2, lam, diff, eps)
    return rnd(out.reshape(T, H * Dv)) @ W["o"].T + W["o.b"]


# ------------------------------------------------------------------------ feed-forward
def route(n, W, router, margins_out=None):
    """ids [T, top] and weights [T, top]: the largest of the softmax over all outputs plus the correction (the lower
    index wins a tie), and the chosen ones' softmax without it, divided by their sum.  margins_out: a list that
    receives, per token, the gap between the last chosen score and the first left out as a share of their softmax scores
    (infinite where all are chosen)."""
    N, top = router["experts"] + router.get("identity", 0), router["top"]
    z = n @ W["router"].T
    s = torch.exp(z - z.max(-1, keepdim=True).values)
    s = s / s.sum(-1, keepdim=True)
    c = s + W["correction"]
    T = n.shape[0]
    ids = torch.zeros(T, top, dtype=torch.long)
    margins = torch.full((T,), math.inf, dtype=F64)
    for t in range(T):
        order = sorted(range(N), key=lambda e: (-c[t, e].item(), e))
        ids[t] = torch.tensor(order[:top])
        if top < N:
            a, b = order[top - 1], order[top]
            margins[t] = (c[t, a] - c[t, b]) / (s[t, a] + s[t, b])
    if margins_out is not None:
        margins_out.append(margins)
    w = torch.gather(s, 1, ids)
    return ids, w / (w.sum(-1, keepdim=True) + 1e-20)


def expert(n, gate, up, down, rnd=_same):
    return rnd(silu(n @ gate.T) * (n @ up.T)) @ down.T


def moe_ff(n, W, spec, rnd=_same, margins_out=None):
    T, d = n.shape
    E = spec["router"]["experts"]
    ids, wts = route(n, W, spec["router"], margins_out)
    out = torch.zeros(T, d, dtype=F64)
    for t in range(T):
        for e, w in zip(ids[t].tolist(), wts[t]):
            y = n[t] if e >= E else expert(n[t], W[f"e{e}.gate"], W[f"e{e}.up"], W[f"e{e}.down"], rnd)
            out[t] = out[t] + w * y
    if spec.get("shared"):
        out = out + expert(n, W["shared.gate"], W["shared.up"], W["shared.down"], rnd)
    return out


# ----------------------------------------------------------------- token input, loop entry
def token_side(x, e, W, eps, rnd=_same):
    """What the per-token vector e [T, dim] adds to the stream: gated by the stream, projected, normed."""
    g = rnd(gelu_tanh(rnd(x) @ W["gate"].T) * e)
    return unit_rms(g @ W["proj"].T, eps) * W["norm"]


def enter_pass(x, x0, w_in, step, rnd=_same):
    """The stream a pass of the loop begins with."""
    return torch.cat([rnd(x), rnd(x0)], dim=-1) @ w_in.T + step


def run_order(cfg):
    """[(layer, pass that begins before it or None)]."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(lp["times"]):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


# ------------------------------------------------------------------------------- model
def _sub(weights, prefix):
    return {k[len(prefix):]: v.to(F64) for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg: dict, weights: dict, tokens, rnd=_same, on_layer=None, margins_out=None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence.  on_layer(i, x): called with the residual stream after every layer run.
    margins_out: see route()."""
    eps = cfg["norm"]["eps"]
    f64 = lambda name: weights[name].to(F64)
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x = x0 = f64("embed")[tokens] * cfg["embedding"]["scale"]
    side = cfg.get("token_side")
    for run, (i, begins) in enumerate(run_order(cfg)):
        layer = cfg["layers"][i]
        if begins is not None:
            x = enter_pass(x, x0, f64("loop.in"), f64("loop.step")[begins], rnd)
        norm = lambda name, y: zero_centred_norm(y, f64(f"l{i}.{name}"), eps)
        x = x + norm("norm1b", attention(rnd(norm("norm1", x)), _sub(weights, f"l{i}.mix."), layer["mixer"], eps, rnd))
        if layer.get("mlp") is not None:
            x = x + norm("norm2b", moe_ff(rnd(norm("norm2", x)), _sub(weights, f"l{i}.mlp."), layer["mlp"], rnd, margins_out))
        if side:
            D = side["dim"]
            x = x + token_side(x, f64("side.embed")[tokens, i * D:(i + 1) * D], _sub(weights, f"l{i}.side."), eps, rnd)
        if on_layer is not None:
            on_layer(run, x)
    return rnd(zero_centred_norm(x, f64("final.norm"), eps)) @ f64("head").T * cfg["logit_scale"]
