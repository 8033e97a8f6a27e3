"""The plain Tobilorn implementation pinned by hand values that a plausible misreading fails, mistakes planted in it that
the tests' weights and lengths must show, and the configuration's refusals, declared tensors and caches.  No GPU."""
import copy
import math

import pytest
import torch

import tobilorn_util as tu
import util
from plain import tobilorn_plain as plain

F64 = torch.float64
t64 = lambda v: torch.tensor(v, dtype=F64)


def test_the_models_norm_has_its_weight_around_zero_and_eps_inside_the_root():
    r = math.sqrt(12.5 + 0.5)
    assert torch.allclose(plain.zero_centred_norm(t64([[3.0, 4.0]]), t64([0.0, 1.0]), 0.5), t64([[3.0 / r, 8.0 / r]]))


def test_rotation_pairs_halves_and_turns_by_position():
    x = torch.zeros(3, 5, dtype=F64)
    x[:, 0], x[:, 3], x[:, 4] = 1.0, 2.0, 9.0                     # dims 4: pairs (0, 2) and (1, 3); channel 4 passes
    got = plain.rotate_halves(x, 100.0, 4)
    for p in range(3):
        a0, a1 = p * 1.0, p * 100.0 ** -0.5
        assert torch.allclose(got[p], t64([math.cos(a0), -2.0 * math.sin(a1), math.sin(a0), 2.0 * math.cos(a1), 9.0]))


def test_a_window_holds_the_token_and_size_minus_one_before_it_and_the_first_tokens_stay():
    ok = plain.visible(8, {"size": 3, "keep_first": 2})
    for i in range(8):
        assert [j for j in range(8) if ok[i, j]] == sorted(set(range(max(0, i - 2), i + 1)) | set(range(min(2, i + 1))))
    assert plain.visible(4, {"size": 1}).equal(torch.eye(4, dtype=torch.bool))
    assert plain.visible(3, None).equal(torch.tril(torch.ones(3, 3, dtype=torch.bool)))


def _mixer(H, G, D, Dv, width, seed=0, **m):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g, dtype=F64)
    W = {"q": r(2 * H * D, width), "k": r(2 * G * D, width), "v": r(G * Dv, width), "o": r(width, H * Dv), "q.b": r(2 * H * D), "k.b": r(2 * G * D),
         "v.b": r(G * Dv), "o.b": r(width), "lq1": 0.5 * r(D), "lk1": r(D), "lq2": 0.5 * r(D), "lk2": r(D)}
    return W, dict(dict(heads=H, kv_heads=G, dim=D, vdim=Dv, scale=0.4, diff=0.3, rot={"base": 50.0, "dims": D}), **m), r


def test_the_second_maps_factor_by_hand():
    W = {"lq1": t64([1.0, 2.0]), "lk1": t64([0.5, -0.25]), "lq2": t64([1.0, 0.0]), "lk2": t64([math.log(3.0), 7.0])}
    assert abs(float(plain.map_weight(W, 0.25)) - (1.0 - 3.0 + 0.25)) < 1e-12


def test_maps_lie_side_by_side_per_head_and_share_their_kv_heads_values():
    """Head by head from the definition: rows [head][map][dim] of q and k, kv head floor(h / (H / G)), both maps on its values."""
    W, m, r = _mixer(4, 2, 6, 5, 9)
    n = r(7, 9)
    got = plain.attention(n, W, m, 1e-3)
    heads = []
    i = 6
    for h in range(4):
        g = h // 2
        maps = []
        for c in (0, 1):
            qrow = slice((2 * h + c) * 6, (2 * h + c + 1) * 6)
            krow = slice((2 * g + c) * 6, (2 * g + c + 1) * 6)
            q = plain.rotate_halves((n @ W["q"][qrow].T + W["q.b"][qrow]), 50.0, 6)[i]
            k = plain.rotate_halves((n @ W["k"][krow].T + W["k.b"][krow]), 50.0, 6)
            p = torch.softmax(k @ q * 0.4, 0)
            maps.append(p @ (n @ W["v"][g * 5:(g + 1) * 5].T + W["v.b"][g * 5:(g + 1) * 5]))
        lam = math.exp(float(W["lq1"] @ W["lk1"])) - math.exp(float(W["lq2"] @ W["lk2"])) + 0.3
        o = maps[0] - lam * maps[1]
        heads.append(o / math.sqrt(float((o * o).mean()) + 1e-3) * 0.7)
    assert torch.allclose(got[i], W["o"] @ torch.cat(heads) + W["o.b"])


def test_equal_maps_leave_one_minus_lambda_of_the_plain_attention_before_the_norm():
    W, m, r = _mixer(1, 1, 4, 3, 8, diff=0.3)
    W = dict(W, q=torch.cat([W["q"][:4]] * 2), k=torch.cat([W["k"][:4]] * 2), **{"q.b": torch.cat([W["q.b"][:4]] * 2), "k.b": torch.cat([W["k.b"][:4]] * 2)},
             o=torch.eye(3, dtype=F64), **{"o.b": torch.zeros(3, dtype=F64)})
    n = r(5, 8)
    got = plain.attention(n, W, m, 1e-12)[4]
    assert abs(float((got * got).mean()) - 0.49) < 1e-6            # unit root mean square times 1 - diff, whatever lambda is
    assert torch.allclose(plain.combine_maps(t64([3.0, 4.0]), t64([1.0, 0.0]), t64(2.0), 0.5, 0.5), t64([1.0, 4.0]) / math.sqrt(8.5 + 0.5) * 0.5)


def test_router_chooses_by_corrected_scores_and_weighs_by_shares_of_the_plain_ones():
    n = t64([[1.0, 0.0]])
    W = {"router": t64([[2.0, 0.0], [-1.0, 0.0], [1.0, 0.0], [0.0, 0.0]]), "correction": t64([-1.0, 0.0, 0.0, 0.5])}
    s = torch.softmax(t64([2.0, -1.0, 1.0, 0.0]), 0)
    ids, wts = plain.route(n, W, {"experts": 3, "top": 2, "identity": 1})
    assert ids.tolist() == [[3, 2]] and torch.allclose(wts[0], s[[3, 2]] / (s[3] + s[2]))       # the largest score is corrected away
    ids, _ = plain.route(n, {"router": t64([[0.3, 0.0]] * 4), "correction": torch.zeros(4, dtype=F64)}, {"experts": 4, "top": 2})
    assert ids.tolist() == [[0, 1]]                              # a tie goes to the lower index


def test_identity_experts_hand_back_their_input_and_the_shared_expert_is_added_as_it_is():
    raw = tu.ONLY["moe"]
    W = {k[len("l0.mlp."):]: v.double() for k, v in tu.make_weights(raw, 0).items() if k.startswith("l0.mlp.")}
    n = torch.randn(3, 48, generator=torch.Generator().manual_seed(0), dtype=F64)
    only_identity = dict(W, correction=torch.cat([torch.full((8,), -9.0, dtype=F64), torch.zeros(3, dtype=F64)]))
    got = plain.moe_ff(n, only_identity, tu.moe(8, 2, 24, identity=3))
    assert torch.allclose(got, n)                                # two identity experts whose weights sum to one
    with_shared, without = plain.moe_ff(n, W, tu.moe(8, 2, 24, 3, 32)), plain.moe_ff(n, W, tu.moe(8, 2, 24, 3))
    g = n @ W["shared.gate"].T
    assert torch.allclose(with_shared - without, (g * torch.sigmoid(g) * (n @ W["shared.up"].T)) @ W["shared.down"].T)


def test_token_side_by_hand():
    x, e = t64([[1.0, -2.0, 0.5]]), t64([[3.0, -1.0]])
    W = {"gate": t64([[1.0, 0.0, 0.0], [0.0, 1.0, 0.0]]), "proj": t64([[1.0, 0.0], [0.0, 1.0], [1.0, 1.0]]), "norm": t64([1.0, 2.0, 3.0])}
    gelu = lambda z: 0.5 * z * (1 + math.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))
    g = [gelu(1.0) * 3.0, gelu(-2.0) * -1.0]
    y = [g[0], g[1], g[0] + g[1]]
    r = math.sqrt(sum(v * v for v in y) / 3 + 0.01)
    assert torch.allclose(plain.token_side(x, e, W, 0.01), t64([[y[0] / r, 2 * y[1] / r, 3 * y[2] / r]]))      # a plain weight


def test_passes_begin_with_stream_and_embedding_and_a_vector_of_their_own():
    assert plain.run_order(dict(layers=[0] * 4, loop=dict(start=1, stop=3, times=2))) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert plain.run_order(dict(layers=[0] * 2)) == [(0, None), (1, None)]
    x, x0 = t64([[1.0, 2.0]]), t64([[10.0, 20.0]])
    got = plain.enter_pass(x, x0, t64([[1.0, 0.0, 0.0, 1.0], [0.0, 3.0, 0.0, 0.0]]), t64([100.0, 200.0]))
    assert torch.equal(got, t64([[1.0 + 20.0 + 100.0, 6.0 + 200.0]]))
    # the model: silent sublayers leave what the entries make of the scaled embedding, pass after pass
    raw = tu.ONLY["loop"]
    w = {k: v.double() for k, v in tu.make_weights(raw, 0).items()}
    for i in range(3):
        w[f"l{i}.norm1b"] = torch.full((48,), -1.0, dtype=F64)
    seen = []
    plain.forward(raw, w, [5, 7], on_layer=lambda i, v: seen.append(v))
    e = w["embed"][[5, 7]] * 3.0
    at = e
    want = [e]
    for t in range(3):
        at = at @ w["loop.in"][:, :48].T + e @ w["loop.in"][:, 48:].T + w["loop.step"][t]
        want += [at, at]
    assert len(seen) == 7 and all(torch.allclose(a, b) for a, b in zip(seen, want))


# ------------------------------------------------------- planted mistakes the tests' inputs must show
ALL = ["mixed", "wide", "odd", "plain"]
LOOPED = ["mixed", "wide", "odd"]


def _masks(change):
    def plant(mp, raw):
        for layer in raw["layers"]:
            if layer["mixer"].get("mask"):
                change(layer["mixer"]["mask"])
    return plant


def _patched(name, make):
    """The function `name` of the plain implementation replaced by make(its true form)."""
    return lambda mp, raw: mp.setattr(plain, name, make(getattr(plain, name)))


def _neighbour_pairs(real):
    def turn(x, base, dims, first=0):
        half = dims // 2
        order = [2 * i for i in range(half)] + [2 * i + 1 for i in range(half)] + list(range(dims, x.shape[-1]))
        back = [order.index(i) for i in range(x.shape[-1])]
        return real(x[..., order], base, dims, first)[..., back]
    return turn


def _maps_apart(real):
    """Rows read as [map][head][dim] instead of [head][map][dim]."""
    def attention(n, W, m, eps, rnd=plain._same):
        D, W = m["dim"], dict(W)
        for k, heads in (("q", m["heads"]), ("k", m["kv_heads"])):
            order = [(c * heads + h) * D + j for h in range(heads) for c in (0, 1) for j in range(D)]
            W[k], W[k + ".b"] = W[k][order], W[k + ".b"][order]
        return real(n, W, m, eps, rnd)
    return attention


def _with(**change):
    return _patched("attention", lambda real: lambda n, W, m, eps, rnd=plain._same: real(n, dict(W, **{k: f(W[k]) for k, f in change.items()}), m, eps, rnd))


def _route(change):
    """change(s, W, ids, wts) -> (ids, wts) on what the true route found; s: the softmax over all outputs."""
    def make(real):
        def route(n, W, router, margins_out=None):
            ids, wts = real(n, W, router, margins_out)
            return change(torch.softmax(n @ W["router"].T, -1), W, ids, wts)
        return route
    return _patched("route", make)


def _uncorrected(real):
    return lambda n, W, router, margins_out=None: real(n, dict(W, correction=torch.zeros_like(W["correction"])), router, margins_out)


def _weights_with_correction(s, W, ids, wts):
    w = torch.gather(s + W["correction"], 1, ids)
    return ids, w / (w.sum(-1, keepdim=True) + 1e-20)


def _no_identity_output(real):
    def moe_ff(n, W, spec, rnd=plain._same, margins_out=None):
        out = real(n, W, spec, rnd, margins_out)
        ids, wts = plain.route(n, W, spec["router"])
        return out - n * (wts * (ids >= spec["router"]["experts"])).sum(-1, keepdim=True)
    return moe_ff


def _softmax_over_experts_alone(real):
    """Identity experts left out of the scores' softmax (their own scores from the logits as they are)."""
    def route(n, W, router, margins_out=None):
        E = router["experts"]
        ids, _ = real(n, W, router, margins_out)
        z = n @ W["router"].T
        s = torch.exp(z)
        s = torch.cat([s[:, :E] / s[:, :E].sum(-1, keepdim=True), s[:, E:] / s.sum(-1, keepdim=True)], dim=-1)
        w = torch.gather(s, 1, ids)
        return ids, w / w.sum(-1, keepdim=True)
    return route


def _side_of(shift):
    """Layer i takes the columns of layer i + shift."""
    def plant(mp, raw):
        real = plain.forward
        n = len(raw["layers"])

        def forward(cfg, weights, tokens, **kw):
            D = cfg["token_side"]["dim"]
            t = weights["side.embed"].reshape(-1, n, D)
            return real(cfg, dict(weights, **{"side.embed": t.roll(shift, dims=1).reshape(-1, n * D)}), tokens, **kw)
        mp.setattr(plain, "forward", forward)
    return plant


def _enter(change):
    return _patched("enter_pass", lambda real: lambda x, x0, w_in, step, rnd=plain._same: change(real, x, x0, w_in, step, rnd))


def _step_of_the_first_pass(mp, raw):
    real = plain.forward
    mp.setattr(plain, "forward", lambda cfg, w, toks, **kw: real(cfg, dict(w, **{"loop.step": w["loop.step"][:1].expand_as(w["loop.step"])}), toks, **kw))


def _entered_between_passes_only(mp, raw):
    real = plain.run_order
    mp.setattr(plain, "run_order", lambda cfg: [(i, None if t == 0 else t) for i, t in real(cfg)])


def _halves_swapped(real, x, x0, w_in, step, rnd):
    return real(x0, x, w_in, step, rnd)


MISTAKES = {
    "window_one_longer": (_masks(lambda m: m.update(size=m["size"] + 1)), ALL),
    "one_more_first_token_kept": (_masks(lambda m: m.update(keep_first=m["keep_first"] + 1)), ALL),
    "no_first_tokens_kept": (_masks(lambda m: m.update(keep_first=0)), ALL),
    "neighbouring_channels_paired": (_patched("rotate_halves", _neighbour_pairs), ALL),
    "whole_maps_rotated": (lambda mp, raw: [l["mixer"]["rot"].update(dims=l["mixer"]["dim"] // 2 * 2) for l in raw["layers"]], ["mixed", "wide", "odd"]),
    "maps_apart_instead_of_side_by_side": (_patched("attention", _maps_apart), ALL),
    "maps_swapped": (_patched("combine_maps", lambda real: lambda a1, a2, *a: real(a2, a1, *a)), ALL),
    "second_map_left_out": (_patched("combine_maps", lambda real: lambda a1, a2, *a: real(a1, torch.zeros_like(a2), *a)), ALL),
    "heads_not_normed": (_patched("combine_maps", lambda real: lambda a1, a2, lam, diff, eps: (a1 - lam * a2) * (1 - diff)), ALL),
    "factor_after_the_heads_norm_left_out_of_diff": (_patched("combine_maps", lambda real: lambda a1, a2, lam, diff, eps: real(a1, a2, lam, 0.0, eps)), ["mixed", "odd"]),
    "diff_left_out_of_the_second_maps_factor": (_patched("map_weight", lambda real: lambda W, diff: real(W, 0.0)), ALL),
    "bias_of_the_values_left_out": (_with(**{"v.b": torch.zeros_like}), ALL),
    "bias_of_the_output_left_out": (_with(**{"o.b": torch.zeros_like}), ALL),
    "bias_of_the_keys_left_out": (_with(**{"k.b": torch.zeros_like}), ALL),
    "choice_without_correction": (_patched("route", _uncorrected), ["wide", "odd", "plain"]),
    "weights_with_correction": (_route(_weights_with_correction), ALL),
    "weights_not_renormalised": (_route(lambda s, W, ids, wts: (ids, torch.gather(s, 1, ids))), ["wide", "odd", "plain"]),
    "identity_experts_silent": (_patched("moe_ff", _no_identity_output), ALL),
    "softmax_without_the_identity_experts": (_patched("route", _softmax_over_experts_alone), ALL),
    "side_vectors_of_the_next_layer": (_side_of(-1), LOOPED),
    "side_norm_around_zero": (_patched("token_side", lambda real: lambda x, e, W, eps, rnd=plain._same: real(x, e, dict(W, norm=1.0 + W["norm"]), eps, rnd)), LOOPED),
    "side_gate_reads_the_normed_stream": (_patched("token_side", lambda real: lambda x, e, W, eps, rnd=plain._same: real(plain.unit_rms(x, eps), e, W, eps, rnd)), LOOPED),
    "exact_gelu": (_patched("gelu_tanh", lambda real: lambda z: 0.5 * z * (1 + torch.erf(z / math.sqrt(2)))), ["mixed", "odd"]),
    "pass_vector_always_the_firsts": (_step_of_the_first_pass, LOOPED),
    "first_pass_without_its_entry": (_entered_between_passes_only, LOOPED),
    "halves_of_the_entry_swapped": (_enter(_halves_swapped), LOOPED),
    "entry_added_to_the_stream": (_enter(lambda real, x, *a: x + real(x, *a)), LOOPED),
    "logits_not_scaled": (lambda mp, raw: raw.update(logit_scale=1.0), ["mixed", "wide", "odd"]),
    "embedding_not_scaled": (lambda mp, raw: raw["embedding"].update(scale=1.0), ["mixed", "wide", "odd"]),
}


@pytest.mark.parametrize("mistake", sorted(MISTAKES))
def test_planted_mistakes_move_the_logits_far_beyond_the_gpu_tests_tolerance(mistake, monkeypatch):
    """A mistake of the oracle shows, in the configurations and at the lengths the GPU tests use, at twenty and more
    times what they allow in float32: a product with that mistake could not pass them."""
    plant, names = MISTAKES[mistake]
    for name in names:
        raw = tu.CONFIGS[name]
        w = tu.make_weights(raw, 0)
        toks = util.rand_tokens(90, raw["vocab"], 0)
        want = plain.forward(raw, w, toks)
        with monkeypatch.context() as mp:
            changed = copy.deepcopy(raw)
            plant(mp, changed)
            got = plain.forward(changed, w, toks)
        over = ((got - want).abs() / (2e-5 + 1e-4 * want.abs())).max()
        assert over > 20.0, (name, float(over))


# ---------------------------------------------------------------------- configuration and caches
def test_configuration_reads_every_size_and_refuses_what_it_cannot_run():
    from tuff_amd.config.base import ConfigError
    from tuff_amd.models.registry import build_model, config_from_dict
    for name, raw in tu.CONFIGS.items():
        cfg = config_from_dict(copy.deepcopy(raw))
        assert cfg.unknown_keys == [] and config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict(), name
        model = build_model(cfg)
        assert [(r.block, r.enter) for r in model.schedule] == plain.run_order(raw), name
        assert model.logit_scale == raw["logit_scale"] and model.embedding_scale == raw["embedding"]["scale"]
        for i, (b, layer) in enumerate(zip(model.blocks, raw["layers"])):
            m, mask = layer["mixer"], layer["mixer"].get("mask") or {}
            assert (b.mixer.heads, b.mixer.Hkv, b.mixer.dim, b.mixer.vd, b.mixer.scale, b.mixer.diff, b.mixer.window, b.mixer.keep_first) == \
                (m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], m["diff"], mask.get("size"), mask.get("keep_first", 0))
            assert (b.mixer.position is None) == (m["rot"]["dims"] == 0)
            if b.mixer.position is not None:
                assert (b.mixer.position.base, b.mixer.position.rotary_dim) == (m["rot"]["base"], m["rot"]["dims"])
            assert b.before1.eps == b.after1.eps == b.mixer.eps == raw["norm"]["eps"] and b.before1.offset == 1.0 and (b.ffn is None) == (layer["mlp"] is None)
            assert (b.side is None) == ("token_side" not in raw)
            if b.side is not None:
                assert (b.side.dim, b.side.col0, b.side.norm.offset) == (raw["token_side"]["dim"], i * raw["token_side"]["dim"], 0.0)
    bad = [
        lambda r: r["layers"][0].update(type="latent_attention"),
        lambda r: r["layers"][0]["mixer"].pop("diff"),
        lambda r: r["layers"][0]["mixer"].update(heads=3),
        lambda r: r["layers"][0]["mixer"].update(dim=0),
        lambda r: r["layers"][0]["mixer"].update(scale=-1.0),
        lambda r: r["layers"][0]["mixer"]["rot"].update(base=0),
        lambda r: r["layers"][0]["mixer"]["rot"].update(dims=7),
        lambda r: r["layers"][0]["mixer"]["rot"].update(dims=18),
        lambda r: r["layers"][0]["mixer"].update(mask={"size": 0}),
        lambda r: r["layers"][0]["mixer"].update(mask={"size": 4, "keep_first": -1}),
        lambda r: r["layers"][0]["mlp"]["router"].update(top=9),
        lambda r: r["layers"][0]["mlp"]["router"].update(identity=-1),
        lambda r: r["layers"][0]["mlp"]["shared"].update(ff=0),
        lambda r: r["layers"][0]["mlp"].update(kind="dense"),
        lambda r: r["layers"][0]["mlp"].pop("expert"),
        lambda r: r["loop"].update(start=3),
        lambda r: r["loop"].update(stop=5),
        lambda r: r["loop"].update(times=0),
        lambda r: r["token_side"].update(dim=0),
        lambda r: r["norm"].update(eps=0),
        lambda r: r.update(logit_scale="big"),
        lambda r: r.pop("vocab"),
    ]
    for i, spoil in enumerate(bad):
        raw = copy.deepcopy(tu.T_MIXED)
        spoil(raw)
        with pytest.raises(ConfigError):
            config_from_dict(raw)
            pytest.fail(f"case {i} was accepted")


def test_declared_tensors_and_caches():
    from tuff_amd.cache.manager import CacheLayout
    from tuff_amd.models.registry import build_model, config_from_dict
    from tuff_amd.parts.base import PagedKV
    model = build_model(config_from_dict(copy.deepcopy(tu.T_MIXED)))
    decls = {d.name: tuple(d.shape) for d in model.weight_decls()}
    assert len(decls) == len(model.weight_decls())
    assert decls["l0.mix.q"] == (2 * 4 * 16, 64) and decls["l0.mix.k"] == (2 * 2 * 16, 64) and decls["l0.mix.v"] == (2 * 24, 64)
    assert decls["l0.mix.o"] == (64, 4 * 24) and decls["l0.mix.o.b"] == (64,) and decls["l0.mix.v.b"] == (48,) and decls["l0.mix.lk2"] == (16,)
    assert decls["l0.mlp.router"] == (4, 64) and decls["l0.mlp.correction"] == (4,) and decls["l0.mlp.e2.down"] == (64, 40)
    assert decls["l0.mlp.shared.gate"] == (48, 64) and "l0.mlp.e3.gate" not in decls and "l3.mlp.shared.up" not in decls
    assert "l1.norm2" not in decls and "l1.norm2b" not in decls and decls["l1.norm1b"] == (64,)
    assert decls["side.embed"] == (211, 64) and decls["l2.side.gate"] == (16, 64) and decls["l2.side.proj"] == (64, 16) and decls["l2.side.norm"] == (64,)
    assert decls["loop.in"] == (64, 128) and decls["loop.step"] == (3, 64)
    # an entry of its own for every run of a looped layer; groups by window and kept first tokens
    layout = CacheLayout.from_specs(model.cache_specs)
    a, b, c, d = PagedKV(2, 32, 20, 24, keep_first=3), PagedKV(1, 16, 33, keep_first=17), PagedKV(2, 48, None, 32), PagedKV(2, 32, 16, 8)
    assert [layout.paged[i] for i in sorted(layout.paged)] == [a, b, c, b, c, b, c, d]
    assert list(zip(layout.group_windows, layout.group_keeps)) == [(20, 3), (33, 17), (None, 0), (16, 0)]
    plain_names = {d.name for d in build_model(config_from_dict(copy.deepcopy(tu.T_PLAIN))).weight_decls()}
    assert not any(n.startswith(("loop.", "side.")) or ".side." in n for n in plain_names)


def test_a_model_with_an_entry_refuses_what_does_not_go_with_it():
    from tuff_amd.models.decoder import DecoderModel, LayerRun
    from tuff_amd.models.registry import build_model, config_from_dict
    base = build_model(config_from_dict(copy.deepcopy(tu.ONLY["loop"])))
    kw = dict(vocab_size=101, hidden_size=48, embedding=base.embedding_decl, blocks=base.blocks, final_norm=base.final_norm, head=base.head_decl)
    with pytest.raises(ValueError, match="without an entry"):
        DecoderModel(schedule=[LayerRun(0, enter=0)], **kw)
    with pytest.raises(ValueError, match="outside 0"):
        DecoderModel(schedule=[LayerRun(0, enter=3)], entry=base.entry, **kw)
    with pytest.raises(ValueError, match="hand on the stream"):
        DecoderModel(schedule=[], entry=base.entry, **dict(kw, blocks=[]))
    assert DecoderModel(schedule=[LayerRun(0), LayerRun(1)], **kw).entry is None


def test_parts_refuse_what_they_cannot_run():
    from tuff_amd.parts.attention import AttentionMixer, DifferentialAttentionMixer
    from tuff_amd.parts.ffn import MoE
    from tuff_amd.parts.rope import Rotary
    names = {k: k for k in ("q", "k", "v", "o", "lq1", "lk1", "lq2", "lk2")}
    kw = dict(names=names, scale=0.5, diff=0.1, norm_eps=1e-5)
    with pytest.raises(ValueError, match="multiple of kv heads"):
        DifferentialAttentionMixer(32, 3, 2, 8, 8, **kw)
    with pytest.raises(ValueError, match="half-split"):
        DifferentialAttentionMixer(32, 2, 2, 8, 8, position=Rotary(8, 100.0, interleaved=True), **kw)
    with pytest.raises(ValueError, match="wide"):
        DifferentialAttentionMixer(32, 2, 2, 330, 8, **kw)
    with pytest.raises(ValueError, match="exact_weights"):
        AttentionMixer(32, 2, 2, 8, names={k: k for k in "qkvo"}, window=8, keep_first=2)
    experts = [("g", "u", "d")] * 3
    with pytest.raises(ValueError, match="softmax"):
        MoE(32, 3, 2, 8, names={"router": "r", "experts": experts}, activation="silu", gated=True, router_weights="sigmoid", scale_input=False, identity=1)
    with pytest.raises(ValueError, match="no groups"):
        MoE(32, 3, 2, 8, names={"router": "r", "experts": experts}, activation="silu", gated=True, router_weights="softmax_share", scale_input=False,
            route_scale=2.0)


def test_random_model_folder_round_trip(tmp_path):
    from tuff_amd.models.registry import build_model, config_from_dict, load_config
    from tuff_amd.weights.loader import Checkpoint
    from tuff_amd.weights.random_init import write_random_model
    cfg = config_from_dict(copy.deepcopy(tu.T_MIXED))
    write_random_model(cfg, str(tmp_path), seed=3)
    assert load_config(str(tmp_path)).to_dict() == cfg.to_dict()
    assert set(Checkpoint(str(tmp_path)).names()) == {d.name for d in build_model(cfg).weight_decls()}
