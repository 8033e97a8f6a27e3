"""The plain Kisutar implementation pinned by hand values that a plausible misreading fails, mistakes planted in it that
the tests' weights and lengths must show, and the configuration's refusals, declared tensors and caches.  No GPU."""
import copy
import math

import pytest
import torch

import kisutar_util as su
import util
from plain import kisutar_plain as plain

F64 = torch.float64
t64 = lambda v: torch.tensor(v, dtype=F64)


def test_rms_norm_has_eps_inside_the_root():
    got = plain.rms_norm(t64([[3.0, 4.0]]), t64([1.0, 2.0]), 0.5)
    r = math.sqrt(12.5 + 0.5)
    assert torch.allclose(got, t64([[3.0 / r, 8.0 / r]]))


def test_token_shift_reads_the_row_before_as_it_was_and_zeros_before_the_first():
    h = t64([[1.0, 10.0], [2.0, 20.0], [4.0, 40.0]])
    got = plain.token_shift(h, t64([0.5, 1.0]))
    # the second channel is the row before outright; the first halfway to the row before as it stood, not as it came out
    assert torch.equal(got, t64([[0.5, 0.0], [1.5, 10.0], [3.0, 20.0]]))
    assert torch.equal(plain.token_shift(h, t64([0.0, -1.0])), t64([[1.0, 20.0], [2.0, 30.0], [4.0, 60.0]]))


def test_depth_average_sums_the_embedding_and_every_result():
    assert torch.equal(plain.depth_average([t64([1.0, 2.0]), t64([10.0, 20.0]), t64([100.0, 200.0])], t64([3.0, 2.0, -1.0])), t64([-77.0, -154.0]))


def test_a_layers_result_is_what_is_kept_and_its_sum_is_what_goes_on():
    """Two layers whose sublayers are silent: X_0 = X_1 = the embedding, so the stream after the first layer is
    (w00 + w01) X_0, the second layer's result is that, and the last stream w10 X_0 + w11 X_0 + w12 (w00 + w01) X_0."""
    raw = su.S_PLAIN
    w = {k: v.double() for k, v in su.make_weights(raw, 0).items()}
    for k in w:
        if k.endswith(".mix.o") or k.endswith(".down"):
            w[k] = torch.zeros_like(w[k])
    seen = []
    plain.forward(raw, w, [5, 7], on_layer=lambda i, x: seen.append(x))
    e, a, b = w["embed"][[5, 7]], w["l0.dwa"], w["l1.dwa"]
    assert torch.allclose(seen[0], (a[0] + a[1]) * e)
    assert torch.allclose(seen[1], (b[0] + b[1] + b[2] * (a[0] + a[1])) * e)


def test_xielu_by_hand_on_both_sides_and_its_numbers_pass_a_softplus():
    p, q = t64(0.3), t64(-0.8)
    sp = lambda v: math.log1p(math.exp(float(v)))
    for z in (2.0, 0.25, 0.0, -0.5, -3.0):
        want = sp(p) * z * z + z / 2 if z > 0 else (0.5 + sp(q)) * (math.exp(z) - 1 - z) + z / 2
        assert abs(float(plain.xielu(t64(z), p, q)) - want) < 1e-12, z
    assert float(plain.xielu(t64(0.0), p, q)) == 0.0


def test_experts_use_the_exact_gelu():
    z = t64([1.0, -0.7])
    want = t64([0.5 * v * (1 + math.erf(v / math.sqrt(2))) for v in (1.0, -0.7)])
    assert torch.allclose(plain.gelu_erf(z), want, atol=1e-14)


def test_rotation_pairs_halves_and_turns_by_position():
    x = torch.zeros(3, 5, dtype=F64)
    x[:, 0], x[:, 3], x[:, 4] = 1.0, 2.0, 9.0                     # dims 4: pairs (0, 2) and (1, 3); channel 4 passes
    got = plain.rotate_halves(x, 100.0, 4)
    for p in range(3):
        a0, a1 = p * 1.0, p * 100.0 ** -0.5
        assert torch.allclose(got[p], t64([math.cos(a0), -2.0 * math.sin(a1), math.sin(a0), 2.0 * math.cos(a1), 9.0]))


def _latent_weights(H, dk, dr, dv, rank, sink, q_rank=None):
    """A mixer whose narrow projections pick columns: a row of the input is [query row | latent | rotated key]."""
    g = torch.Generator().manual_seed(H + dk + dr)
    r = lambda *s: torch.randn(*s, generator=g, dtype=F64)
    q_rank = H * (dk + dr) if q_rank is None else q_rank
    width = q_rank + rank + dr
    eye = torch.eye(width, dtype=F64)
    W = {"dq": eye[:q_rank], "dq.norm": 1.0 + 0.3 * r(q_rank), "uq": torch.eye(q_rank, dtype=F64) if q_rank == H * (dk + dr) else r(H * (dk + dr), q_rank),
         "dkv": eye[q_rank:], "dkv.norm": 1.0 + 0.3 * r(rank), "uk": r(H * dk, rank), "uv": r(H * dv, rank), "sink": t64(sink),
         "o": torch.eye(H * dv, dtype=F64)}
    m = dict(heads=H, dim=dk, rot_dim=dr, vdim=dv, q_rank=q_rank, kv_rank=rank, scale=0.4, rot={"base": 50.0, "dims": dr})
    return W, m, width


def test_sink_counts_once_unscaled_without_a_value_and_the_window_holds_the_token_and_size_minus_one_before_it():
    W, m, width = _latent_weights(1, 2, 2, 3, 2, [math.log(3.0)])
    T = 7
    n = torch.zeros(T, width, dtype=F64)
    n[:, 4:6] = torch.randn(T, 2, generator=torch.Generator().manual_seed(1), dtype=F64)
    rows = plain.latent_rows(n, W, m, 1e-5)
    v = rows[0] @ W["uv"].T
    # zero queries: every score is 0, so the weights are 1 / (keys seen + exp(sink)) = 1 / (seen + 3)
    got = plain.latent_attention(n, rows, W, m, 1e-5)
    for i in range(T):
        assert torch.allclose(got[i], v[:i + 1].sum(0) / (i + 1 + 3.0))
    got = plain.latent_attention(n, rows, W, dict(m, mask={"size": 3}), 1e-5)
    for i in range(T):
        lo = max(0, i - 2)
        assert torch.allclose(got[i], v[lo:i + 1].sum(0) / (i + 1 - lo + 3.0))
    assert torch.allclose(plain.latent_attention(n, rows, W, dict(m, mask={"size": 1}), 1e-5), v / 4.0)


def test_queries_and_latents_are_normed_before_their_expansions_the_rotated_key_is_not_and_both_parts_are_scaled():
    W, m, width = _latent_weights(2, 3, 4, 2, 5, [-30.0, -30.0], q_rank=6)            # sinks that hold nothing
    n = torch.randn(4, width, generator=torch.Generator().manual_seed(2), dtype=F64)
    eps = 0.1
    rows = plain.latent_rows(n, W, m, eps)
    raw = n[:, 6:11]
    assert torch.allclose(rows[0], raw / torch.sqrt((raw * raw).mean(-1, keepdim=True) + eps) * W["dkv.norm"])
    assert torch.allclose(rows[1], plain.rotate_halves(n[:, 11:], 50.0, 4))
    cq = n[:, :6] / torch.sqrt((n[:, :6] ** 2).mean(-1, keepdim=True) + eps) * W["dq.norm"]
    got = plain.latent_attention(n, rows, W, m, eps)[3]
    for h in range(2):
        q = W["uq"][7 * h:7 * h + 7] @ cq[3]
        qr = plain.rotate_halves(q[None, 3:], 50.0, 4, first=3)[0]
        s = ((rows[0] @ W["uk"][3 * h:3 * h + 3].T) @ q[:3] + rows[1] @ qr) * 0.4
        p = torch.softmax(s, 0)
        assert torch.allclose(got[2 * h:2 * h + 2], p @ (rows[0] @ W["uv"][2 * h:2 * h + 2].T), atol=1e-10)
    # carrying the queries into the latent space is the same function
    assert torch.allclose(plain.latent_attention(n, rows, W, m, eps, absorbed=True)[3], got, atol=1e-12)


def test_a_layer_reads_the_rows_of_the_layer_it_names():
    raw = su.ONLY["latent_shared"]
    w = {k: v.double() for k, v in su.make_weights(raw, 0).items()}
    assert "l1.mix.dkv" not in w and "l1.mix.uk" in w and "l2.mix.uv" in w and "l1.mix.dq" in w
    silent = dict(w)
    silent["l0.mix.o"] = torch.zeros_like(w["l0.mix.o"])
    a = plain.forward(raw, silent, [3, 9, 27, 81, 5])
    other = dict(silent)
    other["l0.mix.dkv"] = w["l0.mix.dkv"].flip(0)               # the first layer's own output is gone: only its readers move
    assert (plain.forward(raw, other, [3, 9, 27, 81, 5]) - a).abs().max() > 1e-6


def test_router_weights_are_shares_of_the_softmax_over_all_experts():
    n = t64([[1.0, 0.0]])
    W = {"router": t64([[2.0, 0.0], [-1.0, 0.0], [1.0, 0.0], [0.0, 0.0]])}
    s = torch.softmax(t64([2.0, -1.0, 1.0, 0.0]), 0)
    ids, wts = plain.route(n, W, su.moe(4, 2, 8))
    assert ids.tolist() == [[0, 2]] and torch.allclose(wts[0], s[[0, 2]]) and float(wts.sum()) < 0.99
    ids, _ = plain.route(n, {"router": t64([[0.3, 0.0]] * 4)}, su.moe(4, 2, 8))
    assert ids.tolist() == [[0, 1]]                              # a tie goes to the lower index


def test_the_shared_expert_runs_for_every_token_and_is_added_as_it_is():
    raw = su.ONLY["moe"]
    W = {k[len("l0.mlp."):]: v.double() for k, v in su.make_weights(raw, 0).items() if k.startswith("l0.mlp.")}
    n = torch.randn(3, 48, generator=torch.Generator().manual_seed(0), dtype=F64)
    with_shared, without = plain.moe_ff(n, W, su.moe(8, 2, 24, 32)), plain.moe_ff(n, W, su.moe(8, 2, 24))
    want = plain.gelu_erf(n @ W["shared.up"].T) @ W["shared.down"].T
    assert torch.allclose(with_shared - without, want)


# ------------------------------------------------------- planted mistakes the tests' inputs must show
def _window(change):
    def plant(mp, raw):
        for layer in raw["layers"]:
            if layer["mixer"].get("mask"):
                layer["mixer"]["mask"]["size"] += change
    return plant


def _patched(name, fn):
    return lambda mp, raw: mp.setattr(plain, name, fn)


def _shift_of_the_shifted(h, mix):
    out = torch.zeros_like(h)
    prev = torch.zeros_like(h[0])
    for t in range(h.shape[0]):
        out[t] = h[t] + (prev - h[t]) * mix
        prev = out[t]
    return out


def _shift_lost_at(place):
    real = plain.token_shift

    def lost(h, mix):
        out = real(h, mix)
        if h.shape[0] > place:
            out[place] = h[place] - h[place] * mix
        return out
    return lost


def _neighbour_pairs(x, base, dims, first=0):
    half = dims // 2
    order = [2 * i for i in range(half)] + [2 * i + 1 for i in range(half)] + list(range(dims, x.shape[-1]))
    back = [order.index(i) for i in range(x.shape[-1])]
    return _real_rotate(x[..., order], base, dims, first)[..., back]


_real_rotate = plain.rotate_halves
_real_average = plain.depth_average


def _no_sinks(mp, raw):
    real = plain.latent_attention
    mp.setattr(plain, "latent_attention", lambda n, rows, W, m, eps, *a: real(n, rows, dict(W, sink=W["sink"] - 50.0), m, eps, *a))


def _readers_take_the_writers_window(mp, raw):
    for layer in raw["layers"]:
        src = layer["mixer"].get("kv_from")
        if src is not None:
            layer["mixer"]["mask"] = raw["layers"][src]["mixer"].get("mask")


def _softmax_over_the_chosen(mp, raw):
    real = plain.route

    def route(*a, **kw):
        ids, wts = real(*a, **kw)
        return ids, wts / wts.sum(-1, keepdim=True)
    mp.setattr(plain, "route", route)


MISTAKES = {
    "window_one_longer": (_window(1), ["mixed", "wide", "odd", "plain"]),
    "no_sinks": (_no_sinks, ["mixed", "wide", "odd", "plain"]),
    "shift_of_the_shifted_row": (_patched("token_shift", _shift_of_the_shifted), ["mixed", "wide", "odd", "plain"]),
    "shift_left_out": (_patched("token_shift", lambda h, mix: h), ["mixed", "wide", "odd", "plain"]),
    "shift_state_lost_in_one_place": (_patched("token_shift", _shift_lost_at(40)), ["mixed", "wide", "odd", "plain"]),
    "neighbouring_channels_paired": (_patched("rotate_halves", _neighbour_pairs), ["mixed", "wide", "odd", "plain"]),
    "positions_one_off_in_queries_and_keys_apart": (_patched("queries", lambda n, W, m, eps, rnd=plain._same: _late_queries(n, W, m, eps, rnd)),
                                                    ["mixed", "wide", "odd", "plain"]),
    "the_embedding_left_out_of_the_sums": (_patched("depth_average", lambda xs, w: _real_average(xs[1:], w[1:])), ["mixed", "wide", "odd", "plain"]),
    "readers_take_the_writers_window": (_readers_take_the_writers_window, ["mixed", "wide", "odd"]),
    "weights_renormalised": (_softmax_over_the_chosen, ["wide", "odd", "plain"]),
    "tanh_gelu": (_patched("gelu_erf", lambda z: 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))), ["mixed", "wide", "odd", "plain"]),
    "activation_numbers_swapped": (lambda mp, raw: mp.setattr(plain, "xielu", _swapped(plain.xielu)), ["mixed", "wide", "odd", "plain"]),
}


def _swapped(real):
    return lambda z, p, q: real(z, q, p)


def _late_queries(n, W, m, eps, rnd):
    H, dk, dr = m["heads"], m["dim"], m["rot_dim"]
    q = (plain.rms_norm(n @ W["dq"].T, W["dq.norm"], eps) @ W["uq"].T).view(-1, H, dk + dr)
    return torch.cat([q[..., :dk], plain.rotate_halves(q[..., dk:], m["rot"]["base"], m["rot"]["dims"], first=1)], dim=-1)


@pytest.mark.parametrize("mistake", sorted(MISTAKES))
def test_planted_mistakes_move_the_logits_far_beyond_the_gpu_tests_tolerance(mistake, monkeypatch):
    """A mistake of the oracle shows, in the configurations and at the lengths the GPU tests use, at twenty and more
    times what they allow in float32: a product with that mistake could not pass them."""
    plant, names = MISTAKES[mistake]
    for name in names:
        raw = su.CONFIGS[name]
        w = su.make_weights(raw, 0)
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
    for name, raw in su.CONFIGS.items():
        cfg = config_from_dict(copy.deepcopy(raw))
        assert cfg.unknown_keys == [] and config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict(), name
        model = build_model(cfg)
        assert len(model.schedule) == len(raw["layers"]), name
        for b, layer in zip(model.blocks, raw["layers"]):
            m = layer["mixer"]
            assert (b.mixer.H, b.mixer.dk, b.mixer.dr, b.mixer.dv, b.mixer.rank, b.mixer.q_rank, b.mixer.window, b.mixer.scale, b.mixer.rot_base) == \
                (m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"], (m.get("mask") or {}).get("size"), m["scale"], m["rot"]["base"])
            assert b.norm1.eps == b.mixer.eps == raw["norm"]["eps"] and (b.ffn is None) == (layer["mlp"] is None)
    bad = [
        lambda r: r["layers"][0].update(type="attention"),
        lambda r: r["layers"][0]["mixer"].pop("q_rank"),
        lambda r: r["layers"][0]["mixer"].pop("rot"),
        lambda r: r["layers"][0]["mixer"].update(heads=0),
        lambda r: r["layers"][0]["mixer"].update(scale=-1.0),
        lambda r: r["layers"][0]["mixer"]["rot"].update(base=0),
        lambda r: r["layers"][0]["mixer"]["rot"].update(dims=7),
        lambda r: r["layers"][0]["mixer"]["rot"].update(dims=10),
        lambda r: r["layers"][0]["mixer"].update(mask={"size": 0}),
        lambda r: r["layers"][2]["mixer"].update(kv_from=2),
        lambda r: r["layers"][3]["mixer"].update(kv_from=2),           # a layer without latent rows of its own
        lambda r: r["layers"][2]["mixer"].update(kv_rank=32),          # not the rank of the rows it reads
        lambda r: r["layers"][2]["mixer"]["rot"].update(base=3.0),     # not their rotation
        lambda r: r["layers"][1]["mlp"]["router"].update(top=9),
        lambda r: r["layers"][1]["mlp"]["shared"].update(ff=0),
        lambda r: r["layers"][0]["mlp"].update(kind="gated"),
        lambda r: r["layers"][0]["mlp"].pop("ff"),
        lambda r: r["norm"].update(eps=0),
        lambda r: r.pop("vocab"),
    ]
    for i, spoil in enumerate(bad):
        raw = copy.deepcopy(su.S_MIXED)
        spoil(raw)
        with pytest.raises(ConfigError):
            config_from_dict(raw)
            pytest.fail(f"case {i} was accepted")


def test_declared_tensors_and_caches():
    from tuff_amd.cache.manager import CacheLayout
    from tuff_amd.models.registry import build_model, config_from_dict
    from tuff_amd.parts.base import FixedState, PagedKV
    model = build_model(config_from_dict(copy.deepcopy(su.S_MIXED)))
    decls = {d.name: tuple(d.shape) for d in model.weight_decls()}
    assert decls["l0.mix.dq"] == (24, 64) and decls["l0.mix.dq.norm"] == (24,) and decls["l0.mix.uq"] == (2 * 24, 24)
    assert decls["l0.mix.dkv"] == (40, 64) and decls["l0.mix.dkv.norm"] == (32,) and decls["l0.mix.sink"] == (2,)
    assert decls["l0.mix.uk"] == (32, 32) and decls["l0.mix.uv"] == (48, 32) and decls["l0.mix.o"] == (64, 48)
    assert decls["l0.shift"] == (64,) and decls["l0.dwa"] == (2,) and decls["l4.dwa"] == (6,)
    assert decls["l0.mlp.up"] == (40, 64) and decls["l0.mlp.act"] == (2,)
    assert decls["l1.mlp.e3.up"] == (40, 64) and decls["l1.mlp.router"] == (4, 64) and decls["l1.mlp.shared.down"] == (64, 56)
    assert "l2.norm2" not in decls and "l2.mix.dkv" not in decls and "l2.mix.dkv.norm" not in decls and decls["l2.mix.dq"] == (16, 64)
    assert "l3.mlp.shared.up" not in decls and "l1.mlp.act" not in decls
    # a paged entry a writer, kept for the widest window of the runs that read it; a row of state for every run
    layout = CacheLayout.from_specs(model.cache_specs)
    assert layout.paged == {0: PagedKV(1, 40, 48, 32), 1: PagedKV(1, 40, None, 24), 4: PagedKV(1, 24, 16, 16)}
    assert model.schedule[3].cache == 0 and not model.schedule[3].writes
    assert layout.states == {("run", i): FixedState((64,)) for i in range(5)}
    # a reader with a narrower window leaves the writer's
    plain_model = build_model(config_from_dict(copy.deepcopy(su.S_WIDE)))
    assert plain_model.cache_specs[1] == PagedKV(1, 80, None, 48) and plain_model.cache_specs[0] == PagedKV(1, 64, 40, 48)


def test_a_model_with_sums_over_its_layers_refuses_what_does_not_go_with_them():
    from tuff_amd.models.decoder import DecoderModel, LayerRun
    from tuff_amd.models.registry import build_model, config_from_dict
    from tuff_amd.parts.base import WeightDecl
    base = build_model(config_from_dict(copy.deepcopy(su.S_PLAIN)))
    kw = dict(vocab_size=101, hidden_size=48, embedding=base.embedding_decl, blocks=base.blocks, final_norm=base.final_norm, head=base.head_decl)
    runs = [LayerRun(0, cache=0), LayerRun(1, cache=0, writes=False)]
    with pytest.raises(ValueError, match="i \\+ 2 numbers"):
        DecoderModel(schedule=runs, depth_average=[WeightDecl("a", (2,)), WeightDecl("b", (2,))], **kw)
    with pytest.raises(ValueError, match="one residual stream"):
        DecoderModel(schedule=runs, streams=2, depth_average=[WeightDecl("a", (2,)), WeightDecl("b", (3,))], **dict(kw, blocks=[]))
    assert DecoderModel(schedule=runs, **kw).depth_decls is None      # the blocks alone: plain residual sums


def test_random_model_folder_round_trip(tmp_path):
    from tuff_amd.models.registry import build_model, config_from_dict, load_config
    from tuff_amd.weights.loader import Checkpoint
    from tuff_amd.weights.random_init import write_random_model
    cfg = config_from_dict(copy.deepcopy(su.S_MIXED))
    write_random_model(cfg, str(tmp_path), seed=3)
    assert load_config(str(tmp_path)).to_dict() == cfg.to_dict()
    assert set(Checkpoint(str(tmp_path)).names()) == {d.name for d in build_model(cfg).weight_decls()}
