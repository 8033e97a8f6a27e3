"""Tobilorn on the GPU against the plain implementation (tests/plain/tobilorn_plain.py): every mechanism alone, whole
prompts against token-by-token decoding, portions down to two tokens, batches of unequal requests, pages and slots used
again, keys far away, at page borders, just inside and outside every window and among and just beyond the first tokens
that stay, first tokens, long decoding, sizes nobody tuned the kernels for, and greedy generation through the scheduler,
the command line and the trace runner."""
import functools
import math
import os
import subprocess
import sys

import pytest
import torch

import tobilorn_util as tu
import util
from plain import tobilorn_plain as plain

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]
WHOLE = ["mixed", "wide", "odd", "plain"]
PEAKY = 3.0          # factor on W_q in the runs where single keys are to hold the weight


@functools.lru_cache(maxsize=None)
def model(name: str, seed: int = 0, peaky: bool = False):
    raw = tu.CONFIGS[name]
    w = tu.make_weights(raw, seed)
    if peaky:
        for i in range(len(raw["layers"])):
            for k in ("q", "q.b"):
                w[f"l{i}.mix.{k}"] = (w[f"l{i}.mix.{k}"].float() * PEAKY).to(torch.bfloat16)
    folder = os.path.join(util._TMP.name, f"tobilorn_{name}_{seed}_{int(peaky)}")
    return tu.write_folder(raw, w, folder), raw, w


@functools.lru_cache(maxsize=512)
def _plain(name, seed, peaky, tokens, scale):
    _, raw, w = model(name, seed, peaky)
    if scale is None:
        return plain.forward(raw, w, list(tokens))
    return plain.forward(raw, w, list(tokens), rnd=lambda t: plain.bf16_round(t * scale) / scale)


@functools.lru_cache(maxsize=64)
def _float32_error(name, seed, peaky, tokens):
    """Per row: the most that rounding the plain implementation's activations to float32 moves a logit, the mean of three
    realizations."""
    _, raw, w = model(name, seed, peaky)
    want = _plain(name, seed, peaky, tokens, None)
    rounded = [plain.forward(raw, w, list(tokens), rnd=lambda t: (t * s).float().double() / s) for s in util.REALIZATION_SCALES]
    return torch.stack([(r - want).abs().amax(1) for r in rounded]).mean(0)


CLOSE_CALL = 0.03       # of the two scores' sum: below it, bfloat16 rounding may choose another expert


@functools.lru_cache(maxsize=512)
def rows_before_a_close_call(name, seed, peaky, tokens) -> int:
    _, raw, w = model(name, seed, peaky)
    margins = []
    plain.forward(raw, w, list(tokens), margins_out=margins)
    n = len(tokens)
    for m in margins:
        close = torch.nonzero(m < CLOSE_CALL)
        if len(close):
            n = min(n, int(close[0]))
    return n


def expected(name, tokens, seed=0, peaky=False) -> util.Expected:
    tokens = tuple(tokens)
    return util.Expected(_plain(name, seed, peaky, tokens, None),
                         [_plain(name, seed, peaky, tokens, s) for s in util.REALIZATION_SCALES])


def engine(name, dtype, seed=0, peaky=False, **kw):
    from tuff_amd.engine.engine import Engine
    folder, _, _ = model(name, seed, peaky)
    kw.setdefault("page_size", 16)
    kw.setdefault("max_tokens", 1024)
    kw.setdefault("max_requests", 4)
    return Engine.from_folder(folder, dtype=dtype, poison_cache=True, **kw)


def requests(name, lengths, seed=0):
    V = tu.CONFIGS[name]["vocab"]
    return {f"r{i}": util.rand_tokens(n, V, seed * 100 + i) for i, n in enumerate(lengths)}


def check(name, dtype, plan, reqs, seed=0, peaky=False, **kw):
    eng = engine(name, dtype, seed, peaky, **kw)
    got = util.run_plan(eng, plan)
    eng.manager.check()
    assert not eng.manager.live()
    compare(name, dtype, got, reqs, seed, peaky=peaky)
    return eng, got


def compare(name, dtype, got, reqs, seed=0, what="", peaky=False):
    """float32: every request against the exact logits (with scaled-up queries a score of tens hangs on angles of hundreds of
    radians, which float32 holds to 2e-5, so a weight moves by 1e-4 where two keys compete: ten times the tolerance there,
    where a key more or less moves the logits by tenths; a row may be off by what roundings to float32 alone do to it in the
    plain implementation besides, four times over: a head whose two maps nearly cancel is normed after the difference, and a
    looped layer carries what that magnifies from pass to pass, in single rows of hundreds).  bfloat16: the rows of all requests together against the rounding
    model's error, each request up to its first token at which a router's choice hangs on less than rounding moves (float32
    covers the rest); a single row has a heavier tail with scaled-up queries, where two keys that compete for a row's
    weight change places under rounding, and where a head's two maps nearly cancel before the head is normed."""
    exp = {rid: expected(name, toks, seed, peaky) for rid, toks in reqs.items()}
    if dtype == "float32":
        for rid in reqs:
            err, want = (got[rid].double() - exp[rid].want).abs(), exp[rid].want
            tol = (2e-5 + 1e-4 * want.abs()) * (10.0 if peaky else 1.0)
            if not (err <= tol).all():
                tol = tol + 4.0 * _float32_error(name, seed, peaky, tuple(reqs[rid]))[:, None]
            assert torch.isfinite(got[rid]).all(), f"{what} {name} {rid}"
            assert (err <= tol).all(), (f"{what} {name} {rid}: {int((err > tol).sum())} elements differ, max err {float(err.max()):.3e}, first wrong "
                                        f"token {int(torch.nonzero((err > tol).any(-1))[0])}")
        return
    rids = list(reqs)
    keep = {r: rows_before_a_close_call(name, seed, peaky, tuple(reqs[r])) for r in rids}
    for r in rids:
        assert torch.isfinite(got[r]).all(), f"{what} {name} {r}: non-finite logits"
    if sum(keep.values()) < 8:
        return
    want = util.Expected(torch.cat([exp[r].want[:keep[r]] for r in rids]),
                         [torch.cat([exp[r].rounded[i][:keep[r]] for r in rids]) for i in range(len(util.REALIZATION_SCALES))])
    mine, yard = util.row_errors(torch.cat([got[r][:keep[r]] for r in rids]), want.want), want.yardstick()
    ratio = float(mine.mean() / yard.mean())
    assert ratio <= util.BF16_MEAN_RATIO, f"{what} {name}: mean relative RMS error {float(mine.mean()):.5f} is {ratio:.2f} times the rounding model's"
    per_row = mine / torch.maximum(yard, yard.mean())
    assert per_row.max() <= (10.0 if peaky else 3.5), f"{what} {name}: row {int(per_row.argmax())} is {float(per_row.max()):.2f} times the rounding model's"


def all_single(reqs):
    return util.plan_tail(reqs, tail=10 ** 6)


# ------------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", [n for n in tu.CONFIGS if n.startswith("only_")])
def test_each_mechanism_alone(gpu, name, dtype):
    reqs = requests(name, [37, 1, 9])
    check(name, dtype, util.plan_whole(reqs), reqs)
    check(name, dtype, util.plan_chunks(reqs, sizes=(2, 5, 1, 3, 16, 2)), reqs)
    check(name, dtype, util.plan_tail(reqs, tail=20), reqs)


def test_the_stream_after_every_layer_run(gpu):
    """What every layer run hands on (before the next pass's entry), from a prompt and from single tokens."""
    from tuff_amd.engine.batch import StepEntry
    for name in ("mixed", "odd", "plain", "only_loop", "only_side"):
        _, raw, w = model(name)
        toks = util.rand_tokens(30, raw["vocab"], 4)
        want = {}
        plain.forward(raw, w, toks, on_layer=lambda i, x: want.__setitem__(i, x))
        eng = engine(name, "float32")
        got = {i: [] for i in want}
        eng.model.on_layer = lambda i, x: got[i].append(x.double().cpu())
        eng.use_graphs = eng.record_portions = False
        eng.begin("a")
        for part in (toks[:25], toks[25:26], toks[26:28], toks[28:29], toks[29:]):
            eng.step([StepEntry("a", part, [])])
        for i in want:
            x = torch.cat(got[i])
            assert (x - want[i]).abs().max() < 2e-5 * max(1.0, float(want[i].abs().max())), (name, i)


# -------------------------------------------------------------- whole models under every plan
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", WHOLE)
def test_whole_prompts(gpu, name, dtype):
    reqs = requests(name, [90, 1, 2, 33])
    check(name, dtype, util.plan_whole(reqs), reqs)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", WHOLE)
def test_prompt_then_single_tokens_and_single_tokens_from_the_start(gpu, name, dtype):
    reqs = requests(name, [70, 40], seed=6)
    check(name, dtype, util.plan_tail(reqs, tail=32), reqs, seed=1)
    first = requests(name, [24], seed=2)                 # the first tokens of a sequence, one by one
    check(name, dtype, all_single(first), first, seed=1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", WHOLE)
def test_portions_of_changing_size(gpu, name, dtype):
    reqs = requests(name, [150, 61], seed=3)
    check(name, dtype, util.plan_chunks(reqs), reqs)
    small = {"r1": reqs["r1"]}
    check(name, dtype, util.plan_chunks(small, sizes=(2, 2, 3, 2, 1, 2)), small)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide", "odd", "only_attention_keep_many"])
def test_batches_of_unequal_requests_with_pages_and_slots_used_again(gpu, name, dtype):
    reqs = requests(name, [5, 77, 130, 2, 40, 64, 19, 95, 33], seed=4)
    plan = util.plan_mixed(reqs, seed=4, max_live=3)
    peak = util.live_tokens_peak(plan)
    eng, got = check(name, dtype, plan, reqs, max_tokens=peak, max_requests=3)
    again = util.run_plan(eng, plan)                       # every page and slot has been used before
    for g in eng.manager.groups:
        assert g.pool.allocations > g.pool.num_pages       # pages came back and went out again
    if dtype == "float32":
        for rid in reqs:
            assert torch.equal(again[rid], got[rid]), rid
    else:
        compare(name, dtype, again, reqs, what="second run")


@pytest.mark.parametrize("page_size", [1, 7, 8, 48, 64])
def test_other_page_sizes(gpu, page_size):
    """Pages off the kernels' own borders and larger than windows and than what is kept of the first tokens."""
    reqs = requests("mixed", [70, 33, 9], seed=11)
    for dtype in DTYPES:
        check("mixed", dtype, util.plan_mixed(reqs, seed=3), reqs, page_size=page_size)
        if page_size in (48, 64):
            more = requests("only_attention_keep_many", [230, 60], seed=12)
            check("only_attention_keep_many", dtype, util.plan_chunks(more), more, page_size=page_size)


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_float32_logits_do_not_depend_on_the_plan(gpu, name):
    """The same bits whether a prompt comes whole, in portions, token by token or beside other requests, with
    recorded steps or without."""
    reqs = requests(name, [83, 30, 47], seed=5)
    plans = [util.plan_whole(reqs), util.plan_chunks(reqs), all_single(reqs), util.plan_mixed(reqs, seed=1)]
    base = util.run_plan(engine(name, "float32"), plans[0])
    for i, plan in enumerate(plans[1:]):
        for graphs in (True, False):
            got = util.run_plan(engine(name, "float32", use_graphs=graphs), plan)
            for rid in reqs:
                assert torch.equal(got[rid], base[rid]), f"plan {i + 1}, graphs {graphs}, {rid}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, dtype):
    """Hundreds of single tokens through recorded steps: windows move on over decoded tokens, their pages go back and
    out again, the first tokens' pages stay."""
    reqs = requests("mixed", [330], seed=8)
    eng, _ = check("mixed", dtype, util.plan_tail(reqs, tail=325), reqs)
    assert eng.graph_replays > 0                           # steps of single tokens were recorded and replayed


@pytest.mark.parametrize("name, dtype, size", [("mixed", "float32", 8), ("mixed", "bfloat16", 16), ("only_loop", "float32", 16)])
def test_steps_of_portions_recorded_in_sections(gpu, name, dtype, size):
    """Steps of one size that keep coming are recorded in sections and replayed: four requests side by side, with tokens of
    their own for the side path's table at every replay."""
    reqs = requests(name, [160, 160, 160, 160], seed=7)
    plan = [{"step": k, "entries": [{"id": rid, "tokens": toks[k * size:(k + 1) * size], "want": list(range(size))} for rid, toks in reqs.items()],
             "end": list(reqs) if (k + 1) * size == 160 else []} for k in range(160 // size)]
    eng, _ = check(name, dtype, plan, reqs)
    assert eng.section_replays > 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", [n for n in tu.CONFIGS if n.startswith("only_attention")])
def test_peaky_attention_far_keys_in_prompts_and_in_decoding(gpu, name, dtype):
    """Queries scaled up: a few keys hold the weight, anywhere in hundreds; a key lost, taken twice, seen beyond its
    window or read from a neighbour's page moves the logits."""
    reqs = requests(name, [420, 300], seed=8)
    check(name, dtype, util.plan_tail(reqs, tail=70), reqs, peaky=True)
    check(name, dtype, util.plan_chunks(reqs, sizes=(15, 1, 16, 17, 2, 31, 33, 64, 63, 65)), reqs, peaky=True)


def _drawn(seed: int) -> dict:
    """A configuration with every size drawn, multiples of 8 in half of them."""
    import random
    r = random.Random(seed)
    even = seed % 2 == 0
    size = lambda lo, hi: (lambda v: max(8, v // 8 * 8) if even else v)(r.randint(lo, hi))
    layers = []
    for _ in range(r.randint(2, 4)):
        G = r.randint(1, 3)
        dim = size(4, 70)
        window = r.choice([None, 1, r.randint(2, 40), r.randint(2, 40), r.randint(41, 200), 16, 64])
        keep = r.choice([0, 1, r.randint(1, 20), r.randint(10, 100)])
        rot = r.choice([dim // 2 * 2, 2 * r.randint(0, dim // 2)])
        mixer = tu.attention(G * r.randint(1, 5), G, dim, size(3, 130), r.uniform(0.1, 0.6), r.uniform(-0.5, 0.8), window, keep,
                             r.choice([30.0, 1000.0, 50000.0]), rot)
        E, identity = r.randint(1, 10), r.choice([0, 0, 1, 3])
        mlp = r.choice([None, *[tu.moe(E, r.randint(1, E + identity), size(5, 60), identity, r.choice([None, size(5, 60)]))] * 2])
        layers.append(tu.layer(mixer, mlp))
    a = r.randint(0, len(layers) - 1)
    loop = r.choice([None, (a, r.randint(a + 1, len(layers)), r.randint(1, 3))])
    return tu.config(size(20, 160), r.randint(30, 400), layers, loop, r.choice([None, size(4, 40)]), r.choice([1.0, 3.7]), r.choice([1.0, 0.3]),
                     eps=r.choice([1e-6, 1e-5, 1e-3]))


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(gpu, seed):
    name = f"drawn_{seed}"
    tu.CONFIGS[name] = _drawn(seed)
    reqs = requests(name, [61, 140, 7, 30], seed=seed)
    for dtype in DTYPES:
        check(name, dtype, util.plan_mixed(reqs, seed=seed, max_live=3), reqs, max_requests=3)
        check(name, dtype, util.plan_tail(reqs, tail=16), reqs)


# ------------------------------------------------------------ one key made to stand out
def _bound_mixer(gpu, dtype, H, G, D, Dv, scale, window, keep):
    """A differential attention mixer whose projections pick columns of its input: a row is [queries | keys | values], no
    biases, no rotation (a key lines up with a query wherever it lies)."""
    from tuff_amd.parts.attention import DifferentialAttentionMixer
    from tuff_amd.parts.base import Runtime
    from tuff_amd.parts.linear import Linear
    nq, nk, nv = 2 * H * D, 2 * G * D, G * Dv
    width = nq + nk + nv
    mixer = DifferentialAttentionMixer(width, H, G, D, Dv, scale=scale, diff=0.3, norm_eps=1e-5, window=window, keep_first=keep,
                                       names={k: k for k in ("q", "k", "v", "o", "lq1", "lk1", "lq2", "lk2")})
    mixer.out = Linear("o", H * Dv, H * Dv)
    eye = torch.eye(width)
    g = torch.Generator().manual_seed(H + D)
    weights = {"q": eye[:nq], "k": eye[nq:nq + nk], "v": eye[nq + nk:], "o": torch.eye(H * Dv)}
    weights.update({k: torch.randn(D, generator=g) * 0.5 / math.sqrt(math.sqrt(D)) for k in ("lq1", "lk1", "lq2", "lk2")})
    mixer.bind({n: t.to(dtype).to(gpu) for n, t in weights.items()}, Runtime(gpu, dtype))
    m = dict(heads=H, kv_heads=G, dim=D, vdim=Dv, scale=scale, diff=0.3)
    if window is not None:
        m["mask"] = {"size": window, "keep_first": keep}
    W = {n: t.to(dtype).double() for n, t in weights.items()}
    zero = torch.zeros(1, dtype=torch.float64)
    W.update({"q.b": zero, "k.b": zero, "v.b": zero, "o.b": zero})
    return mixer, width, m, W


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, G, D, Dv, window, keep", [(4, 2, 16, 24, None, 0), (2, 1, 64, 128, 100, 4), (3, 1, 20, 5, 33, 17), (6, 3, 32, 8, 64, 70),
                                                       (1, 1, 8, 8, 16, 1), (2, 2, 144, 16, 50, 3), (24, 1, 24, 40, 17, 130)])
def test_one_key_stands_out_at_every_edge(gpu, H, G, D, Dv, window, keep, dtype):
    """One key is lined up with the last query's first map so that it would hold nearly all its weight, and placed at the
    start, last and first beyond the kept tokens, far back, on both sides of a page's border, last, and just inside and
    just outside the window; the last query sees it from a prompt's portion, as a single token and after portions.  Pages
    are scattered and everything else in the pool is NaN."""
    from tuff_amd.cache.manager import CacheLayout, CacheManager
    from tuff_amd.cache.storage import CacheStorage
    from tuff_amd.engine.batch import StepEntry, build_context
    ps, scale = 16, 5.0 / math.sqrt(D)
    gen = torch.Generator().manual_seed(H + D + Dv)
    mixer, width, m, W = _bound_mixer(gpu, dtype, H, G, D, Dv, scale, window, keep)
    layout = CacheLayout.from_specs({0: mixer.cache_spec()})
    tol = 5e-5 if dtype == torch.float32 else 6e-2
    for n in (1, 17, 130, 300):
        places = {n - 1, 0, (n - 1) // 16 * 16, max(0, (n - 1) // 16 * 16 - 1), n // 2, min(n - 1, 127), min(n - 1, 128)}
        places |= {min(n - 1, max(0, keep - 1)), min(n - 1, keep)}
        if window is not None:
            places |= {max(0, n - window), max(0, n - window - 1), max(0, n - window + 1)}
        for special in sorted(places):
            mgr = CacheManager(layout, ps, 64, 2)
            store = CacheStorage(mgr, dtype, gpu, poison=True)
            mgr.admit("pad")
            mgr.extend("pad", 40)                               # the request's pages do not start at page 0
            x = torch.randn(n, width, generator=gen) * 0.5
            x[special, 2 * H * D:2 * H * D + D] = x[n - 1, :D] * 2.0      # the special key lines up with the last query's first map
            x = x.to(dtype)
            rnd = plain.bf16_round if dtype == torch.bfloat16 else plain._same
            want = plain.attention(x.double(), W, m, 1e-5, rnd)
            for cut in ([n], [n - min(3, n - 1)] + [1] * min(3, n - 1), [n - 2 * (n // 5)] + [n // 5] * 2):
                mgr.admit("a")
                at = 0
                for c in (c for c in cut if c):
                    mgr.extend("a", c)
                    ctx = build_context([StepEntry("a", [0] * c, [])], mgr, gpu, 10)
                    res = torch.zeros(c, H * Dv, dtype=torch.float32, device=gpu)
                    mixer.forward(x[at:at + c].to(gpu).contiguous(), ctx, store.views[0], res)
                    err = (res.double().cpu() - want[at:at + c]).abs().max()
                    assert err <= tol * max(1.0, float(want.abs().max())), (n, special, cut, at, float(err))
                    at += c
                mgr.release("a")


# ----------------------------------------------------------------------- kernels alone
def _paged(g, n, Hkv, hd, vd, ps, extra=7):
    """Keys and values of n positions on pages scattered among NaN: (K, V, key cache, value cache, table)."""
    blocks = -(-n // ps)
    perm = torch.randperm(blocks + extra, generator=g)[:blocks]
    K, V = (torch.randn(n, Hkv, w, generator=g).to(torch.bfloat16) for w in (hd, vd))
    kc = torch.full((blocks + extra, Hkv, ps, hd), float("nan"), dtype=torch.bfloat16)
    vc = torch.full((blocks + extra, Hkv, vd, ps), float("nan"), dtype=torch.bfloat16)
    for b in range(blocks):
        m = min(ps, n - b * ps)
        kc[perm[b], :, :m] = K[b * ps:b * ps + m].transpose(0, 1)
        vc[perm[b], :, :, :m] = V[b * ps:b * ps + m].permute(1, 2, 0)
    return K, V, kc, vc, perm.to(torch.int32)


def _kernel_rows(gpu, H, Hkv, dim, vd, maps, window, keep, positions, n, seed, ps=16):
    """Queries at `positions`, their cache and the exact outputs of every map [T, H, vd] (H counts maps)."""
    g = torch.Generator().manual_seed(seed)
    K, V, kc, vc, perm = _paged(g, n, Hkv, maps * dim, vd, ps)
    scale = 4.0 / math.sqrt(dim)
    q = torch.randn(len(positions), H, dim, generator=g)
    for i, p in enumerate(positions):                     # edges made to stand out: the window's, the kept tokens'
        lo = max(0, p - window + 1) if window else 0
        for h, j in ((0, lo), (1 % H, max(0, lo - 1)), (2 % H, min(p, max(0, keep - 1))), (3 % H, min(p, keep))):
            part = (h % maps) * dim
            q[i, h] = K[j, h // (H // Hkv), part:part + dim].float() * 0.5
    q = q.to(torch.bfloat16)
    want = torch.zeros(len(positions), H, vd, dtype=torch.float64)
    for i, p in enumerate(positions):
        j = torch.arange(p + 1)
        ok = (p - j < window) | (j < keep) if window else j >= 0
        for h in range(H):
            kh, part = h // (H // Hkv), (h % maps) * dim
            s = (K[:p + 1, kh, part:part + dim].double() @ q[i, h].double()) * scale
            want[i, h] = torch.softmax(s.masked_fill(~ok, -math.inf), 0) @ V[:p + 1, kh].double()
    dev = lambda t: t.to(gpu).contiguous()
    kw = dict(Hkv=Hkv, vd=vd, page_size=ps, window=window, scale=scale, keep_first=keep, block_table=dev(perm[None]))
    return dev(q.reshape(len(positions), -1)), dev(kc), dev(vc), want, kw


POSITIONS = [0, 1, 4, 15, 16, 127, 128, 129, 255, 256, 500, 700, 1023, 1024, 1500]


@pytest.mark.parametrize("H, Hkv, dim, vd, window, keep", [(8, 2, 64, 128, 100, 4), (6, 1, 40, 40, 0, 0), (4, 2, 128, 256, 300, 130), (2, 1, 8, 8, 1, 9),
                                                          (48, 1, 24, 40, 128, 1), (16, 4, 32, 64, 1024, 300)])
def test_single_token_attention_with_maps_and_kept_tokens_alone(gpu, H, Hkv, dim, vd, window, keep):
    """Two maps a head combined in the merge, at positions on both sides of every border of blocks, parts, pages and
    windows; the general kernel and its combination give the same."""
    from tuff_amd.csrc import ops
    n = max(POSITIONS) + 1
    q, kc, vc, want, kw = _kernel_rows(gpu, H, Hkv, dim, vd, 2, window, keep, POSITIONS, n, H + dim)
    combine = (0.8, 1e-5, 0.7)
    heads = plain.combine_maps(want[:, 0::2], want[:, 1::2], 0.8, 0.3, 1e-5).reshape(len(POSITIONS), -1)
    T = len(POSITIONS)
    kw.update(req_of_token=torch.zeros(T, dtype=torch.int32, device=gpu), positions=torch.tensor(POSITIONS, dtype=torch.int32, device=gpu), H=H, hd=2 * dim)
    for dt, tol in ((torch.float32, 2e-4), (torch.bfloat16, 1e-2)):
        out = torch.zeros(T, H // 2 * vd, dtype=dt, device=gpu)
        ops.attention_single(q, kc, vc, out, max_ctx_len=n, combine=combine, **kw)
        err = (out.double().cpu() - heads).abs().amax(1)
        assert (err < tol * float(heads.abs().max())).all(), err
    maps = torch.zeros(T, H * vd, device=gpu)
    ops.attention_general(q, kc, vc, maps, maps=2, **kw)
    assert (maps.view(T, H, vd).double().cpu() - want).abs().max() < 2e-5 * float(want.abs().max())
    ops.diff_combine(maps, out := torch.zeros(T, H // 2 * vd, device=gpu), H=H // 2, vd=vd, combine=combine)
    assert (out.double().cpu() - heads).abs().max() < 2e-4 * float(heads.abs().max())
    # every plan holds every key that is seen, whatever the context
    for T in (1, 8, 64, 300):
        for ctx in (1, 16, 1000, 8192, 131072, 1 << 20):
            pk, slots = ops.attention_single_plan(T, H, Hkv, ctx, window, keep if window else 0)
            assert pk % 128 == 0 and 1 <= slots <= 64
            for pos in (0, ctx // 2, ctx - 1):
                lo = max(0, pos - window + 1) if window else 0
                kept = min(-(-(keep if window else 0) // pk), lo // pk)
                assert kept + pos // pk - lo // pk + 1 <= slots, (T, ctx, pos)


@pytest.mark.parametrize("H, Hkv, hd, vd, window, keep", [(8, 2, 64, 128, 100, 4), (4, 4, 40, 24, 33, 70), (20, 1, 192, 128, 64, 1)])
def test_kept_first_tokens_with_one_map_a_head(gpu, H, Hkv, hd, vd, window, keep):
    """The window that keeps first tokens in plain attention with float32 weights: single tokens, portions and the
    general kernel."""
    from tuff_amd.csrc import ops
    positions = list(range(700, 860))
    n, T = 860, 160
    q, kc, vc, want, kw = _kernel_rows(gpu, H, Hkv, hd, vd, 1, window, keep, positions, n, hd)
    kw.update(H=H, hd=hd)
    each = dict(req_of_token=torch.zeros(T, dtype=torch.int32, device=gpu), positions=torch.tensor(positions, dtype=torch.int32, device=gpu))
    flat = want.reshape(T, -1)
    out = torch.zeros(T, H * vd, device=gpu)
    ops.attention_single(q, kc, vc, out, max_ctx_len=n, **each, **kw)
    assert (out.double().cpu() - flat).abs().max() < 4e-5 * float(flat.abs().max())
    a, b = (torch.zeros(T, H * vd, dtype=torch.bfloat16, device=gpu) for _ in range(2))
    ops.attention_general(q, kc, vc, b, **each, **kw)
    nb = ops.attention_prefill_block_columns(max(hd, vd)) // 16
    ops.attention_prefill_wide(q, kc, vc, a, blocks=torch.from_numpy(ops.query_blocks([T], H // Hkv, nb, [n])).to(gpu), max_ctx_len=n,
                               req_info=torch.tensor([[0, T, 700, n]], dtype=torch.int32, device=gpu), **kw)
    for o in (a, b):
        assert (o.double().cpu() - flat).abs().max() < 5e-3 * float(flat.abs().max())


@pytest.mark.parametrize("ps", [16, 48, 64])
@pytest.mark.parametrize("dim, vd", [(8, 8), (32, 64), (24, 128), (32, 256), (64, 64), (56, 128), (64, 200), (96, 128), (80, 192), (96, 256), (128, 128), (120, 256)])
def test_prompt_attention_with_maps_of_every_tile_width(gpu, dim, vd, ps):
    """The prompt kernel's tiles come in several widths: a portion far into a request and one from its start, with windows
    that keep none to hundreds of first tokens (jumps from the kept steps to the window's on and off borders of pages)."""
    from tuff_amd.csrc import ops
    combine = (0.9, 1e-5, 0.6)
    for heads, Hkv, window, keep, past, T in ((4, 2, 0, 0, 83, 90), (3, 1, 70, 5, 400, 70), (2, 2, 33, 200, 380, 40), (5, 1, 16, 64, 0, 150), (2, 1, 100, 17, 331, 3)):
        positions = list(range(past, past + T))
        n = past + T
        q, kc, vc, want, kw = _kernel_rows(gpu, 2 * heads, Hkv, dim, vd, 2, window, keep, positions, n, dim + vd + T, ps)
        want = plain.combine_maps(want[:, 0::2], want[:, 1::2], 0.9, 0.4, 1e-5).reshape(T, -1)
        out = torch.zeros(T, heads * vd, dtype=torch.bfloat16, device=gpu)
        nb = ops.attention_prefill_diff_block_columns() // 16
        ops.attention_prefill_diff(q, kc, vc, out, blocks=torch.from_numpy(ops.query_blocks([T], heads // Hkv, nb, [n])).to(gpu), heads=heads, dim=dim,
                                   req_info=torch.tensor([[0, T, past, n]], dtype=torch.int32, device=gpu), max_ctx_len=n, combine=combine, **kw)
        err = (out.double().cpu() - want).abs().max()
        assert err < 1e-2 * float(want.abs().max()), (heads, window, keep, past, float(err))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, Hk, hd, maps, vd, dims, ps", [(8, 4, 32, 2, 64, 32, 16), (6, 2, 20, 2, 24, 8, 16), (3, 1, 5, 1, 7, 4, 4), (4, 4, 64, 2, 100, 0, 16),
                                                           (2, 2, 130, 2, 70, 130, 48), (5, 5, 16, 1, 16, 16, 16)])
def test_rotate_and_write_kernel_alone(gpu, H, Hk, hd, maps, vd, dims, ps, dtype):
    """Biases, rotation and both cache writes out of a product's float32 sums: tokens in runs of sixteen slots and scattered
    ones, positions inside and beyond the table of angles, with and without a bias and a cache."""
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(H + hd)
    G, T, pages = Hk // maps, 41, 8
    width = (H + Hk) * hd + G * vd
    x, bias = torch.randn(T, width, generator=g), torch.randn(width, generator=g)
    pos = torch.cat([torch.arange(100, 116), torch.randint(0, 3000, (25,), generator=g)]).to(torch.int32)
    first = torch.arange(16) + (16 if ps % 16 == 0 else ps)
    rest = torch.tensor([s for s in torch.randperm(pages * ps, generator=g).tolist() if s not in set(first.tolist())][:25]) if pages * ps >= 41 else None
    if rest is None:
        pages = 16
        rest = torch.tensor([s for s in torch.randperm(pages * ps, generator=g).tolist() if s not in set(first.tolist())][:25])
    slots = torch.cat([first, rest]).to(torch.int32)
    inv_freq = torch.tensor([300.0 ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    dev = lambda t: t.to(gpu).contiguous()
    inv = dev(inv_freq.float()) if dims else None
    table = ops.rope_table(inv, 1000) if dims else None
    for b in (bias, None):
        y = x.double() + (0 if b is None else b.double())
        heads = y[:, :(H + Hk) * hd].reshape(T, H + Hk, hd).clone()
        a = pos.double()[:, None, None] * inv_freq
        u, v = heads[..., :dims // 2].clone(), heads[..., dims // 2:dims].clone()
        heads[..., :dims // 2], heads[..., dims // 2:dims] = u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin()
        for write in (True, False):
            q = torch.zeros(T, H * hd, dtype=dtype, device=gpu)
            kc = torch.full((pages, G, ps, maps * hd), 7.0, dtype=dtype, device=gpu)
            vc = torch.full((pages, G, vd, ps), 7.0, dtype=dtype, device=gpu)
            wr = dict(k_cache=kc, v_cache=vc, slot_mapping=dev(slots)) if write else {}
            ops.qkv_rotate_write(dev(x), q, H=H, Hk=Hk, hd=hd, maps=maps, vd=vd, positions=dev(pos), bias=None if b is None else dev(b), inv_freq=inv,
                                 rotary_dim=dims, angles=table, page_size=ps, **wr)
            tol = 5e-4 if dtype == torch.float32 else 2e-2
            assert (q.double().cpu() - heads[:, :H].reshape(T, -1)).abs().max() < tol * float(heads.abs().max())
            kf = kc.permute(0, 2, 1, 3).reshape(pages * ps, Hk, hd).double().cpu()
            vf = vc.permute(0, 3, 1, 2).reshape(pages * ps, G * vd).double().cpu()
            untouched = torch.ones(pages * ps, dtype=torch.bool)
            if write:
                assert (kf[slots.long()] - heads[:, H:]).abs().max() < tol * float(heads.abs().max())
                assert (vf[slots.long()] - y[:, (H + Hk) * hd:]).abs().max() < tol * float(y.abs().max())
                untouched[slots.long()] = False
            assert (kf[untouched] == 7.0).all() and (vf[untouched] == 7.0).all()


@pytest.mark.parametrize("d, N, identity, top", [(44, 6, 2, 2), (64, 8, 0, 8), (256, 16, 3, 5), (40, 5, 1, 1), (48, 130, 7, 12), (40, 60, 10, 64)])
def test_router_with_a_corrected_choice(gpu, d, N, identity, top):
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(d + N)
    for T in (300, 1100):                                   # one and four tokens a workgroup
        h = torch.randn(T, d, generator=g).to(torch.bfloat16)
        out = N + identity
        W = {"router": torch.randn(out, d, generator=g).double() * 2.0 / math.sqrt(d), "correction": torch.randn(out, generator=g).double() * 0.5 / out}
        margins = []
        ids, wts = plain.route(h.double(), {k: v.float().double() for k, v in W.items()}, {"experts": N, "identity": identity, "top": top}, margins)
        for corrected in (True, False):
            if not corrected:
                margins = []
                ids, wts = plain.route(h.double(), {"router": W["router"].float().double(), "correction": torch.zeros(out).double()},
                                       {"experts": N, "identity": identity, "top": top}, margins)
            z = torch.zeros(T, out, device=gpu)
            idg, wtg = torch.zeros(T, top, dtype=torch.int32, device=gpu), torch.zeros(T, top, device=gpu)
            ops.moe_router(h.to(gpu), W["router"].float().to(gpu), z, idg, wtg, E=out, top=top, weights="softmax_share",
                           correction=W["correction"].float().to(gpu) if corrected else None)
            # (the order among the chosen may turn on less than float32 holds; as a set they are the same)
            got, want = torch.zeros(T, out).double(), torch.zeros(T, out).double()
            got.scatter_(1, idg.cpu().long(), wtg.double().cpu())
            want.scatter_(1, ids, wts)
            ok = margins[0].abs() > 1e-4
            assert ok.sum() > T // 2 and (got[ok] - want[ok]).abs().max() < 1e-5
            assert (wtg.sum(1) - 1).abs().max() < 1e-5


@pytest.mark.parametrize("dtype, d, F, E, top, T", [(torch.float32, 44, 20, 6, 3, 9), (torch.bfloat16, 64, 40, 5, 3, 9), (torch.bfloat16, 64, 40, 4, 2, 400),
                                                    (torch.bfloat16, 44, 20, 6, 3, 9), (torch.bfloat16, 64, 24, 4, 4, 60)])
def test_experts_with_identity_choices_alone(gpu, dtype, d, F, E, top, T):
    """Choices beyond the last expert add the weight times the input, in every form of the experts' kernels; tokens with
    none, some and only such choices."""
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(d + T)
    N = E + 4
    h = torch.randn(T, d, generator=g).to(dtype)
    gate, up = (torch.randn(E, F, d, generator=g).to(dtype) / math.sqrt(d) for _ in range(2))
    down = torch.randn(E, d, F, generator=g).to(dtype) / math.sqrt(F)
    ids = torch.stack([torch.randperm(N, generator=g)[:top] for _ in range(T)]).to(torch.int32)
    ids[0] = torch.arange(E, E + top)                       # identity experts only
    ids[1] = torch.arange(top)
    wts = torch.rand(T, top, generator=g)
    rnd = plain.bf16_round if dtype == torch.bfloat16 else plain._same
    want = torch.ones(T, d, dtype=torch.float64)
    for t in range(T):
        for e, w in zip(ids[t].tolist(), wts[t].double()):
            want[t] += w * (h[t].double() if e >= E else plain.expert(h[t].double(), gate[e].double(), up[e].double(), down[e].double(), rnd))
    dev = lambda t: t.to(gpu).contiguous()
    got = torch.ones(T, d, device=gpu)
    kw = dict(activation="silu", scale_input=False, gated=True)
    ops.moe_experts(dev(h), dev(torch.cat([gate, up], 1)), dev(down), dev(ids), dev(wts), got, **kw)
    tol = 2e-5 if dtype == torch.float32 else 1e-2
    assert (got.double().cpu() - want).abs().max() < tol * float(want.abs().max())
    if not ops.moe_grouped_supported(dtype, d, F, E):
        return
    tiles = [ops.tile_experts([ops.interleave_gate_up(dev(a), dev(b)) for a, b in zip(gate, up)]), ops.tile_experts([dev(w) for w in down])]
    seen = []
    for tiled_from in (96, 1, 10 ** 6):
        old = ops.load("moe").tuff_moe_grouped_tiled_from(tiled_from)
        try:
            got = torch.ones(T, d, device=gpu)
            ops.moe_experts_grouped(dev(h), *tiles, dev(ids), dev(wts), got, F=F, **kw)
        finally:
            ops.load("moe").tuff_moe_grouped_tiled_from(old)
        assert (got.double().cpu() - want).abs().max() < tol * float(want.abs().max()), tiled_from
        seen.append(got)
    assert torch.equal(seen[1], seen[2])                    # the block tiles give the bits of the kernel without them


@pytest.mark.parametrize("d", [24, 200, 52, 1024, 1030, 2048, 5001, 9000])
def test_join_kernel_with_a_bias_of_its_input_a_row_and_plain_rows(gpu, d):
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(d)
    T = 5
    x, y, extra = (torch.randn(T, d, generator=g) for _ in range(3))
    w, b, row, nw = (torch.randn(d, generator=g) for _ in range(4))
    dev = lambda t: t.to(gpu).contiguous()
    v = y.double() + b.double()
    joined = x.double() + plain.unit_rms(v, 1e-3) * w.double()
    tol = lambda want: 1e-5 * float(want.abs().max())
    # a bias of y, then x itself in both types
    for dt in (torch.float32, torch.bfloat16):
        xg, yg, h = dev(x), dev(y), torch.zeros(T, d, dtype=dt, device=gpu)
        ops.post_norm_add(xg, y=yg, w=dev(w), eps=1e-3, mult=1.0, y_bias=dev(b), clear_y=True, h_out=h)
        assert (xg.double().cpu() - joined).abs().max() < tol(joined) and not yg.any()
        assert torch.equal(h, xg.to(dt))
    # the entry of a pass: another tensor and a row, then the next norm
    xg, h = dev(x), torch.zeros(T, d, device=gpu)
    ops.post_norm_add(xg, extra=dev(extra), row=dev(row), next_w=dev(nw), next_eps=1e-3, h_out=h)
    want = x.double() + extra.double() + row.double()
    assert (xg.double().cpu() - want).abs().max() < tol(want)
    want = plain.unit_rms(want, 1e-3) * nw.double()
    assert (h.double().cpu() - want).abs().max() < tol(want)
    xg = dev(x)
    ops.post_norm_add(xg, row=dev(row))
    assert torch.equal(xg.cpu(), x + row)
    with pytest.raises(ops.KernelError):
        ops.post_norm_add(xg, y_bias=dev(b))


@pytest.mark.parametrize("N, wide, col0", [(24, 24, 48), (20, 24, 20), (5, 8, 3), (8, 8, 0)])
def test_activation_times_looked_up_vectors(gpu, N, wide, col0):
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(N)
    u, table = torch.randn(9, N, generator=g) * 2, torch.randn(31, 96, generator=g)
    toks = torch.tensor([0, 30, 7, 7, 1, 2, 29, 11, 0], dtype=torch.int32)
    for tdt in (torch.float32, torch.bfloat16):
        want = plain.gelu_tanh(u.double()) * table.to(tdt).double()[toks.long(), col0:col0 + N]
        for dt, tol in ((torch.float32, 2e-6), (torch.bfloat16, 8e-3)):
            out = torch.full((9, wide), 7.0, dtype=dt, device=gpu)
            ops.act_lookup(u.to(gpu), table.to(tdt).to(gpu), toks.to(gpu), out, "gelu_tanh", col0)
            assert (out[:, :N].double().cpu() - want).abs().max() < tol * float(want.abs().max()) and not out[:, N:].any()
    with pytest.raises(ops.KernelError):
        ops.act_lookup(u.to(gpu), table.to(gpu), toks.to(gpu), out, "gelu_tanh", 96 - N + 1)


def test_an_attention_mixer_that_keeps_first_tokens(gpu):
    """The window that keeps first tokens is an option of the attention mixer too: against itself without a window on the
    keys that are seen, in both types, from a prompt and from single tokens."""
    from tuff_amd.cache.manager import CacheLayout, CacheManager
    from tuff_amd.cache.storage import CacheStorage
    from tuff_amd.engine.batch import StepEntry, build_context
    from tuff_amd.parts.attention import AttentionMixer
    from tuff_amd.parts.base import Runtime
    g = torch.Generator().manual_seed(3)
    d, H, G, hd, window, keep, n = 32, 4, 2, 16, 20, 5, 75
    weights = {"q": torch.randn(H * hd, d, generator=g), "k": torch.randn(G * hd, d, generator=g), "v": torch.randn(G * hd, d, generator=g),
               "o": torch.randn(d, H * hd, generator=g) / 8}
    x = torch.randn(n, d, generator=g)
    for dtype, tol in ((torch.float32, 3e-5), (torch.bfloat16, 4e-2)):
        mixer = AttentionMixer(d, H, G, hd, names={k: k for k in "qkvo"}, window=window, keep_first=keep, exact_weights=True, scale=0.1)
        mixer.bind({k: v.to(dtype).to(gpu) for k, v in weights.items()}, Runtime(gpu, dtype))
        W = {k: v.to(dtype).double() for k, v in weights.items()}
        xd = x.to(dtype).double()
        q, k, v = ((xd @ W[c].T).view(n, -1, hd) for c in "qkv")
        ok = plain.visible(n, {"size": window, "keep_first": keep})
        want = torch.cat([plain.softmax_map(q[:, h], k[:, h // 2], 0.1, ok) @ v[:, h // 2] for h in range(H)], dim=1) @ W["o"].T
        layout = CacheLayout.from_specs({0: mixer.cache_spec()})
        assert layout.group_keeps == [keep]
        mgr = CacheManager(layout, 16, 8, 1)
        store = CacheStorage(mgr, dtype, gpu, poison=True)
        mgr.admit("a")
        at, rows = 0, []
        for c in [50] + [1] * 8 + [n - 58]:
            mgr.extend("a", c)
            ctx = build_context([StepEntry("a", [0] * c, [])], mgr, gpu, 10)
            res = torch.zeros(c, d, device=gpu)
            mixer.forward(x[at:at + c].to(dtype).to(gpu).contiguous(), ctx, store.views[0], res)
            rows.append(res.double().cpu())
            at += c
        assert (torch.cat(rows) - want).abs().max() < tol * float(want.abs().max())


# ------------------------------------------------------------------- generation, command line
def _plain_greedy(name, prompt, n_new, seed=0):
    _, raw, w = model(name, seed)
    toks = list(prompt)
    for _ in range(n_new):
        toks.append(int(plain.forward(raw, w, toks)[-1].argmax()))
    return toks[len(prompt):]


def test_greedy_generation_through_the_scheduler(gpu):
    from tuff_amd.engine.llm import LLM
    from tuff_amd.sampling.params import SamplingParams
    reqs = requests("mixed", [5, 21, 1, 12, 30, 8], seed=9)
    eng = engine("mixed", "float32", max_tokens=512, max_requests=3)
    llm = LLM(engine=eng, max_num_seqs=3, max_batched_tokens=16, ctx_size=128, ignore_eos=True)
    outs = llm.generate(list(reqs.values()), SamplingParams(temp=0.0, max_new_tokens=30, ignore_eos=True))
    for g, prompt in zip(outs, reqs.values()):
        assert list(g.token_ids) == _plain_greedy("mixed", prompt, 30), prompt
    eng.manager.check()
    assert not eng.manager.live()


def test_command_line_and_trace_replay(gpu, tmp_path):
    folder, raw, _ = model("wide")
    prompt = util.rand_tokens(9, raw["vocab"], 3)
    p = subprocess.run([sys.executable, os.path.join(util.ROOT, "bin", "tuff"), "--model", folder, "--prompt-ids",
                        ",".join(map(str, prompt)), "--dump-tokens", "-n", "6", "--dtype", "fp32", "--temp", "0"],
                       capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [int(x) for x in p.stdout.split()] == _plain_greedy("wide", prompt, 6)
    q = subprocess.run([sys.executable, os.path.join(util.ROOT, "bin", "tuff"), "--model", folder, "--inspect"],
                       capture_output=True, text=True, timeout=300)
    assert q.returncode == 0, q.stderr[-2000:]
    for word in ("SandwichBlock", "DifferentialAttentionMixer", "MoE", "keep_first", "TokenSide", "PassEntry"):
        assert word in q.stdout, q.stdout[-2000:]
    # the trace runner: a mixed plan through a child process, four slots, a pool no larger than the plan's peak
    reqs = requests("wide", [50, 3, 70, 20, 31], seed=10)
    plan = util.plan_mixed(reqs, seed=2)
    for dtype in DTYPES:
        got = util.run_trace_run(folder, dtype, plan, util.live_tokens_peak(plan), str(tmp_path / dtype))
        compare("wide", dtype, got, reqs, what="trace runner")
