"""Kisutar on the GPU against the plain implementation (tests/plain/kisutar_plain.py): every mechanism alone, whole
prompts against token-by-token decoding, portions down to two tokens, batches of unequal requests, pages and slots used
again, keys far away, at page borders and just inside and outside every window, readers whose windows are not the
writer's, first tokens, long decoding, sizes nobody tuned the kernels for, and greedy generation through the scheduler,
the command line and the trace runner."""
import copy
import functools
import math
import os
import subprocess
import sys

import pytest
import torch

import kisutar_util as su
import util
from plain import kisutar_plain as plain

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]
WHOLE = ["mixed", "wide", "odd", "plain"]
PEAKY = 3.0          # factor on W_uq in the runs where single keys are to hold the weight


@functools.lru_cache(maxsize=None)
def model(name: str, seed: int = 0, peaky: bool = False):
    raw = su.CONFIGS[name]
    w = su.make_weights(raw, seed)
    if peaky:
        for i in range(len(raw["layers"])):
            w[f"l{i}.mix.uq"] = (w[f"l{i}.mix.uq"].float() * PEAKY).to(torch.bfloat16)
    folder = os.path.join(util._TMP.name, f"kisutar_{name}_{seed}_{int(peaky)}")
    return su.write_folder(raw, w, folder), raw, w


@functools.lru_cache(maxsize=512)
def _plain(name, seed, peaky, tokens, scale):
    _, raw, w = model(name, seed, peaky)
    if scale is None:
        return plain.forward(raw, w, list(tokens))
    # (the roundings of the form the engine computes: queries carried into the latent space, sums of latent rows)
    return plain.forward(raw, w, list(tokens), rnd=lambda t: plain.bf16_round(t * scale) / scale, absorbed=True)


CLOSE_CALL = 0.05       # of the router logits' spread: below it, bfloat16 rounding may choose another expert


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
    V = su.CONFIGS[name]["vocab"]
    return {f"r{i}": util.rand_tokens(n, V, seed * 100 + i) for i, n in enumerate(lengths)}


def check(name, dtype, plan, reqs, seed=0, peaky=False, **kw):
    eng = engine(name, dtype, seed, peaky, **kw)
    got = util.run_plan(eng, plan)
    eng.manager.check()
    assert not eng.manager.live()
    compare(name, dtype, got, reqs, seed, peaky=peaky)
    return eng, got


def compare(name, dtype, got, reqs, seed=0, what="", peaky=False):
    """float32: every request against the exact logits (with scaled-up queries a score of tens hangs on angles of hundreds
    of radians, which float32 holds to 2e-5, so a weight moves by 1e-4 where two keys compete, in single rows of hundreds:
    ten times the tolerance there, where a key more or less moves the logits by tenths).  bfloat16: the rows of all requests together against the rounding model's
    error, each request up to its first token at which a router's choice hangs on less than rounding moves (float32 covers
    the rest); a single row has a heavier tail with scaled-up queries, where two keys that compete for a row's weight
    change places under rounding."""
    exp = {rid: expected(name, toks, seed, peaky) for rid, toks in reqs.items()}
    if dtype == "float32":
        for rid in reqs:
            err, want = (got[rid].double() - exp[rid].want).abs(), exp[rid].want
            tol = (2e-5 + 1e-4 * want.abs()) * (10.0 if peaky else 1.0)
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
@pytest.mark.parametrize("name", [n for n in su.CONFIGS if n.startswith("only_")])
def test_each_mechanism_alone(gpu, name, dtype):
    reqs = requests(name, [37, 1, 9])
    check(name, dtype, util.plan_whole(reqs), reqs)
    check(name, dtype, util.plan_chunks(reqs, sizes=(2, 5, 1, 3, 16, 2)), reqs)
    check(name, dtype, util.plan_tail(reqs, tail=20), reqs)


def test_the_stream_after_every_layer(gpu):
    """What every layer hands on (after its sum over the layers), from a prompt and from single tokens."""
    for name in ("mixed", "odd", "only_deep"):
        _, raw, w = model(name)
        toks = util.rand_tokens(30, raw["vocab"], 4)
        want = {}
        plain.forward(raw, w, toks, on_layer=lambda i, x: want.__setitem__(i, x))
        eng = engine(name, "float32")
        got = {i: [] for i in want}
        eng.model.on_layer = lambda i, x: got[i].append(x.double().cpu())
        eng.use_graphs = eng.record_portions = False
        from tuff_amd.engine.batch import StepEntry
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
@pytest.mark.parametrize("name", ["mixed", "wide", "odd", "only_latent_shared"])
def test_batches_of_unequal_requests_with_pages_and_slots_used_again(gpu, name, dtype):
    reqs = requests(name, [5, 77, 130, 2, 40, 64, 19, 95, 33], seed=4)
    plan = util.plan_mixed(reqs, seed=4, max_live=3)
    peak = util.live_tokens_peak(plan)
    eng, got = check(name, dtype, plan, reqs, max_tokens=peak, max_requests=3)
    for g in eng.manager.groups:
        assert g.pool.allocations > g.pool.num_pages       # pages came back and went out again
    again = util.run_plan(eng, plan)                       # every page and slot has been used before
    if dtype == "float32":
        for rid in reqs:
            assert torch.equal(again[rid], got[rid]), rid
    else:
        compare(name, dtype, again, reqs, what="second run")


@pytest.mark.parametrize("page_size", [1, 7, 8, 64])
def test_other_page_sizes(gpu, page_size):
    """Pages off the kernels' own borders and larger than windows."""
    reqs = requests("mixed", [70, 33, 9], seed=11)
    for dtype in DTYPES:
        check("mixed", dtype, util.plan_mixed(reqs, seed=3), reqs, page_size=page_size)


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
    out again, the shifted rows move on in their slots."""
    reqs = requests("mixed", [330], seed=8)
    eng, _ = check("mixed", dtype, util.plan_tail(reqs, tail=325), reqs)
    assert eng.graph_replays > 0                           # steps of single tokens were recorded and replayed


@pytest.mark.parametrize("name, dtype, size", [("mixed", "float32", 8), ("mixed", "bfloat16", 16), ("only_latent_shared", "float32", 16)])
def test_steps_of_portions_recorded_in_sections(gpu, name, dtype, size):
    """Steps of one size that keep coming are recorded in sections and replayed: four requests side by side, their
    shifted rows carried from replay to replay."""
    reqs = requests(name, [160, 160, 160, 160], seed=7)
    plan = [{"step": k, "entries": [{"id": rid, "tokens": toks[k * size:(k + 1) * size], "want": list(range(size))} for rid, toks in reqs.items()],
             "end": list(reqs) if (k + 1) * size == 160 else []} for k in range(160 // size)]
    eng, _ = check(name, dtype, plan, reqs)
    assert eng.section_replays > 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["only_latent", "only_latent_window", "only_latent_wide", "only_latent_shared", "only_latent_many_heads"])
def test_peaky_attention_far_keys_in_prompts_and_in_decoding(gpu, name, dtype):
    """Queries scaled up: a few keys hold the weight, anywhere in hundreds; a key lost, taken twice, seen beyond its
    window or read from a neighbour's page moves the logits.  Also through layers that read another layer's rows."""
    reqs = requests(name, [420, 300], seed=8)
    check(name, dtype, util.plan_tail(reqs, tail=70), reqs, peaky=True)
    check(name, dtype, util.plan_chunks(reqs, sizes=(15, 1, 16, 17, 2, 31, 33, 64, 63, 65)), reqs, peaky=True)


def _drawn(seed: int) -> dict:
    """A configuration with every size drawn, multiples of 8 in half of them."""
    import random
    r = random.Random(seed)
    even = seed % 2 == 0
    size = lambda lo, hi: (lambda v: max(8, v // 8 * 8) if even else v)(r.randint(lo, hi))
    layers, kept = [], []
    for i in range(r.randint(2, 5)):
        src = r.choice(kept) if kept and r.random() < 0.4 else None
        if src is None:
            rank, rot, base = size(8, 300 if r.random() < 0.2 else 90), 2 * r.randint(1, 20), r.choice([30.0, 1000.0, 50000.0])
            rot = rot // 8 * 8 + 8 if even else rot
        else:
            m = layers[src]["mixer"]
            rank, rot, base = m["kv_rank"], m["rot_dim"], m["rot"]["base"]
        window = r.choice([None, 1, r.randint(2, 40), r.randint(2, 40), r.randint(41, 200), 16, 64])
        mixer = su.latent(r.randint(1, 12), size(3, 50), rot, size(3, 50), size(5, 70), rank, r.uniform(0.1, 0.5), window, base, src)
        E = r.randint(1, 12)
        mlp = r.choice([None, su.dense(size(5, 120)), su.dense(size(5, 120)), su.moe(E, r.randint(1, E), size(5, 60), r.choice([None, size(5, 60)]))])
        if src is None:
            kept.append(i)
        layers.append(su.layer(mixer, mlp))
    return su.config(size(20, 160), r.randint(30, 400), layers, eps=r.choice([1e-6, 1e-5, 1e-3]))


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(gpu, seed):
    name = f"drawn_{seed}"
    su.CONFIGS[name] = _drawn(seed)
    reqs = requests(name, [61, 140, 7, 30], seed=seed)
    for dtype in DTYPES:
        check(name, dtype, util.plan_mixed(reqs, seed=seed, max_live=3), reqs, max_requests=3)
        check(name, dtype, util.plan_tail(reqs, tail=16), reqs)


# ------------------------------------------------------------ one key made to stand out
def _bound_latent(gpu, dtype, H, rank, dr, dv, scale, window, sinks):
    """A latent mixer whose projections pick columns of its input: a row is [query row | raw latent | rotated key]; the
    query row goes through as it is (W_uq the identity), W_uk of every head is the identity, W_uv of head a picks dv
    channels from a on, the norm weights are one."""
    from tuff_amd.parts.base import Runtime
    from tuff_amd.parts.latent import LatentAttentionMixer
    from tuff_amd.parts.linear import Linear
    q_rank = H * (rank + dr)
    width = q_rank + rank + dr
    mixer = LatentAttentionMixer(width, H, rank, dr, dv, rank, norm_eps=1e-6, scale=scale, rot_base=100.0, rot_halves=True, window=window,
                                 q_rank=q_rank, exact_weights=True,
                                 names={k: k for k in ("dq", "dq.norm", "uq", "dkv", "dkv.norm", "uk", "uv", "sink", "o")})
    mixer.out = Linear("o", H * dv, H * dv)
    eye = torch.eye(width)
    uv = torch.cat([torch.eye(rank)[[(a + j) % rank for j in range(dv)]] for a in range(H)])
    weights = {"dq": eye[:q_rank], "dq.norm": torch.ones(q_rank), "uq": torch.eye(q_rank), "dkv": eye[q_rank:], "dkv.norm": torch.ones(rank),
               "uk": torch.eye(rank).repeat(H, 1), "uv": uv, "sink": sinks, "o": torch.eye(H * dv)}
    mixer.bind({n: t.to(dtype).to(gpu) for n, t in weights.items()}, Runtime(gpu, dtype))
    m = dict(heads=H, dim=rank, rot_dim=dr, vdim=dv, q_rank=q_rank, kv_rank=rank, scale=scale, rot={"base": 100.0, "dims": dr})
    if window is not None:
        m["mask"] = {"size": window}
    W = {n: t.to(dtype).double() for n, t in weights.items()}
    return mixer, width, m, W


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, rank, dr, dv, window", [(4, 16, 8, 16, None), (2, 64, 16, 24, 100), (3, 20, 2, 5, 33), (6, 32, 32, 8, 256),
                                                     (1, 8, 8, 8, 16), (2, 272, 16, 16, 50), (24, 24, 8, 8, 17)])
def test_latent_attention_one_key_stands_out_at_every_edge(gpu, H, rank, dr, dv, window, dtype):
    """One latent row is lined up with the last query's first head so that it would hold nearly all the weight, and
    placed at the start, far back, on both sides of a page's border, last, and just inside and just outside the window;
    the heads' sinks hold a share that the plain softmax knows; the last query sees it from a prompt's portion, as a
    single token and after portions.  Pages are scattered and everything else in the pool is NaN."""
    from tuff_amd.cache.manager import CacheLayout, CacheManager
    from tuff_amd.cache.storage import CacheStorage
    from tuff_amd.engine.batch import StepEntry, build_context
    ps, scale = 16, 5.0 / math.sqrt(rank)
    gen = torch.Generator().manual_seed(H + rank + dv)
    sinks = 1.0 + torch.randn(H, generator=gen)
    mixer, width, m, W = _bound_latent(gpu, dtype, H, rank, dr, dv, scale, window, sinks)
    layout = CacheLayout.from_specs({0: mixer.cache_spec()})
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    for n in (1, 17, 130, 300):
        places = {n - 1, 0, (n - 1) // 16 * 16, max(0, (n - 1) // 16 * 16 - 1), n // 2, min(n - 1, 255), min(n - 1, 256)}
        if window is not None:
            places |= {max(0, n - window), max(0, n - window - 1), max(0, n - window + 1)}
        for special in sorted(places):
            mgr = CacheManager(layout, ps, 64, 2)
            store = CacheStorage(mgr, dtype, gpu, poison=True)
            mgr.admit("pad")
            mgr.extend("pad", 40)                               # the request's pages do not start at page 0
            x = torch.randn(n, width, generator=gen) * 0.5
            x[special, H * (rank + dr):H * (rank + dr) + rank] = x[n - 1, :rank] * 2.0   # the special row lines up with the last query's first head
            x = x.to(dtype)
            rnd = plain.bf16_round if dtype == torch.bfloat16 else plain._same
            rows = plain.latent_rows(x.double(), W, m, 1e-6, rnd)
            want = plain.latent_attention(x.double(), rows, W, m, 1e-6, rnd, absorbed=True)
            for cut in ([n], [n - min(3, n - 1)] + [1] * min(3, n - 1), [n - 2 * (n // 5)] + [n // 5] * 2):
                mgr.admit("a")
                at = 0
                for c in (c for c in cut if c):
                    mgr.extend("a", c)
                    ctx = build_context([StepEntry("a", [0] * c, [])], mgr, gpu, 10)
                    res = torch.zeros(c, H * dv, dtype=torch.float32, device=gpu)
                    mixer.forward(x[at:at + c].to(gpu).contiguous(), ctx, store.views[0], res)
                    err = (res.double().cpu() - want[at:at + c]).abs().max()
                    assert err <= tol * max(1.0, float(want.abs().max())), (n, special, cut, at, float(err))
                    at += c
                mgr.release("a")


# ----------------------------------------------------------------------- kernels alone
@pytest.mark.parametrize("d", [24, 200, 52, 1024, 1030, 2048, 3000, 4100, 7, 6144, 9000, 5001])
def test_depth_average_kernel_alone(gpu, d):
    """The sum over one to nineteen streams, its norm in both types, the rows' inverse root mean squares, and the shift of
    single tokens between slots of NaN; long and short steps give a row the same bits."""
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(d)
    T, eps = 9, 1e-3
    dev = lambda t: t.to(gpu).contiguous()
    nw, mix = torch.randn(d, generator=g), torch.rand(d, generator=g)
    for n in (1, 2, 8, 9, 19):
        xs, w = torch.randn(n, T, d, generator=g), torch.randn(n, generator=g)
        want = plain.depth_average(list(xs.double()), w.double())
        want_h = plain.rms_norm(want, nw.double(), eps)
        buf = dev(torch.cat([xs, torch.zeros(1, T, d)]))
        x = buf[n]
        scale = float(want.abs().max())
        ops.depth_average(x, xs=buf[:n], w=dev(w))
        assert (x.double().cpu() - want).abs().max() < 1e-5 * scale
        summed = x.clone()
        inv = torch.zeros(T, device=gpu)
        ops.depth_average(x, xs=buf[:n], w=dev(w), eps=eps, inv_out=inv)
        assert (inv.double().cpu() - 1 / torch.sqrt((want * want).mean(-1) + eps)).abs().max() < 1e-5 * float(inv.max())
        for dt in (torch.float32, torch.bfloat16):
            h = torch.zeros(T, d, dtype=dt, device=gpu)
            x.zero_()
            ops.depth_average(x, xs=buf[:n], w=dev(w), norm_w=dev(nw), eps=eps, h_out=h)
            assert torch.equal(x, summed)
            assert (h.double().cpu() - want_h).abs().max() < (2e-5 if dt == torch.float32 else 8e-3) * float(want_h.abs().max())
        assert torch.equal(buf[:n].cpu(), xs)
        slots = torch.tensor([2 * i + 1 for i in range(T)][::-1], dtype=torch.int32)
        state = torch.full((2 * T + 1, d), float("nan"))
        prev = torch.randn(T, d, generator=g)
        state[slots.long()] = prev
        st, h = dev(state), torch.zeros(T, d, device=gpu)
        ops.depth_average(x, norm_w=dev(nw), eps=eps, h_out=h, mix=dev(mix), state=st, req_of_token=torch.arange(T, dtype=torch.int32, device=gpu),
                          state_slot=dev(slots))                    # (without streams: x as it is)
        assert torch.equal(x, summed)
        want_s = want_h + (prev.double() - want_h) * mix.double()
        assert (h.double().cpu() - want_s).abs().max() < 2e-5 * float(want_s.abs().max())
        assert (st.cpu()[slots.long()].double() - want_h).abs().max() < 2e-5 * float(want_h.abs().max())
        assert torch.isnan(st[0::2]).all()
    ones = torch.zeros(1, T, d)
    copy_of = torch.zeros(T, d, device=gpu)
    ops.depth_average(copy_of, xs=dev(ones + 3.0))                    # no weights: the sum as it is
    assert torch.equal(copy_of.cpu(), torch.full((T, d), 3.0))


@pytest.mark.parametrize("d", [24, 52, 7, 1024, 1030, 2500])
def test_norm_shift_kernel_alone_across_cuts(gpu, d):
    """Two requests in slots between slots of NaN, cut into steps of one, two and more tokens, against the plain shift; the
    single-token kernel and this one leave the same bits."""
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(d)
    lens_all, eps = [23, 9], 1e-3
    dev = lambda t: t.to(gpu).contiguous()
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=gpu)
    xs = [torch.randn(n, d, generator=g) for n in lens_all]
    nw, mix = torch.randn(d, generator=g), torch.randn(d, generator=g)
    want = [plain.token_shift(plain.rms_norm(x.double(), nw.double(), eps), mix.double()) for x in xs]
    seen = {}
    for cuts in ([23], [1, 1, 2, 3, 8, 8], [2] * 11 + [1], [1] * 23):
        for fused in (False, True):
            state = torch.full((5, d), float("nan"), device=gpu)
            state[1].zero_()
            state[3].zero_()
            done, got = [0, 0], [torch.zeros(n, d) for n in lens_all]
            for c in cuts:
                lens = [min(c, lens_all[r] - done[r]) for r in (0, 1)]
                live = [r for r in (0, 1) if lens[r] > 0]
                starts = [sum(lens[q] for q in live[:k]) for k in range(len(live))]
                x = dev(torch.cat([xs[r][done[r]:done[r] + lens[r]] for r in live]))
                out = torch.zeros(x.shape[0], d, device=gpu)
                req_of = i32([k for k, r in enumerate(live) for _ in range(lens[r])])
                slot = i32([[3, 1][r] for r in live])
                if fused and max(lens) == 1:
                    ops.depth_average(x, norm_w=dev(nw), eps=eps, h_out=out, mix=dev(mix), state=state, req_of_token=req_of, state_slot=slot)
                else:
                    inv = torch.zeros(x.shape[0], device=gpu)
                    ops.depth_average(x, eps=eps, inv_out=inv)
                    ops.norm_shift(x, inv, dev(nw), dev(mix), state, out, req_of_token=req_of, q_start=i32(starts),
                                   q_len=i32([lens[r] for r in live]), state_slot=slot)
                for k, r in enumerate(live):
                    got[r][done[r]:done[r] + lens[r]] = out[starts[k]:starts[k] + lens[r]].cpu()
                    done[r] += lens[r]
            for r in (0, 1):
                assert (got[r].double() - want[r]).abs().max() < 2e-5 * float(want[r].abs().max()), (cuts, fused, r)
                assert torch.equal(seen.setdefault(r, got[r]), got[r]), (cuts, fused, r)
            assert torch.isnan(state[0]).all() and torch.isnan(state[2]).all() and torch.isnan(state[4]).all()


@pytest.mark.parametrize("H, Hkv, hd, vd, window, copies", [(6, 1, 40, 40, 100, 1), (32, 1, 224, 224, 1024, 1), (17, 1, 136, 64, 0, 1),
                                                           (8, 4, 64, 128, 1, 1), (40, 2, 256, 256, 300, 1), (3, 3, 8, 8, 129, 1),
                                                           (16, 1, 128, 96, 0, 40), (32, 1, 64, 64, 700, 60)])
def test_single_token_attention_with_float32_weights_alone(gpu, H, Hkv, hd, vd, window, copies):
    """Tokens at positions on both sides of every border of blocks, parts, pages and windows, pages scattered among NaN,
    a key beside the window's edge and a far one made to stand out; `copies`: enough rows that the plan takes longer parts."""
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(H + hd)
    ps, scale = 16, 4.0 / math.sqrt(hd)
    pos_all = [0, 1, 15, 16, 127, 128, 129, 255, 256, 700, 1023, 1024, 1500, 2047]
    n = max(pos_all) + 1
    blocks = -(-n // ps)
    P = blocks + 7
    perm = torch.randperm(P, generator=g)[:blocks]
    K, V = (torch.randn(n, Hkv, w, generator=g).to(torch.bfloat16) for w in (hd, vd))
    sinks, slopes = torch.randn(H, generator=g) + 1.0, torch.rand(H, generator=g) * 0.01
    q = torch.randn(len(pos_all), H, hd, generator=g)
    for i, p in enumerate(pos_all):                       # one head looks at the oldest key it sees, one at the newest one it does not
        lo = max(0, p - window + 1) if window else 0
        q[i, 0] = K[lo, 0].float() * 0.5
        q[i, H - 1] = K[max(0, lo - 1), Hkv - 1].float() * 0.5
    q = q.to(torch.bfloat16)
    kc = torch.full((P, Hkv, ps, hd), float("nan"), dtype=torch.bfloat16)
    vc = torch.full((P, Hkv, vd, ps), float("nan"), dtype=torch.bfloat16)
    for b in range(blocks):
        m = min(ps, n - b * ps)
        kc[perm[b], :, :m] = K[b * ps:b * ps + m].transpose(0, 1)
        vc[perm[b], :, :, :m] = V[b * ps:b * ps + m].permute(1, 2, 0)
    table = torch.stack([perm, perm]).to(torch.int32)
    want = torch.zeros(len(pos_all), H, vd, dtype=torch.float64)
    for i, p in enumerate(pos_all):
        lo = max(0, p - window + 1) if window else 0
        for h in range(H):
            kh = h // (H // Hkv)
            s = (K[lo:p + 1, kh].double() @ q[i, h].double()) * scale - slopes[h].double() * (p - torch.arange(lo, p + 1).double())
            top = max(float(s.max()), float(sinks[h]))
            e = torch.exp(s - top)
            want[i, h] = (e @ V[lo:p + 1, kh].double()) / (e.sum() + math.exp(float(sinks[h]) - top))
    dev = lambda t: t.to(gpu).contiguous()
    T = len(pos_all) * copies
    pk, slots = ops.attention_single_plan(T, H, Hkv, n, window)
    assert (pk > 128) == (copies > 1) and slots <= 64
    out = torch.zeros(T, H * vd, device=gpu)
    ops.attention_single(dev(q.reshape(-1, H * hd).repeat(copies, 1)), dev(kc), dev(vc), out, block_table=dev(table),
                         req_of_token=torch.tensor([i % 2 for i in range(T)], dtype=torch.int32, device=gpu),
                         positions=torch.tensor(pos_all * copies, dtype=torch.int32, device=gpu), H=H, Hkv=Hkv, hd=hd, vd=vd, page_size=ps,
                         max_ctx_len=n, window=window, scale=scale, sinks=dev(sinks), slopes=dev(slopes))
    got = out.view(copies, len(pos_all), H, vd).double().cpu()
    err = (got - want).abs().amax(dim=(0, 2, 3))
    assert (err < 4e-5 * float(want.abs().max())).all(), (pos_all, err)
    # every plan: from one token to as many as there are, at contexts up to a million positions
    for T in (1, 8, 64, 300):
        for ctx in (1, 16, 1000, 8192, 131072, 1 << 20):
            pk, slots = ops.attention_single_plan(T, H, Hkv, ctx, window)
            assert pk % 128 == 0 and 1 <= slots <= 64 and pk * (slots if not window else max(slots, 2)) >= min(ctx, window or ctx)


@pytest.mark.parametrize("hd, vd", [(136, 64), (192, 128), (160, 136), (192, 192), (200, 192), (224, 192), (232, 40), (256, 192), (208, 208), (64, 256)])
def test_prompt_attention_of_every_tile_width_against_the_single_token_kernel(gpu, hd, vd):
    """The prompt kernel's tiles come in several widths: a portion's rows against the same rows taken one by one, with and
    without a window, sinks beside."""
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(hd + vd)
    H, T, past, ps = 5, 150, 83, 16
    n = T + past
    P = -(-n // ps)
    dev = lambda t: t.to(gpu).contiguous()
    q = dev(torch.randn(T, H * hd, generator=g).to(torch.bfloat16))
    k = dev(torch.randn(P, 1, ps, hd, generator=g).to(torch.bfloat16))
    v = dev(torch.randn(P, 1, vd, ps, generator=g).to(torch.bfloat16))
    table = torch.randperm(P, generator=g).to(torch.int32)[None].to(gpu)
    sinks = dev(torch.randn(H, generator=g))
    for window in (0, 70):
        kw = dict(H=H, Hkv=1, hd=hd, vd=vd, page_size=ps, max_ctx_len=n, window=window, scale=2.0 / math.sqrt(hd), sinks=sinks, block_table=table)
        a, b = (torch.zeros(T, H * vd, dtype=torch.bfloat16, device=gpu) for _ in range(2))
        nb = ops.attention_prefill_block_columns(max(hd, vd)) // 16
        ops.attention_prefill_wide(q, k, v, a, blocks=torch.from_numpy(ops.query_blocks([T], H, nb, [n])).to(gpu),
                                   req_info=torch.tensor([[0, T, past, n]], dtype=torch.int32, device=gpu), **kw)
        ops.attention_single(q, k, v, b, req_of_token=torch.zeros(T, dtype=torch.int32, device=gpu),
                             positions=torch.arange(past, n, dtype=torch.int32, device=gpu), **kw)
        assert torch.isfinite(a).all() and (a.float() - b.float()).abs().max() < 1e-2 * float(b.float().abs().max()), window


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, dk, dr, rank, dims", [(3, 8, 8, 24, 8), (1, 5, 6, 11, 4), (20, 16, 64, 192, 64), (2, 4, 2, 8, 0)])
def test_latent_post_kernel_halves_separate_rows_and_readers(gpu, H, dk, dr, rank, dims, dtype):
    """The cache row from float32 sums beside queries of the compute type, pairs of halves, the rows once more page-wise
    transposed; a reader's queries alone, with nothing written."""
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(H + rank)
    T, ps, pages, eps = 11, 4, 6, 1e-4
    lat = rank + dr
    dev = lambda t: t.to(gpu).contiguous()
    q = torch.randn(T, H * (dk + dr), generator=g).to(dtype)
    raw = torch.randn(T, 5 + lat, generator=g)
    nw = torch.randn(rank, generator=g).to(dtype)
    pos = torch.tensor([0, 1, 7, 100, 3000, 12, 13, 14, 15, 16, 17], dtype=torch.int32)
    slots = torch.randperm(pages * ps, generator=g)[:T].to(torch.int32)
    inv_freq = torch.tensor([300.0 ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    half = dims // 2

    def turned(x):                                          # [T, n]
        a = pos.double()[:, None] * inv_freq
        u, v = x[:, :half], x[:, half:dims]
        return torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), x[:, dims:]], dim=1)
    want_row = torch.cat([plain.rms_norm(raw[:, 5:5 + rank].double(), nw.double(), eps), turned(raw[:, 5 + rank:].double())], dim=1)
    want_q = torch.stack([turned(q[:, h * (dk + dr) + dk:(h + 1) * (dk + dr)].double()) for h in range(H)], dim=1)
    tol = 2e-4 if dtype == torch.float32 else 2e-2
    for reader, t_ch in ((False, lat), (False, rank), (True, lat)):
        cache = torch.full((pages, 1, ps, lat), 7.0, dtype=dtype, device=gpu)
        cache_t = torch.full((pages, 1, t_ch, ps), 7.0, dtype=dtype, device=gpu)
        q_lat = torch.full((T, H * lat), 5.0, dtype=dtype, device=gpu)
        ops.latent_post(dev(q), q_lat, cache, q_off=0, ckr=dev(raw), ckr_off=None if reader else 5, norm_w=None if reader else dev(nw), eps=eps,
                        inv_freq=dev(inv_freq.float()) if dims else None, rot_dims=dims, halves=True, positions=dev(pos),
                        slot_mapping=None if reader else dev(slots), H=H, dim=dk, rot=dr, rank=rank, cache_t=None if reader else cache_t)
        ql = q_lat.view(T, H, lat).double().cpu()
        assert (ql[:, :, :rank] == 5.0).all()
        assert (ql[:, :, rank:] - want_q).abs().max() < tol * max(1.0, float(want_q.abs().max()))
        flat = cache.view(-1, lat).double().cpu()
        untouched = torch.ones(pages * ps, dtype=torch.bool)
        if not reader:
            assert (flat[slots.long()] - want_row).abs().max() < tol * max(1.0, float(want_row.abs().max()))
            untouched[slots.long()] = False
            assert torch.equal(cache_t.transpose(2, 3), cache[..., :t_ch])
        assert (flat[untouched] == 7.0).all()


def test_activations_and_the_strided_norm(gpu):
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(3)
    z = torch.cat([torch.randn(7, 40, generator=g) * 3, torch.linspace(-1e-3, 1e-3, 40)[None], torch.linspace(-40, 40, 40)[None]])
    p, q = 0.37, -1.2
    ab = torch.tensor([math.log1p(math.exp(p)), math.log1p(math.exp(q))])
    for act, params, want in (("xielu", ab.to(gpu), plain.xielu(z.double(), torch.tensor(p), torch.tensor(q))), ("gelu_erf", None, plain.gelu_erf(z.double()))):
        out = torch.zeros(z.shape, device=gpu)
        ops.act_rows(z.to(gpu), out, act, params=params)
        assert ((out.double().cpu() - want).abs() <= 1e-6 * (z.abs() + want.abs())).all(), act
    with pytest.raises(ops.KernelError):
        ops.act_rows(z.to(gpu), out, "xielu")
    # the norm of a column range of a wider row, on and off 16-byte borders, and the product with the norm inside
    for lo, n in ((0, 24), (4, 24), (3, 24), (0, 21)):
        wide = torch.randn(5, 40, generator=g)
        w = torch.randn(n, generator=g)
        want = plain.rms_norm(wide[:, lo:lo + n].double(), w.double(), 1e-3)
        out = torch.zeros(5, n, device=gpu)
        ops.rmsnorm(wide.to(gpu)[:, lo:lo + n], w.to(gpu), out, 1e-3)
        assert (out.double().cpu() - want).abs().max() < 1e-5
        if n % 8 == 0 and lo % 4 == 0:
            W = torch.randn(19, n, generator=g).to(torch.bfloat16)
            y = torch.zeros(5, 19, device=gpu)
            ops.gemm_normed(wide.to(gpu)[:, lo:lo + n], w.to(gpu), 1e-3, W.to(gpu), y)
            assert (y.double().cpu() - want @ W.double().T).abs().max() < 2e-2 * float((want @ W.double().T).abs().max())


@pytest.mark.parametrize("d, E, top", [(44, 6, 2), (64, 8, 8), (256, 16, 3), (40, 5, 1), (48, 130, 4)])
def test_router_with_the_softmax_over_all_experts(gpu, d, E, top):
    from tuff_amd.csrc import ops
    g = torch.Generator().manual_seed(d + E)
    T = 300
    h = torch.randn(T, d, generator=g).to(torch.bfloat16)
    router = torch.randn(E, d, generator=g) * 2.0 / math.sqrt(d)
    margins = []
    ids, wts = plain.route(h.double(), {"router": router.double()}, su.moe(E, top, 8), margins)
    z = torch.zeros(T, E, device=gpu)
    idg, wtg = torch.zeros(T, top, dtype=torch.int32, device=gpu), torch.zeros(T, top, device=gpu)
    ops.moe_router(h.to(gpu), router.to(gpu), z, idg, wtg, E=E, top=top, weights="softmax_all")
    ok = margins[0] > 1e-4
    assert ok.sum() > T // 2 and torch.equal(idg.cpu()[ok].long(), ids[ok])
    assert (wtg.double().cpu()[ok] - wts[ok]).abs().max() < 1e-5


def test_the_shift_without_sums_over_the_layers(gpu):
    """The block in a model that keeps plain residual sums: the same parts, another model."""
    from tuff_amd.engine.batch import StepEntry
    from tuff_amd.engine.engine import Engine
    from tuff_amd.models.decoder import DecoderModel, LayerRun
    from tuff_amd.models.registry import build_model, config_from_dict
    raw = su.S_PLAIN
    w = su.make_weights(raw, 2)
    base = build_model(config_from_dict(copy.deepcopy(raw)))
    m = DecoderModel(vocab_size=101, hidden_size=48, embedding=base.embedding_decl, blocks=base.blocks, final_norm=base.final_norm,
                     head=base.head_decl, schedule=[LayerRun(0, cache=0), LayerRun(1, cache=0, writes=False)])
    for i in range(2):                                    # a sum that takes the last result alone is the plain stream
        w[f"l{i}.dwa"] = torch.zeros(i + 2, dtype=torch.bfloat16)
        w[f"l{i}.dwa"][i + 1] = 1.0
    toks = util.rand_tokens(50, 101, 1)
    want = plain.forward(raw, w, toks)
    eng = Engine(m, {k: v.float().to(gpu) for k, v in w.items()}, dtype="float32", max_tokens=128, max_requests=2)
    eng.begin("a")
    rows = []
    for lo, hi in ((0, 20), (20, 22), (22, 23), (23, 24), (24, 50)):
        rows.append(eng.step([StepEntry("a", toks[lo:hi], list(range(hi - lo)))]).clone())
    util.assert_close_f32(torch.cat(rows).cpu(), want)


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
    for word in ("TokenShiftBlock", "LatentAttentionMixer", "DenseMLP", "MoE", "FixedState"):
        assert word in q.stdout, q.stdout[-2000:]
    # the trace runner: a mixed plan through a child process, four slots, a pool no larger than the plan's peak
    reqs = requests("wide", [50, 3, 70, 20, 31], seed=10)
    plan = util.plan_mixed(reqs, seed=2)
    for dtype in DTYPES:
        got = util.run_trace_run(folder, dtype, plan, util.live_tokens_peak(plan), str(tmp_path / dtype))
        compare("wide", dtype, got, reqs, what="trace runner")
