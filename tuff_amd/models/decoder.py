"""A decoder as data: an embedding, a set of blocks, the order in which they run, a final norm
and a head.  The run order is a list of LayerRun; it may name a block twice (each run then has
a cache of its own) or let a run read the cache that another run writes.
"""
from __future__ import annotations

import dataclasses
from typing import Optional

import torch

from ..csrc import ops
from ..parts.base import Block, FixedState, Norm, PagedKV, Runtime, WeightDecl, cache_specs_of
from ..parts.block import PLAIN_ROWS
from ..parts.norm import RMSNorm


@dataclasses.dataclass(frozen=True)
class LayerRun:
    block: int                      # index into DecoderModel.blocks
    cache: Optional[int] = None     # cache entry this run uses (default: one of its own)
    writes: bool = True             # False: only reads the entry, which an earlier run writes
    reinject: bool = False          # True: the embedding (as it entered the first run) is added to x before this run
    enter: Optional[int] = None     # the number of the pass that begins with this run (DecoderModel's entry)


class _Head:
    """Stands for the head as the consumer of the final norm."""
    accepts_pending_norm = True


_HEAD = _Head()


def _any_window(spec):
    """A declaration without its window: runs that share an entry may read windows of different widths."""
    return dataclasses.replace(spec, window=None, keep_first=0) if isinstance(spec, PagedKV) else spec


class DecoderModel:
    def __init__(self, *, vocab_size: int, hidden_size: int, embedding: WeightDecl,
                 blocks: list[Block], final_norm: Norm, head: Optional[WeightDecl] = None,
                 schedule: Optional[list[LayerRun]] = None, max_positions: Optional[int] = None,
                 eos_token_id: Optional[int] = None, embedding_scale: float = 1.0,
                 logit_scale: float = 1.0, logit_softcap: Optional[float] = None, pad_hidden: bool = False,
                 streams: Optional[int] = None, depth_average: Optional[list[WeightDecl]] = None, entry=None):
        """head=None: the head is the embedding (tied), as the reference does when the file has
        no output matrix (src/lfm25_model.c:128-131).
        embedding_scale: the embedding rows are multiplied by it on their way into the residual stream.
        logit_scale, logit_softcap: logits = head(norm(x)) * logit_scale, then, with a cap c,
        c * tanh(logits / c).  The reference has none of the three (scale 1, no cap), which are the defaults.
        pad_hidden: a hidden size that is no multiple of 8 is served in bfloat16 too, by zero columns (for a
        model all of whose parts take such a size); without it such a model is refused when it is bound.
        streams: the model keeps that many residual streams [S, T, d], all equal to the embedding at the start
        and summed before the final norm; its blocks are then all of a kind that takes them (multi_stream).
        depth_average: one weight a run, [i + 2] for run i: with X_0 the embedding and X_(i+1) what run i makes of its
        input, what goes on after run i is the sum of weight[j] X_j, j = 0 .. i + 1.
        entry: a parts.loop.PassEntry; before a run with `enter` = t the stream becomes what the entry makes of it, of the
        embedding and of t (blocks of the kind that hand each other their first input only)."""
        self.pad_hidden = bool(pad_hidden)
        self.streams = None if streams is None else int(streams)
        if self.streams is not None and (self.streams < 1 or not all(getattr(b, "multi_stream", False) for b in blocks)):
            raise ValueError("a model with several residual streams needs at least one and blocks that take them")
        if self.streams is None and any(getattr(b, "multi_stream", False) for b in blocks):
            raise ValueError("a block over several residual streams in a model that keeps one")
        self.depth_decls = None if depth_average is None else list(depth_average)
        if self.depth_decls is not None:
            if self.streams is not None or not blocks or not all(hasattr(b, "enter") for b in blocks):
                raise ValueError("sums over the layers go with one residual stream and blocks that enter through them")
            runs = schedule if schedule is not None else [LayerRun(i) for i in range(len(blocks))]
            if [tuple(w.shape) for w in self.depth_decls] != [(i + 2,) for i in range(len(runs))] or any(r.reinject for r in runs):
                raise ValueError("sums over the layers need a weight of i + 2 numbers for every run i, and no reinjection")
        #: every block hands the next one its first normed input (Block.carries_norm): the kernel that adds a block's
        #: last output into the stream also reads the stream for whoever comes next
        self.carries = bool(blocks) and all(getattr(b, "carries_norm", False) for b in blocks)
        runs_ = schedule if schedule is not None else []
        self.entry = entry
        if entry is None and any(r.enter is not None for r in runs_):
            raise ValueError("a run begins a pass of a model without an entry")
        if entry is not None:
            if not self.carries or not all(getattr(b, "hands_plain_rows", False) for b in blocks):
                raise ValueError("passes with an entry need blocks that hand on the stream itself")
            if any(r.enter is not None and (r.reinject or not 0 <= r.enter < entry.times) for r in runs_):
                raise ValueError(f"a run begins a pass outside 0 .. {entry.times - 1}, or takes the embedding twice")
        #: debugging aid: called as on_layer(run index, x [T, d] or xs [S, T, d]) after every layer run; while it
        #: is set no step is recorded into a graph
        self.on_layer = None
        self.vocab_size, self.hidden_size = int(vocab_size), int(hidden_size)
        self.embedding_decl, self.head_decl = embedding, head
        self.blocks, self.final_norm = list(blocks), final_norm
        self.max_positions, self.eos_token_id = max_positions, eos_token_id
        self.embedding_scale, self.logit_scale = float(embedding_scale), float(logit_scale)
        self.logit_softcap = None if not logit_softcap else float(logit_softcap)
        runs = schedule if schedule is not None else [LayerRun(i) for i in range(len(self.blocks))]
        self.schedule: list[LayerRun] = []
        next_id = 0
        used = {r.cache for r in runs if r.cache is not None}
        for r in runs:
            if not 0 <= r.block < len(self.blocks):
                raise ValueError(f"run order names block {r.block}; there are {len(self.blocks)}")
            cache = r.cache
            if cache is None:
                while next_id in used:
                    next_id += 1
                cache = next_id
                used.add(cache)
            self.schedule.append(LayerRun(r.block, cache, r.writes, r.reinject, r.enter))
        # Every cache entry has exactly one writer, which comes before its readers.  A run's entry is named
        # by LayerRun.cache; a mixer that declares several things to keep has the entries (cache, 0),
        # (cache, 1), ... in the order of its declarations.
        self.cache_specs: dict = {}
        self._run_entries: list = []             # per run: (the mixer declares a tuple, its entry ids)
        written: dict = {}
        self._run_states: list = []              # per run: the entry id of what the block itself keeps, or None
        for i, r in enumerate(self.schedule):
            specs, several = cache_specs_of(self.blocks[r.block].mixer)
            own = self.blocks[r.block].block_state() if hasattr(self.blocks[r.block], "block_state") else None
            self._run_states.append(None if own is None else ("run", i))
            if own is not None:
                self.cache_specs[("run", i)] = own
            ids = tuple((r.cache, j) for j in range(len(specs))) if several else (r.cache,) * len(specs)
            if r.writes:
                if r.cache in written:
                    raise ValueError(f"cache entry {r.cache} has two writers")
                written[r.cache] = specs
                self.cache_specs.update(zip(ids, specs))
            else:
                if r.cache not in written:
                    raise ValueError(f"a run reads cache entry {r.cache} before any run writes it")
                same = lambda a, b: len(a) == len(b) and all(_any_window(u) == _any_window(v) for u, v in zip(a, b))
                if not same(written[r.cache], specs):
                    raise ValueError(f"a run reads cache entry {r.cache} of another shape: "
                                     f"{written[r.cache]} vs {specs}")
                if any(isinstance(s_, FixedState) for s_ in specs):
                    raise ValueError("a fixed-size state cannot be shared between runs")
                # the entry keeps what the widest window of its runs reads
                for e, spec in zip(ids, specs):
                    kept = self.cache_specs[e]
                    if kept.window is None:
                        continue
                    window = None if spec.window is None else max(kept.window, spec.window)
                    keep = 0 if window is None else max(kept.keep_first, spec.keep_first)
                    self.cache_specs[e] = dataclasses.replace(kept, window=window, keep_first=keep)
            self._run_entries.append((several, ids))
        self.embedding: Optional[torch.Tensor] = None
        self.head: Optional[torch.Tensor] = None

    # ------------------------------------------------------------------ description
    def weight_decls(self) -> list[WeightDecl]:
        decls = [self.embedding_decl]
        shared: dict = {}                        # tensors several parts read, once each
        for b in self.blocks:
            decls += b.weight_decls()
            for d in b.shared_decls():
                if shared.setdefault(d.name, d) != d:
                    raise ValueError(f"two parts declare the shared tensor '{d.name}' differently: {shared[d.name]} and {d}")
        decls += list(shared.values())
        if self.entry is not None:
            decls += self.entry.weight_decls()
        decls += self.final_norm.weight_decls()
        decls += self.depth_decls or []
        if self.head_decl is not None:
            decls.append(self.head_decl)
        seen, out = set(), []
        for d in decls:
            if d.name in seen:
                raise ValueError(f"two parts declare the tensor '{d.name}'")
            seen.add(d.name)
            out.append(d)
        return out

    def kernel_modules(self) -> list[str]:
        mods = ["elementwise"] + (["depth"] if self.depth_decls is not None else [])
        for b in self.blocks:
            mods += b.kernel_modules()
        mods += self.final_norm.kernel_modules() + (self.entry.kernel_modules() if self.entry is not None else [])
        return sorted(set(mods))

    def token_inputs(self) -> tuple:
        """What the parts read of a step's tokens beside ids and positions (parts.base.TokenInput), a name once."""
        from ..engine.batch import merge_token_inputs
        return merge_token_inputs([t for b in self.blocks for t in b.token_inputs()])

    def graph_safe(self) -> bool:
        return self.on_layer is None and all(b.graph_safe for b in self.blocks) and self.final_norm.graph_safe

    def records_portions(self) -> bool:
        return self.graph_safe() and all(getattr(b, "records_portions", False) for b in self.blocks)

    def num_parameters(self) -> int:
        n = 0
        for d in self.weight_decls():
            k = 1
            for s in d.shape:
                k *= s
            n += k
        return n

    # ------------------------------------------------------------------------ bind
    def bind(self, weights: dict[str, torch.Tensor], rt: Runtime) -> None:
        self.rt = rt
        self.embedding = weights[self.embedding_decl.name]
        self.head = weights[self.head_decl.name] if self.head_decl is not None else self.embedding
        for b in self.blocks:
            b.bind(weights, rt)
        self.final_norm.bind(weights, rt)
        if self.entry is not None:
            self.entry.bind(weights, rt)
        self._head_cast: Optional[torch.Tensor] = None
        if self.depth_decls is not None:
            self.depth_w = [weights[w.name].float().contiguous() for w in self.depth_decls]
        if self.streams is not None:
            self._ones = torch.ones(self.streams, dtype=torch.float32, device=rt.device)
        if self.head.dtype != rt.dtype and self.head.dtype != torch.float32:
            raise TypeError(f"head weight of type {self.head.dtype} in a {rt.dtype} run")
        self._head_k = self.hidden_size
        if self.head.dtype == torch.bfloat16:
            # the matrix kernels stream a tile-major copy; a tied embedding keeps its rows for the lookup
            head = self.head
            if self.hidden_size % 8 != 0 and not self.pad_hidden:
                raise ValueError(f"the bfloat16 matrix kernels need a hidden size that is a multiple of 8, "
                                 f"got {self.hidden_size}")
            if self.hidden_size % 8 != 0:
                # the kernels read 16 bytes at a time along the inner size: zero columns fill it up, and the
                # normed rows are widened with zeros before the product
                self._head_k = -(-self.hidden_size // 8) * 8
                head = head.new_zeros(self.vocab_size, self._head_k)
                head[:, :self.hidden_size] = self.head
            self.head = ops.tile_weight(head)

    # --------------------------------------------------------------------- forward
    def forward(self, ctx, cache_views: dict[int, object]) -> Optional[torch.Tensor]:
        """Runs the step's tokens through all layers.  Returns float32 logits
        [len(ctx.logit_rows), vocab], or None when no logits are wanted."""
        rt = self.rt
        if self.streams is not None:
            x = self._forward_streams(ctx, cache_views)
            return self._finish(x, ctx, False, False)
        if self.depth_decls is not None:
            x, h = self._forward_depth(ctx, cache_views)
            return self._finish(x, ctx, False, False, h)
        x = torch.empty(ctx.T, self.hidden_size, dtype=torch.float32, device=rt.device)
        ops.embed_rows(self.embedding, ctx.tokens, x, self.embedding_scale)
        x0 = None
        if any(r.reinject for r in self.schedule):
            # the embedding as it entered the first run, for the runs before which it joins the stream again
            x0 = torch.empty_like(x)
            ops.embed_rows(self.embedding, ctx.tokens, x0, self.embedding_scale)
        if self.carries:
            return self._finish(self._forward_carry(x, x0, ctx, cache_views), ctx, False, False)
        head_fused, all_rows = self._head_fused(ctx)
        for i, run in enumerate(self.schedule):
            block = self.blocks[run.block]
            if run.reinject:
                ops.post_norm_add(x, extra=x0)
            own = {} if self._run_states[i] is None else {"state": cache_views[self._run_states[i]]}
            if getattr(block, "takes_next_norm", False):
                if i + 1 < len(self.schedule):
                    nb = self.blocks[self.schedule[i + 1].block]
                    nxt = nb.first_norm_consumer() if hasattr(nb, "first_norm_consumer") else None
                else:
                    nxt = (self.final_norm, _HEAD) if head_fused and all_rows else None
                block.forward(x, ctx, self._views_of(i, cache_views), run.writes, next_norm=nxt, **own)
            else:
                block.forward(x, ctx, self._views_of(i, cache_views), run.writes, **own)
            if self.on_layer is not None:
                self.on_layer(i, x)
        return self._finish(x, ctx, head_fused, all_rows)

    def _forward_depth(self, ctx, cache_views) -> tuple:
        """The layers of a model with sums over the layers; returns the last sum, float32 [T, d], and, where every token's
        logits are wanted and the final norm is an RMS norm, that norm of it (else None).  One buffer holds the
        embedding and every run's stream: a run's place starts as its input, its sublayers add into it, and what stands
        there then is its result X_(i+1), so nothing is copied.  The kernel that sums the results also norms the sum for
        the next run's mixer."""
        last = len(self.schedule) - 1
        xs = torch.empty(last + 3, ctx.T, self.hidden_size, dtype=torch.float32, device=self.rt.device)
        ops.embed_rows(self.embedding, ctx.tokens, xs[0], self.embedding_scale)
        for i, run in enumerate(self.schedule):
            block, x = self.blocks[run.block], xs[i + 1]
            state = cache_views[self._run_states[i]] if self._run_states[i] is not None else None
            h = block.enter(x, ctx, state, xs=xs[:i + 1], w=self.depth_w[i - 1] if i else None)
            if self.on_layer is not None and i:
                self.on_layer(i - 1, x)
            block.forward(x, ctx, self._views_of(i, cache_views), run.writes, h=h)
        x = xs[last + 2]
        h = None
        if self._head_fused(ctx)[1] and isinstance(self.final_norm, RMSNorm):
            h = self.rt.empty(ctx.T, self.hidden_size)
            ops.depth_average(x, xs=xs[:last + 2], w=self.depth_w[last], norm_w=self.final_norm.weight_f32, eps=self.final_norm.eps, h_out=h)
        else:
            ops.depth_average(x, xs=xs[:last + 2], w=self.depth_w[last])
        if self.on_layer is not None:
            self.on_layer(last, x)
        return x, h

    def _forward_carry(self, x, x0, ctx, cache_views) -> torch.Tensor:
        """The layers of a model whose blocks hand each other their first normed input.  The kernel that adds a block's
        last output into x also adds the embedding where the next run takes it again, and norms x for the next block;
        the final norm runs with the head, on the wanted rows."""
        last = len(self.schedule) - 1
        y = torch.empty(ctx.T, self.hidden_size, dtype=torch.float32, device=self.rt.device)
        ops.fill_u32(y, 0)
        carry = z0 = None
        for i, run in enumerate(self.schedule):
            block = self.blocks[run.block]
            nxt = self.schedule[i + 1] if i < last else None
            if run.enter is not None:
                if z0 is None:                                  # (the first pass of the step)
                    rows = self.rt.empty(ctx.T, self.hidden_size)
                    ops.embed_rows(self.embedding, ctx.tokens, rows, self.embedding_scale)
                    z0 = self.entry.embedding_part(rows)
                    if carry is None:                           # nothing ran before: the stream is the embedding
                        carry = rows
                x, carry = self.entry.forward(carry, z0, run.enter, block.first_read())
            extra = x0 if nxt is not None and nxt.reinject else None
            if run.reinject and carry is None:
                ops.post_norm_add(x, extra=x0)              # (nobody before this run could add it)
            if self.on_layer is not None and extra is not None:
                # the hook sees x as the layer leaves it: the embedding joins afterwards, in a launch of its own
                block.forward(x, ctx, self._views_of(i, cache_views), run.writes, carry=carry, next_read=None, y=y)
                self.on_layer(i, x)
                carry = None
                continue
            read = None if nxt is None else PLAIN_ROWS if nxt.enter is not None else self.blocks[nxt.block].first_read()
            carry = block.forward(x, ctx, self._views_of(i, cache_views), run.writes, carry=carry, next_read=read, y=y, extra=extra)
            if self.on_layer is not None:
                self.on_layer(i, x)
        return x

    def _forward_streams(self, ctx, cache_views) -> torch.Tensor:
        """The layers over several residual streams; returns the sum of the streams, float32 [T, d].  The kernel that
        writes a block's last output into the streams also reads the next block's first input (or the final sum)."""
        S = self.streams
        xs = torch.empty(S, ctx.T, self.hidden_size, dtype=torch.float32, device=self.rt.device)
        for s in range(S):
            ops.embed_rows(self.embedding, ctx.tokens, xs[s], self.embedding_scale)
        carry = None
        last = len(self.schedule) - 1
        # what the sublayers add their outputs into: cleared once here, and by the streams' kernel whenever it has read it
        y = torch.empty(ctx.T, self.hidden_size, dtype=torch.float32, device=self.rt.device)
        ops.fill_u32(y, 0)
        for i, run in enumerate(self.schedule):
            block = self.blocks[run.block]
            nxt = self.blocks[self.schedule[i + 1].block].first_read() if i < last else (self._ones, None, 0.0)
            carry = block.forward(xs, ctx, self._views_of(i, cache_views), run.writes, carry=carry, next_read=nxt, y=y)
            if self.on_layer is not None:
                self.on_layer(i, xs)
        if last < 0:
            carry = torch.empty(ctx.T, self.hidden_size, dtype=torch.float32, device=self.rt.device)
            ops.hc_step(xs, in_w=self._ones, u_out=carry)
        return carry

    def _finish(self, x, ctx, head_fused: bool, all_rows: bool, h=None) -> Optional[torch.Tensor]:
        """The final norm and the head over x float32 [T, d].  h: the normed rows, where every row is wanted and they are
        there already."""
        # which rows are wanted is a fact of the step, not of its shape: the head runs outside of what is recorded
        # (a recorder keeps the function and hands back what it returns at each replay)
        # What the last block left for the final norm is taken here, where the step's kernels are issued (or
        # recorded: the tensors are then the recording's own, and every replay's head finds them as the eager
        # step's head does), not inside the function that runs later.
        pre = None
        if head_fused and all_rows and hasattr(self.final_norm, "take_announced"):
            pre = self.final_norm.take_announced(x)
        out: list = []

        def head(c):
            out[:] = [self._head(x, c, pre, h)]
            return out[0]

        ctx.run_eagerly(head)
        for part in self.blocks + [self.final_norm]:
            if hasattr(part, "forget"):                # what a product left for a norm that never asked for it
                part.forget()
        return out[0] if out else None

    def recording_key(self, ctx) -> tuple:
        """What forward() reads of a step outside of ctx.run_eagerly and bakes into its launches: a
        recording of a step in sections is valid for steps with the same key."""
        head_fused, all_rows = self._head_fused(ctx)
        return (ctx.T, bool((head_fused or self.depth_decls is not None) and all_rows))

    def _views_of(self, i: int, cache_views: dict):
        """What run i's mixer is handed as `cache`: None, a view, or a tuple of views."""
        several, ids = self._run_entries[i]
        if several:
            return tuple(cache_views[e] for e in ids)
        return cache_views[ids[0]] if ids else None

    def _head_fused(self, ctx) -> tuple:
        all_rows = ctx.n_logits == ctx.T and bool(ctx.host.get("logit_rows_identity", False))
        # the final norm inside the head's product (at most 16 rows), or, when every row is wanted,
        # from the row scales the last block leaves (at most 64)
        fused = (hasattr(self.final_norm, "pending") and self.head.dtype == torch.bfloat16
                 and self.hidden_size % 8 == 0 and ctx.n_logits > 0
                 and (ctx.n_logits <= ops.NORMED_MAX_ROWS and self.hidden_size <= ops.NORMED_MAX_K
                      or all_rows and ctx.n_logits <= ops.EMIT_MAX_ROWS))
        return fused, all_rows

    def _head(self, x, ctx, pre=None, h=None) -> Optional[torch.Tensor]:
        logits = self._head_product(x, ctx, pre, h)
        if logits is not None and (self.logit_scale != 1.0 or self.logit_softcap is not None):
            ops.scale_cap(logits, self.logit_scale, self.logit_softcap or 0.0)
        return logits

    def _head_product(self, x, ctx, pre=None, h=None) -> Optional[torch.Tensor]:
        """h: the final norm's rows, where they are there already.  pre: (xw, ss), the final norm's operand and row sums as
        the last block's product left them, or None."""
        if ctx.n_logits == 0:
            return None
        rt = self.rt
        head_fused, all_rows = self._head_fused(ctx)
        logits = torch.empty(ctx.n_logits, self.vocab_size, dtype=torch.float32, device=rt.device)
        if head_fused and h is None:
            fn = self.final_norm
            if pre is not None and all_rows:
                ops.gemm_scaled(pre[0], pre[1], fn.eps, self.head, logits)
                return logits
            if ctx.n_logits <= ops.NORMED_MAX_ROWS and self.hidden_size <= ops.NORMED_MAX_K:
                ops.gemm_normed(x, fn.weight_f32, fn.eps, self.head, logits, rows=ctx.logit_rows)
                return logits
        if h is None:
            h = self.final_norm.forward(x, rows=ctx.logit_rows)
        if h.dtype != self.head.dtype:
            h32 = torch.empty(h.shape, dtype=torch.float32, device=rt.device)
            ops.cast(h, h32)
            h = h32
        if self._head_k != self.hidden_size:
            h = ops.pad_cols(h, self._head_k)
        ops.gemm(h, self.head, logits)
        return logits
