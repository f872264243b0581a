"""Causal attention over a latent cache: per position one normed latent vector c [kv_rank],
from which every head's unrotated key and its value are up-projections, and one rotated key
part [rot_dim] that all heads share.  The cache holds nothing but c and that part.

With x the mixer's input, head a, W_uk,a [head_dim, kv_rank] and W_uv,a [value_dim, kv_rank]
the head's rows of the two up-projections:

    c_q      = rmsnorm(W_dq x) * w_dq                     the queries' latent
    q_a      = (W_uq c_q)_a = [q_plain (head_dim) | q_turn (rot_dim)]
    [c | t]  = W_dkv x;  c <- rmsnorm(c) * w_dkv;  t and q_turn are rotated by the position
    score    = (q_plain . W_uk,a c_j + q_turn . t_j) * scale
             = ((W_uk,a^T q_plain) . c_j + q_turn . t_j) * scale
    out_a    = W_uv,a (sum_j p_j c_j) * sigmoid(w_g,a . x)

so the up-projections never touch the cache: a head's query is carried into the latent's space
([W_uk,a^T q_plain | q_turn], kv_rank + rot_dim wide), attention runs with one shared "kv head"
whose key is the cached row [c | t] and whose value is that row's first kv_rank elements, and
the value up-projection is applied to the head's weighted sum of latents.  The softmax's
denominator may hold a learned sink per head.  Projections of x are one fused matrix
[dq | dkv | g].

Options of the spec: `q_rank` 0: the queries have no latent, q_a = (W_q x)_a, and the fused matrix
is [q | dkv | g]: one launch then stores the latents and turns the queries' rotated parts.
Position kind "rope_half": the pairs of the rotation are (i, i + rot_dim / 2), its frequencies
may be stretched and its cosine and sine multiplied by a magnitude; the projections' rows are put
into neighbouring pairs when the part is built, which leaves every score as it is.  `window`: a
query sees the last positions only.  `output_gate` "element": one gate an element of the
concatenated heads, sigmoid(W_g x), instead of one a head.  `shared_kv`: the part has no latents
of its own and reads those that another run has cached.

Kernels: `csrc/head_ops.hip`; attention in bfloat16 on the matrix cores
(`csrc/attention_wide.hip`: cache rows a multiple of 32 wide, latents a multiple of 16),
otherwise, and in float32, `csrc/attention_generic.hip`.
"""
from __future__ import annotations

import numpy as np
import torch

from ..csrc import lib
from ..csrc.lib import PAGE_TOKENS
from ..weights.loader import ParamSpec
from .attention import MATRIX_CORE_ATTENTION, MAX_SLICES, _decode_items
from .base import KVRequest
from .linear import Linear


class LatentAttention:
    @property
    def capture_safe(self):
        return all(product.capture_safe for product in self._products())

    @property
    def capture_rows(self):
        # (beyond the few-rows products' rows the per-head products are the library's as well)
        return min(*(product.capture_rows for product in self._products()), lib.SKINNY_ROWS)

    def _products(self):
        return [product for product in (self.down, self.up_q, self.o) if product is not None]

    @classmethod
    def parameters(cls, spec, hidden):
        params = {}
        if spec.q_rank:
            params["q_down.weight"] = ParamSpec((spec.q_rank, hidden))
            params["q_down_norm.weight"] = ParamSpec((spec.q_rank,), init="norm")
            params["q_up.weight"] = ParamSpec((spec.q_width, spec.q_rank), scale=0.1)
        else:
            params["q_proj.weight"] = ParamSpec((spec.q_width, hidden))
        if not spec.shared_kv:
            params["kv_down.weight"] = ParamSpec((spec.cache_width, hidden))
            params["kv_down_norm.weight"] = ParamSpec((spec.kv_rank,), init="norm")
        params["k_up.weight"] = ParamSpec((spec.n_heads * spec.head_dim, spec.kv_rank), scale=0.1)
        params["v_up.weight"] = ParamSpec((spec.n_heads * spec.value_dim, spec.kv_rank), scale=0.1)
        params["o_proj.weight"] = ParamSpec((hidden, spec.out_width))
        if spec.sink:
            params["sink"] = ParamSpec((spec.n_heads,), init="uniform", low=-1.0, high=1.0)
        if spec.output_gate:
            rows = spec.out_width if spec.output_gate == "element" else spec.n_heads
            params["gate_proj.weight"] = ParamSpec((rows, hidden))
        return params

    @classmethod
    def cache_request(cls, spec):
        # one row [latent | rotated key part] a position and no value pages: the values are the
        # row's first kv_rank elements
        keep = spec.window
        if spec.cache_span is not None:
            keep = None if spec.cache_span == 0 or keep is None else max(keep, spec.cache_span)
        return KVRequest(n_kv_heads=1, head_dim=spec.cache_width, value_dim=0, window=keep)

    @classmethod
    def on_matrix_cores(cls, spec, dtype) -> bool:
        return MATRIX_CORE_ATTENTION and lib.attention_wide_supported(
            dtype, spec.cache_width, spec.cache_width, spec.kv_rank)

    @classmethod
    def kernel_libraries(cls, spec, dtype):
        attention = "attention_wide" if cls.on_matrix_cores(spec, dtype) else "attention_generic"
        return ("head_ops", attention, *Linear.kernel_libraries(dtype))

    @classmethod
    def check(cls, spec):
        if min(spec.n_heads, spec.head_dim, spec.value_dim, spec.kv_rank) < 1 or spec.q_rank < 0:
            raise ValueError("latent_attention: every size must be positive")
        if spec.rot_dim < 0 or spec.rot_dim % 2:
            raise ValueError("latent_attention: rot_dim must be even")
        if spec.rot_dim and (spec.position.kind not in ("rope_pairs", "rope_half")
                             or spec.position.dim != spec.rot_dim):
            raise ValueError("latent_attention: the rotation is of pairs over the whole rotated part")
        if spec.cache_width > 1024 or spec.kv_rank > 512:
            raise ValueError("latent_attention: kv_rank may be 512 and kv_rank + rot_dim 1024 at "
                             f"most, got {spec.kv_rank} and {spec.cache_width}")
        if spec.window is not None and spec.window < 1:
            raise ValueError("latent_attention: a window must be at least 1")
        if spec.output_gate not in (False, True, "head", "element"):
            raise ValueError(f"latent_attention: unknown output_gate {spec.output_gate!r}")
        if spec.q_rank and (spec.shared_kv or spec.output_gate == "element"):
            raise ValueError("latent_attention: shared latents and a gate an element are "
                             "implemented for queries without a latent of their own")
        if not spec.q_rank and spec.output_gate in (True, "head"):
            raise ValueError("latent_attention: one gate a head is implemented for queries with a "
                             "latent of their own")

    def __init__(self, spec, hidden, params, dtype, device, positions):
        self.check(spec)
        self.spec = spec
        self.dtype = dtype
        H, d, r, e = spec.n_heads, spec.head_dim, spec.rot_dim, spec.value_dim
        q_last = params["q_up.weight" if spec.q_rank else "q_proj.weight"]     # rows: [heads, d + r]
        kv_down = None if spec.shared_kv else params["kv_down.weight"]
        if r and spec.position.kind == "rope_half":
            # pairs (i, i + r/2) become the neighbours (2i, 2i + 1) of permuted rows
            order = [row for i in range(r // 2) for row in (i, i + r // 2)]
            q_last = self._pair_rows(q_last, H, d, order)
            if kv_down is not None:
                kv_down = self._pair_rows(kv_down, 1, spec.kv_rank, order)
        fused = ([params["q_down.weight"]] if spec.q_rank else [q_last]) + \
            ([] if kv_down is None else [kv_down])
        if spec.output_gate:
            fused.append(params["gate_proj.weight"])
        spare = -sum(matrix.shape[0] for matrix in fused) % 8
        if not spec.q_rank and spare:      # (rows of whole 16-byte pieces for the batched products)
            fused.append(q_last.new_zeros((spare, hidden)))
        self.down = Linear(torch.cat(fused, dim=0), dtype, device)
        self.up_q = Linear(q_last, dtype, device) if spec.q_rank else None
        self.o = Linear(params["o_proj.weight"], dtype, device)

        def f32(tensor):
            return tensor.to(device=device, dtype=torch.float32).contiguous()
        self.q_norm = f32(params["q_down_norm.weight"]) if spec.q_rank else None
        self.c_norm = None if spec.shared_kv else f32(params["kv_down_norm.weight"])
        # per head [in, out]: W_uk,a as stored is [head_dim, kv_rank]; W_uv,a is transposed
        self.k_up = params["k_up.weight"].to(device=device, dtype=dtype) \
            .reshape(H, d, spec.kv_rank).contiguous()
        self.v_up = params["v_up.weight"].to(device=device, dtype=dtype) \
            .reshape(H, e, spec.kv_rank).transpose(1, 2).contiguous()
        self.sinks = f32(params["sink"]) if spec.sink else None
        position = positions(spec.position) if r else None
        self.frequencies = position.frequencies if r else None
        self.magnitude = getattr(position, "magnitude", 1.0)
        self.scale = spec.scale if spec.scale is not None else float(d + r) ** -0.5
        # where the fused projection's parts begin without a queries' latent: [q | dkv | g]
        self.latent_column = spec.q_width
        self.gate_column = spec.q_width + (0 if spec.shared_kv else spec.cache_width)
        self.compute_units = lib.compute_units(device)
        self.wide = self.on_matrix_cores(spec, dtype)
        self.positions_per_item = (lib.attention_wide_positions(H) if self.wide
                                   else lib.attention_positions_per_item(H))

    @staticmethod
    def _pair_rows(weight, heads: int, skip: int, order):
        """The last len(order) rows of each of `heads` runs of skip + len(order) rows, reordered."""
        run = skip + len(order)
        index = torch.tensor([h * run + row for h in range(heads)
                              for row in (*range(skip), *(skip + place for place in order))],
                             dtype=torch.long, device=weight.device)
        return weight.index_select(0, index)

    @property
    def plan_key(self):
        return ("latent_attention", self.positions_per_item, self.wide)

    def plan_step(self, plan):
        """Work items of the attention kernel, [3, items]: sequence, first row, positions."""
        if plan.decode:
            return {"attention.decode_items": _decode_items(plan.n_seqs, plan.n_live_seqs)}
        size = self.positions_per_item
        items = []
        for index, seq in enumerate(plan.seqs):
            for p0 in range(0, seq.count, size):
                npos = min(size, seq.count - p0)
                items.append((-(seq.start + p0 + npos), index, seq.row0 + p0, npos))
        items.sort()
        return {f"latent.items{size}": np.asarray([item[1:] for item in items],
                                                  dtype=np.int32).T.copy()}

    def decode_slices(self, n_seqs: int, context: int) -> int:
        """Slices of the key range in a decode step: enough blocks for about two a compute
        unit, never more than there are pages."""
        if self.spec.window is not None:
            context = min(context, self.spec.window + PAGE_TOKENS - 1)
        pages = max(1, (context + PAGE_TOKENS - 1) // PAGE_TOKENS)
        if self.wide:         # blocks of up to 64 heads, about two a compute unit
            blocks = n_seqs * ((self.spec.n_heads + 63) // 64)
            wanted = max(1, 2 * self.compute_units // blocks)
        else:
            blocks = n_seqs * ((self.spec.n_heads + 15) // 16)
            wanted = (2 * self.compute_units + blocks - 1) // blocks
        return max(1, min(wanted, pages, MAX_SLICES))

    def _by_library(self, rows: int, *sizes) -> bool:
        """Whether per-head products of so many rows are the library's batched ones (as the
        framework's other bfloat16 products of many rows; even sizes, which the kernel that
        brings their rows together wants)."""
        return (self.dtype == torch.bfloat16 and rows > lib.SKINNY_ROWS
                and all(size % 2 == 0 for size in sizes))

    def _batched(self, ctx, x, matrices, x_head, x_first, name):
        """[heads, rows, out] = x[n, h, x_first ..] . matrices[h], by the library."""
        heads, inner, outer = matrices.shape
        rows = x.shape[0]
        taken = x[:, :heads * x_head].view(rows, heads, x_head)[:, :, x_first:x_first + inner]
        made = ctx.buffer(name, (heads, rows, outer))
        torch.bmm(taken.transpose(0, 1), matrices, out=made)
        return made

    def _values(self, ctx, mixed, slices, gate_rows):
        """The heads' values [N, heads * value_dim] from their weighted sums of latents `mixed` (or
        the slices of them), gated element by element where the spec says so (`gate_rows` holds
        the logits)."""
        spec = self.spec
        n = gate_rows.shape[-2]
        out = ctx.buffer("latent.out", (n, spec.out_width))
        gate = None
        if spec.output_gate == "element":
            gate = lib.Columns(gate_rows, self.gate_column, spec.out_width)
        if slices is None and self._by_library(n, spec.value_dim) and \
                (gate is None or gate.dtype == self.dtype):
            made = self._batched(ctx, mixed, self.v_up, spec.kv_rank, 0, "latent.v_made")
            lib.heads_to_rows(made, out, spec.value_dim, gate=gate)
            ctx.release(made)
        else:
            lib.head_matmul(mixed, self.v_up, out, spec.n_heads, x_head=spec.kv_rank, x_first=0,
                            y_head=spec.value_dim, y_first=0, gate=gate, slices=slices)
        return out

    def _attend(self, ctx, q_wide, k_pages, page_table, gate):
        """(the heads' weighted sums of latents [N, heads * kv_rank], None), or, where the kernel that
        takes them can merge the slices of the key range itself, (None, (sums, weights, slices))."""
        spec, meta = self.spec, ctx.meta
        H, rank = spec.n_heads, spec.kv_rank
        n = q_wide.shape[0]
        common = dict(window=spec.window, scale=self.scale, value_dim=rank, sinks=self.sinks,
                      values_in_keys=True, gate=gate)
        part_o = part_ml = None
        if ctx.decode:
            splits = self.decode_slices(ctx.n_seqs, ctx.context_bound)
            if splits > 1:
                part_o = ctx.buffer("latent.part_o", (n * H * splits * rank,), torch.float32)
                part_ml = ctx.buffer("latent.part_ml", (n * H * splits * 2,), torch.float32)
            section = meta.section("attention.decode_items")
            common.update(n_splits=splits, part_o=part_o, part_ml=part_ml)
        else:
            section = meta.section(f"latent.items{self.positions_per_item}")
        slices = None
        if part_o is not None and self.wide and gate is None:
            slices = (part_o, part_ml, splits)
            common["merge"] = False
        # (the slices stand for it where they are merged later)
        mixed = ctx.buffer("latent.mixed", (n, H * rank))
        count = section.numel() // 3
        kernel = lib.attention_wide if self.wide else lib.attention
        kernel(q_wide, k_pages, None, section[:count], section[count:2 * count],
               section[2 * count:], count, meta.row_pos, meta.row_seq, page_table, mixed,
               H, 1, spec.cache_width, **common)
        ctx.release(q_wide, gate)
        if slices is None:
            ctx.release(part_o, part_ml)
            return mixed, None
        ctx.release(mixed)
        return None, slices

    def forward(self, ctx, x, entry):
        spec, meta = self.spec, ctx.meta
        if entry.writes_cache == spec.shared_kv:
            raise ValueError("latent_attention: a part writes the cache unless it has no latents "
                             "of its own")
        n = x.shape[0]
        group_index, k_pages, _ = ctx.cache.kv(entry.cache)
        page_table = meta.page_table(group_index)
        down = self.down.forward(ctx, x, "latent.down")
        q_wide = ctx.buffer("latent.q_wide", (n, spec.n_heads * spec.cache_width))
        store = self._store_with_latent if spec.q_rank else self._store_direct
        gate = store(ctx, down, q_wide, k_pages, page_table, entry)
        mixed, slices = self._attend(ctx, q_wide, k_pages, page_table, gate)
        out = self._values(ctx, mixed, slices, down)
        ctx.release(mixed, down, *(slices or ())[:2])
        delta = self.o.forward(ctx, out, "latent.o")
        ctx.release(out)
        return delta

    def _store_with_latent(self, ctx, down, q_wide, k_pages, page_table, entry):
        """Queries that pass a latent of their own: the latents stored, `q_wide` made; returns the
        heads' gate logits or None."""
        spec, meta = self.spec, ctx.meta
        H, d, r, rank = spec.n_heads, spec.head_dim, spec.rot_dim, spec.kv_rank
        n = q_wide.shape[0]
        n_gate = H if spec.output_gate else 0
        q_latent = ctx.buffer("latent.cq", (n, spec.q_rank))
        gate = ctx.buffer("latent.gate", (n, H), torch.float32) if n_gate else None
        lib.latent_down_store(down, self.q_norm, self.c_norm, spec.norm_eps, self.frequencies,
                              meta.row_pos, meta.row_seq, page_table, q_latent, k_pages, gate,
                              spec.q_rank, rank, r, n_gate, write_cache=entry.writes_cache,
                              turn_scale=self.magnitude)
        q = self.up_q.forward(ctx, q_latent, "latent.q")
        ctx.release(q_latent)
        if self._by_library(n, rank) and q.dim() == 2:
            made = self._batched(ctx, q, self.k_up, d + r, 0, "latent.q_made")
            lib.heads_to_rows(made, q_wide, spec.cache_width)
            ctx.release(made)
        else:
            lib.head_matmul(q, self.k_up, q_wide, H, x_head=d + r, x_first=0,
                            y_head=spec.cache_width, y_first=0)
        if r:
            lib.rotate_pairs(q, self.frequencies, meta.row_pos, q_wide, H, r, x_head=d + r,
                             x_first=d, y_head=spec.cache_width, y_first=rank,
                             turn_scale=self.magnitude)
        ctx.release(q)
        return gate

    def _store_direct(self, ctx, down, q_wide, k_pages, page_table, entry):
        """Queries that are columns of the projection itself: one launch stores the latents (unless
        they are another run's) and turns the queries' rotated parts, a second carries the rest
        into the latent's space."""
        spec, meta = self.spec, ctx.meta
        H, d, r, rank = spec.n_heads, spec.head_dim, spec.rot_dim, spec.kv_rank
        n = q_wide.shape[0]
        library = self._by_library(n, rank) and down.dim() == 2
        # with the library's product the kernel that brings its rows together turns them as well
        turns_there = library and r and self.frequencies.dtype == torch.float64
        turns = (d, H, d + r, q_wide, rank, spec.cache_width) if r and not turns_there else None
        if entry.writes_cache:
            lib.latent_down_store(lib.Columns(down, self.latent_column, spec.cache_width), None,
                                  self.c_norm, spec.norm_eps, self.frequencies, meta.row_pos,
                                  meta.row_seq, page_table, None, k_pages, None, 0, rank, r, 0,
                                  turn_scale=self.magnitude, turns=turns)
        elif turns is not None:
            lib.latent_down_store(down, None, None, spec.norm_eps, self.frequencies, meta.row_pos,
                                  meta.row_seq, page_table, None, k_pages, None, 0, 0, r, 0,
                                  write_cache=False, turn_scale=self.magnitude, turns=turns)
        if library:
            made = self._batched(ctx, down, self.k_up, d + r, 0, "latent.q_made")
            more = dict(turns=(down, d, d + r), frequencies=self.frequencies,
                        turn_scale=self.magnitude, row_pos=meta.row_pos) if turns_there else {}
            lib.heads_to_rows(made, q_wide, spec.cache_width, **more)
            ctx.release(made)
        else:
            lib.head_matmul(down, self.k_up, q_wide, H, x_head=d + r, x_first=0,
                            y_head=spec.cache_width, y_first=0)
        return None
