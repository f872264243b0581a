"""Gated delta rule: a recurrent mixer with one state matrix per head and sequence.

For token t, value head h and its query/key head h // (heads / kv_heads), with x the
mixer's input (all of the recurrence in float32):

    q, k, v  = silu(conv(W_q x)), silu(conv(W_k x)), silu(conv(W_v x))    short causal
               convolutions over time, one filter a channel, zeros before the sequence
    q, k     = unit vectors per head (x / sqrt(sum x^2 + unit_eps)); q also / sqrt(key_dim)
    beta     = sigmoid(W_beta x)                                          one per head
    g        = exp(-exp(decay_log_rate) * softplus(W_decay x + decay_bias))
    S       <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
    y        = W_o (o / sqrt(mean(o^2) + eps) * out_norm * silu(W_gate x))

Options of the spec: `decay_rank` > 0: the decay is one number per head and key channel,
g = exp(-exp(decay_log_rate_h) * softplus(W_d2 (W_d1 x) + decay_bias)) with decay_bias [heads *
key_dim], and acts on the rows of S that belong to key channels; the read-out's gate is then
W_g2 (W_g1 x), of rank `gate_rank`.  `gate_activation`: "silu" or "sigmoid".

The six input projections are one fused matrix [q | k | v | beta | decay | gate] (of low rank:
[q | k | v | W_d1 | W_g1 | beta]; the second matrices of a step of few rows are applied by the
convolution's launch, in a step of many rows by one library product of the block-diagonal
matrix of both).  Per
sequence the cache holds one float32 row (`StateRequest`): S of every head, then the last
taps - 1 inputs of every convolved channel, so a prompt may arrive whole, in portions of
any size or token by token.  The row has two versions: a step reads one and writes the whole
other one, and the session makes that one current when the step is committed, so a failed
step costs nothing and no copy of the state is ever taken.  Kernels: `csrc/delta_rule.hip`.
"""
from __future__ import annotations

import torch

from ..csrc import lib
from ..weights.loader import ParamSpec
from .base import StateRequest
from .linear import Linear


class GatedDelta:
    @property
    def capture_safe(self):
        """Only this library's kernels, nothing allocated per step, what varies read from the
        step's metadata on the device: as long as its products say the same."""
        return self.proj.capture_safe and self.o.capture_safe

    @property
    def capture_rows(self):
        return min(self.proj.capture_rows, self.o.capture_rows)

    @classmethod
    def shape_of(cls, spec) -> lib.DeltaShape:
        return lib.DeltaShape(spec.n_heads, spec.n_kv_heads, spec.key_dim, spec.value_dim,
                              spec.conv_taps, spec.decay_rank, spec.gate_rank)

    @classmethod
    def parameters(cls, spec, hidden):
        taps = spec.conv_taps
        if spec.decay_rank:
            return cls._low_rank_parameters(spec, hidden)
        return {
            "q_proj.weight": ParamSpec((spec.qk_width, hidden)),
            "k_proj.weight": ParamSpec((spec.qk_width, hidden)),
            "v_proj.weight": ParamSpec((spec.v_width, hidden)),
            "q_conv.weight": ParamSpec((spec.qk_width, taps), scale=0.5),
            "k_conv.weight": ParamSpec((spec.qk_width, taps), scale=0.5),
            "v_conv.weight": ParamSpec((spec.v_width, taps), scale=0.5),
            "beta_proj.weight": ParamSpec((spec.n_heads, hidden)),
            "decay_proj.weight": ParamSpec((spec.n_heads, hidden)),
            "decay_log_rate": ParamSpec((spec.n_heads,), init="uniform", low=-3.0, high=0.5),
            "decay_bias": ParamSpec((spec.n_heads,), init="uniform", low=-4.0, high=0.0),
            "gate_proj.weight": ParamSpec((spec.v_width, hidden)),
            "out_norm.weight": ParamSpec((spec.value_dim,), init="norm"),
            "o_proj.weight": ParamSpec((hidden, spec.v_width)),
        }

    @classmethod
    def _low_rank_parameters(cls, spec, hidden):
        taps, decays = spec.conv_taps, spec.n_heads * spec.key_dim
        return {
            "q_proj.weight": ParamSpec((spec.qk_width, hidden)),
            "k_proj.weight": ParamSpec((spec.qk_width, hidden)),
            "v_proj.weight": ParamSpec((spec.v_width, hidden)),
            "q_conv.weight": ParamSpec((spec.qk_width, taps), scale=0.5),
            "k_conv.weight": ParamSpec((spec.qk_width, taps), scale=0.5),
            "v_conv.weight": ParamSpec((spec.v_width, taps), scale=0.5),
            "beta_proj.weight": ParamSpec((spec.n_heads, hidden)),
            "decay_down.weight": ParamSpec((spec.decay_rank, hidden)),
            "decay_up.weight": ParamSpec((decays, spec.decay_rank), scale=0.1),
            "decay_log_rate": ParamSpec((spec.n_heads,), init="uniform", low=-3.0, high=0.5),
            "decay_bias": ParamSpec((decays,), init="uniform", low=-4.0, high=0.0),
            "gate_down.weight": ParamSpec((spec.gate_rank, hidden)),
            "gate_up.weight": ParamSpec((spec.v_width, spec.gate_rank), scale=0.1),
            "out_norm.weight": ParamSpec((spec.value_dim,), init="norm"),
            "o_proj.weight": ParamSpec((hidden, spec.v_width)),
        }

    @classmethod
    def cache_request(cls, spec):
        # (S is a megabyte a layer and sequence at real sizes: two versions instead of copies)
        return StateRequest(shape=(cls.shape_of(spec).state_floats,), two_versions=True)

    @classmethod
    def kernel_libraries(cls, spec, dtype):
        return ("delta_rule", *Linear.kernel_libraries(dtype))

    @classmethod
    def check(cls, spec):
        if spec.n_heads < 1 or spec.n_kv_heads < 1 or spec.n_heads % spec.n_kv_heads:
            raise ValueError("gated_delta: n_heads must be a multiple of n_kv_heads")
        if not 1 <= spec.key_dim <= 256:
            raise ValueError(f"gated_delta: key_dim must lie in 1..256, got {spec.key_dim}")
        if spec.value_dim < 1:
            raise ValueError("gated_delta: value_dim must be positive")
        if not 1 <= spec.conv_taps <= 32:
            raise ValueError(f"gated_delta: conv_taps must lie in 1..32, got {spec.conv_taps}")
        if (spec.decay_rank > 0) != (spec.gate_rank > 0):
            raise ValueError("gated_delta: decay and gate are both of low rank, or neither is")
        if spec.gate_activation not in ("silu", "sigmoid"):
            raise ValueError(f"gated_delta: unknown gate activation '{spec.gate_activation}'")

    def __init__(self, spec, hidden, params, dtype, device, positions=None):
        self.check(spec)
        self.spec = spec
        self.shape = self.shape_of(spec)
        if self.shape.low_rank:
            fused = self._low_rank_rows(params)
            up_decay, up_gate = (params[f"{name}.weight"].to(device=device, dtype=dtype)
                                 for name in ("decay_up", "gate_up"))
            # for few rows each matrix as [rank, out]; for many both as one [out, rank]
            self.w_decay, self.w_gate = up_decay.t().contiguous(), up_gate.t().contiguous()
            self.w_both = torch.block_diag(up_decay, up_gate).contiguous() \
                if dtype == torch.bfloat16 else None
        else:
            fused = torch.cat([params[f"{name}.weight"] for name in
                               ("q_proj", "k_proj", "v_proj", "beta_proj", "decay_proj",
                                "gate_proj")], dim=0)
        self.proj = Linear(fused, dtype, device)
        self.o = Linear(params["o_proj.weight"], dtype, device)

        def f32(tensor):
            return tensor.to(device=device, dtype=torch.float32).contiguous()
        self.conv_w = f32(torch.cat([params["q_conv.weight"], params["k_conv.weight"],
                                     params["v_conv.weight"]], dim=0))
        self.decay_log_rate = f32(params["decay_log_rate"])
        self.decay_bias = f32(params["decay_bias"])
        self.out_norm = f32(params["out_norm.weight"])
        self.q_scale = float(spec.key_dim) ** -0.5

    def _low_rank_rows(self, params):
        """The fused projection's rows where `DeltaShape` places them, zeros between."""
        shape = self.shape
        weights = {name: params[f"{name}.weight"] for name in
                   ("q_proj", "k_proj", "v_proj", "decay_down", "gate_down", "beta_proj")}
        fused = weights["q_proj"].new_zeros((shape.width, weights["q_proj"].shape[1]))
        at = {"q_proj": 0, "k_proj": shape.qk_width, "v_proj": 2 * shape.qk_width,
              "decay_down": shape.low_col, "gate_down": shape.gate_low_col,
              "beta_proj": shape.beta_col}
        for name, weight in weights.items():
            fused[at[name]:at[name] + weight.shape[0]] = weight
        return fused

    def input_product(self):
        """The product of x that a caller may make together with others."""
        return self.proj

    def use_input_product(self, product):
        self.proj = product

    def _convolved(self, ctx, proj, state, renew):
        """The convolved channels (and behind them, with a decay per key channel, the decays) and
        what holds the gate's logits (None: the projection itself)."""
        shape, meta = self.shape, ctx.meta
        rows, first = (proj.rows, proj.first) if isinstance(proj, lib.Columns) else (proj, 0)
        n = rows.shape[-2]
        conv = ctx.buffer("delta.conv", (n, shape.conv_width), torch.float32)
        where = (meta.row_pos, meta.row_seq, meta.seq_state_in, meta.seq_state_out, meta.seq_start)
        if not shape.low_rank:
            lib.delta_conv(proj, self.conv_w, state, shape, *where, conv, renew_tail=renew)
            return conv, None, None
        if proj.dtype == torch.float32:
            gate = ctx.buffer("delta.gate", (n, shape.v_width), torch.float32)
            lib.delta_prepare(proj, self.conv_w, state, shape, *where, conv, self.decay_log_rate,
                              self.decay_bias, self.w_decay, self.w_gate, gate, renew_tail=renew)
            return conv, gate, gate
        # a bfloat16 step of many rows: decays' and gate's logits as one library product
        both = ctx.buffer("delta.low", (n, shape.decay_width + shape.v_width))
        torch.matmul(rows[:, first + shape.low_col:first + shape.beta_col], self.w_both.t(), out=both)
        lib.delta_conv(proj, self.conv_w, state, shape, *where, conv, renew_tail=renew,
                       decay_logits=both, a_log=self.decay_log_rate, dt_bias=self.decay_bias)
        return conv, lib.Columns(both, shape.decay_width, shape.v_width), both

    def forward(self, ctx, x, entry, projected=None):
        """The mixer's rows; `projected`: the input product's rows, made by the caller."""
        if not entry.writes_cache:
            raise ValueError("gated_delta: a run that only reads another run's state is not "
                             "implemented")
        shape, meta = self.shape, ctx.meta
        n = x.shape[0]
        state = ctx.cache.state(entry.cache)                 # [2 (slots + 1), state_floats]
        rows_in = meta.seq_state_in                          # a sequence's state, and the row
        rows_out = meta.seq_state_out                        # the step writes
        proj = self.proj.forward(ctx, x, "delta.proj") if projected is None else projected
        # a decode step (one row a sequence) renews the convolution's tails in the same kernel
        renew = ctx.decode and shape.taps <= lib.DELTA_FEW_TAPS
        conv, gate, held = self._convolved(ctx, proj, state, renew)
        if not renew:
            lib.delta_tail(proj, state, shape, n, rows_in, rows_out, meta.seq_count,
                           meta.seq_row0)
        o_raw = ctx.buffer("delta.o_raw", (n, shape.v_width), torch.float32)
        rates = (None, None) if shape.low_rank else (self.decay_log_rate, self.decay_bias)
        lib.delta_rule(conv, proj, *rates, state, shape,
                       rows_in, rows_out, meta.seq_count, meta.seq_row0, o_raw, self.q_scale,
                       self.spec.unit_eps)
        ctx.release(conv)
        gated = ctx.buffer("delta.gated", (n, shape.v_width))
        lib.delta_out(o_raw, proj, self.out_norm, self.spec.out_norm_eps, shape, meta.row_seq,
                      gated, sigmoid_gate=self.spec.gate_activation == "sigmoid", gate_logits=gate)
        ctx.release(o_raw, proj if projected is None else None, held)
        delta = self.o.forward(ctx, gated, "delta.o")
        ctx.release(gated)
        return delta
