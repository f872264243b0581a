"""Routed feed-forward: a mixture of experts.

For every row x: router logits z = W_router x in float32 (the router matrix is kept in
float32; x is read as the step stores it), the `top` experts with the largest logits, their
weights p = softmax over the chosen logits alone, and

    y = sum over the chosen e of p_e W_down,e (silu(W_gate,e x) * (W_up,e x)).

With `scoring = "softmax_all"` the scores are the softmax over all router outputs, the choice
goes by score plus a learned `correction` per output (where the spec has one), and the weights
are the chosen scores themselves; with `identity = I` the router has I outputs beyond the
experts, and one of them chosen adds p x itself.

With `scoring = "sigmoid"` the scores are sigmoid(z); the experts are cut into `group_count`
runs of equal length, of which the `group_keep` whose two best scores add up to most take part, and the weights are the chosen scores over their sum, times `weight_scale`.  An expert's
activation may be the clamped swish of `parts.mlp`; `shared` is a gated feed-forward of its own
size that every row passes, whose rows the kernel that sums the experts' outputs adds.

The experts' matrices are stacked when the part is built (gate and up [E, F, H], down
[E, H, F]); routing stays on the device, so a step with this part is captured like any
other.  In bfloat16 with widths that are multiples of 64 the experts run as grouped matrix
products on the matrix cores (the pairs of (row, choice) laid out by expert on the device);
for few rows every expert's blocks find their pairs themselves and leave a slice a choice;
otherwise, and in float32, a kernel takes one pair at a time.  Kernels: `csrc/moe.hip`.
"""
from __future__ import annotations

import torch

from ..csrc import lib
from ..weights.loader import ParamSpec
from .mlp import GatedMLP


class RoutedMLP:
    @property
    def capture_safe(self):
        """Only this library's kernels, nothing read back, no allocation, as long as the shared
        expert's products do the same."""
        return self.shared is None or self.shared.capture_safe

    @property
    def capture_rows(self):
        return (1 << 30) if self.shared is None else self.shared.capture_rows

    @classmethod
    def kernel_libraries(cls, spec, dtype):
        shared = getattr(spec, "shared", None)
        return ("moe", "rowwise", *(() if shared is None else GatedMLP.kernel_libraries(shared, dtype)))

    @classmethod
    def parameters(cls, spec, hidden):
        outputs = spec.n_experts + getattr(spec, "identity", 0)
        params = {"router.weight": ParamSpec((outputs, hidden), scale=0.2)}
        if getattr(spec, "correction", False):
            params["router.correction"] = ParamSpec((outputs,), scale=0.05)
        for expert in range(spec.n_experts):
            prefix = f"experts.{expert}."
            params[prefix + "gate_proj.weight"] = ParamSpec((spec.intermediate_size, hidden))
            params[prefix + "up_proj.weight"] = ParamSpec((spec.intermediate_size, hidden))
            params[prefix + "down_proj.weight"] = ParamSpec((hidden, spec.intermediate_size))
        if getattr(spec, "shared", None) is not None:
            for name, param in GatedMLP.parameters(spec.shared, hidden).items():
                params["shared." + name] = param
        return params

    @classmethod
    def check(cls, spec):
        if not 1 <= spec.n_experts <= 512:
            raise ValueError(f"routed_mlp: 1 to 512 experts, got {spec.n_experts}")
        identity = getattr(spec, "identity", 0)
        if identity < 0 or spec.n_experts + identity > 512:
            raise ValueError("routed_mlp: a router has at most 512 outputs")
        if not 1 <= spec.top <= min(spec.n_experts + identity, 64):
            raise ValueError(f"routed_mlp: top must lie in 1..min(router outputs, 64), got {spec.top}")
        if getattr(spec, "scoring", "softmax_chosen") not in lib.ROUTER_SCORINGS:
            raise ValueError(f"routed_mlp: unknown scoring '{spec.scoring}'")
        if getattr(spec, "correction", False) and spec.scoring != "softmax_all":
            raise ValueError("routed_mlp: a correction belongs to the scoring 'softmax_all'")
        groups, keep = getattr(spec, "group_count", 1), getattr(spec, "group_keep", 1)
        if groups < 1 or not 1 <= keep <= groups or spec.n_experts % groups:
            raise ValueError(f"routed_mlp: {groups} groups of which {keep} are kept do not fit "
                             f"{spec.n_experts} experts")
        if groups > 1 and spec.scoring != "sigmoid":
            raise ValueError("routed_mlp: groups of experts belong to the scoring 'sigmoid'")
        if getattr(spec, "scoring", None) == "sigmoid" and \
                (identity or spec.top > spec.n_experts // groups * keep):
            raise ValueError("routed_mlp: the scoring 'sigmoid' has no identity experts, and the "
                             "kept groups must hold enough experts to choose from")
        if getattr(spec, "activation", "silu") not in lib.EXPERT_ACTIVATIONS:
            raise ValueError(f"routed_mlp: unknown activation '{spec.activation}'; "
                             f"known: {sorted(lib.EXPERT_ACTIVATIONS)}")
        if spec.intermediate_size < 1:
            raise ValueError("routed_mlp: an expert's width must be positive")

    def __init__(self, spec, hidden, params, dtype, device):
        self.check(spec)
        self.spec = spec
        self.hidden = hidden

        def stacked(name):
            return torch.stack([params[f"experts.{expert}.{name}.weight"]
                                for expert in range(spec.n_experts)]).to(
                                    device=device, dtype=dtype).contiguous()
        self.w_gate, self.w_up, self.w_down = stacked("gate_proj"), stacked("up_proj"), stacked("down_proj")
        self.router = params["router.weight"].to(device=device, dtype=torch.float32).contiguous()
        self.scoring = getattr(spec, "scoring", "softmax_chosen")
        self.correction = None
        if getattr(spec, "correction", False):
            self.correction = params["router.correction"].to(device=device, dtype=torch.float32).contiguous()
        self.routing = dict(scoring=self.scoring, correction=self.correction,
                            groups=getattr(spec, "group_count", 1), keep=getattr(spec, "group_keep", 1),
                            weight_scale=getattr(spec, "weight_scale", 1.0))
        self.act = dict(activation=getattr(spec, "activation", "silu"),
                        limit=getattr(spec, "limit", 0.0), alpha=getattr(spec, "alpha", 1.0))
        self.shared = None
        if getattr(spec, "shared", None) is not None:
            self.shared = GatedMLP(spec.shared, hidden,
                                   {name[len("shared."):]: tensor for name, tensor in params.items()
                                    if name.startswith("shared.")}, dtype, device)
        self.grouped = lib.moe_grouped_supported(dtype, hidden, spec.intermediate_size,
                                                 spec.n_experts)
        if self.grouped:       # (those forms take the matrices in operand order; no other copy is kept)
            self.w_gate, self.w_up, self.w_down = (
                lib.pack_experts(w) for w in (self.w_gate, self.w_up, self.w_down))

    def forward(self, ctx, x):
        spec = self.spec
        n = x.shape[0]
        if self.grouped and n <= lib.MOE_FEW_ROWS:
            slices = self._few_rows(ctx, x)
            if slices is not None:
                return slices
        shared = None if self.shared is None else self.shared.forward(ctx, x)
        expert = ctx.buffer("moe.expert", (n, spec.top), torch.int32)
        weight = ctx.buffer("moe.weight", (n, spec.top), torch.float32)
        lib.moe_route(x, self.router, ctx.meta.row_seq, expert, weight, **self.routing)
        act = ctx.buffer("moe.act", (n * spec.top, spec.intermediate_size))
        out = ctx.buffer("moe.out", (n, self.hidden), torch.float32)
        if self.grouped:
            pairs = n * spec.top
            order = ctx.buffer("moe.order", (2 * pairs + spec.n_experts + 1,), torch.int32)
            sums = ctx.buffer("moe.sums", (pairs, self.hidden), torch.float32)
            lib.moe_experts_grouped(x, self.w_gate, self.w_up, self.w_down, expert, weight,
                                    order[:pairs], order[pairs:2 * pairs], order[2 * pairs:], act,
                                    sums, out, extra=shared, **self.act)
            ctx.release(order, sums)
        else:
            lib.moe_experts(x, self.w_gate, self.w_up, self.w_down, expert, weight, act, out,
                            extra=shared, **self.act)
        ctx.release(shared, expert, weight, act)
        return out

    def _few_rows(self, ctx, x):
        """The rows of a step of few rows as float32 slices, one a choice, followed by those of the
        shared expert's last product: whoever reads the rows adds them up (None where the shared
        expert's product does not come in slices)."""
        spec = self.spec
        n = x.shape[0]
        if self.shared is None:
            slices = ctx.buffer("moe.slices.f32", (spec.top, n, self.hidden), torch.float32)
        else:
            slices = self.shared.slices_behind(ctx, x, "moe.slices", spec.top)
            if slices is None:
                return None
        expert = ctx.buffer("moe.expert", (n, spec.top), torch.int32)
        weight = ctx.buffer("moe.weight", (n, spec.top), torch.float32)
        lib.moe_route(x, self.router, ctx.meta.row_seq, expert, weight, **self.routing)
        act = ctx.buffer("moe.act", (n * spec.top, spec.intermediate_size))
        lib.moe_experts_few(x, self.w_gate, self.w_up, self.w_down, expert, weight, ctx.meta.row_seq,
                            act, slices[:spec.top], identity=getattr(spec, "identity", 0), **self.act)
        ctx.release(expert, weight, act)
        return slices
