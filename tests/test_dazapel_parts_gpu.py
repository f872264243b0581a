"""The mechanisms of the Dazapel layers alone, each against its plain function: the store kernel
with a projection's bias, a rotation with stretched frequencies and a magnitude and unit RMS
behind it; the router's choice within groups; clamped-swish experts beside a shared one; window
attention that keeps the first tokens, with keys made to stand out just inside and just outside
the window and the kept tokens, far keys among hundreds, gates on every element, in every form of
the kernels; and the vector added before each pass of a loop."""
import math

import pytest
import torch

import plain_dazapel as plain
from helpers import assert_close_bf16, assert_close_f32

pytestmark = pytest.mark.gpu
DEV = "cuda"
HIDDEN, VOCAB, EPS = 48, 31, 1e-5


def exact(shape, generator, scale=1.0):
    """Random float32 values that bfloat16 holds exactly."""
    return (torch.randn(shape, generator=generator) * scale).to(torch.bfloat16).float()


def i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


# -- the store kernel ---------------------------------------------------------------------------
@pytest.mark.parametrize("dim, vdim, rot, eps", [
    (16, 24, (10000.0, 16, (4.0, 40, 8.0, 1.0)), 1e-5),      # 16-byte pieces, the whole head
    (64, 64, (300000.0, 32, (6.0, 384, 24.0, 1.5)), 1e-6),   # half the head
    (40, 8, (100.0, 16, None), 0.3),                         # an eps that shows; 5 of 8 lanes work
    (10, 7, (3000.0, 6, (3.0, 25, 6.0, 1.5)), 1e-5),         # an element a lane
    (72, 16, (500.0, 72, None), 1e-5),                       # two elements a lane
    (24, 32, None, 1e-5)])                                   # no rotation: the norm alone
@pytest.mark.parametrize("slices", [0, 1, 3])
def test_store_with_bias_magnitude_and_unit_norm(dim, vdim, rot, eps, slices):
    from edge_infer_amd.config.specs import PositionSpec, YarnScaling
    from edge_infer_amd.csrc import lib
    from edge_infer_amd.parts.rope import RotaryHalfFrequencies
    heads, kv_heads, tail = 6, 2, 8
    g = torch.Generator().manual_seed(dim)
    positions = [0, 1, 63, 64, 1000, 123456, 1000000]
    n, width = len(positions), heads * dim + kv_heads * (dim + vdim) + tail
    shape = (n, width) if slices == 0 else (slices, n, width)
    proj = exact(shape, g)
    bias = exact((width,), g, 0.5)
    summed = (proj if slices == 0 else proj.double().sum(0)).double() + bias.double()
    magnitude, frequencies, rot_cfg = 1.0, None, None
    if rot is not None:
        scaling = None if rot[2] is None else YarnScaling(*rot[2])
        table = RotaryHalfFrequencies(PositionSpec(kind="rope_half", theta=rot[0], dim=rot[1],
                                                   scaling=scaling), DEV)
        frequencies, magnitude = table.frequencies, table.magnitude
        rot_cfg = {"base": rot[0], "dims": rot[1]}
        if rot[2] is not None:
            rot_cfg["scaling"] = dict(zip(("factor", "original", "fast", "slow"), rot[2]))
            assert magnitude > 1.05
    k_pages = torch.full((n, kv_heads, 64, dim), 9.0, device=DEV)
    v_pages = torch.full((n, kv_heads, 64, vdim), 9.0, device=DEV)
    # every row a sequence of its own whose current page is page `row`
    table_width = max(positions) // 64 + 1
    pages = torch.full((n, table_width), -1, dtype=torch.int32)
    for row, p in enumerate(positions):
        pages[row, p // 64] = row
    q = torch.empty(n, heads * dim, device=DEV)
    lib.head_store(proj.to(DEV), None, None, eps, frequencies, i32(positions), i32(list(range(n))),
                   pages.to(DEV), q, k_pages, v_pages, heads, kv_heads, dim, vdim,
                   bias=bias.to(DEV), turn_scale=magnitude, unit_norm=True)
    at = torch.tensor(positions)

    def turned(first, count):
        x = summed[:, first:first + count * dim].reshape(n, count, dim)
        return plain.unit_rms(plain.rotate_halves(x, at, rot_cfg), eps)
    assert_close_f32(q.reshape(n, heads, dim), turned(0, heads), "queries")
    slot = at % 64
    got_k = torch.stack([k_pages[row, :, slot[row]] for row in range(n)])
    got_v = torch.stack([v_pages[row, :, slot[row]] for row in range(n)])
    assert_close_f32(got_k, turned(heads * dim, kv_heads), "keys")
    first = (heads + kv_heads) * dim
    assert_close_f32(got_v, summed[:, first:first + kv_heads * vdim].reshape(n, kv_heads, vdim), "values")
    assert (k_pages == 9.0).sum().item() == k_pages.numel() - n * kv_heads * dim
    # into bfloat16, rounded once
    q16 = torch.empty(n, heads * dim, device=DEV, dtype=torch.bfloat16)
    k16, v16 = k_pages.to(torch.bfloat16), v_pages.to(torch.bfloat16)
    lib.head_store(proj.to(DEV), None, None, eps, frequencies, i32(positions), i32(list(range(n))),
                   pages.to(DEV), q16, k16, v16, heads, kv_heads, dim, vdim, bias=bias.to(DEV),
                   turn_scale=magnitude, unit_norm=True)
    assert (q16.float() - q).abs().max().item() <= 2.0 ** -8 * q.abs().max().item()


def test_a_bias_follows_its_rows_when_neighbouring_pairs_are_reordered():
    """A part whose rotation turns neighbouring pairs reorders the rows of its projections, and
    their biases with them: scores do not change, so neither does the output."""
    from edge_infer_amd.config.specs import AttentionSpec, PositionSpec
    mixer = AttentionSpec(n_heads=4, n_kv_heads=2, head_dim=8, value_dim=8, qkv_bias=True, o_bias=True,
                          scale=0.5, position=PositionSpec(kind="rope_pairs", theta=100.0, dim=8))
    spec = one_layer(mixer)
    params = params_for(spec, seed=3)
    model, session = session_for(spec, params)
    torch.manual_seed(1)
    T = 30
    x = torch.randn(T, HIDDEN).to(torch.bfloat16).float()
    t = tensors_of(params)

    def project(name, heads):
        rows = plain.linear(x, t["m." + name], t["m." + name + ".b"]).reshape(T, heads, 8)
        if name == "v":
            return rows
        out = rows.clone()
        for i in range(4):
            a = torch.arange(T, dtype=torch.float64) * 100.0 ** (-2.0 * i / 8)
            c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
            u, v = rows[..., 2 * i], rows[..., 2 * i + 1]
            out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
        return out
    want = plain.softmax_attention(project("q", 4), project("k", 2), project("v", 2), 0.5,
                                   lambda i: list(range(i + 1))).reshape(T, -1)
    want = plain.linear(want, t["m.o"], t["m.o.b"])
    for cuts in ([T], [2] * 5 + [20]):
        got = in_cuts(session, model.layers[0].mixer, x, cuts)
        assert_close_f32(got, want, f"neighbouring pairs with biases, cuts {cuts[:3]}")


# -- the router and the experts ------------------------------------------------------------------
@pytest.mark.parametrize("experts, groups, keep, top, width", [
    (20, 4, 3, 3, 48), (8, 2, 1, 3, 64), (5, 5, 3, 2, 50), (65, 13, 4, 4, 96), (12, 3, 3, 5, 48),
    (7, 1, 1, 7, 33), (1, 1, 1, 1, 16), (512, 64, 9, 8, 64), (128, 2, 1, 6, 40), (192, 96, 5, 4, 40)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_router_choice_within_groups(experts, groups, keep, top, width, dtype):
    from edge_infer_amd.csrc import lib
    g = torch.Generator().manual_seed(experts + groups)
    rows = 40
    x = exact((rows, width), g)
    tensors = {"r.router": exact((experts, width), g, 1.5 / width ** 0.5)}
    router = {"top": top, "scale": 1.7, "groups": {"count": groups, "keep": keep}}
    chosen, weights, scores = plain.route(x, tensors, "r.", router)
    clear = torch.tensor([plain.margin_of(row, router) > 2e-6 for row in scores])
    assert clear.sum() >= 30
    expert = torch.full((rows + 1, top), 77, dtype=torch.int32, device=DEV)
    weight = torch.full((rows + 1, top), 77.0, device=DEV)
    row_seq = i32([0] * rows + [-1])
    padded = torch.cat([x, torch.zeros(1, width)]).to(DEV).to(dtype)
    lib.moe_route(padded, tensors["r.router"].to(DEV), row_seq, expert, weight, scoring="sigmoid",
                  groups=groups, keep=keep, weight_scale=1.7)
    # (the order of the chosen is by score; where two chosen ones tie nearly they may change places)
    assert expert[:rows].cpu()[clear].sort(-1).values.tolist() == chosen[clear].sort(-1).values.tolist()
    order_got, order_want = expert[:rows].cpu()[clear].argsort(-1), chosen[clear].argsort(-1)
    assert_close_f32(torch.gather(weight[:rows].cpu()[clear], 1, order_got),
                     torch.gather(weights[clear], 1, order_want), "renormalised, scaled scores")
    assert torch.allclose(weight[:rows].sum(-1), torch.full((rows,), 1.7, device=DEV), rtol=1e-5)
    assert weight[rows].abs().max().item() == 0.0         # a padding row takes nothing
    if keep < groups and experts > groups:                # the groups matter
        free = torch.topk(scores, top, dim=-1).indices.sort(-1).values
        assert (free != chosen.sort(-1).values).any()


def test_equal_scores_and_equal_groups_go_to_the_lower_index():
    from edge_infer_amd.csrc import lib
    x = torch.ones(1, 16, device=DEV)
    router_w = torch.zeros(12, 16, device=DEV)            # every score is 1/2
    expert = torch.empty(1, 3, dtype=torch.int32, device=DEV)
    weight = torch.empty(1, 3, device=DEV)
    lib.moe_route(x, router_w, None, expert, weight, scoring="sigmoid", groups=4, keep=2)
    assert expert.cpu().tolist() == [[0, 1, 2]]
    router_w[7] = 1.0                                     # its group (2) comes first, then group 0
    lib.moe_route(x, router_w, None, expert, weight, scoring="sigmoid", groups=4, keep=2)
    assert expert.cpu().tolist() == [[7, 0, 1]]


def test_a_groups_score_is_the_sum_of_its_two_largest():
    """The best single expert's group loses against two good ones."""
    from edge_infer_amd.csrc import lib
    logit = torch.tensor([3.0, -4.0, -4.0, 1.0, 0.9, -3.0, -2.0, -3.0, -3.0])
    x = torch.zeros(1, 16, device=DEV)
    x[0, 0] = 1.0
    router_w = torch.zeros(9, 16, device=DEV)
    router_w[:, 0] = logit.to(DEV)
    expert = torch.empty(1, 2, dtype=torch.int32, device=DEV)
    weight = torch.empty(1, 2, device=DEV)
    lib.moe_route(x, router_w, None, expert, weight, scoring="sigmoid", groups=3, keep=1)
    assert expert.cpu().tolist() == [[3, 4]]
    lib.moe_route(x, router_w, None, expert, weight, scoring="sigmoid", groups=3, keep=2)
    assert expert.cpu().tolist() == [[0, 3]]
    s = torch.sigmoid(logit[[0, 3]].double())
    assert_close_f32(weight[0], s / s.sum(), "weights over the chosen scores' sum")


@pytest.mark.parametrize("experts, groups, keep, top, inter, shared, width, rows, dtype", [
    (6, 3, 2, 2, 40, 56, 48, 9, "float32"), (5, 1, 1, 3, 13, 11, 50, 7, "float32"),
    (4, 2, 1, 2, 24, None, 48, 20, "float32"), (8, 4, 2, 2, 64, 96, 64, 1, "bfloat16"),
    (8, 4, 2, 2, 64, 96, 64, 50, "bfloat16"), (8, 4, 3, 3, 128, 64, 128, 300, "bfloat16"),
    (4, 1, 1, 2, 256, 256, 256, 2, "bfloat16"), (20, 4, 2, 4, 64, None, 192, 40, "bfloat16"),
    (6, 2, 1, 2, 192, 40, 64, 16, "bfloat16"), (6, 2, 2, 3, 128, 33, 64, 30, "bfloat16"),
    (70, 7, 3, 5, 64, 64, 128, 64, "bfloat16"), (33, 3, 2, 2, 64, None, 64, 200, "bfloat16"),
    (3, 1, 1, 2, 192, 64, 64, 700, "bfloat16"), (5, 5, 4, 3, 64, None, 320, 1000, "bfloat16"),
    (5, 1, 1, 3, 24, 40, 48, 30, "bfloat16")])
def test_clamped_experts_beside_a_shared_one(experts, groups, keep, top, inter, shared, width, rows, dtype):
    """The routed feed-forward part through the pair-at-a-time kernels, the matrix-core ones of few
    rows (which leave a slice a choice) and the grouped ones (small and large tiles), the shared
    expert's rows as slices and as one tensor; limits that clamp many activations on both sides."""
    from edge_infer_amd.config.specs import GatedMLPSpec, RoutedMLPSpec
    from edge_infer_amd.parts import RoutedMLP
    g = torch.Generator().manual_seed(inter + rows)
    swish = dict(activation="clamped_swish", alpha=1.702)
    spec = RoutedMLPSpec(n_experts=experts, top=top, intermediate_size=inter, scoring="sigmoid",
                         weight_scale=1.3, group_count=groups, group_keep=keep, limit=0.8,
                         shared=None if shared is None else
                         GatedMLPSpec(intermediate_size=shared, limit=1.1, bias=False, **swish), **swish)
    # (few close calls: router rows of large size)
    tensors = {"f.router": exact((experts, width), g, 1.5 / width ** 0.5)}
    names = [(f"e{e}.", f"experts.{e}.", inter) for e in range(experts)]
    if shared is not None:
        names.append(("shared.", "shared.", shared))
    params = {"router.weight": tensors["f.router"]}
    for short, long, ff in names:
        for name, shape in (("gate", (ff, width)), ("up", (ff, width)), ("down", (width, ff))):
            tensors["f." + short + name] = params[f"{long}{name}_proj.weight"] = \
                exact(shape, g, shape[1] ** -0.5)
    part = RoutedMLP(spec, width, params, torch.float32 if dtype == "float32" else torch.bfloat16, DEV)
    assert part.grouped == (dtype == "bfloat16" and inter % 64 == 0 and width % 64 == 0)
    x = exact((rows, width), g, 1.5)
    mlp = {"expert": {"ff": inter, "limit": 0.8},
           "router": {"top": top, "scale": 1.3, "groups": {"count": groups, "keep": keep}}}
    if shared is not None:
        mlp["shared"] = {"ff": shared, "limit": 1.1}
    margins = []
    want = plain.routed_feed_forward(x, tensors, "f.", mlp, margins)
    clear = margins[0] > 1e-5

    class Context:
        class meta:
            row_seq = torch.zeros(rows, dtype=torch.int32, device=DEV)

        @staticmethod
        def buffer(name, shape, kind=None):
            return torch.empty(shape, device=DEV, dtype=kind or part.w_gate.dtype)

        @staticmethod
        def release(*buffers):
            pass
    got = part.forward(Context, x.to(DEV).to(part.w_gate.dtype))
    if got.dim() == 3:              # (few rows: a slice a choice, then the shared product's)
        assert part.grouped and rows <= 64
        got = got.sum(0)
    assert clear.sum() >= 0.9 * rows
    got, want = got[clear.to(DEV)], want[clear]
    if dtype == "float32":
        assert_close_f32(got, want, "clamped experts")
    else:
        assert_close_bf16(got, want, "clamped experts", rms_rel=1.5e-2, max_rel=2e-2)
    if shared is not None:          # it shows
        without = plain.routed_feed_forward(x, tensors, "f.", {k: v for k, v in mlp.items() if k != "shared"})
        assert (without[clear] - want).abs().max() > 0.1 * want.abs().max()


# -- attention ------------------------------------------------------------------------------------
def one_layer(mixer):
    from edge_infer_amd.config.specs import LayerSpec, ModelSpec, NormSpec, ScheduleEntry
    norm = NormSpec(eps=EPS)
    return ModelSpec(architecture="test", vocab_size=VOCAB, hidden_size=HIDDEN,
                     layers=(LayerSpec(block="prenorm", norm=norm, mixer=mixer, feed_forward=None),),
                     schedule=(ScheduleEntry(layer=0, cache=0),), final_norm=norm,
                     tie_word_embeddings=False, max_position_embeddings=1 << 20,
                     bos_token_id=None, eos_token_id=None)


def params_for(spec, seed):
    from edge_infer_amd.engine.model import model_parameters
    g = torch.Generator().manual_seed(seed)
    out = {}
    for path, param in model_parameters(spec).items():
        if param.optional:
            continue
        shape = tuple(param.shape)
        value = torch.randn(shape, generator=g)
        if param.init == "norm":
            value = 1 + 0.1 * value
        elif len(shape) == 2:
            value = value / shape[1] ** 0.5
        else:
            value = value * 0.4
        out[path] = value.to(torch.bfloat16).float()
    return out


def session_for(spec, params, dtype="float32", max_tokens=1024, max_seqs=4):
    from edge_infer_amd.engine import DecoderModel, Session
    model = DecoderModel(spec, params, dtype, DEV)
    return model, Session(model, max_tokens=max_tokens, max_seqs=max_seqs, graphs=False)


def run_part(session, part, pieces):
    """`pieces`: (slot, start, x rows) per sequence of one step; the part's output rows."""
    from edge_infer_amd.engine.batch import SeqStep
    seqs = [SeqStep(slot=slot, start=start, tokens=[0] * x.shape[0]) for slot, start, x in pieces]
    session.cache.grow([(s.slot, s.start + s.count) for s in seqs])
    ctx, _ = session.context_for(seqs)
    rows = torch.cat([x for _, _, x in pieces]).contiguous().to(DEV).to(session.dtype)
    out = part.forward(ctx, rows, session.model.spec.schedule[0])
    out = (out.sum(0) if out.dim() == 3 else out).float().clone()
    session.cache.commit([(s.slot, s.start + s.count) for s in seqs])
    return out


def in_cuts(session, part, x, cuts):
    slot = session.begin()
    rows, at = [], 0
    for take in cuts:
        rows.append(run_part(session, part, [(slot, at, x[at:at + take])]))
        at += take
    assert at == x.shape[0]
    session.end(slot)
    return torch.cat(rows)


NAMES = {"q_proj": "q", "k_proj": "k", "v_proj": "v", "gate_proj": "g", "o_proj": "o"}


def tensors_of(params):
    out = {}
    for path, value in params.items():
        if path.startswith("layers.0.mixer."):
            name, kind = path[len("layers.0.mixer."):].split(".")
            out["m." + NAMES[name] + (".b" if kind == "bias" else "")] = value
    return out


def kept_spec(heads, kv_heads, dim, vdim, scale, window, keep, rot):
    from edge_infer_amd.config.specs import AttentionSpec, PositionSpec, YarnScaling
    position = PositionSpec(kind="none") if rot is None else \
        PositionSpec(kind="rope_half", theta=rot[0], dim=rot[1],
                     scaling=None if rot[2] is None else YarnScaling(*rot[2]))
    return AttentionSpec(n_heads=heads, n_kv_heads=kv_heads, head_dim=dim, value_dim=vdim,
                         qkv_bias=True, o_bias=True, scale=scale, window=window, keep_first=keep,
                         position=position, qk_unit_norm=True, qk_norm_eps=EPS, output_gate=True)


def plain_kept(params, spec, x):
    mixer = {"heads": spec.n_heads, "kv_heads": spec.n_kv_heads, "dim": spec.head_dim,
             "vdim": spec.v_dim, "scale": spec.scale}
    if spec.window is not None:
        mixer["mask"] = {"size": spec.window, "keep_first": spec.keep_first}
    if spec.position.kind != "none":
        mixer["rot"] = {"base": spec.position.theta, "dims": spec.position.dim}
        s = spec.position.scaling
        if s is not None:
            mixer["rot"]["scaling"] = {"factor": s.factor, "original": s.original, "fast": s.fast, "slow": s.slow}
    return plain.attention_mixer(x.double(), tensors_of(params), "m.", mixer, EPS, torch.arange(x.shape[0]))


def close(dtype, got, want, what):
    if dtype == "float32":
        assert_close_f32(got, want, what)
    else:
        assert_close_bf16(got, want, what, rms_rel=2e-2, max_rel=4e-2)


@pytest.mark.parametrize("shape", [
    dict(heads=4, kv_heads=2, dim=16, vdim=24, scale=0.6, window=20, keep=5, rot=(100.0, 8, (4.0, 40, 8.0, 1.0))),
    dict(heads=6, kv_heads=1, dim=10, vdim=6, scale=0.8, window=None, keep=0, rot=(50.0, 10, None)),
    dict(heads=2, kv_heads=2, dim=64, vdim=64, scale=0.3, window=64, keep=64, rot=(1e4, 32, (8.0, 64, 16.0, 1.0))),
    dict(heads=8, kv_heads=2, dim=64, vdim=64, scale=0.3, window=3, keep=70, rot=None),
    dict(heads=6, kv_heads=3, dim=64, vdim=64, scale=0.3, window=70, keep=1, rot=(1e4, 64, None)),
    dict(heads=20, kv_heads=1, dim=64, vdim=64, scale=0.3, window=33, keep=17, rot=(1e4, 64, None)),
    dict(heads=4, kv_heads=1, dim=128, vdim=128, scale=0.2, window=65, keep=130, rot=(1e4, 128, (2.0, 30, 4.0, 0.5))),
    dict(heads=3, kv_heads=3, dim=128, vdim=128, scale=0.2, window=1, keep=0, rot=None),
    dict(heads=2, kv_heads=1, dim=64, vdim=32, scale=0.3, window=30, keep=9, rot=(1e4, 64, None))])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_window_attention_that_keeps_the_first_tokens_alone(shape, dtype):
    """Whole, in portions down to two tokens and token by token; head sizes 64 and 128 with
    values as wide take the matrix-core kernels in bfloat16."""
    mixer = kept_spec(**shape)
    params = params_for(one_layer(mixer), seed=5)
    model, session = session_for(one_layer(mixer), params, dtype)
    part = model.layers[0].mixer
    assert part.matrix_cores == (dtype == "bfloat16" and shape["dim"] >= 64 and shape["vdim"] == shape["dim"])
    torch.manual_seed(8)
    T = 210
    x = torch.randn(T, HIDDEN).to(torch.bfloat16).float()
    want = plain_kept(params, mixer, x)
    for cuts in ([T], [2] * 10 + [T - 20], [63, 2, 65, 80], [T - 60] + [1] * 60):
        close(dtype, in_cuts(session, part, x, cuts), want, f"attention {shape}, cuts {cuts[:3]}")
    session.cache.check()


@pytest.mark.parametrize("dtype, dim", [("float32", 16), ("bfloat16", 64), ("bfloat16", 128), ("bfloat16", 16)])
@pytest.mark.parametrize("window, keep", [(5, 3), (64, 64), (65, 1), (100, 70), (20, 130), (64, 16)])
def test_keys_that_stand_out_at_the_edges(window, keep, dtype, dim):
    """A key is made to dominate the last position's softmax (its input is the query's, and the
    keys are made with the queries' matrix): the oldest token of the window and the last kept
    token show, the token just before the window and the first one that is not kept do not.  In
    prompts, in portions that end at the edge, and decoded."""
    mixer = kept_spec(2, 2, dim, dim if dim >= 64 else 8, 6.0 / dim, window, keep, None)
    params = params_for(one_layer(mixer), seed=9)
    pre = "layers.0.mixer."
    params[pre + "k_proj.weight"] = params[pre + "q_proj.weight"].clone()
    params[pre + "k_proj.bias"] = params[pre + "q_proj.bias"].clone()
    model, session = session_for(one_layer(mixer), params, dtype)
    part = model.layers[0].mixer
    T = 240
    last = T - 1
    torch.manual_seed(6)
    base = torch.randn(T, HIDDEN).to(torch.bfloat16).float()
    # what stands behind one key of the many: the value is made to differ much from the others'
    cases = [(last - window + 1, True), (last - window, last - window < keep), (keep - 1, True),
             (keep, last - keep < window), (0, True)]
    quiet = plain_kept(params, mixer, base)
    for place, seen in cases:
        x = base.clone()
        x[place] = x[last] if place != last else x[place]
        want = plain_kept(params, mixer, x)
        moved = (want[-1] - quiet[-1]).abs().max().item() / want[-1].abs().max().item()
        assert (moved > 0.02) == seen, f"the key at {place} does not stand out as meant ({moved:.2e})"
        for cuts in ([T], [T - 1, 1], [place + 1, T - place - 1], [T - 30] + [1] * 30):
            close(dtype, in_cuts(session, part, x, cuts), want,
                  f"window {window}, keep {keep}, key at {place}, cuts {cuts[:3]}")


@pytest.mark.parametrize("dim, heads, kv_heads", [(64, 8, 2), (128, 4, 1), (64, 3, 3)])
def test_kept_tokens_in_the_form_whose_waves_take_whole_pages(dim, heads, kv_heads):
    """A prompt of few blocks lets two waves share every page's keys; one of many blocks gives
    a wave the whole page.  The second form is asked for here on a short prompt."""
    mixer = kept_spec(heads, kv_heads, dim, dim, 0.3, 40, 66, (1e4, dim // 2, (4.0, 64, 8.0, 1.0)))
    params = params_for(one_layer(mixer), seed=17)
    model, session = session_for(one_layer(mixer), params, "bfloat16")
    part = model.layers[0].mixer
    part.prefill_key_ways = lambda counts: 1
    torch.manual_seed(3)
    T = 250
    x = torch.randn(T, HIDDEN).to(torch.bfloat16).float()
    want = plain_kept(params, mixer, x)
    for cuts in ([T], [70, 180], [T - 3, 1, 1, 1]):
        close("bfloat16", in_cuts(session, part, x, cuts), want, f"one wave a page, cuts {cuts}")


@pytest.mark.parametrize("dtype, dim", [("float32", 16), ("bfloat16", 64)])
@pytest.mark.parametrize("splits", [1, 2, 5, 16])
def test_slices_of_a_decode_step_over_kept_tokens_and_window(dtype, dim, splits):
    """However many slices the kept tokens and the window are cut into, decoded rows are those
    of the prompt; with one slice the kernel applies the gates itself, with more the merge does."""
    mixer = kept_spec(4, 2, dim, dim, 2.5 / dim ** 0.5, 150, 90, (1e4, dim, None))
    params = params_for(one_layer(mixer), seed=23)
    model, session = session_for(one_layer(mixer), params, dtype)
    part = model.layers[0].mixer
    launch = part.decode_launch
    part.decode_launch = lambda n, context: (splits, *launch(n, context)[1:])
    torch.manual_seed(4)
    T = 420
    x = torch.randn(T, HIDDEN).to(torch.bfloat16).float()
    want = plain_kept(params, mixer, x)
    for first in (T - 12, 86, 60):
        got = in_cuts(session, part, x[:first + 12], [first] + [1] * 12)
        close(dtype, got, want[:first + 12], f"{splits} slices from position {first}")


@pytest.mark.parametrize("sequences", [40, 70])
def test_many_sequences_decoded_together(sequences):
    """Enough (sequence, kv head) pairs for the decode kernel's blocks of 8 and of 4 waves: every
    sequence's row is what it is alone."""
    mixer = kept_spec(8, 8, 64, 64, 0.3, 30, 9, (1e4, 32, (4.0, 64, 8.0, 1.0)))
    params = params_for(one_layer(mixer), seed=29)
    model, session = session_for(one_layer(mixer), params, "bfloat16", max_tokens=64 * 160,
                                 max_seqs=sequences)
    part = model.layers[0].mixer
    assert part.decode_launch(sequences, 128)[1] == (8 if sequences == 40 else 4)
    torch.manual_seed(5)
    lengths = [3, 12, 45, 70, 100]
    xs = [torch.randn(n + 4, HIDDEN).to(torch.bfloat16).float() for n in lengths]
    wants = [plain_kept(params, mixer, x) for x in xs]
    slots = [session.begin() for _ in range(sequences)]
    which = [s % len(lengths) for s in range(sequences)]
    run_part(session, part, [(slots[s], 0, xs[which[s]][:lengths[which[s]]]) for s in range(sequences)])
    for k in range(4):
        got = run_part(session, part, [(slots[s], lengths[which[s]] + k,
                                        xs[which[s]][lengths[which[s]] + k:][:1]) for s in range(sequences)])
        want = torch.stack([wants[which[s]][lengths[which[s]] + k] for s in range(sequences)])
        close("bfloat16", got, want, f"{sequences} sequences, token {k}")


@pytest.mark.parametrize("dtype, dim", [("float32", 16), ("bfloat16", 64)])
def test_a_far_kept_key_among_hundreds(dtype, dim):
    """Position 3 of 700 repeats the last position's input, and the window is 300: the kept key
    takes a weight that shows, position 8's (not kept) would not; whole, in portions and decoded,
    long after the pages between have been given back."""
    mixer = kept_spec(2, 1, dim, dim, 10.0 / dim, 300, 5, None)
    params = params_for(one_layer(mixer), seed=13)
    pre = "layers.0.mixer."
    params[pre + "k_proj.weight"] = params[pre + "q_proj.weight"][:dim].clone()
    params[pre + "k_proj.bias"] = params[pre + "q_proj.bias"][:dim].clone()
    model, session = session_for(one_layer(mixer), params, dtype)
    part = model.layers[0].mixer
    torch.manual_seed(10)
    T = 700
    base = torch.randn(T, HIDDEN).to(torch.bfloat16).float()
    quiet = plain_kept(params, mixer, base)
    x = base.clone()
    x[3] = x[T - 1]
    want = plain_kept(params, mixer, x)
    moved = (quiet[-1] - want[-1]).abs().max() / want[-1].abs().max()
    assert moved > 0.05, f"the far key does not show ({moved:.2e})"
    other = base.clone()
    other[8] = other[T - 1]
    assert torch.equal(plain_kept(params, mixer, other)[-1], quiet[-1])
    for cuts in ([T], [T - 1, 1], [2, 2, 300, T - 304 - 40] + [1] * 40):
        close(dtype, in_cuts(session, part, x, cuts), want, f"far key, cuts {cuts[:4]}")


def test_the_gates_reach_every_element():
    """Gates of very unequal size, made by a gate matrix whose rows differ by orders of magnitude:
    rows of a prompt of more than 256 rows (one bfloat16 tensor), of fewer (float32 slices) and
    decoded."""
    mixer = kept_spec(4, 2, 64, 64, 0.3, 50, 3, None)
    params = params_for(one_layer(mixer), seed=31)
    g = params["layers.0.mixer.gate_proj.weight"]
    params["layers.0.mixer.gate_proj.weight"] = (g * torch.logspace(-1, 1, g.shape[0])[:, None]).to(
        torch.bfloat16).float()
    model, session = session_for(one_layer(mixer), params, "bfloat16")
    part = model.layers[0].mixer
    torch.manual_seed(14)
    T = 330
    x = torch.randn(T, HIDDEN).to(torch.bfloat16).float()
    want = plain_kept(params, mixer, x)
    for cuts in ([T], [300, 29, 1], [100, 100, 100, 28, 1, 1]):
        close("bfloat16", in_cuts(session, part, x, cuts), want, f"gates, cuts {cuts}")


# -- the loop ----------------------------------------------------------------------------------------
@pytest.mark.parametrize("start, stop, times", [(0, 2, 2), (1, 2, 3), (0, 1, 1)])
def test_a_vector_is_added_once_before_each_pass(start, stop, times):
    """With layers whose sublayers add nothing (a multiplier of 0) the stream is the embedding row
    plus every pass's vector, once."""
    import edge_infer_amd as ei
    from dazapel_helpers import attention, model, sharp_weights
    from edge_infer_amd.config import DazapelConfig
    raw = model(50, 64, 1e-6, 0.0, (start, stop, times),
                [attention(2, 1, 16, 16, 0.5, None, None, None) for _ in range(2)])
    tensors = sharp_weights(raw, seed=4)
    cfg = DazapelConfig.from_dict(raw)
    entry = ei.config.resolve_architecture(raw)
    for dtype in ("float32", "bfloat16"):
        made = ei.build_model(entry, cfg, dict(tensors), dtype)
        session = ei.Session(made, max_tokens=128)
        slot = session.begin()
        got = torch.cat([session.step([(slot, [5, 7, 9], [0, 1, 2])]), session.step([(slot, [11], [0])])])
        x = tensors["embed"][[5, 7, 9, 11]].double() + tensors["loop.step"].double().sum(0)
        want = plain.linear(plain.rms_norm(x, tensors["final.norm"], 1e-6), tensors["embed"])
        assert torch.allclose(plain.forward(raw, tensors, [5, 7, 9, 11]), want, atol=1e-9)
        if dtype == "float32":
            assert_close_f32(got, want, "stream after the passes")
        else:
            assert_close_bf16(got, want, "stream after the passes")


def test_experts_of_few_rows_leave_padding_rows_out():
    """A step padded to a fixed batch: padding rows (in between and at the end) take no expert and
    do not disturb the others; a weight of exactly 0 still writes its slice."""
    from edge_infer_amd.csrc import lib
    g = torch.Generator().manual_seed(2)
    rows, top, experts, inter, width = 24, 2, 4, 64, 128
    x = exact((rows, width), g)
    w = [exact((experts, inter, width), g, width ** -0.5), exact((experts, inter, width), g, width ** -0.5),
         exact((experts, width, inter), g, inter ** -0.5)]
    expert = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(rows)]).to(torch.int32)
    weight = torch.rand(rows, top, generator=g)
    weight[5, 1] = 0.0
    row_seq = torch.arange(rows, dtype=torch.int32)
    dead = [3, 22, 23]
    row_seq[dead] = -1
    expert[dead], weight[dead] = 0, 0.0
    act = torch.empty(rows * top, inter, device=DEV, dtype=torch.bfloat16)
    out = torch.full((top, rows, width), 5.0, device=DEV)
    dev = [lib.pack_experts(m.to(DEV).to(torch.bfloat16)) for m in w]
    lib.moe_experts_few(x.to(DEV).to(torch.bfloat16), *dev, expert.to(DEV), weight.to(DEV),
                        row_seq.to(DEV), act, out, activation="clamped_swish", limit=0.9, alpha=1.702)
    for r in range(rows):
        if r in dead:
            assert bool((out[:, r] == 5.0).all())
            continue
        for k in range(top):
            e = int(expert[r, k])
            t = {"gate": w[0][e], "up": w[1][e], "down": w[2][e]}
            want = weight[r, k].double() * plain.clamped_expert(x[r:r + 1], t, "", 0.9)[0]
            assert torch.allclose(out[k, r].double().cpu(), want, atol=2e-2)
