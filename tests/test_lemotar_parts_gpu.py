"""The mechanisms of the Lemotar layers alone, each against its plain function: the norm over the
scaled stream and a sublayer's output, with and without normed branches; stretched frequencies;
window attention whose values are its keys, with a cap on the scores and a one in the softmax's
denominator, and keys made to stand out just inside and just outside the window; latent attention
with a window, a sink, a gate an element and rotated halves, keys that stand out, and a layer that
reads another layer's latents; the delta rule with a decay per key channel; and the two side by
side from one input product."""
import dataclasses

import pytest
import torch

import plain_lemotar as plain
from helpers import assert_close_bf16, assert_close_f32

pytestmark = pytest.mark.gpu
DEV = "cuda"
HIDDEN, VOCAB, EPS = 48, 31, 1e-5
PRE = "layers.0.mixer."


def layers_of(*mixers, ffn=None, alpha=1.0, hidden=HIDDEN, readers=()):
    """A model of the given mixers; `readers`: layer -> the layer whose cache it reads."""
    from edge_infer_amd.config.specs import LayerSpec, ModelSpec, NormSpec, ScheduleEntry
    norm = NormSpec(eps=EPS, weight_offset=1.0)
    readers = dict(readers)
    return ModelSpec(architecture="test", vocab_size=VOCAB, hidden_size=hidden,
                     layers=tuple(LayerSpec(block="postnorm", norm=norm, mixer=mixer, feed_forward=ffn,
                                            stream_scale=alpha) for mixer in mixers),
                     schedule=tuple(ScheduleEntry(layer=i, cache=readers.get(i, i),
                                                  writes_cache=i not in readers)
                                    for i in range(len(mixers))),
                     final_norm=norm, tie_word_embeddings=False, max_position_embeddings=1 << 20,
                     bos_token_id=None, eos_token_id=None)


def params_for(spec, seed):
    """Order-one parameters by parameter path, float32 values that bfloat16 holds exactly."""
    from edge_infer_amd.engine.model import model_parameters
    g = torch.Generator().manual_seed(seed)
    out = {}
    for path, param in model_parameters(spec).items():
        if param.optional:
            continue
        shape = tuple(param.shape)
        if param.init == "norm":
            value = 1 + 0.4 * (torch.rand(shape, generator=g) - 0.5)
        elif param.init == "uniform":
            value = param.low + (param.high - param.low) * torch.rand(shape, generator=g)
        elif "conv" in path:
            value = torch.randn(shape, generator=g) * 0.7
        elif len(shape) == 2:
            value = torch.randn(shape, generator=g) / shape[1] ** 0.5
        else:
            value = torch.randn(shape, generator=g) * 0.5
        out[path] = value.to(torch.bfloat16).float()
    return out


def session_for(spec, params, dtype="float32", max_tokens=1024, max_seqs=4):
    from edge_infer_amd.engine import DecoderModel, Session
    model = DecoderModel(spec, params, dtype, DEV)
    return model, Session(model, max_tokens=max_tokens, max_seqs=max_seqs, graphs=False)


def run_parts(session, spec, parts, pieces):
    """`pieces`: (slot, start, x rows) per sequence of one step; every part's output rows."""
    from edge_infer_amd.engine.batch import SeqStep
    seqs = [SeqStep(slot=slot, start=start, tokens=[0] * x.shape[0]) for slot, start, x in pieces]
    session.cache.grow([(s.slot, s.start + s.count) for s in seqs])
    ctx, _ = session.context_for(seqs)
    x = torch.cat([x for _, _, x in pieces]).contiguous().to(DEV)
    outs = []
    for part, entry in zip(parts, spec.schedule):
        out = part.forward(ctx, x, entry)
        out = out.sum(0) if out.dim() == 3 else out
        outs.append(out.float().clone())
    session.cache.commit([(s.slot, s.start + s.count) for s in seqs])
    return outs


def in_cuts(session, spec, parts, x, cuts):
    """The rows of `x` through the parts in steps of the given sizes, as one sequence."""
    slot = session.begin()
    rows, at = [], 0
    for take in cuts:
        rows.append(run_parts(session, spec, parts, [(slot, at, x[at:at + take])]))
        at += take
    assert at == x.shape[0]
    session.end(slot)
    return [torch.cat(outs) for outs in zip(*rows)]


def close(dtype, got, want, what, rms=2e-2, top=5e-2):
    if dtype == "float32":
        return assert_close_f32(got, want, what)
    return assert_close_bf16(got, want, what, rms_rel=rms, max_rel=top)


def rows_of(count, seed, size=1.0):
    g = torch.Generator().manual_seed(seed)
    return (size * torch.randn(count, HIDDEN, generator=g)).to(torch.bfloat16).float()


def under(params, prefix, names):
    return {short: params[prefix + long] for short, long in names.items()}


# -- the norm over the sum ---------------------------------------------------------------------
@pytest.mark.parametrize("alpha", [1.0, 2.7])
@pytest.mark.parametrize("width, rows", [(48, 3), (50, 2), (1000, 1), (2048, 600), (4100, 5)])
def test_norm_over_the_scaled_stream_and_a_delta(width, rows, alpha):
    from edge_infer_amd.csrc import lib
    g = torch.Generator().manual_seed(width)
    stream, delta = torch.randn(rows, width, generator=g), torch.randn(3, rows, width, generator=g) * 2
    weight = 0.6 * torch.rand(width, generator=g) - 0.3
    want = plain.offset_norm(alpha * stream.double() + delta.double().sum(0), weight, 1e-2)
    residual = stream.to(DEV)
    low = torch.empty(rows, width, device=DEV, dtype=torch.bfloat16)
    lib.post_norm(residual, delta.to(DEV), alpha, 1.0 + weight.to(DEV), 1e-2, cast_out=low)
    assert_close_f32(residual, want, "norm over the sum of stream and slices")
    assert torch.equal(low, residual.to(torch.bfloat16))
    narrow = delta[0].to(torch.bfloat16)
    want = plain.offset_norm(alpha * stream.double() + narrow.double(), weight, 1e-2)
    residual = stream.to(DEV)
    lib.post_norm(residual, narrow.to(DEV), alpha, 1.0 + weight.to(DEV), 1e-2)
    assert_close_f32(residual, want, "norm over the sum of stream and a bfloat16 delta")


@pytest.mark.parametrize("width, rows", [(48, 3), (50, 2), (1000, 1), (2048, 600), (4100, 5)])
def test_norm_over_the_stream_and_the_mean_of_normed_branches(width, rows):
    from edge_infer_amd.csrc import lib
    g = torch.Generator().manual_seed(width + 1)
    stream = torch.randn(rows, width, generator=g)
    one = torch.randn(2, rows, width, generator=g)
    two = (torch.randn(rows, width, generator=g) * 9).to(torch.bfloat16)
    w1, w2 = (1 + 0.5 * torch.randn(width, generator=g) for _ in range(2))
    weight = 0.6 * torch.rand(width, generator=g) - 0.3
    mean = 0.5 * (plain.rms_norm(one.double().sum(0), w1, EPS) + plain.rms_norm(two, w2, EPS))
    want = plain.offset_norm(1.4 * stream.double() + mean, weight, 1e-3)
    residual = stream.to(DEV)
    low = torch.empty(rows, width, device=DEV, dtype=torch.bfloat16)
    lib.post_norm(residual, [one.to(DEV), two.to(DEV)], 1.4, 1.0 + weight.to(DEV), 1e-3, cast_out=low,
                  branch_weights=[w1.to(DEV), w2.to(DEV)], branch_eps=EPS)
    assert_close_f32(residual, want, "norm over the stream and the branches' mean")
    assert torch.equal(low, residual.to(torch.bfloat16))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("with_ffn", [True, False])
def test_block_norms_the_sums(dtype, with_ffn):
    """norm1(alpha x + mixer(x)), then norm2(alpha x + ff(x)), weights stored around zero, on a
    model of one layer; a layer without a feed-forward has no second norm."""
    from edge_infer_amd.config.specs import GatedMLPSpec
    mixer = delta_spec(n_heads=2, n_kv_heads=1, key_dim=16, value_dim=16, conv_taps=3)
    ffn = GatedMLPSpec(intermediate_size=72, activation="silu", bias=False) if with_ffn else None
    spec = layers_of(mixer, ffn=ffn, alpha=1.7)
    params = params_for(spec, 11)
    assert ("layers.0.norm2.weight" in params) == with_ffn
    model, session = session_for(spec, params, dtype)
    tokens = [3, 30, 7, 7, 12, 0, 19, 4]
    x = params["embed.weight"][tokens].double()
    x = plain.offset_norm(1.7 * x + plain_delta(params, PRE, mixer, x), params["layers.0.norm1.weight"], EPS)
    if with_ffn:
        matrices = under(params, "layers.0.ffn.", {"gate": "gate_proj.weight", "up": "up_proj.weight",
                                                   "down": "down_proj.weight"})
        x = plain.offset_norm(1.7 * x + plain.dense_feed_forward(x, matrices, ""),
                              params["layers.0.norm2.weight"], EPS)
    want = plain.linear(plain.offset_norm(x, params["final_norm.weight"], EPS), params["head.weight"])
    slot = session.begin()
    logits = session.step([(slot, tokens[:5], list(range(5)))])
    logits = torch.cat([logits, session.step([(slot, tokens[5:], [0, 1, 2])])])
    close(dtype, logits, want, "block")


# -- rotation ------------------------------------------------------------------------------------
@pytest.mark.parametrize("base, dims, scaling", [
    (10000.0, 32, (4.0, 100, 8.0, 1.0)), (250.0, 6, (16.0, 30, 2.0, 0.5)),
    (10000.0, 64, (1.0, 4096, 32.0, 1.0)), (500000.0, 16, (8.0, 12, 64.0, 32.0)),
    (10000.0, 2, (8.0, 4096, 32.0, 1.0)), (7000.0, 8, None)])
def test_stretched_frequencies(base, dims, scaling):
    """Ramps of ordinary width, of no width, cut at either end, and a factor of one."""
    from edge_infer_amd.config.specs import PositionSpec, YarnScaling
    from edge_infer_amd.parts.rope import RotaryHalfFrequencies
    rot = {"base": base, "dims": dims}
    made = None
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
        made = YarnScaling(**rot["scaling"])
    got = RotaryHalfFrequencies(PositionSpec(kind="rope_half", theta=base, dim=dims, scaling=made), DEV)
    want, magnitude = plain.stretched_frequencies(rot)
    want = torch.tensor(want, dtype=torch.float64)
    assert ((got.frequencies.cpu() - want).abs() <= 1e-12 * want).all()
    assert abs(got.magnitude - magnitude) < 1e-12


# -- window attention whose values are its keys --------------------------------------------------
def keyed_spec(n_heads, n_kv_heads, dim, scale, softcap, window, rot):
    from edge_infer_amd.config.specs import AttentionSpec, PositionSpec
    return AttentionSpec(n_heads=n_heads, n_kv_heads=n_kv_heads, head_dim=dim, value_dim=dim,
                         qkv_bias=False, o_bias=False, qk_norm=True, qk_norm_scope="projection",
                         qk_norm_eps=EPS, values_from_keys=True, scale=scale, softcap=softcap,
                         window=window, unit_sink=True,
                         position=PositionSpec(kind="rope_pairs", theta=rot[0], dim=rot[1]))


def plain_keyed(params, prefix, mixer, x):
    tensors = under(params, prefix, {"q": "q_proj.weight", "k": "k_proj.weight", "o": "o_proj.weight",
                                     "q.norm": "q_norm.weight", "k.norm": "k_norm.weight"})
    m = {"heads": mixer.n_heads, "kv_heads": mixer.n_kv_heads, "dim": mixer.head_dim,
         "scale": mixer.scale, "softcap": mixer.softcap,
         "rot": {"base": mixer.position.theta, "dims": mixer.position.dim},
         "mask": None if mixer.window is None else {"size": mixer.window}}
    return plain.shared_value_attention(x, tensors, "", m, EPS, torch.arange(x.shape[0]))


@pytest.mark.parametrize("shape", [
    (6, 3, 16, 0.7, 4.0, 20, (10000.0, 8)), (5, 1, 10, 0.9, 1.5, 1, (100.0, 10)),
    (4, 4, 40, 0.3, 50.0, 65, (700.0, 2)), (8, 1, 24, 0.5, 3.0, None, (10000.0, 24)),
    # the matrix-core kernels in bfloat16: groups of 1, 3, 4 and 8, windows about the page of 64
    (4, 4, 64, 0.3, 5.0, 64, (10000.0, 32)), (6, 2, 64, 0.3, 2.0, 63, (10000.0, 64)),
    (8, 2, 128, 0.2, 8.0, 100, (500.0, 16)), (8, 1, 64, 0.35, 30.0, None, (10000.0, 16)),
    (2, 1, 128, 0.2, 4.0, 2, (10000.0, 128)), (3, 3, 64, 0.3, 6.0, 130, (10000.0, 2))])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_window_attention_with_keys_as_values_alone(shape, dtype):
    """Whole, in portions and token by token, over the window's edge and two page borders."""
    mixer = keyed_spec(*shape)
    spec = layers_of(mixer)
    params = params_for(spec, seed=7)
    model, session = session_for(spec, params, dtype)
    part = model.layers[0].mixer
    assert part.matrix_cores == (dtype == "bfloat16" and mixer.head_dim in (64, 128))
    x = rows_of(150, 5)
    want = plain_keyed(params, PRE, mixer, x.double())
    for cuts in ([150], [60, 2, 3, 64, 21], [100] + [1] * 50):
        got, = in_cuts(session, spec, [part], x.to(model.dtype), cuts)
        close(dtype, got, want, f"keys as values {shape} {cuts[:3]}")
    session.cache.check()


@pytest.mark.parametrize("heads, kv_heads, dim", [(6, 2, 64), (8, 8, 64), (4, 1, 128)])
def test_capped_attention_over_a_long_prompt_on_the_matrix_cores(heads, kv_heads, dim):
    """Prompts of many blocks and of few, in a batch, a window of several pages, then decoding
    together (key ranges cut into slices)."""
    mixer = keyed_spec(heads, kv_heads, dim, 0.25, 5.0, 300, (10000.0, dim // 2))
    spec = layers_of(mixer)
    params = params_for(spec, seed=8)
    model, session = session_for(spec, params, "bfloat16", max_tokens=2048)
    part = model.layers[0].mixer
    lengths = [700, 65, 330]
    xs = [rows_of(n, 50 + n) for n in lengths]
    wants = [plain_keyed(params, PRE, mixer, x.double()) for x in xs]
    slots = [session.begin() for _ in xs]
    cuts = [n - 4 for n in lengths]
    got, = run_parts(session, spec, [part], [(s, 0, x[:c].bfloat16()) for s, x, c in zip(slots, xs, cuts)])
    close("bfloat16", got, torch.cat([w[:c] for w, c in zip(wants, cuts)]), "prompts")
    for t in range(4):
        got, = run_parts(session, spec, [part], [(s, c + t, x[c + t:c + t + 1].bfloat16())
                                                 for s, x, c in zip(slots, xs, cuts)])
        close("bfloat16", got, torch.stack([w[c + t] for w, c in zip(wants, cuts)]), f"token {t}")


@pytest.mark.parametrize("dim, dtype", [(16, "float32"), (64, "float32"), (64, "bfloat16"), (128, "bfloat16")])
@pytest.mark.parametrize("window", [5, 64, 65, 100])
def test_a_key_that_stands_out_at_the_windows_edge(window, dim, dtype):
    """Queries and keys are made by one matrix and one element of two turns, so a row that is a
    multiple of the last position's has a key like the query's own and a value of another
    size.  Just outside the window it must change nothing; just inside it takes a share of the
    weight that shows."""
    mixer = keyed_spec(2, 2, dim, 8.0 / dim, 9.0, window, (1e4, 2))
    spec = layers_of(mixer)
    params = params_for(spec, seed=9)
    params[PRE + "k_proj.weight"] = params[PRE + "q_proj.weight"].clone()
    params[PRE + "k_norm.weight"] = params[PRE + "q_norm.weight"].clone()
    model, session = session_for(spec, params, dtype)
    part = model.layers[0].mixer
    T = 180
    base = rows_of(T, 6)
    for offset, seen in ((window, False), (window - 1, True)):
        x = base.clone()
        x[T - 1 - offset] = 3.0 * x[T - 1]
        want = plain_keyed(params, PRE, mixer, x.double())
        calm = x.clone()
        calm[T - 1 - offset] = base[T - 1 - offset]
        quiet = plain_keyed(params, PRE, mixer, calm.double())
        moved = (want[-1] - quiet[-1]).abs().max().item() / want[-1].abs().max().item()
        assert (moved > 0.15) == seen, f"the test's key does not stand out as meant ({moved:.2e})"
        for cuts in ([T], [T - 1, 1], [T - offset - 1, 1, offset], [T - 30] + [1] * 30):
            got, = in_cuts(session, spec, [part], x.to(model.dtype), cuts)
            close(dtype, got[-1:], want[-1:], f"window {window}, key at distance {offset}, cuts {cuts[:3]}",
                  rms=3e-2, top=6e-2)


def test_cap_and_the_softmaxs_one_show():
    """The first positions: with the one in the denominator a lone key of a small score takes half
    the weight; the cap, left out or halved, moves the output by far more than the tolerance."""
    mixer = keyed_spec(4, 2, 16, 0.9, 3.0, 40, (1e4, 4))
    spec = layers_of(mixer)
    params = params_for(spec, seed=10)
    x = rows_of(60, 7)
    wants = {}
    for cap in (3.0, 1.5, 1e6):
        capped = dataclasses.replace(mixer, softcap=cap)
        wants[cap] = plain_keyed(params, PRE, capped, x.double())
        for dtype in ("float32", "bfloat16"):
            model, session = session_for(layers_of(capped), params, dtype)
            got, = in_cuts(session, spec, [model.layers[0].mixer], x.to(model.dtype), [1, 1, 40, 18])
            close(dtype, got, wants[cap], f"cap {cap}")
    top = wants[3.0].abs().max()
    assert all((wants[3.0] - wants[cap]).abs().max() > 0.02 * top for cap in (1.5, 1e6))
    quiet = dataclasses.replace(mixer, scale=1e-6)
    want = plain_keyed(params, PRE, quiet, x.double())
    values = plain.linear(x[:1], params[PRE + "k_proj.weight"]).reshape(1, 2, 16)
    lone = plain.linear(0.5 * values.repeat_interleave(2, dim=1).reshape(1, 64), params[PRE + "o_proj.weight"])
    assert torch.allclose(want[:1], lone, rtol=1e-4, atol=1e-5)
    model, session = session_for(layers_of(quiet), params)
    got, = in_cuts(session, spec, [model.layers[0].mixer], x, [60])
    assert_close_f32(got, want, "scores of nothing")


# -- latent attention -----------------------------------------------------------------------------
def latent_spec(n_heads, dim, rot, vdim, rank, scale, window, shared=False, span=None):
    from edge_infer_amd.config.specs import LatentAttentionSpec, PositionSpec, YarnScaling
    scaling = None if rot[2] is None else YarnScaling(*(float(v) for v in rot[2]))
    return LatentAttentionSpec(n_heads=n_heads, head_dim=dim, rot_dim=rot[1], value_dim=vdim,
                               kv_rank=rank, q_rank=0, scale=scale, norm_eps=EPS, sink=True,
                               output_gate="element", window=window, shared_kv=shared, cache_span=span,
                               position=PositionSpec(kind="rope_half", theta=rot[0], dim=rot[1],
                                                     scaling=scaling))


def plain_latent(params, prefix, mixer, x, shared=None):
    names = {"q": "q_proj.weight", "uk": "k_up.weight", "uv": "v_up.weight", "sink": "sink",
             "g": "gate_proj.weight", "o": "o_proj.weight"}
    if shared is None:
        names.update({"dkv": "kv_down.weight", "dkv.norm": "kv_down_norm.weight"})
    rot = {"base": mixer.position.theta, "dims": mixer.rot_dim}
    if mixer.position.scaling is not None:
        rot["scaling"] = dataclasses.asdict(mixer.position.scaling)
    m = {"heads": mixer.n_heads, "dim": mixer.head_dim, "rot_dim": mixer.rot_dim,
         "vdim": mixer.value_dim, "kv_rank": mixer.kv_rank, "scale": mixer.scale, "rot": rot,
         "mask": None if mixer.window is None else {"size": mixer.window}}
    return plain.latent_attention(x, under(params, prefix, names), "", m, EPS,
                                  torch.arange(x.shape[0]), shared)


YARN = (4.0, 60, 8.0, 1.0)


@pytest.mark.parametrize("shape", [
    (3, 16, (1e4, 8, YARN), 24, 40, 0.25, 21), (1, 32, (500.0, 16, None), 40, 24, 0.2, 64),
    (20, 8, (1e4, 2, YARN), 8, 72, 0.3, 65), (5, 7, (1e4, 6, (2.0, 400, 30.0, 4.0)), 9, 13, 0.3, 1),
    (6, 24, (1e5, 32, YARN), 12, 264, 0.1, None),
    # cache rows that the matrix-core kernel for wide keys takes in bfloat16
    (3, 16, (1e4, 16, YARN), 24, 48, 0.25, 17), (20, 8, (1e4, 32, YARN), 8, 96, 0.2, 63),
    (8, 32, (1e4, 32, YARN), 32, 64, 0.15, 100), (70, 8, (1e4, 32, None), 4, 32, 0.2, None),
    (16, 64, (1e4, 64, YARN), 64, 256, 0.09, 130)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_latent_attention_alone(shape, dtype):
    """Whole, in portions and token by token; with a sink that outweighs the first keys."""
    mixer = latent_spec(*shape)
    spec = layers_of(mixer)
    params = params_for(spec, seed=11)
    params[PRE + "sink"][0] = 3.0
    model, session = session_for(spec, params, dtype)
    part = model.layers[0].mixer
    assert part.wide == (dtype == "bfloat16" and mixer.cache_width % 32 == 0 and mixer.kv_rank % 16 == 0)
    x = rows_of(150, 8)
    want, _ = plain_latent(params, PRE, mixer, x.double())
    for cuts in ([150], [60, 2, 3, 64, 21], [100] + [1] * 50):
        got, = in_cuts(session, spec, [part], x.to(model.dtype), cuts)
        close(dtype, got, want, f"latent attention {shape} {cuts[:3]}")
    session.cache.check()


@pytest.mark.parametrize("rank, rot_dim, dtype", [(40, 4, "float32"), (64, 32, "float32"), (64, 32, "bfloat16")])
@pytest.mark.parametrize("window", [5, 64, 65, 100])
def test_a_latent_that_stands_out_at_the_windows_edge(window, rank, rot_dim, dtype):
    """Queries are carried by the matrices that make the keys, so an earlier row's latent that is
    the last position's outscores every other; the values are made from the latent, whose
    weight in the sum shows.  Outside the window it must change nothing."""
    dim = 16
    mixer = latent_spec(2, dim, (1e9, rot_dim, None), 12, rank, 0.2, window)
    spec = layers_of(mixer)
    params = params_for(spec, seed=13)
    # q_plain = U down x and k = U c: a row's key is aligned with its own query
    up = torch.randn(2 * dim, rank, generator=torch.Generator().manual_seed(3)) / rank ** 0.5
    params[PRE + "k_up.weight"] = up.to(torch.bfloat16).float()
    q = params[PRE + "q_proj.weight"].reshape(2, dim + rot_dim, HIDDEN)
    q[:, :dim] = (params[PRE + "k_up.weight"] @ params[PRE + "kv_down.weight"][:rank]) \
        .reshape(2, dim, HIDDEN).to(torch.bfloat16).float()
    q[:, dim:] *= 0.1
    model, session = session_for(spec, params, dtype)
    part = model.layers[0].mixer
    T = 180
    base = rows_of(T, 10)
    for offset, seen in ((window, False), (window - 1, True)):
        x = base.clone()
        # (near the last row, so that it scores as high, yet with a latent of its own)
        x[T - 1 - offset] = x[T - 1] + 0.5 * base[3]
        x = x.to(torch.bfloat16).float()
        want, _ = plain_latent(params, PRE, mixer, x.double())
        calm = x.clone()
        calm[T - 1 - offset] = base[5]
        quiet, _ = plain_latent(params, PRE, mixer, calm.double())
        moved = (want[-1] - quiet[-1]).abs().max().item() / want[-1].abs().max().item()
        assert (moved > 0.1) == seen, f"the test's latent does not stand out as meant ({moved:.2e})"
        for cuts in ([T], [T - 1, 1], [T - offset - 1, 1, offset], [T - 30] + [1] * 30):
            got, = in_cuts(session, spec, [part], x.to(model.dtype), cuts)
            close(dtype, got[-1:], want[-1:], f"window {window}, latent at distance {offset}, cuts {cuts[:3]}",
                  rms=4e-2, top=8e-2)


@pytest.mark.parametrize("rank, rot_dim", [(40, 8), (64, 32)])
def test_a_far_latent_among_hundreds_and_the_sink(rank, rot_dim):
    """Position 3 of 700 repeats the last position's input and there is no window: its latent takes
    a weight that shows; with the sink left out the oracle's own output moves as well."""
    dim = 16
    mixer = latent_spec(2, dim, (1e9, rot_dim, None), 16, rank, 1.0, None)
    spec = layers_of(mixer)
    params = params_for(spec, seed=14)
    up = torch.randn(2 * dim, rank, generator=torch.Generator().manual_seed(4)) / rank ** 0.5
    params[PRE + "k_up.weight"] = up.to(torch.bfloat16).float()
    q = params[PRE + "q_proj.weight"].reshape(2, dim + rot_dim, HIDDEN)
    q[:, :dim] = (params[PRE + "k_up.weight"] @ params[PRE + "kv_down.weight"][:rank]) \
        .reshape(2, dim, HIDDEN).to(torch.bfloat16).float()
    q[:, dim:] *= 0.1
    T = 700
    x = rows_of(T, 12)
    x[3] = x[T - 1]

    def reference(tensors, rows):
        return plain_latent(tensors, PRE, mixer, rows.double())[0]
    # a sink of about the own key's score
    latent = plain.rms_norm(plain.linear(x[-1:], params[PRE + "kv_down.weight"][:rank]),
                            params[PRE + "kv_down_norm.weight"], EPS)
    own = (plain.linear(x[-1:], q.reshape(-1, HIDDEN)).reshape(2, -1)[:, :dim]
           * plain.linear(latent, params[PRE + "k_up.weight"]).reshape(2, dim)).sum(1)
    params[PRE + "sink"] = own.to(torch.bfloat16).float()
    want = reference(params, x)
    other = x.clone()
    other[3] = x[4]
    top = want[-1].abs().max()
    assert (reference(params, other)[-1] - want[-1]).abs().max() > 0.05 * top, "the far latent does not show"
    assert (reference({**params, PRE + "sink": torch.full((2,), -30.0)}, x)[-1] - want[-1]).abs().max() \
        > 0.05 * top, "the sink does not show"
    for dtype in ("float32", "bfloat16"):
        model, session = session_for(spec, params, dtype)
        for cuts in ([T], [T - 1, 1], [2, 2, 300, T - 304 - 40] + [1] * 40):
            got, = in_cuts(session, spec, [model.layers[0].mixer], x.to(model.dtype), cuts)
            close(dtype, got, want, f"far latent, cuts {cuts[:4]}", rms=4e-2, top=0.12)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rank, rot_dim", [(40, 8), (64, 32)])
@pytest.mark.parametrize("windows", [(10, 90), (90, 10), (10, None), (None, 33)])
def test_a_layer_that_reads_another_layers_latents(windows, rank, rot_dim, dtype):
    """The second and third mixers have no down-projection: they meet the first one's cached latents
    and rotated parts with queries, up-projections, sinks, windows and head counts of their
    own; the first one's cache keeps what the widest window needs."""
    rot = (500.0, rot_dim, YARN)
    span = 0 if None in windows else max(*windows, 40)
    mixers = [latent_spec(4, 16, rot, 24, rank, 0.3, windows[0], span=span),
              latent_spec(3, 24, rot, 16, rank, 0.25, windows[1], shared=True),
              latent_spec(8, 8, rot, 8, rank, 0.35, 40, shared=True)]
    spec = layers_of(*mixers, readers={1: 0, 2: 0})
    params = params_for(spec, seed=21)
    model, session = session_for(spec, params, dtype)
    parts = [layer.mixer for layer in model.layers]
    assert "kv_down.weight" not in type(parts[1]).parameters(mixers[1], HIDDEN)
    T = 200
    x = rows_of(T, 4)
    first, kept = plain_latent(params, PRE, mixers[0], x.double())
    wants = [first] + [plain_latent(params, f"layers.{i}.mixer.", mixers[i], x.double(), kept)[0]
                       for i in (1, 2)]
    for cuts in ([T], [70, 2, 64, 64], [T - 50] + [1] * 50):
        outs = in_cuts(session, spec, parts, x.to(model.dtype), cuts)
        for index, (got, want) in enumerate(zip(outs, wants)):
            close(dtype, got, want, f"layer {index}, cuts {cuts[:3]}", rms=3e-2, top=8e-2)
    session.cache.check()


@pytest.mark.parametrize("rows, heads, k, j, slices", [(1, 3, 16, 40, 2), (7, 5, 48, 12, 5)])
def test_merged_slices_and_a_gate_in_the_heads_product(rows, heads, k, j, slices):
    """`head_matmul` on what attention over a cut key range leaves: sums weighted by the slices'
    maxima and masses; then a sigmoid an element."""
    from edge_infer_amd.csrc import lib
    g = torch.Generator().manual_seed(rows)
    part_o = torch.randn(rows, heads, slices, k, generator=g)
    part_m = torch.randn(rows, heads, slices, generator=g) * 3
    part_l = torch.rand(rows, heads, slices, generator=g) + 0.1
    matrices = torch.randn(heads, k, j, generator=g) / k ** 0.5
    gate = torch.randn(rows, heads * j, generator=g)
    weight = torch.exp(part_m.double() - part_m.double().max(dim=2, keepdim=True).values)
    merged = (weight[..., None] * part_o.double()).sum(2) / (weight * part_l.double()).sum(2)[..., None]
    want = torch.stack([merged[:, h] @ matrices[h].double() for h in range(heads)], dim=1) \
        .reshape(rows, -1) * plain.sigmoid(gate.double())
    held = torch.cat([torch.full((rows, 5), 9.0), gate], dim=1).to(DEV)
    y = torch.empty(rows, heads * j, device=DEV)
    part_ml = torch.stack([part_m, part_l], dim=3)
    lib.head_matmul(None, matrices.to(DEV), y, heads, x_head=k, x_first=0, y_head=j, y_first=0,
                    gate=lib.Columns(held, 5, heads * j),
                    slices=(part_o.to(DEV).contiguous(), part_ml.to(DEV).contiguous(), slices))
    assert_close_f32(y, want, "merged slices through the heads' product")


# -- the delta rule with a decay per key channel --------------------------------------------------
def delta_spec(**kw):
    from edge_infer_amd.config.specs import GatedDeltaSpec
    base = dict(n_heads=4, n_kv_heads=2, key_dim=24, value_dim=40, conv_taps=4, out_norm_eps=EPS,
                decay_rank=7, gate_rank=11, gate_activation="sigmoid", unit_eps=1e-6)
    base.update(kw)
    return GatedDeltaSpec(**base)


DELTA_NAMES = {"q": "q_proj.weight", "k": "k_proj.weight", "v": "v_proj.weight",
               "q.conv": "q_conv.weight", "k.conv": "k_conv.weight", "v.conv": "v_conv.weight",
               "b": "beta_proj.weight", "a1": "decay_down.weight", "a2": "decay_up.weight",
               "A_log": "decay_log_rate", "dt_bias": "decay_bias", "g1": "gate_down.weight",
               "g2": "gate_up.weight", "norm": "out_norm.weight", "o": "o_proj.weight"}


def plain_delta(params, prefix, mixer, x):
    m = {"heads": mixer.n_heads, "kv_heads": mixer.n_kv_heads, "dim": mixer.key_dim,
         "vdim": mixer.value_dim}
    return plain.delta_mixer(x, under(params, prefix, DELTA_NAMES), "", m, EPS)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [
    dict(), dict(conv_taps=1, n_heads=2, n_kv_heads=2, key_dim=8, value_dim=8, decay_rank=1, gate_rank=1),
    dict(key_dim=144, value_dim=12, n_heads=2, n_kv_heads=1, decay_rank=30),
    dict(key_dim=13, value_dim=5, n_heads=3, n_kv_heads=1, conv_taps=2),
    dict(conv_taps=7, key_dim=64, value_dim=64, n_heads=2, n_kv_heads=2, decay_rank=64, gate_rank=64),
    dict(conv_taps=10, key_dim=16, value_dim=24, n_heads=6, n_kv_heads=2, decay_rank=130, gate_rank=3),
    dict(key_dim=256, value_dim=8, n_heads=1, n_kv_heads=1, conv_taps=3),
    dict(key_dim=128, value_dim=128, n_heads=4, n_kv_heads=4, decay_rank=128, gate_rank=128)])
def test_delta_rule_with_channel_decays_alone(sizes, dtype):
    """Two sequences: whole prompts of unequal lengths, then portions of 2, 1 and 5 rows, then
    single tokens; the state and the convolution's tail carry over every cut."""
    mixer = delta_spec(**sizes)
    spec = layers_of(mixer)
    params = params_for(spec, 8)
    # decays that differ from channel to channel: half of them forget at once, half hardly
    bias = params[PRE + "decay_bias"]
    bias[::2] = 4.0
    bias[1::2] = -6.0
    model, session = session_for(spec, params, dtype)
    part = model.layers[0].mixer
    lengths = [83, 21]
    xs = [rows_of(n, 30 + n) for n in lengths]
    expected = [plain_delta(params, PRE, mixer, x.double()) for x in xs]
    slots = [session.begin() for _ in lengths]
    at = [n - 12 for n in lengths]

    def run(takes, what):
        out, = run_parts(session, spec, [part], [(s, a, x[a:a + t].to(model.dtype))
                                                 for s, x, a, t in zip(slots, xs, at, takes)])
        close(dtype, out, torch.cat([e[a:a + t] for e, a, t in zip(expected, at, takes)]), what,
              rms=3e-2, top=6e-2)
    prompts, at = at, [0, 0]
    run(prompts, f"{sizes}: prompts")
    at = prompts
    for take in (2, 1, 5, 1, 1, 2):
        run([take, take], f"{sizes}: {take} rows at {at}")
        at = [a + take for a in at]
    assert at == lengths


@pytest.mark.parametrize("rows", [300, 20])
def test_delta_rule_of_many_rows_and_few_in_bfloat16(rows):
    """A step of many rows takes the library's product for decays and gate, one of few rows the
    launch that also convolves; both follow the oracle."""
    mixer = delta_spec(key_dim=64, value_dim=64, n_heads=4, n_kv_heads=2, decay_rank=64, gate_rank=32)
    spec = layers_of(mixer)
    params = params_for(spec, 12)
    model, session = session_for(spec, params, "bfloat16")
    x = rows_of(rows, 9)
    want = plain_delta(params, PRE, mixer, x.double())
    got, = in_cuts(session, spec, [model.layers[0].mixer], x.bfloat16(), [rows - 3, 2, 1])
    close("bfloat16", got, want, f"{rows} rows", rms=2e-2, top=5e-2)


def test_channel_decays_act_on_the_rows_of_their_channels():
    """Channels that never forget keep what the third token wrote for 150 tokens; the others lose
    it at once.  Exchanging the two halves of the decays moves the output by far more than the
    tolerance, and the part follows the oracle in each case."""
    mixer = delta_spec(n_heads=2, n_kv_heads=2, key_dim=32, value_dim=16)
    spec = layers_of(mixer)
    params = params_for(spec, 10)
    params[PRE + "decay_up.weight"] *= 0.1
    x = rows_of(153, 6)
    results = []
    for keep in (slice(0, 16), slice(16, 32)):
        bias = torch.full((2, 32), 5.0)
        bias[:, keep] = -30.0
        params[PRE + "decay_bias"] = bias.reshape(-1)
        want = plain_delta(params, PRE, mixer, x.double())
        other = x.clone()
        other[2] = -x[2]
        far = (plain_delta(params, PRE, mixer, other.double())[-1] - want[-1]).abs().max()
        assert far > 1e-3 * want[-1].abs().max(), "what was written long ago does not show"
        model, session = session_for(spec, params)
        got, = in_cuts(session, spec, [model.layers[0].mixer], x, [70, 80, 1, 1, 1])
        assert_close_f32(got, want, f"channels {keep} keep")
        results.append(want)
    assert (results[0] - results[1]).abs().max() > 0.1 * results[0].abs().max()


def test_delta_rule_from_the_first_token_and_in_a_slot_used_again():
    """Single tokens from position 0 (the convolution sees zeros before the start), then the
    slot is given back and taken again: the new sequence starts from an empty state."""
    mixer = delta_spec()
    spec = layers_of(mixer)
    params = params_for(spec, 9)
    for dtype in ("float32", "bfloat16"):
        model, session = session_for(spec, params, dtype, max_seqs=1)
        for trial in range(2):
            x = rows_of(9, 70 + trial)
            got, = in_cuts(session, spec, [model.layers[0].mixer], x.to(model.dtype), [1] * 9)
            close(dtype, got, plain_delta(params, PRE, mixer, x.double()), f"trial {trial}",
                  rms=3e-2, top=6e-2)


# -- side by side ---------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("softmax, delta", [
    ((6, 3, 16, 0.7, 4.0, 20, (1e4, 8)), dict()),
    ((4, 2, 64, 0.3, 6.0, 65, (1e4, 32)), dict(key_dim=64, value_dim=32, decay_rank=64, gate_rank=32)),
    ((3, 1, 10, 0.9, 2.0, None, (1e3, 2)), dict(n_heads=3, n_kv_heads=1, key_dim=7, value_dim=9))])
def test_the_two_mixers_side_by_side_from_one_input_product(softmax, delta, dtype):
    """Half the sum of the normed outputs; the input projections of both are one product, and each
    branch reads its own columns of it."""
    from edge_infer_amd.config.specs import ParallelSpec
    mixer = ParallelSpec(branches=(keyed_spec(*softmax), delta_spec(**delta)), names=("left", "right"),
                         norm_eps=EPS)
    spec = layers_of(mixer)
    params = params_for(spec, seed=17)
    model, session = session_for(spec, params, dtype)
    part = model.layers[0].mixer
    assert part.proj is not None and len(part.columns) == 2
    for lengths in ([150], [270]):
        x = rows_of(lengths[0], 15)
        want = 0.5 * (plain.rms_norm(plain_keyed(params, PRE + "left.", mixer.branches[0], x.double()),
                                     params[PRE + "left_out.weight"], EPS)
                      + plain.rms_norm(plain_delta(params, PRE + "right.", mixer.branches[1], x.double()),
                                       params[PRE + "right_out.weight"], EPS))
        for cuts in ([len(x)], [60, 2, 3, len(x) - 65], [len(x) - 20] + [1] * 20):
            got, = in_cuts(session, spec, [part], x.to(model.dtype), cuts)
            close(dtype, got, want, f"side by side, cuts {cuts[:3]}", rms=3e-2, top=8e-2)
    session.cache.check()
