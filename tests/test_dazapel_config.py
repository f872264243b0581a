"""The Dazapel configuration: what config.json gives, the spec it becomes, the checkpoint's
names, what is refused and what may be absent, the stretched frequencies, and the pages of kept
first tokens (no GPU).  The oracle's own mechanisms are pinned by closed forms."""
import copy
import math

import pytest
import torch

import plain_dazapel as plain
from dazapel_helpers import CONFIGS, TWINS, sharp_weights, tensor_shapes


def config_of(raw):
    from edge_infer_amd.config import DazapelConfig
    return DazapelConfig.from_dict(raw)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_round_trip_and_spec(name):
    from edge_infer_amd.config.specs import RoutedMLPSpec, YarnScaling
    raw = CONFIGS[name]
    cfg = config_of(raw)
    assert config_of(cfg.to_dict()) == cfg
    spec = cfg.model_spec()
    assert spec.tie_word_embeddings and spec.final_norm.kind == "rmsnorm"
    assert spec.final_norm.eps == raw["norm"]["eps"]
    runs = plain.layer_runs(raw)
    assert [entry.layer for entry in spec.schedule] == [layer for layer, _ in runs]
    assert len({entry.cache for entry in spec.schedule}) == len(runs)     # a cache a run
    if raw["loop"] is None:
        assert spec.loop is None
    else:
        assert not spec.loop.remix and spec.loop.times == raw["loop"]["times"]
    for layer, made in zip(raw["layers"], spec.layers):
        assert made.block == "sandwich" and made.residual_scale == raw["residual_mult"]
        mixer, got = layer["mixer"], made.mixer
        assert (got.n_heads, got.n_kv_heads, got.head_dim, got.v_dim, got.scale) == \
            tuple(mixer[k] for k in ("heads", "kv_heads", "dim", "vdim", "scale"))
        assert got.qk_unit_norm and got.qk_norm_eps == raw["norm"]["eps"] and not got.qk_norm
        assert got.qkv_bias is True and got.o_bias is True and got.output_gate is True
        mask = mixer.get("mask") or {}
        assert got.window == mask.get("size") and got.keep_first == mask.get("keep_first", 0)
        rot = mixer.get("rot")
        if rot is None:
            assert got.position.kind == "none"
        else:
            assert (got.position.kind, got.position.theta, got.position.dim) == \
                ("rope_half", rot["base"], rot["dims"])
            scaling = rot.get("scaling")
            assert got.position.scaling == (None if scaling is None else YarnScaling(**scaling))
        mlp, ffn = layer["mlp"], made.feed_forward
        if mlp is None:
            assert ffn is None
            continue
        router = mlp["router"]
        groups = router.get("groups") or {"count": 1, "keep": 1}
        assert isinstance(ffn, RoutedMLPSpec) and ffn.scoring == "sigmoid"
        assert (ffn.n_experts, ffn.top, ffn.weight_scale, ffn.group_count, ffn.group_keep) == \
            (router["experts"], router["top"], router["scale"], groups["count"], groups["keep"])
        assert (ffn.activation, ffn.limit, ffn.alpha) == ("clamped_swish", mlp["expert"]["limit"], 1.702)
        assert (ffn.shared is None) == ("shared" not in mlp)
        if ffn.shared is not None:
            assert (ffn.shared.intermediate_size, ffn.shared.limit, ffn.shared.alpha, ffn.shared.bias) == \
                (mlp["shared"]["ff"], mlp["shared"]["limit"], 1.702, False)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_checkpoint_names_and_shapes(name):
    from edge_infer_amd.engine.model import expected_parameters
    from edge_infer_amd.weights import match_parameters
    cfg = config_of(CONFIGS[name])
    expected = expected_parameters(cfg.model_spec(), cfg.checkpoint_name)
    shapes = {key: tuple(shape) for key, (shape, _) in tensor_shapes(CONFIGS[name]).items()}
    needed = {ck: tuple(param.shape) for path, (ck, param) in expected.items()
              if not param.optional and path != "head.weight"}
    assert needed == shapes
    params = match_parameters(expected, sharp_weights(CONFIGS[name], 1),
                              optional={"head.weight": "embed.weight"})
    assert params["head.weight"] is params["embed.weight"]
    assert "loop.in.weight" not in params


def test_norms_of_a_layer_without_a_feed_forward_may_be_stored():
    from edge_infer_amd.engine.model import expected_parameters
    from edge_infer_amd.weights import match_parameters
    cfg = config_of(CONFIGS["A"])
    tensors = sharp_weights(CONFIGS["A"], 1)
    tensors["l1.norm2"] = tensors["l1.norm2b"] = torch.ones(64, dtype=torch.bfloat16)
    match_parameters(expected_parameters(cfg.model_spec(), cfg.checkpoint_name), tensors,
                     optional={"head.weight": "embed.weight"})


def test_registry_finds_the_architecture():
    from edge_infer_amd.config import DazapelConfig, resolve_architecture
    assert resolve_architecture({"architecture": "Dazapel"}).config_class is DazapelConfig
    assert resolve_architecture({"model_type": "dazapel"}).config_class is DazapelConfig


def changed(path, value):
    raw = copy.deepcopy(CONFIGS["A"])
    at = raw
    for key in path[:-1]:
        at = at[key]
    if value is KeyError:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return raw


@pytest.mark.parametrize("path, value, message", [
    (("layers", 0, "type"), "mamba2", "type must be one of"),
    (("layers", 0, "mixer", "heads"), 5, "multiple of kv_heads"),
    (("layers", 0, "mixer", "sink"), True, "does not know"),
    (("layers", 0, "mixer", "rot", "dims"), 7, "even and at most dim"),
    (("layers", 0, "mixer", "rot", "dims"), 18, "even and at most dim"),
    (("layers", 0, "mixer", "rot", "scaling", "low"), 1.0, "does not know"),
    (("layers", 0, "mixer", "rot", "scaling", "fast"), KeyError, "lacks 'fast'"),
    (("layers", 0, "mixer", "rot", "base"), 1.0, "no wavelengths"),
    (("layers", 0, "mixer", "mask", "keep_first"), -1, "at least 0"),
    (("layers", 0, "mixer", "mask", "pool"), 4, "does not know"),
    (("layers", 0, "mlp", "kind"), "dense", "must be 'moe'"),
    (("layers", 0, "mlp", "router", "top"), 5, "above the experts of the kept groups"),
    (("layers", 0, "mlp", "router", "groups", "count"), 4, "do not fit 6 experts"),
    (("layers", 0, "mlp", "router", "groups", "keep"), 4, "do not fit 6 experts"),
    (("layers", 0, "mlp", "router", "scale"), KeyError, "lacks 'scale'"),
    (("layers", 0, "mlp", "expert", "limit"), 0.0, "above 0"),
    (("layers", 0, "mlp", "shared", "bias"), True, "does not know"),
    (("loop", "stop"), 5, "loop.start < loop.stop <= 4"),
    (("residual_mult",), KeyError, "lacks 'residual_mult'"),
])
def test_refusals(path, value, message):
    from edge_infer_amd.config.dazapel import DazapelConfigError
    with pytest.raises(DazapelConfigError, match=message):
        config_of(changed(path, value))


def test_what_may_be_absent():
    raw = changed(("layers", 0, "mixer", "mask"), {"size": 9})
    assert config_of(raw).model_spec().layers[0].mixer.keep_first == 0
    raw = changed(("layers", 0, "mixer", "mask"), None)
    assert config_of(raw).model_spec().layers[0].mixer.window is None
    raw = changed(("layers", 0, "mixer", "rot"), KeyError)
    assert config_of(raw).model_spec().layers[0].mixer.position.kind == "none"
    raw = changed(("layers", 0, "mlp", "router", "groups"), None)
    assert config_of(raw).model_spec().layers[0].feed_forward.group_count == 1
    raw = changed(("layers", 0, "mlp", "shared"), KeyError)
    assert config_of(raw).model_spec().layers[0].feed_forward.shared is None
    raw = changed(("loop",), KeyError)
    assert config_of(raw).model_spec().loop is None


def test_spec_options_that_do_not_go_together():
    """The attention part refuses kept first tokens with chunks or pooled blocks, the routed part
    groups under another scoring."""
    import dataclasses
    from edge_infer_amd.config.specs import AttentionSpec, PositionSpec, RoutedMLPSpec
    from edge_infer_amd.parts import Attention, RoutedMLP
    good = AttentionSpec(n_heads=2, n_kv_heads=1, head_dim=8, window=5, keep_first=2,
                         qk_unit_norm=True, position=PositionSpec(kind="none"))
    Attention.check(good)
    for change in (dict(chunk=4), dict(pool=2), dict(keep_first=-1)):
        with pytest.raises(ValueError):
            Attention.check(dataclasses.replace(good, **change))
    routed = RoutedMLPSpec(n_experts=6, top=2, intermediate_size=8, scoring="sigmoid",
                           group_count=3, group_keep=1)
    RoutedMLP.check(routed)
    for change in (dict(scoring="softmax_all"), dict(group_count=4), dict(top=3), dict(group_keep=4),
                   dict(activation="relu")):
        with pytest.raises(ValueError):
            RoutedMLP.check(dataclasses.replace(routed, **change))


@pytest.mark.parametrize("base, dims, scaling", [
    (10000.0, 64, (6.0, 384, 24.0, 1.5)), (300000.0, 128, (4.0, 4096, 16.0, 2.0)),
    (100.0, 6, (2.0, 20, 3.0, 1.0)), (500.0, 16, (16.0, 7, 32.0, 1.0)),
    (10.0, 8, (2.0, 100000, 2.0, 1.0))])
def test_stretched_frequencies(base, dims, scaling):
    """Against the oracle's own, pair by pair; the first and last pairs are as said where the
    ramp does not reach them."""
    from edge_infer_amd.config.specs import PositionSpec, YarnScaling
    from edge_infer_amd.parts.rope import rotation_magnitude, scaled_frequencies
    factor, original, fast, slow = scaling
    spec = PositionSpec(kind="rope_half", theta=base, dim=dims,
                        scaling=YarnScaling(factor, original, fast, slow))
    rot = {"base": base, "dims": dims,
           "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow}}
    got, want = scaled_frequencies(spec), torch.tensor(plain.frequencies(rot), dtype=torch.float64)
    assert torch.allclose(got, want, rtol=1e-13, atol=0.0)
    assert rotation_magnitude(spec) == pytest.approx(0.1 * math.log(factor) + 1.0, rel=1e-15)
    assert rotation_magnitude(PositionSpec(kind="rope_half", theta=base, dim=dims)) == 1.0
    unscaled = torch.tensor(plain.frequencies({"base": base, "dims": dims}), dtype=torch.float64)
    assert bool(((got <= unscaled * (1 + 1e-12)) & (got >= unscaled / factor * (1 - 1e-12))).all())


def test_yarn_ramp_in_closed_form():
    """base e, 14 dims and an original length of 2 pi e^1.5: pairs 0 to 4 keep their frequency,
    5 and 6 lie on the ramp."""
    rot = {"base": math.e, "dims": 14,
           "scaling": {"factor": 4.0, "original": 2 * math.pi * math.exp(1.5),
                       "fast": math.exp(0.9), "slow": math.exp(0.6)}}
    # index = 14 ln(original / (2 pi t)) / 2 = 7 (1.5 - ln t): fast 4.2 -> 4, slow 6.3 -> 7
    got = plain.frequencies(rot)
    for i in range(7):
        f = math.exp(-2.0 * i / 14)
        ramp = min(max((i - 4) / 3.0, 0.0), 1.0)
        assert got[i] == pytest.approx(f / 4.0 * ramp + f * (1 - ramp), rel=1e-12)


def test_the_oracles_mechanisms_in_closed_form():
    mask = {"size": 3, "keep_first": 2}
    assert plain.visible_keys(6, mask) == [0, 1, 4, 5, 6]
    assert plain.visible_keys(2, mask) == [0, 1, 2]
    assert plain.visible_keys(3, {"size": 1, "keep_first": 0}) == [3]
    assert plain.visible_keys(3, None) == [0, 1, 2, 3]
    # unit RMS after a rotation of part of the head: the magnitude changes the ratio of the parts
    rot = {"base": 10.0, "dims": 2, "scaling": {"factor": math.e, "original": 10.0, "fast": 2.0, "slow": 1.0}}
    x = torch.tensor([[[3.0, 4.0, 2.0]]], dtype=torch.float64)
    turned = plain.rotate_halves(x, torch.tensor([0]), rot)
    assert torch.allclose(turned, torch.tensor([[[3.3, 4.4, 2.0]]], dtype=torch.float64))
    assert plain.unit_rms(turned, 0.0).pow(2).mean().item() == pytest.approx(1.0)
    # a group is scored by its two largest: the best single expert's group may be left out
    scores = torch.tensor([0.9, 0.1, 0.0, 0.6, 0.55, 0.2, 0.5, 0.45, 0.44], dtype=torch.float64)
    router = {"top": 2, "groups": {"count": 3, "keep": 1}}
    assert plain.choose(scores, router) == [3, 4]
    assert plain.choose(scores, {"top": 3, "groups": {"count": 3, "keep": 2}}) == [0, 3, 4]
    assert plain.choose(scores, {"top": 3}) == [0, 3, 4]
    assert plain.choose(torch.full((4,), 0.5), {"top": 2, "groups": {"count": 2, "keep": 1}}) == [0, 1]
    assert plain.layer_runs({"loop": {"start": 1, "stop": 3, "times": 2}, "layers": [0] * 4}) == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]


def test_cache_requests_and_kept_pages():
    from edge_infer_amd.cache.allocator import PagePool, SequencePages
    from edge_infer_amd.cache.storage import CacheLayout
    from edge_infer_amd.parts.base import KVRequest
    layout = CacheLayout(config_of(CONFIGS["B"]).model_spec())
    requests = [request for request, _ in layout.kv_groups]
    assert KVRequest(n_kv_heads=2, head_dim=64, window=64, keep_first=5) in requests
    assert KVRequest(n_kv_heads=1, head_dim=64, window=65, keep_first=70) in requests
    pool = PagePool(16)
    pages = SequencePages(pool, 1, window=65, keep_first=70)
    pages.open(0)
    pages.grow(0, 500)
    pages.trim(0, 500)
    # the next query (500) sees 436 .. 500 and 0 .. 69: pages 0, 1 and 6, 7
    assert [p >= 0 for p in pages.row(0)] == [True, True, False, False, False, False, True, True]
    assert pool.n_free == 12
    pages.grow(0, 700)
    pages.trim(0, 700)
    assert [i for i, p in enumerate(pages.row(0)) if p >= 0] == [0, 1, 9, 10]
    pages.close(0)
    pool.check()
    assert pool.n_free == 16
    # a page that is given back may go to another sequence while the first one's kept page stays
    one = SequencePages(PagePool(4), 2, window=1, keep_first=1)
    one.open(0), one.open(1)
    one.grow(0, 200)
    one.trim(0, 200)
    assert [p >= 0 for p in one.row(0)] == [True, False, False, True]
    one.grow(1, 128)
    assert not set(p for p in one.row(0) if p >= 0) & set(one.row(1))
    one.close(0), one.close(1)
    one.pool.check()


def test_twins_leave_no_choice():
    for cfg in TWINS.values():
        for layer in cfg["layers"]:
            if layer["mlp"] is not None:
                assert layer["mlp"]["router"]["experts"] == layer["mlp"]["router"]["top"]
        config_of(cfg)
