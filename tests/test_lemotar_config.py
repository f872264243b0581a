"""The Lemotar configuration: what config.json gives, the spec it becomes, the ranks that only the
checkpoint tells, the checkpoint's names, what is refused and what may be absent (no GPU)."""
import copy

import pytest
import torch

import plain_lemotar as plain
from lemotar_helpers import CONFIGS, ranks, sharp_weights, tensor_shapes


def config_of(raw):
    from edge_infer_amd.config import LemotarConfig
    return LemotarConfig.from_dict(raw)


def sized(raw):
    return config_of(raw).sized_by({name: shape for name, (shape, _) in tensor_shapes(raw).items()})


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_round_trip_and_spec(name):
    from edge_infer_amd.config.specs import (AttentionSpec, GatedDeltaSpec, GatedMLPSpec,
                                             LatentAttentionSpec, ParallelSpec, YarnScaling)
    raw = CONFIGS[name]
    cfg = config_of(raw)
    assert config_of(cfg.to_dict()) == cfg
    spec = sized(raw).model_spec()
    assert spec.embedding_scale == raw["embedding"]["scale"] and not spec.tie_word_embeddings
    norm = spec.final_norm
    assert (norm.kind, norm.eps, norm.weight_offset) == ("rmsnorm", raw["norm"]["eps"], 1.0)
    for index, (layer, made) in enumerate(zip(raw["layers"], spec.layers)):
        assert made.block == "postnorm" and made.stream_scale == raw["postln_alpha"]
        assert made.norm == norm
        mixer, entry = layer["mixer"], spec.schedule[index]
        if layer["type"] == "parallel":
            assert isinstance(made.mixer, ParallelSpec) and made.mixer.names == ("left", "right")
            left, right = made.mixer.branches
            assert isinstance(left, AttentionSpec) and isinstance(right, GatedDeltaSpec)
            assert (left.n_heads, left.n_kv_heads, left.head_dim, left.v_dim, left.scale, left.softcap) \
                == tuple(mixer["left"][k] for k in ("heads", "kv_heads", "dim", "vdim", "scale", "softcap"))
            assert left.values_from_keys and left.unit_sink and left.qk_norm_scope == "projection"
            assert left.window == (mixer["left"].get("mask") or {}).get("size")
            rot = mixer["left"]["rot"]
            assert (left.position.kind, left.position.theta, left.position.dim) == \
                ("rope_pairs", rot["base"], rot["dims"])
            assert (right.n_heads, right.n_kv_heads, right.key_dim, right.value_dim, right.conv_taps) \
                == tuple(mixer["right"][k] for k in ("heads", "kv_heads", "dim", "vdim", "conv"))
            assert (right.decay_rank, right.gate_rank) == ranks(raw, index)
            assert right.gate_activation == "sigmoid" and right.unit_eps == 1e-6
        else:
            latent = made.mixer
            assert isinstance(latent, LatentAttentionSpec) and latent.q_rank == 0 and latent.sink
            assert latent.output_gate == "element"
            assert (latent.n_heads, latent.head_dim, latent.rot_dim, latent.value_dim, latent.kv_rank,
                    latent.scale) == tuple(mixer[k] for k in ("heads", "dim", "rot_dim", "vdim",
                                                              "kv_rank", "scale"))
            assert latent.window == (mixer.get("mask") or {}).get("size")
            scaling = mixer["rot"].get("scaling")
            assert latent.position.kind == "rope_half"
            assert latent.position.scaling == (None if scaling is None else YarnScaling(**scaling))
            assert latent.shared_kv == ("kv_from" in mixer)
            assert (entry.cache, entry.writes_cache) == \
                ((mixer["kv_from"], False) if "kv_from" in mixer else (index, True))
        if layer["mlp"] is None:
            assert made.feed_forward is None
        else:
            assert isinstance(made.feed_forward, GatedMLPSpec) and made.feed_forward.bias is False
            assert made.feed_forward.intermediate_size == layer["mlp"]["ff"]


def test_what_a_shared_cache_keeps():
    """A layer whose latents other layers read keeps what the widest of their windows needs; all
    of it when a reader has no window.  Latents have no value pages."""
    from edge_infer_amd.cache.storage import CacheLayout
    for name, source, window in (("A", 1, 50), ("B", 2, 70), ("C", 1, None), ("D", 0, 130)):
        layout = CacheLayout(sized(CONFIGS[name]).model_spec())
        request, = [request for request, entries in layout.kv_groups if source in entries]
        assert request.window == window and request.value_dim == 0
    layout = CacheLayout(sized(CONFIGS["B"]).model_spec())
    assert {request.window for request, entries in layout.kv_groups if 0 in entries} == {64}


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_checkpoint_names_and_shapes(name):
    from edge_infer_amd.engine.model import expected_parameters
    cfg = sized(CONFIGS[name])
    expected = expected_parameters(cfg.model_spec(), cfg.checkpoint_name)
    shapes = {key: shape for key, (shape, _) in tensor_shapes(CONFIGS[name]).items()}
    needed = {ck: tuple(param.shape) for ck, param in expected.values() if not param.optional}
    assert needed == {key: tuple(shape) for key, shape in shapes.items()}
    with pytest.raises(KeyError):
        cfg.checkpoint_name("layers.0.mixer.nothing.weight")


def test_registry_finds_the_architecture():
    from edge_infer_amd.config import LemotarConfig, resolve_architecture
    assert resolve_architecture({"architecture": "Lemotar"}).config_class is LemotarConfig
    assert resolve_architecture({"model_type": "lemotar"}).config_class is LemotarConfig


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
    (("layers", 0, "type"), "delta", "type must be one of"),
    (("layers", 0, "mixer", "left", "heads"), 5, "multiple of kv_heads"),
    (("layers", 0, "mixer", "left", "vdim"), 24, "values are the keys"),
    (("layers", 0, "mixer", "left", "rot", "dims"), 18, "even and at most 16"),
    (("layers", 0, "mixer", "left", "rot", "scaling"), {}, "does not know"),
    (("layers", 0, "mixer", "right", "kv_heads"), 2, "multiple of kv_heads"),
    (("layers", 0, "mixer", "right", "rank"), 3, "does not know"),
    (("layers", 1, "mixer", "rot", "dims"), 4, "must be rot_dim"),
    (("layers", 1, "mixer", "rot", "scaling", "slow"), KeyError, "lacks 'slow'"),
    (("layers", 1, "mixer", "q_rank"), 8, "does not know"),
    (("layers", 2, "mixer", "kv_from"), 2, "earlier layer"),
    (("layers", 2, "mixer", "kv_from"), 0, "latents of its own"),
    (("layers", 2, "mixer", "kv_rank"), 32, "latents or rotations differ"),
    (("layers", 2, "mixer", "rot", "base"), 6000.0, "latents or rotations differ"),
    (("layers", 0, "mlp", "kind"), "moe", "must be 'dense'"),
    (("postln_alpha",), KeyError, "lacks 'postln_alpha'"),
    (("embedding", "scale"), "big", "must be a number"),
])
def test_refusals(path, value, message):
    from edge_infer_amd.config.lemotar import LemotarConfigError
    with pytest.raises(LemotarConfigError, match=message):
        config_of(changed(path, value))


def test_what_may_be_absent():
    raw = changed(("layers", 0, "mixer", "left", "softcap"), KeyError)
    del raw["layers"][0]["mixer"]["left"]["mask"]
    left = config_of(raw).model_spec().layers[0].mixer.branches[0]
    assert left.softcap is None and left.window is None
    # without a checkpoint the ranks are a head's sizes
    right = config_of(raw).model_spec().layers[0].mixer.branches[1]
    assert (right.decay_rank, right.gate_rank) == (right.key_dim, right.value_dim)


def test_the_plain_implementation_is_causal():
    """Logits at a position are those of the sequence cut behind it, and the stretched frequencies
    keep fast pairs and divide slow ones."""
    cfg = CONFIGS["A"]
    tensors = sharp_weights(cfg, seed=1)
    tokens = [5, 17, 3, 200, 44, 9]
    whole = plain.forward(cfg, tensors, tokens)
    assert torch.allclose(whole[:4], plain.forward(cfg, tensors, tokens[:4]), rtol=1e-9, atol=1e-9)
    freqs, magnitude = plain.stretched_frequencies({"base": 1e4, "dims": 64, "scaling": {
        "factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}})
    plain_ones = plain.plain_frequencies(1e4, 64)
    assert freqs[0] == plain_ones[0] and abs(freqs[-1] * 8.0 - plain_ones[-1]) < 1e-12
    assert abs(magnitude - (1.0 + 0.1 * 2.0794415416798357)) < 1e-12
