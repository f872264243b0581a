"""Small Lemotar configurations and weights for the tests.

The configurations differ from each other in every size and option: head sizes 64 and 128 (the
matrix-core attention kernels in bfloat16) and others, group ratios 1 to 8, windows of one token,
below, at and just above the cache's page of 64 tokens and none, rotations of a part of the head,
of the whole head and none, stretched frequencies or plain ones, caps that bite and caps that
hardly do, latents whose cached rows the matrix-core kernel takes and others, layers that read an
earlier layer's latents with a window of their own or none, delta-rule key heads of 6 to 256
elements shared by one to three value heads, 1 to 9 taps, decay and gate of different ranks,
layers without a feed-forward.  The weights are drawn so that signals are of order one; they are
rounded to bfloat16, so that both precisions and the oracle see the same numbers.
"""
import json
from pathlib import Path

import torch


def rotation(rot):
    """rot: (base, dims) or (base, dims, (factor, original, fast, slow))."""
    out = {"base": rot[0], "dims": rot[1]}
    if len(rot) > 2 and rot[2] is not None:
        out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), rot[2]))
    return out


def mlp(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def parallel(left, right, ff):
    """left: (heads, kv_heads, dim, scale, softcap, window or None, rot); right: (heads, kv_heads,
    dim, vdim, taps)."""
    heads, kv_heads, dim, scale, softcap, window, rot = left
    softmax = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale,
               "softcap": softcap, "rot": rotation(rot)}
    if window is not None:
        softmax["mask"] = {"size": window}
    delta = dict(zip(("heads", "kv_heads", "dim", "vdim", "conv"), right))
    return {"type": "parallel", "mixer": {"left": softmax, "right": delta}, "mlp": mlp(ff)}


def latent(heads, dim, rot, vdim, kv_rank, scale, window, ff, kv_from=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot[1], "vdim": vdim, "kv_rank": kv_rank,
             "scale": scale, "rot": rotation(rot)}
    if window is not None:
        mixer["mask"] = {"size": window}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp(ff)}


def model(vocab, width, eps, embedding_scale, alpha, layers):
    return {"architecture": "Lemotar", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": embedding_scale}, "postln_alpha": alpha, "layers": layers}


YARN = (4.0, 60, 8.0, 1.0)
CONFIG_A = model(211, 64, 1e-5, 2.0, 1.6, [
    parallel((6, 3, 16, 0.7, 4.0, 20, (10000.0, 8)), (3, 1, 12, 24, 3), 96),
    latent(5, 12, (5000.0, 8, YARN), 9, 40, 0.6, 17, 72),
    latent(5, 20, (5000.0, 8, YARN), 14, 40, 0.5, 50, None, kv_from=1),
    parallel((4, 1, 24, 0.6, 30.0, None, (500.0, 24)), (4, 2, 32, 20, 4), 80)])
# head sizes 64 and 128 and cached rows of 96 and 160 elements: the matrix-core kernels in bfloat16
CONFIG_B = model(97, 128, 1e-6, 1.0, 2.2, [
    latent(8, 32, (10000.0, 32, (8.0, 100, 16.0, 2.0)), 32, 64, 0.35, 64, 160),
    parallel((8, 2, 64, 0.35, 6.0, 65, (10000.0, 32)), (4, 4, 64, 64, 4), None),
    latent(4, 48, (300.0, 32, None), 64, 128, 0.3, 10, 128),
    latent(16, 16, (300.0, 32, None), 16, 128, 0.35, 70, 96, kv_from=2),
    parallel((4, 4, 128, 0.25, 15.0, 64, (200.0, 128)), (6, 2, 32, 48, 2), 128)])
# key heads of 160 and 256 elements (32 lanes a column), one tap and more than eight, windows of one
# and two tokens, a reader without a window
CONFIG_C = model(150, 96, 1e-6, 0.5, 0.8, [
    parallel((5, 1, 40, 0.5, 2.0, 1, (100.0, 2)), (2, 2, 160, 24, 1), None),
    latent(3, 24, (100.0, 16, YARN), 40, 48, 0.5, 2, 56),
    latent(6, 8, (100.0, 16, YARN), 8, 48, 0.6, None, 40, kv_from=1),
    parallel((8, 1, 64, 0.4, 50.0, 100, (1000.0, 16)), (3, 1, 256, 10, 9), 104)])
# sizes that are multiples of nothing: no vector kernel and no few-rows product applies
CONFIG_D = model(101, 50, 1e-5, 5.0, 3.1, [
    latent(3, 7, (3000.0, 6, YARN), 5, 13, 0.9, 7, 30),
    parallel((6, 2, 10, 0.9, 3.0, 33, (3000.0, 6)), (3, 3, 6, 7, 2), 30),
    latent(2, 9, (3000.0, 6, YARN), 3, 13, 0.8, 130, None, kv_from=0)])
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C, "D": CONFIG_D}


def ranks(cfg, index):
    """(rank of the decay, rank of the gate) of a parallel layer: no keys of the configuration."""
    right = cfg["layers"][index]["mixer"]["right"]
    return 3 + right["dim"] // 4 + index, 2 + right["vdim"] // 3


def tensor_shapes(cfg):
    """name -> (shape, law) of every tensor of a model of `cfg`."""
    w = cfg["width"]
    out = {"embed": ((cfg["vocab"], w), "table"), "final.norm": ((w,), "offset"),
           "head": ((cfg["vocab"], w), "matrix")}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        out[p + "norm1"] = ((w,), "offset")
        if layer["type"] == "parallel":
            left, right = m["left"], m["right"]
            q, k = left["heads"] * left["dim"], left["kv_heads"] * left["dim"]
            s = p + "mix.left."
            out[s + "q"], out[s + "k"] = ((q, w), "matrix"), ((k, w), "matrix")
            out[s + "q.norm"], out[s + "k.norm"] = ((q,), "norm"), ((k,), "norm")
            out[s + "o"] = ((w, q), "matrix")
            out[s + "out"] = ((w,), "norm")
            s = p + "mix.right."
            qk, v = right["kv_heads"] * right["dim"], right["heads"] * right["vdim"]
            decays = right["heads"] * right["dim"]
            decay_rank, gate_rank = ranks(cfg, i)
            for name, size in (("q", qk), ("k", qk), ("v", v)):
                out[s + name] = ((size, w), "matrix")
                out[s + name + ".conv"] = ((size, right["conv"]), "filter")
            out[s + "b"] = ((right["heads"], w), "matrix")
            out[s + "A_log"] = ((right["heads"],), "rate")
            out[s + "dt_bias"] = ((decays,), "shift")
            out[s + "a1"], out[s + "a2"] = ((decay_rank, w), "matrix"), ((decays, decay_rank), "matrix")
            out[s + "g1"], out[s + "g2"] = ((gate_rank, w), "matrix"), ((v, gate_rank), "matrix")
            out[s + "norm"] = ((right["vdim"],), "norm")
            out[s + "o"] = ((w, v), "matrix")
            out[s + "out"] = ((w,), "norm")
        else:
            s = p + "mix."
            H, e = m["heads"], m["vdim"]
            out[s + "q"] = ((H * (m["dim"] + m["rot_dim"]), w), "matrix")
            if m.get("kv_from") is None:
                out[s + "dkv"] = ((m["kv_rank"] + m["rot_dim"], w), "matrix")
                out[s + "dkv.norm"] = ((m["kv_rank"],), "norm")
            out[s + "uk"] = ((H * m["dim"], m["kv_rank"]), "matrix")
            out[s + "uv"] = ((H * e, m["kv_rank"]), "matrix")
            out[s + "sink"] = ((H,), "sink")
            out[s + "g"] = ((H * e, w), "matrix")
            out[s + "o"] = ((w, H * e), "matrix")
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out[p + "norm2"] = ((w,), "offset")
            for name, shape in (("gate", (ff, w)), ("up", (ff, w)), ("down", (w, ff))):
                out[p + "mlp." + name] = (shape, "matrix")
    return out


def sharp_weights(cfg, seed):
    """Tensors of order-one signal, bfloat16: single keys stand out of the softmax, heads of the
    delta rule forget within a few tokens or hardly at all, and a key's channels unequally."""
    g = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, (shape, law) in tensor_shapes(cfg).items():
        if law == "matrix":
            value = torch.randn(shape, generator=g) / shape[1] ** 0.5
        elif law == "table":
            value = torch.randn(shape, generator=g)
        elif law == "norm":
            value = 1.0 + (torch.rand(shape, generator=g) * 0.6 - 0.3)
        elif law == "offset":
            value = torch.rand(shape, generator=g) * 0.6 - 0.3
        elif law == "filter":
            value = torch.randn(shape, generator=g) * 0.8
        elif law == "rate":
            value = torch.rand(shape, generator=g) * 7.0 - 6.5
        elif law == "shift":
            value = torch.rand(shape, generator=g) * 4.0 - 3.0
        elif law == "sink":
            value = torch.randn(shape, generator=g) * 2.0
        tensors[name] = value.to(torch.bfloat16)
    return tensors


def write_folder(path, cfg, tensors):
    from safetensors.torch import save_file
    path = Path(path)
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg, indent=1))
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(path / "model.safetensors"))
    return path


def ids(vocab, count, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (count,), generator=g).tolist()
