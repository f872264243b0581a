"""Small Dazapel configurations and weights for the tests.

The configurations differ from each other in every size and option: key and value head sizes
that differ or are equal (64 and 64, 128 and 128 take the matrix-core attention kernels in
bfloat16), group ratios 1 to 8, windows below, at and just above the cache's page of 64 tokens
and none, kept first tokens from none to more than a page, rotations of a part of the head, of
the whole head and none, with and without stretched frequencies, loops over some layers, over
all of them and none, run once to three times, layers without a feed-forward, 3 to 65 experts
in groups of one to many of which some or all take part, with and without a shared expert,
limits that many activations pass.  Queries and keys come at unit RMS, so a mixer's `scale` of
about 2.5 / sqrt(dim) spreads the scores by 2.5 and single keys stand out.  The weights are drawn
so that signals are of order one (N(0, 0.02) matrices would hide a wrong key or expert), and are
rounded to bfloat16, so that both precisions and the oracle see the same numbers.
"""
import json
from pathlib import Path

import torch


def moe(ff, limit, experts, top, scale=1.0, groups=None, shared=None):
    """groups: None or (count, keep); shared: None or (ff, limit)."""
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
           "router": {"experts": experts, "top": top, "scale": scale}}
    if groups is not None:
        out["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared is not None:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def attention(heads, kv_heads, dim, vdim, scale, mask, rot, mlp):
    """mask: None or (size, keep_first); rot: None or (base, dims, scaling), scaling None or
    (factor, original, fast, slow)."""
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if mask is not None:
        mixer["mask"] = {"size": mask[0], "keep_first": mask[1]}
    if rot is not None:
        mixer["rot"] = {"base": rot[0], "dims": rot[1]}
        if rot[2] is not None:
            mixer["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), rot[2]))
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def model(vocab, width, eps, mult, loop, layers):
    """loop: None or (start, stop, times)."""
    return {"architecture": "Dazapel", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "residual_mult": mult,
            "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop)),
            "layers": layers}


CONFIG_A = model(211, 64, 1e-5, 0.8, (1, 3, 2), [
    attention(6, 2, 16, 24, 0.6, (20, 3), (10000.0, 8, (4.0, 40, 8.0, 1.0)),
              moe(40, 1.5, 6, 2, 1.7, (3, 2), (56, 0.9))),
    attention(4, 4, 16, 8, 0.7, (33, 1), (500.0, 16, None), None),
    attention(5, 1, 24, 16, 0.5, (7, 10), None, moe(24, 0.7, 5, 3, 0.6, None, (16, 2.0))),
    attention(4, 2, 8, 8, 0.9, None, (10000.0, 4, (32.0, 100, 16.0, 2.0)), moe(32, 3.0, 8, 2, 2.5, (2, 1)))])
# head sizes 64 and 128 with values as wide: the matrix-core kernels in bfloat16; windows of a
# page and of a token more, kept tokens within a page, of one page exactly and of more; the
# grouped products of the experts; no loop
CONFIG_B = model(97, 128, 1e-6, 1.0, None, [
    attention(4, 2, 64, 64, 0.3, (64, 5), (300000.0, 64, (7.0, 80, 20.0, 1.0)),
              moe(64, 1.2, 8, 2, 1.0, (4, 2), (128, 1.0))),
    attention(8, 1, 64, 64, 0.3, (65, 70), (10000.0, 32, None), moe(128, 2.0, 4, 2, 2.0, (2, 2), (64, 2.5))),
    attention(3, 3, 128, 128, 0.2, (10, 64), (10000.0, 128, (2.0, 30, 4.0, 0.5)), None)])
# every layer in a loop of three passes, groups of a single expert, more experts than a wave has
# lanes, a window of one token
CONFIG_C = model(150, 96, 1e-5, 0.5, (0, 3, 3), [
    attention(2, 1, 48, 40, 0.35, (1, 4), (100.0, 48, (1.5, 20, 2.0, 0.25)), moe(16, 1.0, 65, 4, 3.0, (13, 4), (24, 1.1))),
    attention(8, 8, 24, 24, 0.5, (100, 2), (100.0, 22, (16.0, 300, 30.0, 3.0)), None),
    attention(6, 3, 40, 8, 0.4, (40, 0), (5000.0, 6, None), moe(56, 0.5, 5, 2, 1.0, (5, 3)))])
# sizes that are multiples of nothing: no vector kernel and no few-rows product applies; a loop
# over one layer, passed once
CONFIG_D = model(101, 50, 1e-6, 1.3, (1, 2, 1), [
    attention(6, 2, 10, 7, 0.8, (7, 2), (3000.0, 6, (3.0, 25, 6.0, 1.5)), moe(13, 0.8, 3, 1, 1.4, None, (11, 1.3))),
    attention(5, 5, 6, 9, 0.9, (130, 3), (3000.0, 6, None), moe(7, 1.0, 9, 3, 0.5, (3, 2)))])
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C, "D": CONFIG_D}


def routeless_twin(cfg):
    """`cfg` with every router left no choice: as many experts as a token takes, one group.  A
    router chooses by the order of its scores, which any rounding may change where two of them
    nearly tie, and one token routed otherwise changes the rows after it as well; comparisons in
    bfloat16 over whole requests therefore run on models whose tokens take every expert."""
    twin = json.loads(json.dumps(cfg))
    for layer in twin["layers"]:
        if layer["mlp"] is not None:
            router = layer["mlp"]["router"]
            router["experts"] = router["top"]
            router.pop("groups", None)
    return twin


TWINS = {name: routeless_twin(cfg) for name, cfg in CONFIGS.items()}


def tensor_shapes(cfg):
    """name -> (shape, law) of every tensor of a model of `cfg`."""
    w = cfg["width"]
    out = {"embed": ((cfg["vocab"], w), "table"), "final.norm": ((w,), "norm")}
    if cfg.get("loop"):
        out["loop.step"] = ((cfg["loop"]["times"], w), "step")
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        out[p + "norm1"] = out[p + "norm1b"] = ((w,), "norm")
        for name, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]),
                           ("v", m["kv_heads"] * m["vdim"])):
            out[p + "mix." + name] = ((rows, w), "matrix")
            out[p + "mix." + name + ".b"] = ((rows,), "bias")
        out[p + "mix.g"] = ((m["heads"] * m["vdim"], w), "matrix")
        out[p + "mix.o"] = ((w, m["heads"] * m["vdim"]), "matrix")
        out[p + "mix.o.b"] = ((w,), "bias")
        mlp = layer["mlp"]
        if mlp is None:
            continue
        out[p + "norm2"] = out[p + "norm2b"] = ((w,), "norm")
        out[p + "mlp.router"] = ((mlp["router"]["experts"], w), "router")
        experts = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
        if mlp.get("shared"):
            experts.append(("shared.", mlp["shared"]["ff"]))
        for name, ff in experts:
            out[p + "mlp." + name + "gate"] = ((ff, w), "matrix")
            out[p + "mlp." + name + "up"] = ((ff, w), "matrix")
            out[p + "mlp." + name + "down"] = ((w, ff), "matrix")
    return out


def sharp_weights(cfg, seed):
    """Tensors of order-one signal, bfloat16."""
    g = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, (shape, law) in tensor_shapes(cfg).items():
        if law == "matrix":
            value = torch.randn(shape, generator=g) / shape[1] ** 0.5
        elif law == "router":     # scores that spread over most of (0, 1)
            value = torch.randn(shape, generator=g) * 1.5 / shape[1] ** 0.5
        elif law == "table":
            value = torch.randn(shape, generator=g)
        elif law == "norm":
            value = 1.0 + (torch.rand(shape, generator=g) * 0.4 - 0.2)
        elif law == "bias":
            value = torch.randn(shape, generator=g) * 0.3
        elif law == "step":
            value = torch.randn(shape, generator=g) * 0.5
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
