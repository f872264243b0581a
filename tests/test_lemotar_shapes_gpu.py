"""Lemotar models of drawn sizes against the plain implementation: every size, option and the
order of the layers come from a seeded generator, so that nothing rests on the sizes of the
hand-made configurations.  Per model, in float32 and bfloat16: a whole prompt, the prompt cut into
portions, and a batch of unequal requests decoded together."""
import random

import pytest
import torch

import plain_lemotar as plain
from helpers import assert_close_bf16, assert_close_f32
from lemotar_helpers import ids, latent, model, parallel, sharp_weights, write_folder

pytestmark = pytest.mark.gpu
SEEDS = list(range(40))


def drawn_parallel(rng, ff):
    kv_heads = rng.choice([1, 2, 3, 4])
    heads = kv_heads * rng.choice([1, 2, 3, 4, 5])
    dim = rng.choice([8, 10, 16, 24, 32, 48, 64, 64, 128])
    rot = (rng.choice([100.0, 10000.0, 300000.0]),
           rng.choice([d for d in (2, 4, 8, 16, 32, dim) if d <= dim]))
    left = (heads, kv_heads, dim, rng.choice([1.5, 2.5]) / dim ** 0.5, rng.choice([1.5, 5.0, 20.0, 60.0]),
            rng.choice([1, 2, 17, 63, 64, 65, 100, None]), rot)
    shared = rng.choice([1, 2, 3, 5])
    right = (shared * rng.choice([1, 2, 3]), shared, rng.choice([4, 8, 10, 16, 32, 64, 96, 128]),
             rng.choice([4, 7, 8, 16, 32, 64, 128]), rng.choice([1, 2, 3, 4, 5, 8]))
    return parallel(left, right, ff)


def drawn_latent(rng, ff, kv_from=None, like=None):
    heads, dim, vdim = rng.choice([1, 2, 3, 4, 5, 8, 16, 20]), rng.choice([4, 8, 10, 16, 32, 64]), \
        rng.choice([4, 5, 8, 16, 32, 64])
    if like is None:
        fast = rng.choice([2.0, 8.0, 30.0])
        scaling = None if rng.random() < 0.3 else (
            rng.choice([1.0, 2.0, 8.0, 40.0]), rng.choice([16, 64, 400, 4096]), fast,
            fast / rng.choice([2.0, 8.0, 32.0]))
        rot = (rng.choice([100.0, 10000.0, 300000.0]), rng.choice([2, 4, 8, 16, 32, 64]), scaling)
        rank = rng.choice([6, 12, 16, 32, 48, 64, 96, 128])
    else:
        rot, rank = like
    made = latent(heads, dim, rot, vdim, rank, rng.choice([1.0, 1.7]) / (dim + rot[1]) ** 0.5,
                  rng.choice([1, 2, 17, 63, 64, 65, 100, None]), ff, kv_from=kv_from)
    return made, (rot, rank)


def drawn_config(seed):
    rng = random.Random(9000 + seed)
    width = rng.choice([32, 40, 50, 64, 72, 96, 128, 256])
    layers, own = [], []
    for index in range(rng.randint(1, 6)):
        ff = None if rng.random() < 0.2 else rng.choice([8, 24, 50, 64, 96, 128, 200])
        if rng.random() < 0.45:
            layers.append(drawn_parallel(rng, ff))
        elif own and rng.random() < 0.6:
            source, like = rng.choice(own)
            layers.append(drawn_latent(rng, ff, source, like)[0])
        else:
            made, like = drawn_latent(rng, ff)
            own.append((index, like))
            layers.append(made)
    return model(rng.randint(20, 300), width, rng.choice([1e-5, 1e-6]), rng.choice([0.5, 1.0, 4.0]),
                 rng.choice([0.7, 1.0, 1.8, 3.0]), layers)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", SEEDS)
def test_drawn_model(seed, dtype, tmp_path):
    import edge_infer_amd as ei
    cfg = drawn_config(seed)
    tensors = sharp_weights(cfg, seed=seed)
    requests = [ids(cfg["vocab"], n, 50 + n) for n in (150, 1, 37)]
    refs = [plain.forward(cfg, tensors, r) for r in requests]
    session = ei.Session(ei.load_model(write_folder(tmp_path / "m", cfg, tensors), dtype=dtype),
                         max_tokens=64 * 8, max_seqs=3)

    def close(got, want, what):
        if dtype == "float32":
            return assert_close_f32(got, want, what)
        # (bfloat16's roundings add up like a random walk over the layers)
        deeper = max(1.0, len(cfg["layers"]) / 4.0) ** 0.5
        assert_close_bf16(got, want, what, rms_rel=4e-2 * deeper, max_rel=12e-2 * deeper)
    # whole, and in portions
    slot = session.begin()
    close(session.step([(slot, requests[0], list(range(150)))]), refs[0], "whole")
    session.end(slot)
    slot = session.begin()
    rows, at = [], 0
    for take in (2, 3, 60, 1, 70, 14):
        rows.append(session.step([(slot, requests[0][at:at + take], list(range(take)))]))
        at += take
    close(torch.cat(rows), refs[0], "portions")
    session.end(slot)
    # a batch of unequal requests that start together and are decoded together
    slots = [session.begin() for _ in requests]
    cuts = [max(1, len(r) - 12) for r in requests]
    got = [[] for _ in requests]
    logits = session.step([(slots[i], requests[i][:cuts[i]], [cuts[i] - 1]) for i in range(3)])
    for i in range(3):
        got[i].append(logits[i:i + 1])
    at = list(cuts)
    live = [i for i in range(3) if at[i] < len(requests[i])]
    while live:
        logits = session.step([(slots[i], [requests[i][at[i]]], [0]) for i in live])
        for row, i in enumerate(live):
            got[i].append(logits[row:row + 1])
            at[i] += 1
        live = [i for i in live if at[i] < len(requests[i])]
    for i in range(3):
        close(torch.cat(got[i]), refs[i][cuts[i] - 1:], f"request {i} of the batch")
    session.cache.check()
