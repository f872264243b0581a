"""Dazapel models of drawn sizes against the plain implementation: every size, option and the
order of the layers come from a seeded generator, so that nothing rests on the sizes of the
hand-made configurations.  Per model: whole prompts, a prompt cut into portions, a batch of
unequal requests decoded together, in float32; and the twin whose routers have no choice in
bfloat16."""
import random

import pytest
import torch

import plain_dazapel as plain
from helpers import assert_close_bf16, assert_close_f32
from dazapel_helpers import attention, ids, model, moe, routeless_twin, sharp_weights, write_folder

pytestmark = pytest.mark.gpu
SEEDS = list(range(40))


def drawn_config(seed):
    rng = random.Random(7000 + seed)
    width = rng.choice([32, 40, 64, 72, 96, 128, 256])
    layers = []
    for _ in range(rng.randint(1, 5)):
        mlp = None
        if rng.random() < 0.8:
            groups = rng.choice([None, (1, 1), (2, 1), (2, 2), (3, 2), (4, 3), (8, 3)])
            count, keep = groups or (1, 1)
            experts = count * rng.choice([1, 2, 3, 4, 5])
            mlp = moe(rng.choice([8, 24, 64, 96, 128]), rng.choice([0.5, 1.0, 2.0, 7.0]), experts,
                      rng.randint(1, min(experts // count * keep, 4)), rng.choice([0.5, 1.0, 2.5]), groups,
                      None if rng.random() < 0.25 else (rng.choice([16, 33, 64, 100]), rng.choice([0.6, 1.5])))
        kv_heads = rng.choice([1, 2, 3, 4])
        heads = kv_heads * rng.choice([1, 2, 4, 5])
        dim = rng.choice([8, 10, 16, 24, 32, 64, 64, 128])
        vdim = dim if rng.random() < 0.5 else rng.choice([7, 8, 16, 32, 48, 64])
        mask = None
        if rng.random() < 0.8:
            mask = (rng.choice([1, 2, 17, 63, 64, 65, 100]), rng.choice([0, 1, 2, 6, 16, 64, 65, 100]))
        rot = None
        if rng.random() < 0.85:
            scaling = None
            if rng.random() < 0.7:
                fast = rng.choice([2.0, 8.0, 30.0])
                scaling = (rng.choice([1.0, 2.0, 8.0, 40.0]), rng.choice([16, 64, 400, 4096]), fast,
                           fast / rng.choice([2.0, 8.0, 32.0]))
            rot = (rng.choice([100.0, 10000.0, 300000.0]),
                   rng.choice([d for d in (2, 4, 8, 16, 32, dim) if d <= dim]), scaling)
        layers.append(attention(heads, kv_heads, dim, vdim, rng.choice([1.5, 2.5]) / dim ** 0.5, mask, rot, mlp))
    loop = None
    if rng.random() < 0.7:
        start = rng.randrange(len(layers))
        loop = (start, rng.randint(start + 1, len(layers)), rng.choice([1, 2, 2, 3]))
    return model(rng.randint(20, 300), width, rng.choice([1e-5, 1e-6]), rng.choice([1.0, 0.5, 0.7, 1.4]),
                 loop, layers)


def run_all(cfg, tensors, dtype, folder, margin):
    import edge_infer_amd as ei
    vocab = cfg["vocab"]
    requests = [ids(vocab, n, 50 + n) for n in (150, 1, 37)]
    refs = [plain.clear_rows(cfg, tensors, r, margin, carry=True) for r in requests]
    model_ = ei.load_model(write_folder(folder, cfg, tensors), dtype=dtype)
    session = ei.Session(model_, max_tokens=64 * 8, max_seqs=3)

    def close(got, want, clear, what):
        if clear.sum() == 0:
            return
        got, want = got[clear.to(got.device)], want[clear]
        if dtype == "float32":
            assert_close_f32(got, want, what)
        else:
            # (bfloat16's roundings add up like a random walk over the runs of layers: the bound
            # of the hand-made models grows with the root of the depth)
            deeper = max(1.0, len(plain.layer_runs(cfg)) / 5.0) ** 0.5
            assert_close_bf16(got, want, what, rms_rel=4e-2 * deeper, max_rel=12e-2 * deeper)
    # whole, and in portions
    slot = session.begin()
    close(session.step([(slot, requests[0], list(range(150)))]), *refs[0], "whole")
    session.end(slot)
    slot = session.begin()
    rows, at = [], 0
    for take in (2, 3, 60, 1, 70, 14):
        rows.append(session.step([(slot, requests[0][at:at + take], list(range(take)))]))
        at += take
    close(torch.cat(rows), *refs[0], "portions")
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
        want, clear = refs[i]
        close(torch.cat(got[i]), want[cuts[i] - 1:], clear[cuts[i] - 1:], f"request {i} of the batch")
    session.cache.check()
    return sum(int(clear.sum()) for _, clear in refs)


@pytest.mark.parametrize("seed", SEEDS)
def test_drawn_model_in_float32(seed, tmp_path):
    cfg = drawn_config(seed)
    run_all(cfg, sharp_weights(cfg, seed=seed), "float32", tmp_path / "m", 1e-5)


@pytest.mark.parametrize("seed", SEEDS)
def test_drawn_twin_in_bfloat16(seed, tmp_path):
    cfg = routeless_twin(drawn_config(seed))
    assert run_all(cfg, sharp_weights(cfg, seed=seed), "bfloat16", tmp_path / "m", 0.02) == 188
