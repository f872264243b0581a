"""The Lemotar decoder in the engine against the plain implementation (`plain_lemotar`), in
float32 and bfloat16: whole prompts, the stream after every layer, prompts then tokens one by one,
portions down to two tokens, batches of unequal requests with slots and pages used again, long
decoding over window edges and page borders, the first tokens of a sequence, a token far back,
greedy generation through the entry point, the framework's own random-weights folder and the
replay program."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import plain_lemotar as plain
from helpers import assert_close_bf16, assert_close_f32
from lemotar_helpers import CONFIGS, ids, sharp_weights, tensor_shapes, write_folder

pytestmark = pytest.mark.gpu

ROOT = Path(__file__).resolve().parents[1]
DTYPES = ["float32", "bfloat16"]
NAMES = ["A", "B", "C", "D"]
LENGTHS = {"A": [150, 1, 49, 75], "B": [210, 2, 101, 64], "C": [140, 3, 110, 65],
           "D": [150, 1, 5, 66]}
# bfloat16 engine against the float64 oracle on these order-one weights: root-mean-square error
# relative to the logits' root-mean-square, and largest error relative to the largest logit
BF16_RMS, BF16_MAX = 4e-2, 12e-2


def close(dtype, actual, expected, what):
    if dtype == "float32":
        return assert_close_f32(actual, expected, what)
    return assert_close_bf16(actual, expected, what, rms_rel=BF16_RMS, max_rel=BF16_MAX)


@pytest.fixture(scope="module")
def weights():
    return {name: sharp_weights(CONFIGS[name], seed=20 + i) for i, name in enumerate(NAMES)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory, weights):
    root = tmp_path_factory.mktemp("lemotar")
    return {name: write_folder(root / name, CONFIGS[name], weights[name]) for name in NAMES}


@pytest.fixture(scope="module")
def models(folders):
    import edge_infer_amd as ei
    cache = {}

    def get(name, dtype):
        if (name, dtype) not in cache:
            cache[(name, dtype)] = ei.load_model(folders[name], dtype=dtype)
        return cache[(name, dtype)]
    return get


def requests_for(name, seed=5):
    return [ids(CONFIGS[name]["vocab"], n, seed + i) for i, n in enumerate(LENGTHS[name])]


@pytest.fixture(scope="module")
def references(weights):
    return {name: [plain.forward(CONFIGS[name], weights[name], r) for r in requests_for(name)]
            for name in NAMES}


# ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts(models, references, name, dtype):
    import edge_infer_amd as ei
    session = ei.Session(models(name, dtype), max_tokens=512)
    for request, ref in zip(requests_for(name), references[name]):
        slot = session.begin()
        logits = session.step([(slot, request, list(range(len(request))))])
        close(dtype, logits, ref, f"{name} {dtype} whole {len(request)}")
        session.end(slot)
    session.cache.check()


@pytest.mark.parametrize("name", NAMES)
def test_prompts_of_more_rows_than_the_few_rows_product_takes(models, weights, name):
    """A prompt of 420 tokens and one of 300 beside a short one (bfloat16: the library multiplies,
    decays' and gate's logits as one product), then tokens one by one together."""
    import edge_infer_amd as ei
    cfg = CONFIGS[name]
    requests = [ids(cfg["vocab"], n, 60 + n) for n in (425, 305, 9)]
    refs = [plain.forward(cfg, weights[name], r) for r in requests]
    session = ei.Session(models(name, "bfloat16"), max_tokens=1024, max_seqs=3)
    slots = [session.begin() for _ in requests]
    cuts = [len(r) - 5 for r in requests]
    logits = session.step([(s, r[:c], list(range(c))) for s, r, c in zip(slots, requests, cuts)])
    at = 0
    for ref, cut in zip(refs, cuts):
        close("bfloat16", logits[at:at + cut], ref[:cut], f"{name} prompt of {cut} in a batch")
        at += cut
    for k in range(5):
        logits = session.step([(s, r[c + k:c + k + 1], [0]) for s, r, c in zip(slots, requests, cuts)])
        want = torch.stack([ref[cut + k] for ref, cut in zip(refs, cuts)])
        close("bfloat16", logits, want, f"{name} token {k} after the prompts")


@pytest.mark.parametrize("cuts", [[49], [47, 1, 1], [2, 3, 44]])
@pytest.mark.parametrize("name", NAMES)
def test_the_stream_after_every_layer(models, weights, name, cuts):
    """The float32 stream after each layer is the oracle's."""
    import edge_infer_amd as ei
    model = models(name, "float32")
    request = requests_for(name)[0][:49]
    kept = []
    plain.forward(CONFIGS[name], weights[name], request, layer_outputs=kept)
    seen = [[] for _ in kept]
    session = ei.Session(model, max_tokens=256, graphs=False)
    slot = session.begin()
    try:
        for index, layer in enumerate(model.layers):
            def watched(ctx, residual, pending, entry, original=layer.forward, rows=seen[index]):
                out = original(ctx, residual, pending, entry)
                rows.append(residual.clone())
                return out
            layer.forward = watched
        at = 0
        for take in cuts:
            session.step([(slot, request[at:at + take], [])])
            at += take
    finally:
        for layer in model.layers:
            del layer.forward
    for index, (rows, want) in enumerate(zip(seen, kept)):
        assert_close_f32(torch.cat(rows), want, f"stream after layer {index}, cuts {cuts}")


@pytest.mark.parametrize("graphs", [True, False])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prompt_then_tokens_one_by_one(models, references, name, dtype, graphs):
    """The decoded tokens pass window edges and a page border (64, 128)."""
    import edge_infer_amd as ei
    session = ei.Session(models(name, dtype), max_tokens=512, graphs=graphs)
    for request, ref in zip(requests_for(name), references[name]):
        cut = max(1, len(request) - 60)
        slot = session.begin()
        rows = [session.step([(slot, request[:cut], [cut - 1])])]
        rows += [session.step([(slot, [token], [0])]) for token in request[cut:]]
        close(dtype, torch.cat(rows), ref[cut - 1:], f"{name} {dtype} tail of {len(request)}")
        session.end(slot)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("sizes", [(2, 2, 3, 2), (1, 5, 64, 2, 7), (63, 2, 65), (20, 100, 3)])
def test_portions(models, references, name, dtype, sizes):
    """A prompt cut into portions (the given sizes in turn, down to two tokens and one): every
    position's logits are those of the whole prompt."""
    import edge_infer_amd as ei
    session = ei.Session(models(name, dtype), max_tokens=512)
    request, ref = requests_for(name)[0], references[name][0]
    slot = session.begin()
    rows, at, turn = [], 0, 0
    while at < len(request):
        take = min(sizes[turn % len(sizes)], len(request) - at)
        rows.append(session.step([(slot, request[at:at + take], list(range(take)))]))
        at, turn = at + take, turn + 1
    close(dtype, torch.cat(rows), ref, f"{name} {dtype} portions {sizes}")
    session.end(slot)


def test_float32_logits_do_not_depend_on_the_cut(models):
    """Whole, in portions and token by token: the same float32 logits, up to the rounding of a
    few sums that the kernels take in another order for another number of rows (half the
    bound against the oracle)."""
    import edge_infer_amd as ei
    request = requests_for("A")[0][:100]
    session = ei.Session(models("A", "float32"), max_tokens=512)

    def run(sizes):
        slot = session.begin()
        rows, at = [], 0
        for take in sizes:
            rows.append(session.step([(slot, request[at:at + take], list(range(take)))]))
            at += take
        session.end(slot)
        return torch.cat(rows)
    whole = run([100])
    for sizes in ([37, 63], [2] * 50, [99, 1], [1] * 100):
        got = run(sizes)
        assert (got - whole).abs().max().item() <= 1e-5 * whole.abs().max().item(), sizes


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_batches_of_unequal_requests_with_slots_and_pages_used_again(models, references, name, dtype):
    """Requests of unequal lengths start together and are decoded together; the shorter end
    earlier and their slots and pages go back; a second and a third batch then run in what was
    freed (the cache has room for little more than one batch)."""
    import edge_infer_amd as ei
    requests, refs = requests_for(name), references[name]
    tail = 20
    session = ei.Session(models(name, dtype), max_tokens=64 * 12, max_seqs=4)
    for batch in ([0, 1, 2, 3], [3, 2, 0], [1, 0, 3, 2]):
        slots = {i: session.begin() for i in batch}
        cuts = {i: max(1, len(requests[i]) - tail) for i in batch}
        got = {i: [] for i in batch}
        logits = session.step([(slots[i], requests[i][:cuts[i]], [cuts[i] - 1]) for i in batch])
        for row, i in enumerate(batch):
            got[i].append(logits[row:row + 1])
        at = dict(cuts)
        live = [i for i in batch if at[i] < len(requests[i])]
        for i in batch:
            if i not in live:
                session.end(slots[i])
        while live:
            logits = session.step([(slots[i], [requests[i][at[i]]], [0]) for i in live])
            for row, i in enumerate(live):
                got[i].append(logits[row:row + 1])
                at[i] += 1
            for i in [i for i in live if at[i] == len(requests[i])]:
                session.end(slots[i])
                live.remove(i)
        for i in batch:
            close(dtype, torch.cat(got[i]), refs[i][cuts[i] - 1:],
                  f"{name} {dtype} request {i} in batch {batch}")
        session.cache.check()
    assert session.cache.slots.n_free == 4
    assert all(pool.n_free == pool.n_pages for pool in session.cache.kv_pools)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_prompts_portions_and_tokens_mixed_in_one_step(models, references, name, dtype):
    """A step that holds a prompt's portion, another one's first tokens and a third one's next token;
    every request's logits are those of it alone."""
    import edge_infer_amd as ei
    requests, refs = [requests_for(name)[i] for i in (0, 2, 3)], [references[name][i] for i in (0, 2, 3)]
    session = ei.Session(models(name, dtype), max_tokens=512, max_seqs=3)
    slots = [session.begin() for _ in requests]
    got, at = [[] for _ in requests], [0, 0, 0]
    for plan in ([30, 0, 0], [1, 3, 0], [40, 1, 1], [1, 1, 1], [2, 0, 40], [1, 1, 2]):
        entries, members = [], []
        for i, take in enumerate(plan):
            take = min(take, len(requests[i]) - at[i])
            if take > 0:
                entries.append((slots[i], requests[i][at[i]:at[i] + take], list(range(take))))
                members.append((i, take))
        logits = session.step(entries)
        row = 0
        for i, take in members:
            got[i].append(logits[row:row + take])
            row, at[i] = row + take, at[i] + take
    for i, ref in enumerate(refs):
        close(dtype, torch.cat(got[i]), ref[:at[i]], f"{name} {dtype} request {i} of the mixed steps")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_long_decoding_from_the_first_token(models, weights, name, dtype):
    """One token, then 299 more one by one, from graphs where the products allow it: every window's
    edge and four page borders are passed while decoding; pages behind the windows are given
    back, those that a later layer with a wider window reads stay."""
    import edge_infer_amd as ei
    cfg = CONFIGS[name]
    request = ids(cfg["vocab"], 300, 77)
    ref = plain.forward(cfg, weights[name], request)
    session = ei.Session(models(name, dtype), max_tokens=320)
    slot = session.begin()
    rows = [session.step([(slot, [token], [0])]) for token in request]
    close(dtype, torch.cat(rows), ref, f"{name} {dtype} 300 tokens one by one")
    if session.graphs:     # (all but B have products of odd widths, which in bfloat16 the library multiplies)
        assert session.graph_replays > 250
    else:
        assert name != "B" and dtype == "bfloat16"
    for pages, (request_of, _) in zip(session.cache.kv_pages, session.cache.layout.kv_groups):
        if request_of.window is None:
            continue
        held = [i for i, page in enumerate(pages.row(slot)) if page >= 0]
        assert held == [i for i in range(5) if 64 * i + 63 >= 300 - request_of.window + 1]


@pytest.mark.parametrize("graphs", [True, False])
def test_a_failed_step_leaves_the_sequence_as_it_was(models, references, graphs):
    """A step that fails after its layers have run (here the head raises, once in a prompt portion
    and once in a decode step) leaves the sequence at its length and its state as it was, so the
    same step again gives what a run without the failure gives."""
    import edge_infer_amd as ei
    model = models("A", "float32")
    request, ref = requests_for("A")[0], references["A"][0]
    session = ei.Session(model, max_tokens=512, graphs=graphs)
    slot = session.begin()
    rows = [session.step([(slot, request[:40], list(range(40)))])]
    whole = type(model).logits
    failures = []

    def failing(self, ctx, hidden):
        if not failures:
            failures.append(ctx.n_rows)
            raise RuntimeError("forced failure after the layers have run")
        return whole(self, ctx, hidden)
    try:
        type(model).logits = failing
        with pytest.raises(RuntimeError, match="forced failure"):
            session.step([(slot, request[40:90], list(range(50)))])
        assert session.length(slot) == 40
        rows.append(session.step([(slot, request[40:90], list(range(50)))]))
        failures.clear()       # (the first decode step: the one that runs eagerly before a graph is made)
        with pytest.raises(RuntimeError, match="forced failure"):
            session.step([(slot, request[90:91], [0])])
        for t in range(90, 100):
            rows.append(session.step([(slot, request[t:t + 1], [0])]))
    finally:
        type(model).logits = whole
    close("float32", torch.cat(rows), ref[:100], "after failed steps")


@pytest.mark.parametrize("name, place", [("A", 0), ("A", 40), ("C", 1), ("C", 100)])
def test_a_token_far_back_shows(tmp_path, name, place):
    """Two prompts that differ in one early token alone still differ at position 400, by far more
    than the tolerance (through the layers without a window, and the state), and the engine
    follows the oracle for both, whole, in portions and decoded."""
    import edge_infer_amd as ei
    cfg = CONFIGS[name]
    tensors = sharp_weights(cfg, seed=31)
    for key, tensor in tensors.items():     # heads that hardly forget
        if key.endswith("A_log"):
            tensors[key] = (tensor.float() - 3.0).to(torch.bfloat16)
    model = ei.load_model(write_folder(tmp_path / "far", cfg, tensors), dtype="float32")
    base = ids(cfg["vocab"], 401, 3)
    other = list(base)
    other[place] = (base[place] + 1) % cfg["vocab"]
    refs = [plain.forward(cfg, tensors, r)[-1:] for r in (base, other)]
    gap = (refs[0] - refs[1]).abs().max().item() / refs[0].abs().max().item()
    assert gap > 1e-3, f"the test's weights do not carry the token to the end ({gap:.1e})"
    session = ei.Session(model, max_tokens=1024)
    for request, ref in zip((base, other), refs):
        slot = session.begin()
        close("float32", session.step([(slot, request, [400])]), ref, "far token, whole")
        session.end(slot)
        slot = session.begin()
        session.step([(slot, request[:130], [])])
        session.step([(slot, request[130:390], [])])
        for token in request[390:400]:
            session.step([(slot, [token], [])])
        close("float32", session.step([(slot, request[400:], [0])]), ref, "far token, decoded")
        session.end(slot)


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_greedy_generation_through_the_entry_point(models, weights, name):
    """`Session.generate_batch` (the scheduler, sampler and step function together) gives the
    oracle's greedy tokens in float32."""
    import edge_infer_amd as ei
    cfg = CONFIGS[name]
    prompts = [ids(cfg["vocab"], n, 40 + n) for n in (5, 1, 30)]
    session = ei.Session(models(name, "float32"), max_tokens=512, max_seqs=3)
    got = session.generate_batch(prompts, max_new_tokens=12, temperature=0.0)
    for prompt, tokens in zip(prompts, got):
        assert len(tokens) == 12
        logits = plain.forward(cfg, weights[name], list(prompt) + list(tokens[:-1]))[len(prompt) - 1:]
        for token, row in zip(tokens, logits):
            best = row.argmax().item()
            if token != best:       # only a tie within float32's reach may differ
                assert (row[best] - row[token]).item() <= 2e-5 * row.abs().max().item()


def test_model_type_through_the_python_entry_and_the_command_line(folders, weights):
    """`Model.from_pretrained` and `bin/chat` on token ids give the oracle's greedy tokens."""
    from edge_infer_amd.api import Model
    model = Model.from_pretrained(folders["A"], "lemotar_fp32")
    session = model.new_session(capacity=128, max_batch=2)
    prompt = ids(CONFIGS["A"]["vocab"], 9, 1)
    tokens = session.generate(prompt, None, max_length=len(prompt) + 4, temperature=0.0)
    logits = plain.forward(CONFIGS["A"], weights["A"], prompt)[-1]
    assert tokens[0] == logits.argmax().item() and len(tokens) == 4
    with pytest.raises(ValueError, match="names the family"):
        Model.from_pretrained(folders["A"], "qwen3_bf16")
    done = subprocess.run([sys.executable, str(ROOT / "bin" / "chat"), "--model_path",
                           str(folders["A"]), "--model_type", "lemotar_fp32",
                           "--prompt_ids", ",".join(str(t) for t in prompt), "--temperature", "0",
                           "--max_new_tokens", "4"], capture_output=True, text=True, timeout=300)
    assert done.returncode == 0, done.stderr[-2000:]
    for token in tokens:
        assert str(token) in done.stdout


def test_random_weights_folder_of_the_framework(tmp_path):
    """`write_model_folder` writes a Lemotar folder that reads back to the same configuration
    and runs; its tensors carry the checkpoint's names."""
    import edge_infer_amd as ei
    from safetensors.torch import load_file
    cfg = ei.config.LemotarConfig.from_dict(CONFIGS["C"])
    folder = ei.write_model_folder(tmp_path / "random", cfg, seed=2)
    assert ei.read_config(folder)[1] == cfg
    tensors = load_file(str(folder / "model.safetensors"))
    assert set(tensors) == set(tensor_shapes(CONFIGS["C"]))
    model = ei.load_model(folder, dtype="float32")
    session = ei.Session(model, max_tokens=128)
    slot = session.begin()
    request = ids(CONFIGS["C"]["vocab"], 70, 9)
    logits = session.step([(slot, request, list(range(70)))])
    raw = json.loads((folder / "config.json").read_text())
    close("float32", logits, plain.forward(raw, tensors, request), "random folder")


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_replay_program_runs_a_lemotar_folder(folders, weights, tmp_path, dtype):
    """`bin/trace_run` chooses the model class by config.json and writes the step's logits."""
    cfg, tensors = CONFIGS["B"], weights["B"]
    vocab = cfg["vocab"]
    one, two = ids(vocab, 90, 8), ids(vocab, 12, 9)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": one[:88], "want": [0, 87]},
                                     {"id": "y", "tokens": two[:11], "want": [10]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": one[88:89], "want": []},
                                     {"id": "y", "tokens": two[11:], "want": [0]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": one[89:], "want": [0]}], "end": ["x"]}]
    done = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model",
                           str(folders["B"]), "--dtype", dtype, "--out", str(tmp_path),
                           "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps),
                          capture_output=True, text=True, timeout=300)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [l for l in done.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    ref_one, ref_two = plain.forward(cfg, tensors, one), plain.forward(cfg, tensors, two)

    def written(step, rows):
        return torch.from_numpy(np.fromfile(tmp_path / f"{step}.f32", dtype="<f4").reshape(rows, vocab))
    close(dtype, written(0, 3), torch.cat([ref_one[[0, 87]], ref_two[[10]]]), "replayed prompts")
    close(dtype, written(1, 1), ref_two[11:], "replayed token of the short request")
    close(dtype, written(2, 1), ref_one[89:], "replayed token")
