"""Baselix on the GPU against the plain implementation (tests/plain_baselix.py, float64): every mechanism's kernels
alone -- with inputs made so that one key, one edge of a window, the sink or one expert decides the result --, then whole
models: prompts whole, decoded token by token, in portions down to two tokens, unequal requests in one batch, pages and
slots that are used again, long decoding, greedy generation through the entry point and the scheduler -- in 32-bit and in
bfloat16, on configurations that differ in every size (tests/baselix_models.py).

In bfloat16 the whole models run with routers that have nothing to choose (every expert used, weighed by its logit):
where a choice is a close call a rounding turns it, and the rows behind it are then another model's.  The choice itself
is tested on the routing kernel alone, and in 32-bit on the whole models."""
import math
import types

import numpy as np
import pytest
import torch

import baselix_models
import helpers
import plain_baselix as plain

pytestmark = pytest.mark.gpu

# A row of logits may differ from the plain row by this fraction of the plain row's root mean square (the errors' root
# mean square over the vocabulary), and no single logit by more than ten times that.
ROW_RMS = {"float32": 2e-5, "bfloat16": 6e-2}
LENGTHS = {"A": [1, 2, 9, 70, 150], "B": [3, 33, 64, 201], "C": [1, 17, 140], "D": [2, 66, 131, 200], "E": [1, 2, 3, 65, 190],
           "F": [1, 5, 64, 130], "G": [5, 150, 260]}
CLOSE_CALL = 1e-5       # a 32-bit run is held to the plain rows up to a request's first routing margin below this
DEV = "cuda:0"


def close_rows(got, where, plain_logits, dtype, label, factor=1.0, upto=None):
    assert set(got) == set(where), f"{label}: rows produced {len(got)}, rows expected {len(where)}"
    limit, worst = ROW_RMS[dtype] * factor, 0.0
    for key in sorted(where):
        rid, pos = where[key]
        if upto is not None and pos >= upto.get(rid.replace("again", ""), 1 << 30):
            continue
        ref, row = plain_logits[rid][pos], got[key]
        assert np.all(np.isfinite(row)), f"{label}: non-finite logits at step {key[0]}, request {rid}, position {pos}"
        err, size = row - ref, float(np.sqrt(np.mean(ref * ref)))
        rms = float(np.sqrt(np.mean(err * err))) / size
        assert rms <= limit and float(np.abs(err).max()) <= 10 * limit * size, (
            f"{label}: first wrong row at step {key[0]}, request {rid}, position {pos}: errors' rms {rms:.3g} of the "
            f"row's (limit {limit:.3g}), largest {np.abs(err).max():.3g} of {size:.3g}")
        worst = max(worst, rms)
    return worst


def first_close_call(model) -> int:
    margins = model.closest_call()
    if margins is None:
        return 1 << 30
    near = torch.nonzero(margins < CLOSE_CALL)
    return int(near[0]) if len(near) else 1 << 30


def folder_for(tmp, name, dtype):
    if dtype == "bfloat16":
        return baselix_models.write_folder(tmp, name, dtype, config=baselix_models.settled(baselix_models.CONFIGS[name]),
                                           seed=baselix_models.SEEDS[name], tag="_settled")
    return baselix_models.write_folder(tmp, name, dtype)


@pytest.fixture(scope="module")
def setups(tmp_path_factory):
    """(name, dtype) -> (folder, requests, plain logits of every request, first close call of every request)."""
    tmp, made = tmp_path_factory.mktemp("baselix"), {}

    def get(name, dtype):
        key = (name, dtype)
        if key not in made:
            folder = folder_for(tmp, name, dtype)
            model = plain.PlainBaselix(folder)
            requests = {f"r{i}": helpers.random_ids(n, model.cfg["vocab"], 900 + i) for i, n in enumerate(LENGTHS[name])}
            logits, upto = {}, {}
            for rid, ids in requests.items():
                logits[rid] = model.forward(ids).numpy()
                upto[rid] = first_close_call(model)
            made[key] = (folder, requests, logits, upto)
        return made[key]
    return get


def executor(folder, dtype, num_pages, page_tokens, max_requests=4, max_tokens=0, **kw):
    from bare_cuda_4gib_amd.engine import Executor, load_model
    model, _ = load_model(folder, dtype, DEV)
    ex = Executor(model, num_pages=num_pages, max_requests=max_requests, page_tokens=page_tokens, poison=True,
                  max_tokens=min(max_tokens or num_pages * page_tokens, model.max_seq_len), **kw)
    ex.cache.shuffle_free_pages(5)
    return ex


CASES = [(n, d) for n in sorted(baselix_models.CONFIGS) for d in ("float32", "bfloat16")]


@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_prompts(setups, name, dtype):
    folder, requests, logits, upto = setups(name, dtype)
    steps, where = helpers.trace_whole(requests)
    got = helpers.replay_in_process(executor(folder, dtype, 40, 16), steps)
    close_rows(got, where, logits, dtype, f"whole {name} {dtype}", upto=upto)


@pytest.mark.parametrize("name", sorted(baselix_models.CONFIGS))
def test_the_stream_after_every_layer(setups, name):
    """The residual stream behind every layer against the plain one, in 32-bit (the engine keeps it in units of the
    factor on the sublayers' outputs)."""
    from bare_cuda_4gib_amd.engine import StepEntry
    folder, requests, _, upto = setups(name, "float32")
    rid = max(requests, key=lambda r: len(requests[r]))
    ids = requests[rid]
    model = plain.PlainBaselix(folder)
    _, after = model.forward(ids, return_layers=True)
    ex = executor(folder, "float32", 20, 16)
    seen = []
    for layer in ex.model.layers:

        def run(x, ctx, cache, writes=True, _forward=layer.forward):
            _forward(x, ctx, cache, writes)
            seen.append(x.detach().float().cpu().double().clone() * model.cfg["residual_mult"])
        layer.forward = run
    ex.admit(rid)
    ex.step([StepEntry(rid, ids, [len(ids) - 1])])
    assert len(seen) == len(after)
    rows = min(len(ids), upto[rid])
    for n, (mine, theirs) in enumerate(zip(seen, after)):
        size = float(theirs[:rows].pow(2).mean().sqrt())
        assert float((mine[:rows] - theirs[:rows]).abs().max()) <= 2e-4 * size, f"{name}: layer {n}"


@pytest.mark.parametrize("name,dtype", CASES)
def test_prefill_against_decoding_token_by_token(setups, name, dtype):
    """Most of a request in one step, its last 110 tokens one by one: most windows (up to 100 keys) pass over decoded
    tokens."""
    folder, requests, logits, upto = setups(name, dtype)
    steps, where = helpers.trace_tail_one_by_one(requests, tail=110)
    got = helpers.replay_in_process(executor(folder, dtype, 20, 16), steps)
    close_rows(got, where, logits, dtype, f"tail {name} {dtype}", upto=upto)


@pytest.mark.parametrize("name,dtype", CASES)
def test_portions_down_to_two_tokens(setups, name, dtype):
    """Portions are cut in the middle of pages and windows."""
    folder, requests, logits, upto = setups(name, dtype)
    for seed, sizes in ((1, (17, 2, 5, 64, 3, 2, 31, 9)), (2, (2, 2, 3, 16, 15, 1, 33, 70))):
        steps, where = helpers.trace_portions(requests, seed, sizes)
        got = helpers.replay_in_process(executor(folder, dtype, 20, 16), steps)
        close_rows(got, where, logits, dtype, f"portions {name} {dtype} {seed}", upto=upto)


@pytest.mark.parametrize("name,dtype", CASES)
def test_mixed_batches_with_pages_and_slots_used_again(setups, name, dtype):
    """Up to three live requests in three slots and a pool just large enough: portions beside decoded tokens, requests
    left out of steps, pages handed to the next request without being cleared (unowned pages hold NaN)."""
    folder, requests, logits, upto = setups(name, dtype)
    many = dict(requests)
    many.update({rid + "again": ids for rid, ids in requests.items()})            # the same requests once more, in other slots
    plain_logits = dict(logits)
    plain_logits.update({rid + "again": logits[rid] for rid in requests})
    for seed in (3, 4):
        steps, where, peak = helpers.trace_mixed(many, seed, max_live=3, tail=10, page_tokens=16)
        ex = executor(folder, dtype, peak // 16, 16, max_requests=3, max_tokens=272)
        got = helpers.replay_in_process(ex, steps)
        close_rows(got, where, plain_logits, dtype, f"mixed {name} {dtype} {seed}", upto=upto)
        assert ex.cache.pages_in_use() == 0 and ex.cache.free_slots == 3


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_requests_in_one_batch_against_each_alone(setups, dtype):
    from bare_cuda_4gib_amd.engine import StepEntry
    folder, requests, _, _ = setups("A", dtype)
    ex = executor(folder, dtype, 40, 16, max_requests=5)
    alone = {}
    for rid, ids in requests.items():
        ex.admit(rid)
        alone[rid] = ex.step([StepEntry(rid, ids, list(range(len(ids))))]).cpu().numpy()
        ex.release(rid)
    for rid in requests:
        ex.admit(rid)
    together = ex.step([StepEntry(rid, ids, list(range(len(ids)))) for rid, ids in requests.items()]).cpu().numpy()
    at = 0
    for rid, ids in requests.items():
        rows = together[at:at + len(ids)]
        at += len(ids)
        size = float(np.sqrt(np.mean(alone[rid] ** 2)))
        assert float(np.abs(rows - alone[rid]).max()) <= (1e-5 if dtype == "float32" else 5e-2) * size, rid


@pytest.mark.parametrize("name", ["A", "D"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_from_the_first_tokens(setups, name, dtype):
    """Two tokens, then 300 one by one over pages of 16, up to the last position of the table: the windows from the very
    first tokens, and the pages they have left behind."""
    from bare_cuda_4gib_amd.engine import StepEntry
    folder, _, _, _ = setups(name, dtype)
    model = plain.PlainBaselix(folder)
    ids = helpers.random_ids(302, model.cfg["vocab"], 9)
    want = model.forward(ids).numpy()
    upto = {"r": first_close_call(model)}
    ex = executor(folder, dtype, 19, 16, max_requests=2)
    ex.admit("r")
    got = {}
    rows = ex.step([StepEntry("r", ids[:2], [0, 1])]).cpu().numpy()
    got[(0, 0)], got[(0, 1)] = rows[0], rows[1]
    for p in range(2, len(ids)):
        got[(0, p)] = ex.step([StepEntry("r", [ids[p]], [0])]).cpu().numpy()[0]
    where = {(0, p): ("r", p) for p in range(len(ids))}
    close_rows(got, where, {"r": want}, dtype, f"long decoding {name} {dtype}", upto=upto)
    if name == "A":          # (the windows, the widest reader's for a shared stream, have left all but the last pages)
        assert ex.cache.pages_in_use(("window", 23)) <= 3 and ex.cache.pages_in_use(("window", 17)) <= 3


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point_and_the_scheduler(setups, dtype):
    from bare_cuda_4gib_amd.engine import Engine, generate_batch
    folder, _, _, _ = setups("A", dtype)
    model = plain.PlainBaselix(folder)
    prompts = [helpers.random_ids(n, model.cfg["vocab"], 50 + n) for n in (1, 5, 21, 40)]
    engine = Engine(folder, max_tokens=96, max_seqs=3, dtype=dtype, page_tokens=16, prefill_chunk=16)   # four requests, three slots
    together = generate_batch(engine, prompts, 24)
    margin = 1e-4 if dtype == "float32" else 0.3
    for prompt, tokens in zip(prompts, together):
        assert len(tokens) == 24
        full = model.forward(list(prompt) + list(tokens)).numpy()
        turned = first_close_call(model)
        for i, tok in enumerate(tokens):                # every chosen token is the plain best, or within a near-tie of it
            if len(prompt) - 1 + i >= turned:
                break
            row = full[len(prompt) - 1 + i]
            assert float(row.max() - row[tok]) <= margin, f"token {i} ({tok}) lies {row.max() - row[tok]:.4g} below the plain best"
    stats = engine.stats()
    assert stats["kv_pages_used"] == 0 and stats["running"] == 0


def test_the_command_line_generates_from_a_folder(setups):
    """bin/llm-infer over a Baselix folder: the architecture is chosen by config.json, ids in, ids out."""
    import os
    import subprocess
    import sys
    folder, _, _, _ = setups("B", "float32")
    model = plain.PlainBaselix(folder)
    prompt = helpers.random_ids(9, model.cfg["vocab"], 4)
    proc = subprocess.run([sys.executable, os.path.join(helpers.ROOT, "bin", "llm-infer"), "--model", folder, "--prompt",
                           ",".join(map(str, prompt)), "--tokens", "6", "--dtype", "float32"], capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    tokens = [int(t) for t in proc.stdout.strip().splitlines()[-1].split(":", 1)[1].split()]
    assert len(tokens) == 6
    full = model.forward(prompt + tokens).numpy()
    for i, tok in enumerate(tokens):
        row = full[len(prompt) - 1 + i]
        assert float(row.max() - row[tok]) <= 1e-4, (i, tok)


def test_the_replay_program_on_a_mixed_trace(setups, tmp_path):
    folder, requests, logits, upto = setups("A", "float32")
    steps, where, peak = helpers.trace_mixed(requests, 8, max_live=4, tail=6, page_tokens=64)
    got = helpers.replay_subprocess(folder, "float32", steps, str(tmp_path / "out"), peak, baselix_models.CONFIGS["A"]["vocab"])
    close_rows(got, where, logits, "float32", "bin/trace_run", upto=upto)


# ---- the kernels of each mechanism alone ---------------------------------------------------------------------------

def step_context(lengths, cached, slots):
    """What the kernels read of a step's context: request s brings lengths[s] rows after cached[s] tokens, in slot slots[s]."""
    starts = np.concatenate([[0], np.cumsum(lengths)]).astype(np.int32)
    row_seq = np.concatenate([np.full(n, s, dtype=np.int32) for s, n in enumerate(lengths)])
    positions = np.concatenate([np.arange(c, c + n, dtype=np.int32) for c, n in zip(cached, lengths)])
    i32 = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)      # noqa: E731
    return types.SimpleNamespace(
        n_tokens=int(starts[-1]), n_seqs=len(lengths), row_seq=i32(row_seq), positions=i32(positions), token_ids=None,
        seq_start=list(starts), seq_ctx=list(cached), seq_slots=list(slots), seq_start_dev=i32(starts), seq_slots_dev=i32(slots),
        seq_ctx_dev=i32(cached), max_kv_len=int(max(c + n for c, n in zip(cached, lengths))), captured=False)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_embedding_with_a_vector_for_every_position(dtype):
    """Token and position vectors added before the factor, stored or added to what the stream holds; a position that the
    table does not have gives NaN and reads nothing."""
    from bare_cuda_4gib_amd.csrc import ops
    from bare_cuda_4gib_amd.engine.spec import PartSpec
    from bare_cuda_4gib_amd.parts import build_part
    torch.manual_seed(3)
    V, W, N, factor = 30, 44, 12, 2.5
    table, places = torch.randn(V, W).to(dtype), torch.randn(N, W).to(dtype)
    emb = build_part("embedding", PartSpec("embedding", dict(vocab_size=V, hidden_size=W, scale=factor, positions=N)))
    emb.bind({"weight": table.to(DEV), "positions": places.to(DEV)}, None)
    ids, positions = torch.tensor([3, 3, 0, 29, 7], dtype=torch.int32), torch.tensor([0, 11, 4, 4, 1], dtype=torch.int32)
    ctx = types.SimpleNamespace(token_ids=ids.to(DEV), positions=positions.to(DEV))
    want = torch.stack([plain.placed_embedding(table.double(), places.double(), [t], first=int(p))[0] for t, p in zip(ids, positions)]) * factor
    assert torch.allclose(emb.forward(ctx).cpu().double(), want, atol=1e-6, rtol=1e-6)
    x = torch.randn(5, W)
    xs = x.clone().to(DEV)
    emb.add_to(xs, ctx)
    assert torch.allclose(xs.cpu().double(), x.double() + want, atol=1e-6, rtol=1e-6)
    out = ops.embed_placed(table.to(DEV), places.to(DEV), ids.to(DEV), torch.tensor([0, N, -1, 4, 1], dtype=torch.int32).to(DEV)).cpu()
    assert bool(torch.isnan(out[1:3]).all()) and bool(torch.isfinite(out[[0, 3, 4]]).all())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("size", [1, 7, 8, 4096, 100003])
def test_squared_relu_and_capped_logits(dtype, size):
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(size)
    z = (torch.randn(size) * 3.0).to(dtype)
    want = plain.squared_relu(z.double())
    tol = 1e-6 if dtype == torch.float32 else 1e-2
    zd = z.to(DEV)
    assert torch.allclose(ops.squared_relu(zd).cpu().double(), want, atol=tol, rtol=tol)
    assert ops.squared_relu(zd, out=zd) is zd and torch.allclose(zd.cpu().double(), want, atol=tol, rtol=tol)
    logits = torch.randn(size) * 20.0
    for cap in (1.0, 30.0):
        got = ops.softcap(logits.clone().to(DEV), cap).cpu().double()
        assert torch.allclose(got, plain.capped(logits.double(), cap), atol=1e-5, rtol=1e-5)


# rows x outputs x k of the products' forms: the float one (k or dtype no kernel takes), the weight-streaming one, the tiled
# one with operands straight into LDS (k whole steps of 64) and staged through registers, outputs that are no multiple of 8 or 4
@pytest.mark.parametrize("m,n,k", [(3, 40, 36), (1, 64, 64), (7, 50, 128), (40, 96, 64), (64, 33, 192), (130, 448, 192), (300, 100, 128), (200, 90, 72),
                                   (129, 67, 64)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_squared_relu_inside_the_product(dtype, m, n, k):
    """max(x W^T, 0)^2 of plain rows, and of rows whose norm is fused into the product, run before it, or prepared by the
    product that last added to the stream."""
    from bare_cuda_4gib_amd.csrc import ops
    from bare_cuda_4gib_amd.engine.spec import PartSpec
    from bare_cuda_4gib_amd.parts import build_part
    from bare_cuda_4gib_amd.parts.lazy import Normed
    from bare_cuda_4gib_amd.parts.linear import linear_squared_relu
    torch.manual_seed(m + n)
    x, w, g = torch.randn(m, k) * 2.0, (torch.randn(n, k) / math.sqrt(k)).to(dtype), (torch.randn(k) * 0.2).to(dtype)
    sw = ops.StreamedWeight(w.to(DEV))
    h = x.to(dtype)
    tol = 3e-5 if dtype == torch.float32 else 3e-2

    def close(got, rows):
        want = plain.squared_relu(rows.double() @ w.double().T)
        assert got.dtype == dtype and tuple(got.shape) == (m, n)
        assert torch.allclose(got.float().cpu().double(), want, atol=tol * float(want.abs().max()), rtol=tol)
    close(linear_squared_relu(h.to(DEV), sw, dtype), h)
    norm = build_part("norm", PartSpec("rmsnorm", dict(size=k, eps=1e-3, offset=1.0)))
    norm.bind({"weight": g.to(DEV)}, types.SimpleNamespace(act_dtype=dtype, device=DEV))
    close(linear_squared_relu(Normed(x.to(DEV), norm), sw, dtype), plain.norm_about_one(x.double(), g.double(), 1e-3))
    if dtype == torch.bfloat16 and m <= 64:
        stream, o = x.to(DEV).clone(), ops.StreamedWeight((torch.randn(k, 64) / 8).bfloat16().to(DEV))
        a = torch.randn(m, 64).bfloat16().to(DEV)
        if ops.gemm_emit_supported(a, o, stream, norm.weight):
            pre = ops.gemm_accumulate_emit(a, o, stream, norm.weight, norm.eps)
            if ops.gemm_prenormed_supported(pre, sw, ops.EPI_SQUARED_RELU):
                close(linear_squared_relu(Normed(stream, norm, pre=pre), sw, dtype), plain.norm_about_one(stream.cpu().double(), g.double(), 1e-3))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rank", [1, 13, 32, 200])
def test_latent_rows_without_a_rotated_part(dtype, rank):
    """The latent normed and written to its slots; nothing else is touched.  Without a cache there is nothing to do."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(rank)
    T, H, d, P = 5, 3, 6, 4
    both, g = torch.randn(T, H * d + rank).to(dtype), torch.randn(rank)
    slots = torch.tensor([9, 2, 0, 7, 5], dtype=torch.int32)
    cache = torch.zeros(3, P, rank, dtype=dtype, device=DEV)
    wide = both.to(DEV)
    q_lat = torch.full((T, H, rank), 7.0, device=DEV)
    ops.latent_prepare(wide[:, :H * d], wide[:, H * d:], g.to(DEV), 1e-3, None, slots.to(DEV), cache, q_lat, H, d, 0, rank, 0)
    want = plain.unit_rms(both[:, H * d:].double(), 1e-3) * g.double()
    flat, tol = cache.view(-1, rank).cpu().double(), 1e-5 if dtype == torch.float32 else 2e-2
    assert torch.allclose(flat[slots.long()], want, atol=tol, rtol=tol)
    assert float(flat[[1, 3, 4, 6, 8, 10, 11]].abs().max()) == 0.0 and float(q_lat.min()) == 7.0
    ops.latent_prepare(wide[:, :H * d], None, None, 1e-3, None, None, None, q_lat, H, d, 0, rank, 0)
    assert float(q_lat.min()) == 7.0 == float(q_lat.max())


def test_queries_of_a_layer_without_a_latent_are_rotated_alone():
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(1)
    T, H, d, rot, rank = 4, 2, 3, 6, 5
    q, dkv, g = torch.randn(T, H * (d + rot)).to(DEV), torch.randn(T, rank + rot).to(DEV), torch.rand(rank).to(DEV)
    angles = ops.latent_angles(torch.tensor([0, 3, 50, 9], dtype=torch.int32, device=DEV), 4, 30.0)
    cache, slots = torch.zeros(1, 8, rank + rot, device=DEV), torch.arange(4, dtype=torch.int32, device=DEV)
    one, two = torch.zeros(T, H, rank + rot, device=DEV), torch.zeros(T, H, rank + rot, device=DEV)
    ops.latent_prepare(q, dkv, g, 1e-5, angles, slots, cache, one, H, d, rot, rank, 4)
    ops.latent_prepare(q, None, None, 1e-5, angles, None, None, two, H, d, rot, rank, 4)
    assert torch.equal(one, two) and float(one[..., rank:].abs().min()) > 0


def paged(rows, pages, P, dtype, n_pages):
    """A cache [pages, P, size] that holds NaN but for the given rows, laid into the given pages."""
    c = torch.full((n_pages, P, rows.shape[1]), float("nan"), dtype=dtype, device=DEV)
    for j in range(rows.shape[0]):
        if pages[j // P] >= 0:
            c[pages[j // P], j % P] = rows[j].to(dtype).to(DEV)
    return c


def plain_row(q, rows, sink, pos, window, scale):
    """q [H, rank] (absorbed queries), rows [n, rank] -> (weighted sums [H, rank], weights [H, pos + 1]) of the row at ``pos``."""
    n = pos + 1
    s = torch.zeros(q.shape[0], n, n, dtype=torch.float64)
    s[:, -1] = (q.double() @ rows[:n].double().T) * scale
    w = plain.sink_softmax(s, plain.window_mask(n, window), sink.double())[:, -1]
    return w @ rows[:n].double(), w


# heads and latent sizes: beyond what the matrix-core kernel takes (the plain kernel serves bfloat16 too) and all its forms
SIZES = [(3, 20), (1, 32), (5, 96), (16, 64), (20, 128), (2, 250), (32, 512), (1, 1), (9, 13)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", SIZES)
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 100, 129])
@pytest.mark.parametrize("where", ["inside", "outside"])
def test_attention_at_the_edges_of_the_window(dtype, sizes, window, where):
    """A key made to stand out takes the weight as the first key of a row's window and is not seen at all one place further
    back: as a decoded token, in a portion whose rows' windows begin at different keys, and for a portion long enough that
    several tiles of tokens share a workgroup -- over scattered pages of 16, of which those that every row's window has
    passed were given back (they hold NaN and the table has no page for them)."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(window)
    (H, rank), n, P, scale = sizes, 150, 16, 0.3
    rows = (torch.randn(n, rank) * 0.3).to(dtype).float()
    q, sink = torch.randn(H, rank), torch.randn(H)
    at = n - window if where == "inside" else n - 1 - window
    mark = min(1, H - 1)
    rows[at] = (q[mark] / float(q[mark] @ q[mark]) * 14.0 / scale).to(dtype).float()
    pages = torch.randperm(20)[:-(-n // P)]
    for new in (1, 5, 21):
        cached = n - new
        live = pages.clone()
        live[:max(0, cached - window + 1) // P] = -1
        cache = paged(rows, live, P, dtype, 20)
        tensor_cores = ops.attention_latent_mfma_takes(cache, rank, 0)
        tol = 3e-2 if tensor_cores else 3e-5
        ctx = step_context([new], [cached], [0])
        q_lat = q.view(1, H, rank).repeat(new, 1, 1).contiguous().to(DEV)
        got = ops.attention_latent(q_lat, cache, sink.to(DEV), live.to(torch.int32).view(1, -1).to(DEV), ctx, H, rank, 0, P, window,
                                   scale).cpu().double()
        for r in range(new):
            want, w = plain_row(q, rows, sink, cached + r, window, scale)
            assert torch.allclose(got[r], want, atol=tol * max(1.0, float(want.abs().max())), rtol=tol), (new, r)
        if where == "inside":
            assert float(w[mark][at]) > 0.9
        else:
            assert float(w[mark][at]) == 0.0 and int((w[mark] > 0).sum()) == min(window, n)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(3, 20), (4, 96), (16, 512)])
@pytest.mark.parametrize("needle", [0, 15, 16, 31, 32, 120, 199])
def test_attention_finds_one_key_among_hundreds(dtype, sizes, needle):
    """A window wider than the 200 cached keys, and none: one key, far back, at a page's border or the row's own."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(needle)
    (H, rank), n, P, scale = sizes, 200, 8, 0.3
    rows = (torch.randn(n, rank) * 0.3).to(dtype).float()
    q, sink = torch.randn(H, rank), torch.randn(H)
    rows[needle] = (q[1] / float(q[1] @ q[1]) * 14.0 / scale).to(dtype).float()
    pages = torch.randperm(40)[:n // P]
    cache = paged(rows, pages, P, dtype, 40)
    tol = 3e-2 if ops.attention_latent_mfma_takes(cache, rank, 0) else 3e-5
    for new, window in ((1, 0), (1, 250), (6, 0), (6, 201)):
        ctx = step_context([new], [n - new], [0])
        q_lat = q.view(1, H, rank).repeat(new, 1, 1).contiguous().to(DEV)
        got = ops.attention_latent(q_lat, cache, sink.to(DEV), pages.to(torch.int32).view(1, -1).to(DEV), ctx, H, rank, 0, P, window,
                                   scale).cpu().double()
        for r in range(new):
            want, w = plain_row(q, rows, sink, n - new + r, window, scale)
            assert torch.allclose(got[r], want, atol=tol * max(1.0, float(want.abs().max())), rtol=tol), (new, r)
        assert float(w[1][needle]) > 0.9


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(3, 20), (4, 64)])
def test_attention_of_the_first_tokens_unequal_requests_and_sinks(dtype, sizes):
    """Three requests in one step -- the first token of a sequence, a portion from position 0, a decoded token far in --
    each with a block table of its own.  The first token weighs 1 / (1 + exp(sink - score)); a sink far above the scores
    leaves nothing, one far below leaves the plain softmax."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(8)
    (H, rank), P, scale, window = sizes, 4, 0.5, 5
    lengths, cached, n_pages = [1, 9, 1], [0, 0, 30], 24
    perm, tables, seqs, at = torch.randperm(n_pages), torch.full((3, 8), -1, dtype=torch.int32), [], 0
    cache = torch.full((n_pages + 1, P, rank), float("nan"), dtype=dtype, device=DEV)
    for s, (new, old) in enumerate(zip(lengths, cached)):
        rows = (torch.randn(new + old, rank) * 0.5).to(dtype).float()
        pages = perm[at:at + -(-len(rows) // P)]
        at += len(pages)
        tables[s, :len(pages)] = pages.to(torch.int32)
        for j in range(len(rows)):
            cache[pages[j // P], j % P] = rows[j].to(dtype).to(DEV)
        seqs.append(rows)
    q = torch.randn(sum(lengths), H, rank)
    sink = torch.tensor([0.7, 60.0, -60.0, 0.0])[:H]
    tol = 3e-2 if ops.attention_latent_mfma_takes(cache, rank, 0) else 3e-5
    got = ops.attention_latent(q.to(DEV), cache, sink.to(DEV), tables.to(DEV), step_context(lengths, cached, [0, 1, 2]), H, rank, 0, P, window,
                               scale).cpu().double()
    row = 0
    for s, (new, old) in enumerate(zip(lengths, cached)):
        for i in range(new):
            want, w = plain_row(q[row], seqs[s], sink, old + i, window, scale)
            assert torch.allclose(got[row], want, atol=tol, rtol=tol), (s, i)
            assert float(w[1].sum()) < 1e-9 and abs(float(w[2].sum()) - 1.0) < 1e-9
            if s == 0:
                score = float(q[0, 0].double() @ seqs[0][0].double()) * scale
                assert abs(float(w[0][0]) - 1.0 / (1.0 + math.exp(float(sink[0]) - score))) < 1e-9
            row += 1


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("windows", [(6, 40), (40, 6), (6, 0), (0, 6), (17, 17)])
@pytest.mark.parametrize("rank", [20, 32])
def test_a_latent_taken_over_with_another_window(tmp_path, dtype, windows, rank):
    """Two layers over one stream of latents, the second without one of its own: windows narrower and wider than the
    writer's, and none.  The prompt in portions, then decoded past both windows and several pages, with the pages that
    neither reads any more given back and holding NaN."""
    wide = dict(architecture="Baselix", vocab=60, width=40, max_positions=120, norm=dict(eps=1e-5), residual_mult=0.8, logit_softcap=12.0, layers=[
        baselix_models.layer(4, 12, 10, rank, window=windows[0] or None, mlp=None),
        baselix_models.layer(3, 16, 8, rank, window=windows[1] or None, kv_from=0, mlp=None)])
    folder = baselix_models.write_folder(tmp_path, "shared", dtype, config=wide, seed=5, query_factor=4.0)
    ids = helpers.random_ids(110, 60, 3)
    want = {"r": plain.PlainBaselix(folder).forward(ids).numpy()}
    ex = executor(folder, dtype, 14, 8, max_requests=1)
    for steps, where in (helpers.trace_tail_one_by_one({"r": ids}, tail=60), helpers.trace_portions({"r": ids}, 1, (7, 2, 9, 20))):
        close_rows(helpers.replay_in_process(ex, steps), where, want, dtype, f"windows {windows}")
    ex.admit("r")
    from bare_cuda_4gib_amd.engine import StepEntry
    ex.step([StepEntry("r", ids[:100])])
    kept = 100 if 0 in windows else max(windows)
    assert ex.cache.pages_in_use() == -(-100 // 8) - (max(0, 100 - kept + 1) // 8)


@pytest.mark.parametrize("experts,top,factor", [(8, 3, 1.0), (6, 2, 2.5), (5, 5, 0.5), (4, 1, 1.0), (64, 6, 1.5), (1, 1, 2.0), (40, 7, 1.0), (200, 4, 1.0)])
def test_the_router_weighs_the_chosen_logits_alone(experts, top, factor):
    """Logits of many rows with a bias large enough to change the choice; the weights are the softmax over the chosen
    logits; rows whose choice is a close call in 32-bit are left out.  The logits are a part of wider rows, some of them far
    apart (a softmax over all of them would underflow)."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(experts * 10 + top)
    T = 300
    wide = torch.randn(T, experts + 3) * 2.0
    wide[::7] *= 60.0
    bias = torch.randn(experts)
    z = wide[:, :experts]
    chosen, weights, margin = plain.route(z.double() + bias.double(), top)
    got_w, got_c = ops.moe_route(wide.to(DEV)[:, :experts], experts, top, want_chosen=True, factor=factor, bias=bias.to(DEV), over_chosen=True)
    got_w, got_c = got_w.cpu().double(), got_c.cpu().long()
    want_w = torch.zeros(T, experts, dtype=torch.float64).scatter_(1, chosen, weights * factor)
    sure = margin > 1e-4
    assert int(sure.sum()) > T * 0.9
    assert torch.allclose(got_w[sure], want_w[sure], atol=2e-5, rtol=2e-5)
    assert torch.equal(got_c[sure].sort(dim=1).values, chosen[sure].sort(dim=1).values)
    assert torch.allclose(got_w.sum(dim=1), torch.full((T,), factor, dtype=torch.float64), atol=1e-5)
    if 1 < top < experts:         # (the bias matters, in the choice and in the weights)
        other, w2, _ = plain.route(z.double(), top)
        assert not torch.equal(other.sort(dim=1).values, chosen.sort(dim=1).values)
        assert torch.equal(ops.moe_route(z.contiguous().to(DEV), experts, top, over_chosen=True, want_chosen=True)[1].cpu().long()[sure][:3].sort(dim=1).values,
                           other[sure][:3].sort(dim=1).values)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,ff,shared_ff", [(3, 10, 7), (4, 16, 0), (1, 5, 3), (6, 24, 16), (0, 0, 12), (2, 8, 12)])
@pytest.mark.parametrize("gated", [False, True])
def test_weighted_clamped_units_and_the_shared_one(dtype, experts, ff, shared_ff, gated):
    """Every expert's units times the row's weight for it (zero where it was not chosen); the shared unit, with sizes and a
    limit of its own, as it is or times a gate of the row; gates and ups far beyond the limits on both sides."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(experts + ff)
    T, limit, shared_limit = 13, 1.5, 0.6
    gu = (torch.randn(T, 2 * (experts * ff + shared_ff)) * 2.0).to(dtype)
    weights = torch.rand(T, experts) * (torch.rand(T, experts) > 0.4) if experts else None
    gate = torch.randn(T, 1) if gated and shared_ff else None
    want = []
    for j in range(experts):
        part = gu[:, 2 * ff * j:2 * ff * (j + 1)].double()
        want.append(plain.clamped_unit(part[:, :ff], part[:, ff:], limit) * weights[:, j:j + 1].double())
    if shared_ff:
        part = gu[:, 2 * ff * experts:].double()
        unit = plain.clamped_unit(part[:, :shared_ff], part[:, shared_ff:], shared_limit)
        want.append(unit * torch.sigmoid(gate.double()) if gate is not None else unit)
    want = torch.cat(want, dim=1)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    got = ops.routed_glu(gu.to(DEV), weights.float().to(DEV) if experts else None, experts, ff, limit, shared_ff=shared_ff,
                         shared_limit=shared_limit, shared_logit=gate.to(DEV) if gate is not None else None).float().cpu().double()
    assert got.shape == want.shape and torch.allclose(got, want, atol=tol, rtol=tol)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_captured_decode_step_replayed_over_lengths(setups, dtype):
    """One request decoded in captured steps whose graph was made for another context, with eager steps of another request
    in between: every row equals the plain one."""
    from bare_cuda_4gib_amd.engine import StepEntry
    folder, requests, logits, upto = setups("G", dtype)
    (short, long) = sorted(requests, key=lambda r: len(requests[r]))[-2:]
    ex = executor(folder, dtype, 40, 16)
    ex.admit(long), ex.admit(short)
    ids, got, where = requests[long], {}, {}
    ex.step([StepEntry(long, ids[:200])])
    for p in range(200, len(ids)):
        got[(0, p)] = ex.step([StepEntry(long, [ids[p]], [0])]).cpu().numpy()[0].copy()
        where[(0, p)] = (long, p)
        q = 2 * (p - 200)
        if q + 2 <= len(requests[short]):
            rows = ex.step([StepEntry(short, requests[short][q:q + 2], [0, 1])]).cpu().numpy()
            for i in (0, 1):
                got[(1, q + i)], where[(1, q + i)] = rows[i], (short, q + i)
    assert ex.captures >= 1
    close_rows(got, where, logits, dtype, f"captured {dtype}", upto=upto)
