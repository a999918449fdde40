"""Varolix on the GPU against the plain implementation (tests/plain_varolix.py, float64): every mechanism's kernels alone --
with inputs made so that one key, one token of a memory, the step of a temperature or a bias decides the result --, then whole
models: prompts whole, decoded token by token, in portions down to two tokens, unequal requests in one batch, pages and
slots that are used again, long decoding, greedy generation through the entry point and the scheduler -- in 32-bit and in
bfloat16, on configurations that differ in every size (tests/varolix_models.py)."""
import math
import types

import numpy as np
import pytest
import torch

import helpers
import plain_varolix as plain
import varolix_models

pytestmark = pytest.mark.gpu

# A row of logits may differ from the plain row by this fraction of the plain row's root mean square (the errors' root
# mean square over the vocabulary), and no single logit by more than ten times that.  In bfloat16 a row is also allowed three times
# what rounding the plain model's linear maps alone does to it (some rows, an early token's say, are held up by little).
ROW_RMS = {"float32": 3e-5, "bfloat16": 1e-1}
LENGTHS = {"A": [1, 2, 9, 70, 150], "B": [3, 33, 64, 201], "C": [1, 17, 140], "D": [2, 66, 131, 200], "E": [1, 2, 3, 65, 190], "F": [5, 150, 260]}
DEV = "cuda:0"
BOTH = [torch.float32, torch.bfloat16]


def close_rows(got, where, plain_logits, dtype, label, factor=1.0, noise=None):
    assert set(got) == set(where), f"{label}: rows produced {len(got)}, rows expected {len(where)}"
    worst = 0.0
    for key in sorted(where):
        rid, pos = where[key]
        ref, row = plain_logits[rid][pos], got[key]
        limit = max(ROW_RMS[dtype] * factor, 3.0 * float(noise[rid.replace("again", "")][pos]) if noise else 0.0)
        assert np.all(np.isfinite(row)), f"{label}: non-finite logits at step {key[0]}, request {rid}, position {pos}"
        err, size = row - ref, float(np.sqrt(np.mean(ref * ref)))
        rms = float(np.sqrt(np.mean(err * err))) / size
        assert rms <= limit and float(np.abs(err).max()) <= 10 * limit * size, (
            f"{label}: first wrong row at step {key[0]}, request {rid}, position {pos}: errors' rms {rms:.3g} of the "
            f"row's (limit {limit:.3g}), largest {np.abs(err).max():.3g} of {size:.3g}")
        worst = max(worst, rms)
    return worst


def noise_of(folder, requests, logits):
    rough = plain.PlainVarolix(folder, rounded=True)
    return {rid: np.sqrt(np.mean((rough.forward(ids).numpy() - logits[rid]) ** 2, axis=1) / np.mean(logits[rid] ** 2, axis=1))
            for rid, ids in requests.items()}


@pytest.fixture(scope="module")
def setups(tmp_path_factory):
    """(name, dtype) -> (folder, requests, plain logits of every request, what rounding alone does to every row)."""
    tmp, made = tmp_path_factory.mktemp("varolix"), {}

    def get(name, dtype):
        key = (name, dtype)
        if key not in made:
            config = varolix_models.CONFIGS[name]
            folder = varolix_models.write_folder(tmp, name, dtype, config=varolix_models.settled(config) if dtype == "bfloat16" else config)
            model = plain.PlainVarolix(folder)
            requests = {f"r{i}": helpers.random_ids(n, model.cfg["vocab"], 900 + i) for i, n in enumerate(LENGTHS[name])}
            logits, noise = {rid: model.forward(ids).numpy() for rid, ids in requests.items()}, None
            if dtype == "bfloat16":
                noise = noise_of(folder, requests, logits)
            made[key] = (folder, requests, logits, noise)
        return made[key]
    return get


def executor(folder, dtype, num_pages, page_tokens, max_requests=4, max_tokens=0, **kw):
    from bare_cuda_4gib_amd.engine import Executor, load_model
    model, _ = load_model(folder, dtype, DEV)
    ex = Executor(model, num_pages=num_pages, max_requests=max_requests, page_tokens=page_tokens, poison=True,
                  max_tokens=max_tokens or num_pages * page_tokens, **kw)
    ex.cache.shuffle_free_pages(5)
    return ex


CASES = [(n, d) for n in sorted(varolix_models.CONFIGS) for d in ("float32", "bfloat16")]


@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_prompts(setups, name, dtype):
    folder, requests, logits, noise = setups(name, dtype)
    steps, where = helpers.trace_whole(requests)
    got = helpers.replay_in_process(executor(folder, dtype, 40, 16), steps)
    close_rows(got, where, logits, dtype, f"whole {name} {dtype}", noise=noise)


@pytest.mark.parametrize("name", sorted(varolix_models.CONFIGS))
def test_the_stream_after_every_layer_run(setups, name):
    from bare_cuda_4gib_amd.engine import StepEntry
    folder, requests, _, _ = setups(name, "float32")
    rid = max(requests, key=lambda r: len(requests[r]))
    ids = requests[rid]
    _, after = plain.PlainVarolix(folder).forward(ids, return_layers=True)
    ex = executor(folder, "float32", 20, 16)
    seen = []
    for layer in ex.model.layers:

        def run(x, ctx, cache, writes=True, _forward=layer.forward):
            _forward(x, ctx, cache, writes)
            seen.append(x.detach().float().cpu().double().clone())
        layer.forward = run
    ex.admit(rid)
    ex.step([StepEntry(rid, ids, [len(ids) - 1])])
    assert len(seen) == len(after)
    for n, (mine, theirs) in enumerate(zip(seen, after)):
        size = float(theirs.pow(2).mean().sqrt())
        assert float((mine - theirs).abs().max()) <= 2e-4 * size, f"{name}: layer run {n}"


@pytest.mark.parametrize("name,dtype", CASES)
def test_prefill_against_decoding_token_by_token(setups, name, dtype):
    """Most of a request in one step, its last 70 tokens one by one through captured steps."""
    folder, requests, logits, noise = setups(name, dtype)
    steps, where = helpers.trace_tail_one_by_one(requests, tail=70)
    got = helpers.replay_in_process(executor(folder, dtype, 20, 16), steps)
    close_rows(got, where, logits, dtype, f"tail {name} {dtype}", noise=noise)


@pytest.mark.parametrize("name,dtype", CASES)
def test_portions_down_to_two_tokens(setups, name, dtype):
    """Portions are cut in the middle of pages and of the memories' chunks."""
    folder, requests, logits, noise = setups(name, dtype)
    for seed, sizes in ((1, (17, 2, 5, 64, 3, 2, 31, 9)), (2, (2, 2, 3, 33, 32, 1, 65, 70))):
        steps, where = helpers.trace_portions(requests, seed, sizes)
        got = helpers.replay_in_process(executor(folder, dtype, 20, 16), steps)
        close_rows(got, where, logits, dtype, f"portions {name} {dtype} {seed}", noise=noise)


@pytest.mark.parametrize("name,dtype", CASES)
def test_mixed_batches_with_pages_and_slots_used_again(setups, name, dtype):
    """Up to three live requests in three slots and a pool just large enough: portions beside decoded tokens, requests
    left out of steps, pages and slots handed to the next request (unowned pages hold NaN)."""
    folder, requests, logits, noise = setups(name, dtype)
    many = dict(requests)
    many.update({rid + "again": ids for rid, ids in requests.items()})            # the same requests once more, in other slots
    plain_logits = dict(logits)
    plain_logits.update({rid + "again": logits[rid] for rid in requests})
    for seed in (3, 4):
        steps, where, peak = helpers.trace_mixed(many, seed, max_live=3, tail=10, page_tokens=16)
        ex = executor(folder, dtype, peak // 16, 16, max_requests=3, max_tokens=272)
        got = helpers.replay_in_process(ex, steps)
        close_rows(got, where, plain_logits, dtype, f"mixed {name} {dtype} {seed}", noise=noise)
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
        assert float(np.abs(rows - alone[rid]).max()) <= (2e-5 if dtype == "float32" else 8e-2) * size, rid


@pytest.mark.parametrize("name", ["A", "D"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_from_the_first_tokens(setups, name, dtype):
    """Two tokens, then 300 one by one over pages of 16 and several buckets of captured steps."""
    from bare_cuda_4gib_amd.engine import StepEntry
    folder, _, _, _ = setups(name, dtype)
    model = plain.PlainVarolix(folder)
    ids = helpers.random_ids(302, model.cfg["vocab"], 9)
    want = model.forward(ids).numpy()
    ex = executor(folder, dtype, 19, 16, max_requests=2)
    ex.admit("r")
    got = {}
    rows = ex.step([StepEntry("r", ids[:2], [0, 1])]).cpu().numpy()
    got[(0, 0)], got[(0, 1)] = rows[0], rows[1]
    for p in range(2, len(ids)):
        got[(0, p)] = ex.step([StepEntry("r", [ids[p]], [0])]).cpu().numpy()[0]
    where = {(0, p): ("r", p) for p in range(len(ids))}
    close_rows(got, where, {"r": want}, dtype, f"long decoding {name} {dtype}", factor=2.0,
               noise=noise_of(folder, {"r": ids}, {"r": want}) if dtype == "bfloat16" else None)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point_and_the_scheduler(setups, dtype):
    from bare_cuda_4gib_amd.engine import Engine, generate_batch
    folder, _, _, _ = setups("A", dtype)
    model = plain.PlainVarolix(folder)
    prompts = [helpers.random_ids(n, model.cfg["vocab"], 50 + n) for n in (1, 5, 21, 40)]
    engine = Engine(folder, max_tokens=96, max_seqs=3, dtype=dtype, page_tokens=16, prefill_chunk=16)   # four requests, three slots
    together = generate_batch(engine, prompts, 24)
    for prompt, tokens in zip(prompts, together):
        assert len(tokens) == 24
        full = model.forward(list(prompt) + list(tokens)).numpy()
        for i, tok in enumerate(tokens):                # every chosen token is the plain best, or within a near-tie of it
            row = full[len(prompt) - 1 + i]
            margin = (1e-4 if dtype == "float32" else 0.2) * max(1.0, float(np.sqrt(np.mean(row * row))))
            assert float(row.max() - row[tok]) <= margin, f"token {i} ({tok}) lies {row.max() - row[tok]:.4g} below the plain best"
    stats = engine.stats()
    assert stats["kv_pages_used"] == 0 and stats["running"] == 0


def test_the_command_line_generates_from_a_folder(setups):
    """bin/llm-infer over a Varolix folder: the architecture is chosen by config.json, ids in, ids out."""
    import os
    import subprocess
    import sys
    folder, _, _, _ = setups("B", "float32")
    model = plain.PlainVarolix(folder)
    prompt = helpers.random_ids(9, model.cfg["vocab"], 4)
    proc = subprocess.run([sys.executable, os.path.join(helpers.ROOT, "bin", "llm-infer"), "--model", folder, "--prompt",
                           ",".join(map(str, prompt)), "--tokens", "6", "--dtype", "float32"], capture_output=True, text=True, timeout=110)
    assert proc.returncode == 0, proc.stderr[-2000:]
    tokens = [int(t) for t in proc.stdout.strip().splitlines()[-1].split(":", 1)[1].split()]
    assert len(tokens) == 6
    full = model.forward(prompt + tokens).numpy()
    for i, tok in enumerate(tokens):
        row = full[len(prompt) - 1 + i]
        assert float(row.max() - row[tok]) <= 1e-4, (i, tok)


def test_the_replay_program_on_a_mixed_trace(setups, tmp_path):
    folder, requests, logits, noise = setups("A", "float32")
    steps, where, peak = helpers.trace_mixed(requests, 8, max_live=4, tail=6, page_tokens=64)
    got = helpers.replay_subprocess(folder, "float32", steps, str(tmp_path / "out"), peak, varolix_models.CONFIGS["A"]["vocab"])
    close_rows(got, where, logits, "float32", "bin/trace_run")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_captured_decode_step_replayed_over_lengths(setups, dtype):
    """One request decoded in captured steps whose graph was made for another context, with eager steps of another request
    in between: every row equals the plain one."""
    from bare_cuda_4gib_amd.engine import StepEntry
    folder, requests, logits, noise = setups("F", dtype)
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
    close_rows(got, where, logits, dtype, f"captured {dtype}", noise=noise)


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


def run_memory(x, state, lengths, slots, H, d, e, out_dtype, **kw):
    """ops.matrix_memory over one step's rows x = [q | k | v | gate | zi | zf]."""
    from bare_cuda_4gib_amd.csrc import ops
    ctx = step_context(lengths, [0] * len(lengths), slots)
    base, n_chunks = ops.decay_scan_chunks(ctx)
    q, k, v, g, zi, zf = torch.split(x, [H * d, H * d, H * e, H * e, H, H], dim=1)
    return ops.matrix_memory(q, k, v, g, zi, zf, state, ctx, H, d, e, out_dtype=out_dtype, n_chunks=n_chunks,
                             chunk_base=torch.tensor(base, dtype=torch.int32, device=DEV), **kw)


def plain_memory(x, H, d, e, bias_i, bias_f, cap, weight, eps, factor=1.0):
    """One sequence's rows -> [T, H * e] (float64)."""
    x = x.double()
    q, k, v, g, zi, zf = torch.split(x, [H * d, H * d, H * e, H * e, H, H], dim=1)
    T = x.shape[0]
    i, f = plain.log_input_gate(zi + bias_i.double(), cap), plain.log_forget_gate(zf + bias_f.double(), cap)
    o = torch.stack([plain.matrix_memory(q.reshape(T, H, d)[:, a] * d ** -0.5, k.reshape(T, H, d)[:, a], v.reshape(T, H, e)[:, a],
                                         i[:, a], f[:, a])[0] for a in range(H)], dim=1)
    return plain.unit_rms(o, eps).reshape(T, H * e) * weight.double() * torch.sigmoid(g) * factor


def fresh_state(slots, H, d, e):
    return (torch.zeros(slots, H, d, e, device=DEV), torch.zeros(slots, H, d, device=DEV), torch.zeros(slots, H, device=DEV))


# one number of everything; every bucket of the scan's registers; values of one to four waves; sizes of 16-byte pieces and not
MEMORIES = [(1, 1, 2), (3, 5, 3), (2, 16, 16), (3, 17, 64), (3, 40, 36), (2, 64, 128), (1, 100, 130), (2, 128, 128), (1, 200, 256), (2, 256, 65)]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("sizes", MEMORIES)
def test_the_memory_over_portions_in_used_slots(dtype, sizes):
    """Three requests in slots out of order, portions of 1 to 150 rows that end inside, at and behind chunks' borders, then
    steps of one row each; what the other slots hold is not touched; the result goes into a part of wider rows."""
    H, d, e = sizes
    torch.manual_seed(d)
    cap, eps, factor = 7.0, 1e-5, 0.6
    rows = [torch.cat([torch.randn(n, H * (2 * d + 2 * e)), torch.randn(n, 2 * H) * 6.0], dim=1).to(dtype) for n in (190, 99, 40)]
    bi, bf, weight = torch.randn(H), torch.randn(H) + 3.0, torch.randn(H * e) * 0.3 + 1.0
    want = [plain_memory(x, H, d, e, bi, bf, cap, weight, eps, factor) for x in rows]
    slots, state = [4, 0, 2], fresh_state(5, H, d, e)
    state[0][[1, 3]], state[1][[1, 3]], state[2][[1, 3]] = 7.0, 7.0, 7.0
    at, got = [0, 0, 0], [[], [], []]
    for portion in ((1, 33, 2), (31, 1, 32), (150, 64, 1), (3, 1, 2)) + ((1, 0, 1),) * 3 + ((1, 0, 0),) * 2:
        who = [s for s in range(3) if portion[s]]
        x = torch.cat([rows[s][at[s]:at[s] + portion[s]] for s in who]).to(DEV)
        wide = torch.full((x.shape[0], H * e + 5), -3.0, device=DEV)
        out = run_memory(x, state, [portion[s] for s in who], [slots[s] for s in who], H, d, e, torch.float32, bias_i=bi.to(DEV), bias_f=bf.to(DEV),
                         cap=cap, weight=weight.to(DEV), eps=eps, factor=factor, out=wide[:, 2:2 + H * e])
        assert float(wide[:, :2].max()) == -3.0 == float(wide[:, 2 + H * e:].min())
        n = 0
        for s in who:
            got[s].append(out[n:n + portion[s]].cpu().double())
            n, at[s] = n + portion[s], at[s] + portion[s]
    assert at == [190, 99, 40]
    for s in range(3):
        size = float(want[s].pow(2).mean().sqrt())
        err = (torch.cat(got[s]) - want[s]).abs()
        # (a head of two values whose numerator nearly vanishes is a direction of nearly nothing: the norm lifts the rounding)
        assert float((err > 1e-3 * size).double().mean()) < (0.01 if e <= 3 else 1e-9), (s, float(err.max()))
        assert float(err.median()) < 1e-5 * size
    assert all(float(t[[1, 3]].min()) == 7.0 == float(t[[1, 3]].max()) for t in state)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("sizes", [(2, 8, 12), (1, 64, 64), (2, 100, 40)])
@pytest.mark.parametrize("marked", [0, 1, 31, 32, 63, 64, 200])
def test_the_memory_keeps_one_token_among_hundreds(dtype, sizes, marked):
    """One token with an open input gate among tokens with closed ones, forget gates open: rows far behind it, in prompts and
    decoded, read that token's value; rows ahead of it read nothing of it.  A closed forget gate later takes it away."""
    H, d, e = sizes
    torch.manual_seed(marked)
    n, cap = 300, 11.0
    x = torch.randn(n, H * (2 * d + 2 * e) + 2 * H)
    x[:, -2 * H:-H], x[:, -H:] = -40.0, 60.0                      # i near -cap, f near 0
    x[marked, -2 * H:-H] = 40.0                                   # i near cap
    x[280, -H:] = -60.0
    key = x[marked, H * d:2 * H * d].clone()
    x[290 if marked != 200 else 260:, :H * d] = key               # queries that ask for it
    x[250, :H * d] = key
    x = x.to(dtype)
    zero, weight = torch.zeros(H), torch.ones(H * e)
    want = plain_memory(x, H, d, e, zero, zero, cap, weight, 1e-5)
    value = plain.unit_rms(x[marked, 2 * H * d:2 * H * d + H * e].double().reshape(H, e), 1e-5).reshape(-1) * torch.sigmoid(
        x[250, 2 * H * d + H * e:2 * H * d + 2 * H * e].double())
    assert torch.allclose(want[250], value, atol=2e-2, rtol=2e-2)
    assert not torch.allclose(want[295], value, atol=0.3)
    for cut in ([n], [1, 249, 1, 49], [97, 2, 151] + [1] * 50):
        state, got, at = fresh_state(1, H, d, e), [], 0
        for m in cut:
            got.append(run_memory(x[at:at + m].to(DEV), state, [m], [0], H, d, e, torch.float32, bias_i=zero.to(DEV), bias_f=zero.to(DEV), cap=cap,
                                  weight=weight.to(DEV), eps=1e-5).cpu().double())
            at += m
        got = torch.cat(got)
        for t in (marked, 250, 279):
            assert torch.allclose(got[t], want[t], atol=1e-3, rtol=1e-3), (cut[:3], t)


def test_the_memory_s_floor_and_its_first_token():
    """The first token: m is max(f, i), not i; with small gates the denominator is e^(-m), not |n . q|."""
    H, d, e = 1, 4, 4
    for zi, zf in ((-3.0, 0.5), (2.0, -4.0), (0.0, 30.0)):
        x = torch.randn(1, H * (2 * d + 2 * e) + 2 * H)
        x[:, -2], x[:, -1] = zi, zf
        zero, weight = torch.zeros(H), torch.ones(H * e)
        state = fresh_state(1, H, d, e)
        got = run_memory(x.to(DEV), state, [1], [0], H, d, e, torch.float32, bias_i=zero.to(DEV), bias_f=zero.to(DEV), cap=9.0,
                         weight=weight.to(DEV), eps=0.3).cpu().double()          # (an eps that shows the size of what is normed)
        assert torch.allclose(got, plain_memory(x, H, d, e, zero, zero, 9.0, weight, 0.3), atol=1e-6)
        m = max(float(plain.log_input_gate(torch.tensor(zi), 9.0)), float(plain.log_forget_gate(torch.tensor(zf), 9.0)))
        assert abs(float(state[2]) - m) < 1e-5


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("every", [1, 7, 64, 2.5])
def test_queries_normed_per_head_with_a_temperature(dtype, every):
    """Bias, norm per head with a weight all heads share, rotation, then the factor of the position: around every step of it,
    at position 0 and far out; keys get no factor and go to scattered slots."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(3)
    H, G, d, coef, eps = 3, 2, 10, 0.7, 1e-3
    positions = torch.tensor([0, 1, 5, 6, 7, 12, 13, 14, 62, 63, 64, 126, 127, 128, 70001], dtype=torch.int32)
    T = len(positions)
    x = torch.randn(T, (H + G) * d).to(dtype)
    bias, wq, wk = torch.randn((H + G) * d), torch.rand(d) + 0.5, torch.rand(d) + 0.5
    speeds, amp = plain.turning_speeds(6, 50.0)
    table = ops.rotary_table(positions.to(DEV), speeds.to(DEV), amp)
    q_out = torch.empty(T, H, d, device=DEV)
    cache, slots = torch.zeros(8, G, 4, d, device=DEV), torch.randperm(32)[:T].to(torch.int32)
    xd = x.to(DEV)
    bd, wqd, wkd = bias.to(DEV), wq.to(DEV), wk.to(DEV)
    where = positions.to(DEV)
    sd = slots.to(DEV)
    bq, bk = bd[:H * d].contiguous(), bd[H * d:].contiguous()
    ops.heads_prepare_many([
        ops.heads_section(xd[:, :H * d], H, d, q_out, bias=bq, norm_weight=wqd, eps=eps, table=table, temperature=(where, coef, every)),
        ops.heads_section(xd[:, H * d:], G, d, cache, bias=bk, norm_weight=wkd, eps=eps, table=table, slot_map=sd, page_tokens=4)])
    full = x.double() + bias.double()
    q = plain.rms_norm(full[:, :H * d].reshape(T, H, d), wq.double(), eps)
    k = plain.rms_norm(full[:, H * d:].reshape(T, G, d), wk.double(), eps)
    q = plain.turn_halves(q, positions, speeds, amp) * plain.query_temperature(positions, coef, every)[:, None, None]
    k = plain.turn_halves(k, positions, speeds, amp)
    assert torch.allclose(q_out.cpu().double(), q, atol=2e-5, rtol=2e-5)
    flat = cache.permute(0, 2, 1, 3).reshape(32, G, d).cpu().double()
    assert torch.allclose(flat[slots.long()], k, atol=2e-5, rtol=2e-5)


def paged_heads(rows, pages, P, dtype, n_pages):
    """rows [n, G, size] -> a cache [pages, G, P, size] that holds NaN but for them."""
    c = torch.full((n_pages, rows.shape[1], P, rows.shape[2]), float("nan"), dtype=dtype, device=DEV)
    for j in range(rows.shape[0]):
        c[pages[j // P], :, j % P] = rows[j].to(dtype).to(DEV)
    return c


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("sizes", [(4, 2, 12, 10), (8, 4, 64, 128), (6, 6, 32, 64), (3, 1, 130, 70), (16, 4, 128, 128), (2, 1, 96, 48), (8, 1, 16, 16)])
@pytest.mark.parametrize("needle", [0, 15, 16, 31, 32, 63, 64, 120, 299])
def test_attention_over_every_key_finds_one_among_hundreds(dtype, sizes, needle):
    """No window: one key made to stand out, at the sequence's first place, at page and tile borders and the row's own, for
    a decoded token, a short portion and one long enough for whole tiles of rows, grouped heads; the heads times a factor,
    into a part of wider rows."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(needle)
    (H, G, d, e), n, P, scale, factor = sizes, 300, 16, 0.4, 0.7
    k, v = (torch.randn(n, G, d) * 0.3).to(dtype).float(), torch.randn(n, G, e).to(dtype).float()
    q = torch.randn(H, d)
    mark = H - 1
    k[needle, mark // (H // G)] = (q[mark] / float(q[mark] @ q[mark]) * 14.0 / scale).to(dtype).float()
    pages = torch.randperm(40)[:-(-n // P)]
    kc, vc = paged_heads(k, pages, P, dtype, 40), paged_heads(v, pages, P, dtype, 40)
    for new in (1, 5, 70):
        t0 = n - new
        ctx = step_context([new], [t0], [0])
        qs = q.view(1, H, 1, d).repeat(new, 1, 1, 1).contiguous()
        qs[:, :mark] += torch.randn(new, mark, 1, d)                # (every row's other heads are its own)
        wide = torch.full((new, H * e + 9), 5.0, dtype=dtype, device=DEV)
        got = ops.attention_maps(qs.to(DEV), kc, vc, pages.to(torch.int32).view(1, -1).to(DEV), ctx, dtype, H, G, 1, d, e, 0, 0, scale,
                                 out=wide[:, 4:4 + H * e], factor=factor).float().cpu().double()
        assert float(wide[:, :4].min()) == 5.0 == float(wide[:, 4 + H * e:].max())
        tol = 3e-5 if dtype == torch.float32 else 1e-2
        for r in range(new):
            seen = t0 + r + 1
            for a in range(H):
                s = (qs[r, a, 0].double() @ k[:seen, a // (H // G)].double().T) * scale
                w = torch.softmax(s, dim=0)
                want = (w @ v[:seen, a // (H // G)].double()) * factor
                assert torch.allclose(got[r, a * e:(a + 1) * e], want, atol=tol * max(1.0, float(want.abs().max())), rtol=tol), (new, r, a)
            if needle < seen:
                assert float(w[needle]) > 0.9


def plain_heads(q, k, v, positions, window, sink, scale, factor):
    """q [T, H, d], one request's k [n, G, d], v [n, G, e]; row t stands at positions[t] -> [T, H * e] (float64)."""
    T, H = q.shape[:2]
    hg = H // k.shape[1]
    out = []
    for t in range(T):
        p = int(positions[t])
        lo = max(0, p - window + 1) if window else 0
        row = []
        for a in range(H):
            s = (k[lo:p + 1, a // hg].double() @ q[t, a].double()) * scale
            top = max(float(s.max()), float(sink[a]) if sink is not None else -math.inf)
            e = torch.exp(s - top)
            total = e.sum() + (math.exp(float(sink[a]) - top) if sink is not None else 0.0)
            row.append((e @ v[lo:p + 1, a // hg].double()) / total * factor)
        out.append(torch.cat(row))
    return torch.stack(out)


# heads, key/value heads, key and value sizes: every form of the matrix-core kernel, sizes it fills and sizes it pads, groups of
# heads that do not divide sixteen rows
FORMS = [(4, 4, 8, 8), (6, 2, 32, 40), (8, 1, 24, 128), (3, 1, 64, 200), (4, 2, 40, 24), (5, 5, 64, 64), (12, 3, 56, 128), (2, 1, 48, 256),
         (4, 2, 128, 16), (7, 1, 104, 64), (8, 2, 128, 128), (2, 2, 72, 136), (3, 3, 256, 32), (4, 1, 136, 48), (6, 2, 200, 104), (20, 1, 256, 256)]


@pytest.mark.parametrize("sizes", FORMS)
@pytest.mark.parametrize("window,page", [(0, 16), (0, 12), (1, 16), (33, 8), (64, 64), (100, 16)])
def test_attention_of_prompt_portions_on_the_matrix_cores_is_32_bit(sizes, window, page):
    """Three requests in one step -- a whole prompt, a portion far in whose windows have left pages behind (NaN, no page in
    the table), two rows -- against float64 at float32's accuracy, though the cache is bfloat16: large scores, a sink that
    takes some of the weight and heads without one; the plain kernel computes the same."""
    from bare_cuda_4gib_amd.csrc import ops
    H, G, d, e = sizes
    torch.manual_seed(d + window)
    lengths, cached, scale, factor, n_pages = [90, 77, 2], [0, 140, 50], 0.6, 1.7, 60
    perm, tables, seqs, at = torch.randperm(n_pages), torch.full((3, 30), -1, dtype=torch.int32), [], 0
    kc = torch.full((n_pages, G, page, d), float("nan"), dtype=torch.bfloat16)
    vc = torch.full((n_pages, G, page, e), float("nan"), dtype=torch.bfloat16)
    for s, (new, old) in enumerate(zip(lengths, cached)):
        k, v = (torch.randn(new + old, G, d) * (6.0 / math.sqrt(d))).bfloat16(), torch.randn(new + old, G, e).bfloat16()
        pages = perm[at:at + -(-(new + old) // page)]
        at += len(pages)
        gone = (max(0, old - window + 1) // page) if window else 0
        for j in range(gone * page, new + old):
            kc[pages[j // page], :, j % page], vc[pages[j // page], :, j % page] = k[j], v[j]
        tables[s, :len(pages)] = pages.to(torch.int32)
        tables[s, :gone] = -1
        seqs.append((k, v))
    q = torch.randn(sum(lengths), H, d)
    sink = torch.randn(H) * 3.0 + 4.0
    ctx = step_context(lengths, cached, [0, 1, 2])
    operands = q.view(-1, H, 1, d).to(DEV), kc.to(DEV), vc.to(DEV), tables.to(DEV)
    for sk in (None, sink):
        how = dict(sink=sk.to(DEV) if sk is not None else None, factor=factor)
        got = ops.attention_maps(*operands, ctx, torch.float32, H, G, 1, d, e, window, 0, scale, **how).cpu().double()
        other = ops.attention_maps(*operands, ctx, torch.float32, H, G, 1, d, e, window, 0, scale, waves=1, **how).cpu().double()
        assert window == 1 or not torch.equal(got, other)       # (two kernels; with one key there is one sum)
        row = 0
        for s, (new, old) in enumerate(zip(lengths, cached)):
            some = sorted({0, 1, new - 1, new // 2, min(new - 1, 63), min(new - 1, 31)})
            want = plain_heads(q[[row + t for t in some]], *seqs[s], [old + t for t in some], window, sk, scale, factor)
            for a, b in ((got, 1e-5), (other, 1e-5)):
                assert torch.allclose(a[[row + t for t in some]], want, atol=b, rtol=b), (s, sk is not None)
            row += new


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("sizes", [(3, 8, 6, 20, 14), (2, 4, 2, 9, 300), (4, 16, 32, 64, 24)])
def test_latents_turned_in_halves_and_the_queries_own_latent(dtype, sizes):
    """Both latents normed by one launch (the cache row and the queries' latent), then the queries' turned part."""
    from bare_cuda_4gib_amd.csrc import ops
    H, d, r, rank, low = sizes
    torch.manual_seed(rank)
    T, P, eps = 6, 4, 1e-3
    both = torch.randn(T, low + rank + r + H).to(dtype)
    g, gq, q = torch.rand(rank) + 0.5, torch.rand(low) + 0.5, torch.randn(T, H * (d + r)).to(dtype)
    positions = torch.tensor([0, 1, 7, 63, 64, 50001], dtype=torch.int32)
    angles = ops.latent_angles(positions.to(DEV), r, 30.0)
    slots = torch.tensor([9, 2, 0, 7, 5, 11], dtype=torch.int32)
    cache = torch.zeros(3, P, rank + r, dtype=dtype, device=DEV)
    wide = both.to(DEV)
    got_low = ops.latent_prepare(None, wide[:, low:low + rank + r], g.to(DEV), eps, angles, slots.to(DEV), cache, None, H, d, r, rank, r, halves=True,
                                 low=wide[:, :low], low_g=gq.to(DEV))
    q_lat = torch.full((T, H, rank + r), 7.0, device=DEV)
    ops.latent_prepare(q.to(DEV), None, None, eps, angles, None, None, q_lat, H, d, r, rank, r, halves=True)
    x = both.double()
    speeds, _ = plain.turning_speeds(r, 30.0)
    want_row = torch.cat([plain.rms_norm(x[:, low:low + rank], g.double(), eps), plain.turn_halves(x[:, low + rank:low + rank + r], positions, speeds)], dim=1)
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    flat = cache.view(-1, rank + r).cpu().double()
    assert torch.allclose(flat[slots.long()], want_row, atol=tol, rtol=tol)
    assert float(flat[[1, 3, 4, 6, 8, 10]].abs().max()) == 0.0
    assert got_low.dtype == dtype and torch.allclose(got_low.cpu().double(), plain.rms_norm(x[:, :low], gq.double(), eps), atol=tol, rtol=tol)
    turned = plain.turn_halves(q.double().view(T, H, d + r)[..., d:], positions, speeds)
    assert torch.allclose(q_lat[..., rank:].cpu().double(), turned, atol=2e-5, rtol=2e-5) and float(q_lat[..., :rank].min()) == 7.0


@pytest.mark.parametrize("a_dtype", BOTH)
@pytest.mark.parametrize("w_dtype", BOTH)
@pytest.mark.parametrize("t,h,n,k", [(1, 3, 10, 20), (5, 4, 16, 64), (40, 2, 48, 32), (70, 6, 33, 24)])
def test_a_gate_a_head_behind_the_values_up_projection(a_dtype, w_dtype, t, h, n, k):
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(t)
    a, w, z = torch.randn(t, h, k).to(a_dtype), (torch.randn(h, n, k) / math.sqrt(k)).to(w_dtype), torch.randn(t, h + 3) * 3.0
    want = torch.stack([a[:, i].double() @ w[i].double().T for i in range(h)], dim=1) * torch.sigmoid(z[:, 2:2 + h].double())[:, :, None]
    out = torch.empty(t, h, n, device=DEV)
    ops.heads_gemm(a.to(DEV), w.to(DEV), out, k=k, n=n, gate=z.to(DEV)[:, 2:2 + h])
    tol = 2e-5 if torch.float32 == w_dtype else 2e-2
    assert torch.allclose(out.cpu().double(), want, atol=tol, rtol=tol)


# rows x outputs x k of the products' forms: the float one (k or dtype no kernel takes), the weight-streaming one, the tiled
# one with operands straight into LDS and staged through registers, outputs that are no multiple of 8 or 4
PRODUCTS = [(3, 40, 36), (1, 64, 64), (7, 50, 128), (40, 96, 64), (64, 33, 192), (130, 448, 192), (300, 100, 128), (200, 90, 72), (129, 67, 64)]


@pytest.mark.parametrize("m,n,k", PRODUCTS)
@pytest.mark.parametrize("dtype", BOTH)
def test_a_bias_with_every_form_of_the_product_that_adds_to_the_stream(dtype, m, n, k):
    """x += a W^T + b where nothing follows, where the product prepares the next norm, where its parts are added up by the kernel that norms
    them, and where there is nothing to add to yet."""
    from bare_cuda_4gib_amd.csrc import ops
    from bare_cuda_4gib_amd.engine.spec import PartSpec
    from bare_cuda_4gib_amd.parts import build_part
    from bare_cuda_4gib_amd.parts.lazy import NormHandoff, Normed
    from bare_cuda_4gib_amd.parts.linear import linear
    torch.manual_seed(m + n)
    a, w, x, b = torch.randn(m, k).to(dtype), (torch.randn(n, k) / math.sqrt(k)).to(dtype), torch.randn(m, n), torch.randn(n) * 3.0
    sw, bd = ops.StreamedWeight(w.to(DEV)), b.to(DEV)
    want = x.double() + a.double() @ w.double().T + b.double()
    tol = 3e-5 if dtype == torch.float32 else 5e-3
    got = x.to(DEV)
    linear(a.to(DEV), sw, accumulate_into=got, bias=bd)
    assert torch.allclose(got.cpu().double(), want, atol=tol, rtol=tol)
    fresh = ops.Fresh()
    linear(a.to(DEV), sw, accumulate_into=fresh, bias=bd)
    assert torch.allclose(fresh.tensor.cpu().double(), want - x.double(), atol=tol, rtol=tol)
    norm = build_part("norm", PartSpec("rmsnorm", dict(size=n, eps=1e-3)))
    g = (torch.rand(n) + 0.5).to(dtype)
    norm.bind({"weight": g.to(DEV)}, types.SimpleNamespace(act_dtype=dtype, device=DEV))
    ctx = types.SimpleNamespace(handoff=NormHandoff())
    got = x.to(DEV)
    with ctx.handoff.reader(norm, True):
        linear(a.to(DEV), sw, accumulate_into=got, ctx=ctx, bias=bd)
    assert torch.allclose(got.cpu().double(), want, atol=tol, rtol=tol)
    left = ctx.handoff.take(norm)
    normed = plain.rms_norm(want, g.double(), 1e-3)
    if isinstance(left, ops.Finished):
        assert torch.allclose(left.tensor.float().cpu().double(), normed, atol=3e-2, rtol=3e-2)
    elif left is not None:
        v = ops.StreamedWeight((torch.randn(24, n) / math.sqrt(n)).to(dtype).to(DEV))
        after = linear(Normed(got, norm, pre=left), v, out_dtype=torch.float32)
        assert torch.allclose(after.cpu().double(), normed @ ops._rows(v).cpu().double().T, atol=5e-2, rtol=5e-2)


def test_a_bias_where_k_is_cut_into_parts():
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(2)
    m, n, k = 100, 128, 1024
    a, w, x, b, g = torch.randn(m, k).bfloat16(), (torch.randn(n, k) / 32).bfloat16(), torch.randn(m, n), torch.randn(n) * 3.0, (torch.rand(n) + 0.5).bfloat16()
    sw, got = ops.StreamedWeight(w.to(DEV)), x.to(DEV)
    assert ops.gemm_parts_supported(a.to(DEV), sw, got, g.to(DEV))
    done = ops.gemm_parts_accumulate_norm(a.to(DEV), sw, got, g.to(DEV), 1e-4, bias=b.to(DEV))
    want = x.double() + a.double() @ w.double().T + b.double()
    assert torch.allclose(got.cpu().double(), want, atol=5e-3, rtol=5e-3)
    assert torch.allclose(done.tensor.float().cpu().double(), plain.rms_norm(want, g.double(), 1e-4), atol=3e-2, rtol=3e-2)


@pytest.mark.parametrize("m,inter,k", [(3, 20, 36), (1, 32, 64), (7, 24, 128), (40, 48, 64), (64, 16, 192), (130, 224, 192), (300, 56, 128), (200, 40, 72), (129, 33, 64)])
@pytest.mark.parametrize("dtype", BOTH)
def test_gelu_gated_units_inside_the_product(dtype, m, inter, k):
    """gelu(x Wg^T) * (x Wu^T) of plain rows, and of rows whose norm is fused into the product, run before it, or prepared by
    the product that last added to the stream; gates far out on both sides."""
    from bare_cuda_4gib_amd.csrc import ops
    from bare_cuda_4gib_amd.engine.spec import PartSpec
    from bare_cuda_4gib_amd.parts import build_part
    from bare_cuda_4gib_amd.parts.lazy import Normed
    torch.manual_seed(m + inter)
    x, g = torch.randn(m, k) * 2.0, (torch.rand(k) + 0.5).to(dtype)
    gate, up = (torch.randn(inter, k) * 2.0 / math.sqrt(k)).to(dtype), (torch.randn(inter, k) / math.sqrt(k)).to(dtype)
    gate[0] *= 20.0
    rt = types.SimpleNamespace(act_dtype=dtype, device=DEV)
    ffn = build_part("feedforward", PartSpec("swiglu", dict(hidden_size=k, intermediate_size=inter, act="gelu_tanh")))
    down = torch.eye(inter, dtype=dtype) if inter == k else (torch.randn(k, inter) / math.sqrt(inter)).to(dtype)
    ffn.bind({"gate_proj.weight": gate.to(DEV), "up_proj.weight": up.to(DEV), "down_proj.weight": down.to(DEV)}, rt)
    norm = build_part("norm", PartSpec("rmsnorm", dict(size=k, eps=1e-3)))
    norm.bind({"weight": g.to(DEV)}, rt)
    from bare_cuda_4gib_amd.parts.linear import linear_swiglu
    tol = 3e-5 if dtype == torch.float32 else 3e-2

    def close(got, rows):
        want = plain.gelu_by_tanh(rows.double() @ gate.double().T) * (rows.double() @ up.double().T)
        assert got.dtype == dtype and tuple(got.shape) == (m, inter)
        assert torch.allclose(got.float().cpu().double(), want, atol=tol * float(want.abs().max()), rtol=tol)
    h = x.to(dtype)
    close(linear_swiglu(h.to(DEV), ffn.w_gu, ffn.interleaved, "gelu_tanh"), h)
    close(linear_swiglu(Normed(x.to(DEV), norm), ffn.w_gu, ffn.interleaved, "gelu_tanh"), plain.rms_norm(x.double(), g.double(), 1e-3))
    if dtype == torch.bfloat16 and ffn.interleaved:
        stream, o, a = x.to(DEV).clone(), ops.StreamedWeight((torch.randn(k, 64) / 8).bfloat16().to(DEV)), torch.randn(m, 64).bfloat16().to(DEV)
        if ops.gemm_emit_supported(a, o, stream, norm.weight):
            pre = ops.gemm_accumulate_emit(a, o, stream, norm.weight, norm.eps)
            if ops.gemm_prenormed_supported(pre, ffn.w_gu, ops.EPI_GEGLU):
                close(linear_swiglu(Normed(stream, norm, pre=pre), ffn.w_gu, True, "gelu_tanh"), plain.rms_norm(stream.cpu().double(), g.double(), 1e-3))
    # the part as a whole
    y = torch.zeros(m, k, device=DEV)
    ffn.forward(h.to(DEV), types.SimpleNamespace(handoff=types.SimpleNamespace(reading_next=None)), y)
    want = (plain.gelu_by_tanh(h.double() @ gate.double().T) * (h.double() @ up.double().T)) @ down.double().T
    assert torch.allclose(y.cpu().double(), want, atol=tol * max(1.0, float(want.abs().max())), rtol=tol)


def test_a_prepared_norm_finished_in_the_tiled_gated_product():
    """The gelu's form of the tiled product that finishes a prepared norm, where the plan sends a wide weight there."""
    from bare_cuda_4gib_amd.csrc import ops
    torch.manual_seed(1)
    m, width, n2 = 40, 64, 8192
    x, o, a, g = torch.randn(m, width) * 2.0, ops.StreamedWeight((torch.randn(width, 64) / 8).bfloat16().to(DEV)), torch.randn(m, 64).bfloat16().to(DEV), (torch.rand(width) + 0.5)
    gu = (torch.randn(n2, width) / 8).bfloat16()
    w = ops.StreamedWeight(gu.to(DEV))
    stream = x.to(DEV)
    pre = ops.gemm_accumulate_emit(a, o, stream, g.to(DEV), 1e-4)
    assert not ops.streams_weights(m, n2, width) and ops.gemm_prenormed_supported(pre, w, ops.EPI_GEGLU)
    got = ops.gemm_prenormed(pre, w, ops.EPI_GEGLU).float().cpu().double()
    z = plain.rms_norm(stream.cpu().double(), g.double(), 1e-4) @ gu.double().T
    z = z.view(m, n2 // 16, 2, 8)
    want = (plain.gelu_by_tanh(z[:, :, 0]) * z[:, :, 1]).reshape(m, n2 // 2)
    assert torch.allclose(got, want, atol=3e-2 * float(want.abs().max()), rtol=3e-2)
