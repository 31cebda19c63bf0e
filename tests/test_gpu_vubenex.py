"""The Vubenex design in the engine against the plain implementation (`plain_vubenex.py`): each kernel alone, then whole models of
four small configurations under every way of cutting the work into steps, and generation through the entry point and the
scheduler.  In float32 the engine's logits must not depend on the cutting at all (equal bits); in bfloat16 they must lie as close
to the exact model as rounding alone explains."""
import copy
import random

import pytest
import torch

import plain_vubenex as P
from model_folders import assert_within_bfloat16_noise, relative_error
from vubenex_folders import CONFIGS, PAGE_SIZE, random_weights, write_model

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F64 = torch.float64


def _prompt(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("vubenex")
    out = {}
    for name, cfg in CONFIGS.items():
        write_model(root / name, cfg, seed=61 + ord(name))
        out[name] = root / name
    return out


_plain_cache = {}


def plain_logits(folders, name, tokens, rounded=False, dtype=F64):
    key = (str(folders[name]), tuple(tokens), rounded, dtype)
    if key not in _plain_cache:
        _plain_cache[key] = P.PlainVubenex(folders[name], dtype=dtype, storage=torch.bfloat16 if rounded else None).logits(tokens)
    return _plain_cache[key]


def make_runner(folders, name, dtype, **kw):
    from geneinfer_amd.engine import Runner, load_model
    model = load_model(folders[name], dtype, DEV)
    kw.setdefault("page_size", PAGE_SIZE.get(name, 16))
    kw.setdefault("max_tokens", 1024)
    kw.setdefault("max_requests", 4)
    return Runner(model, **kw)


def feed(runner, request, tokens, cuts):
    """The request's tokens in portions of the sizes in `cuts` (the rest one by one); logits of every position, on the host."""
    from geneinfer_amd.engine import StepEntry
    rows, at = [], 0
    sizes = list(cuts) + [1] * (len(tokens) - sum(cuts))
    for n in sizes:
        rows.append(runner.step([StepEntry(request, tokens[at:at + n], tuple(range(n)))]).cpu())
        at += n
    return torch.cat(rows)


def check_against_plain(folders, name, dtype, tokens, got, what):
    exact = plain_logits(folders, name, tokens)
    if dtype == "float32":            # within 4 times what the plain model itself loses in 32-bit
        single = plain_logits(folders, name, tokens, dtype=torch.float32)
        noise = max(relative_error(single[p], exact[p]) for p in range(len(tokens)))
        err = max(relative_error(got[p], exact[p]) for p in range(len(tokens)))
        assert err < 4 * noise + 1e-5, f"{what}: float32 logits differ from the plain implementation by {err:.2e} (the plain model in 32-bit: {noise:.2e})"
    else:
        rounded = plain_logits(folders, name, tokens, rounded=True)
        assert_within_bfloat16_noise({p: got[p] for p in range(len(tokens))}, lambda p: exact[p], lambda p: rounded[p], what)


# =============================================================================================== kernels alone
def _ints(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


def _lightning_rows(g, T, H, dk, dv, pad=3):
    """Projections [q | k | v | some columns more] of T rows and the plain statement's three operands."""
    proj = torch.randn(T, 2 * H * dk + H * dv + pad, generator=g)
    d = P.silu(proj.double())
    return proj, d[:, :H * dk].reshape(T, H, dk), d[:, H * dk:2 * H * dk].reshape(T, H, dk), d[:, 2 * H * dk:2 * H * dk + H * dv].reshape(T, H, dv)


def _scan(proj, seg, slots, state, H, dk, dv, decay, chunks):
    """seg: [(first row, rows, slot)]."""
    from geneinfer_amd.kernels import ops
    rows = proj.shape[0]
    row_slot = [0] * rows
    for t0, n, s in seg:
        row_slot[t0:t0 + n] = [s] * n
    out = torch.full((rows, H * dv), float("nan"), device=DEV)
    ops.lightning_scan(proj.to(DEV), (0, H * dk, 2 * H * dk), ops.lightning_powers(decay, DEV), _ints([t for t, _, _ in seg]), _ints([n for _, n, _ in seg]), _ints(row_slot), state,
                       out, H, dk, dv, rows_per_request=[n for _, n, _ in seg] if chunks else None)
    return out.cpu()


SIZES = [(1, 5, 7), (3, 8, 12), (2, 64, 64), (4, 32, 96), (2, 33, 17), (1, 130, 70), (5, 16, 1), (2, 1, 40), (1, 300, 20), (1, 512, 33)]


@pytest.mark.parametrize("H, dk, dv", SIZES)
def test_fading_memories_token_by_token_do_not_depend_on_the_cut(H, dk, dv):
    """Two requests in used slots of a wider state tensor, their rows in portions over several steps in changing order: every row as the
    plain statement's, the same bits for every cut, the other slots untouched."""
    g = torch.Generator().manual_seed(H * dk + dv)
    decay = [0.97, 0.6, 1.0, 0.0, 0.999][:H]
    lengths, slot_of = {"a": 41, "b": 23}, {"a": 3, "b": 0}
    made = {r: _lightning_rows(g, L, H, dk, dv) for r, L in lengths.items()}
    want = {r: P.fading_memory_as_weights(q, k, v, decay).reshape(lengths[r], H * dv) for r, (_, q, k, v) in made.items()}
    results = []
    for steps in ([[("a", 41), ("b", 23)]], [[("b", 2), ("a", 1)], [("a", 9)], [("a", 17), ("b", 1)], [("b", 20), ("a", 2)], [("a", 12)]],
                  [[("a", 1), ("b", 1)]] * 23 + [[("a", 1)]] * 18):
        state = torch.full((5, H * dk * dv + 6), 7.0, device=DEV)
        for s in slot_of.values():
            state[s] = 0
        at, got = {r: 0 for r in lengths}, {r: [] for r in lengths}
        for step in steps:
            proj = torch.cat([made[r][0][at[r]:at[r] + n] for r, n in step])
            seg, t0 = [], 0
            for r, n in step:
                seg.append((t0, n, slot_of[r]))
                t0 += n
            out = _scan(proj, seg, slot_of, state, H, dk, dv, decay, chunks=False)
            for (r, n), (t0, _, _) in zip(step, seg):
                got[r].append(out[t0:t0 + n])
                at[r] += n
        results.append({r: torch.cat(got[r]) for r in lengths})
        for r in lengths:
            assert relative_error(results[-1][r], want[r]) < 5e-6, r
            assert torch.equal(results[-1][r], results[0][r]), f"{r}: another cut gave other bits"
        assert bool((state[[1, 2, 4]] == 7.0).all()) and bool((state[:, H * dk * dv:].cpu()[[1, 2, 4]] == 7.0).all())


@pytest.mark.parametrize("H, dk, dv", SIZES)
@pytest.mark.parametrize("lens", [[200], [64, 1, 33], [65, 2], [31, 128, 63, 5]])
def test_fading_memories_in_chunks(H, dk, dv, lens):
    """Long runs cut into chunks that run at once, several requests side by side, each from a state that holds something, then a
    second step on top: the same results and states as token by token, up to rounding."""
    g = torch.Generator().manual_seed(sum(lens) + dk)
    decay = [0.97, 0.6, 1.0, 0.0, 0.999][:H]
    slots = [4, 0, 2, 5][:len(lens)]
    start = torch.randn(6, H * dk * dv, generator=g)
    states = {c: start.to(DEV).clone() for c in (False, True)}
    for extra in (0, 40):
        seg, t0 = [], 0
        for n, s in zip(lens, slots):
            seg.append((t0, n + extra, s))
            t0 += n + extra
        proj = _lightning_rows(g, t0, H, dk, dv)[0]
        plain = _scan(proj, seg, slots, states[False], H, dk, dv, decay, chunks=False)
        chunked = _scan(proj, seg, slots, states[True], H, dk, dv, decay, chunks=True)
        assert relative_error(chunked, plain) < 5e-6
        assert relative_error(states[True], states[False]) < 5e-6
    untouched = [s for s in range(6) if s not in slots]
    assert torch.equal(states[True][untouched].cpu(), start[untouched])


@pytest.mark.parametrize("T, far, chunks", [(300, 0, True), (300, 63, True), (300, 64, True), (257, 1, True), (129, 127, True), (90, 0, False)])
def test_a_far_row_that_stands_out_in_a_memory_that_never_fades(T, far, chunks):
    """The row `far` has a key along the last row's query, a hundred times the others' and a value of its own: the last row reads that
    value across every chunk between them; with a decay of 1/2 nothing of it is left."""
    H, dk, dv = 2, 32, 16
    g = torch.Generator().manual_seed(T + far)
    proj, *_ = _lightning_rows(g, T, H, dk, dv)
    for a in range(H):
        proj[T - 1, a * dk:(a + 1) * dk] = 4.0
        proj[far, (H + a) * dk:(H + a + 1) * dk] = 300.0
    d = P.silu(proj.double())
    q, k, v = (d[:, s:s + H * w].reshape(T, H, w) for s, w in ((0, dk), (H * dk, dk), (2 * H * dk, dv)))
    decay = [1.0, 0.5]
    want = P.fading_memory_as_weights(q, k, v, decay)
    got = _scan(proj, [(0, T, 0)], [0], torch.zeros(1, H * dk * dv, device=DEV), H, dk, dv, decay, chunks).reshape(T, H, dv)
    mine = 32 * 300.0 * q[T - 1, 0, 0] * v[far, 0]
    assert relative_error(want[T - 1, 0], mine) < 0.2 and (T - far < 40 or float(want[T - 1, 1].abs().max()) < 0.01 * float(mine.abs().max()))
    for a in range(H):
        assert relative_error(got[:, a], want[:, a]) < 5e-6 and relative_error(got[T - 1, a], want[T - 1, a]) < 5e-5


@pytest.mark.parametrize("dim", [1, 7, 36, 192, 1000, 1024, 1028, 3000, 4096, 8192, 8196, 9001])
@pytest.mark.parametrize("wdtype, odtype", [(torch.float32, torch.float32), (torch.bfloat16, torch.bfloat16), (torch.float32, torch.bfloat16), (torch.bfloat16, torch.float32)])
def test_a_norm_over_the_whole_row_times_its_gate(dim, wdtype, odtype):
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(dim)
    wide = torch.randn(5, 3 * dim + 4, generator=g)
    o, gate, w = wide[:, :dim], wide[:, dim + 1:2 * dim + 1], (1 + 0.1 * torch.randn(dim, generator=g)).to(wdtype)
    want = P.rms_norm(o.double(), w.double(), 1e-3) * torch.sigmoid(gate.double())
    wd = wide.to(DEV)
    out = ops.row_norm_gate(wd[:, :dim], wd[:, dim + 1:2 * dim + 1], w.to(DEV), 1e-3, torch.empty(5, dim, dtype=odtype, device=DEV))
    tol = 2e-6 if odtype == torch.float32 else 6e-3
    assert relative_error(out, want) < tol
    aligned = ops.row_norm_gate(wd[:, :dim].contiguous(), wd[:, dim + 1:2 * dim + 1].contiguous(), w.to(DEV), 1e-3, torch.empty(5, dim, dtype=odtype, device=DEV))
    assert relative_error(aligned, want) < tol


@pytest.mark.parametrize("dim", [3, 50, 192, 1024, 2052, 4096, 8192, 8200])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_start_of_the_stream_and_a_sublayer_s_output_normed_and_added(dim, dtype):
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(dim)
    table, where = torch.randn(30, dim, generator=g).to(dtype), torch.randn(9, dim, generator=g).to(dtype)
    tokens, pos = [3, 29, 0, 3, 7], [0, 8, 1, 3, 8]
    want = table.double()[tokens] * 1.7 + where.double()[pos]
    x, low = torch.empty(5, dim, device=DEV), torch.empty(5, dim, dtype=torch.bfloat16, device=DEV)
    ops.embed_positioned(table.to(DEV), _ints(tokens), 1.7, where.to(DEV), _ints(pos), x, low)
    assert relative_error(x, want) < 1e-6 and torch.equal(low, x.to(torch.bfloat16))
    y = ops.add_position_rows(ops.embed(table.to(DEV), _ints(tokens), torch.empty(5, dim, device=DEV)), where.to(DEV), _ints(pos))
    assert relative_error(y, table.double()[tokens] + where.double()[pos]) < 1e-6
    # the norm behind a sublayer: added onto the stream, and the stream as the next product reads it
    x0, sub, w = torch.randn(5, dim, generator=g), 3 * torch.randn(5, dim, generator=g), (1 + 0.1 * torch.randn(dim, generator=g)).to(dtype)
    x, low = x0.to(DEV), torch.empty(5, dim, dtype=torch.bfloat16, device=DEV)
    ops.rmsnorm_add_store(sub.to(DEV), w.to(DEV), 1e-4, x, low)
    assert relative_error(x, x0.double() + P.rms_norm(sub.double(), w.double(), 1e-4)) < 1e-6 and torch.equal(low, x.to(torch.bfloat16))


@pytest.mark.parametrize("d", [24, 16, 32, 64, 128, 256])
@pytest.mark.parametrize("every", [1, 2.5, 3, 64, 1000])
def test_queries_that_grow_and_keys_that_serve_as_values(every, d):
    """The kernels that norm and store (the one for heads of any size, the one for powers of two): queries at the positions around every
    step of their growth, keys normed, and the page's values the keys before their norm."""
    from geneinfer_amd.kernels import ops
    H, G, page, eps, coef = 6, 3, 8, 1e-4, 0.8
    g = torch.Generator().manual_seed(int(every * 10))
    edges = sorted({max(0, int(n * every) + o) for n in (0, 1, 2, 3, 7) for o in (-2, -1, 0, 1)})
    T = len(edges)
    proj = torch.randn(T, (H + G) * d, generator=g)
    q_w, k_w = 1 + 0.2 * torch.randn(d, generator=g), 1 + 0.2 * torch.randn(d, generator=g)
    qd, kd = proj.double()[:, :H * d].reshape(T, H, d), proj.double()[:, H * d:].reshape(T, G, d)
    grow = torch.tensor([P.query_growth(p, coef, every) for p in edges], dtype=F64)
    want_q = P.rms_norm(qd, q_w.double(), eps) * grow[:, None, None]
    assert len(set(grow.tolist())) >= 4
    n_pages = -(-(max(edges) + 1) // page)
    cache = torch.zeros(n_pages, G * page * 2 * d, device=DEV)
    table, pos, slot = torch.arange(n_pages, dtype=torch.int32, device=DEV).reshape(1, -1), _ints(edges), _ints([0] * T)
    pd = proj.to(DEV)
    q, k = pd[:, :H * d], pd[:, H * d:]
    out = torch.empty(T, H * d, device=DEV)
    ops.norm_rope_store(q, k, k, q_w.to(DEV), k_w.to(DEV), eps, None, None, 0, pos, slot, table, out, cache, page, H, G, d, d, query_growth=(coef, every))
    assert relative_error(out, want_q.reshape(T, H * d)) < 2e-6
    for t, p in enumerate(edges):
        mine = cache[p // page].cpu().double()
        keys, values = mine[:G * page * d].reshape(G, page, d)[:, p % page], mine[G * page * d:].reshape(G, d, page)[:, :, p % page]
        assert relative_error(keys, P.rms_norm(kd[t], k_w.double(), eps)) < 2e-6 and torch.equal(values, kd[t])


@pytest.mark.parametrize("H, G, d, page, T", [(4, 4, 16, 16, 5), (5, 1, 64, 16, 37), (32, 8, 64, 16, 70), (3, 3, 128, 32, 9), (2, 1, 256, 8, 3), (7, 7, 32, 5, 1)])
def test_heads_normed_and_stored_without_a_rotation(H, G, d, page, T):
    """Rows of two requests in bfloat16, values of their own with a weight on them, pages in falling order: against the plain statement, and
    against the same kernel's general form (which a rotation by no angle makes it take)."""
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(H * d + T)
    proj = torch.randn(T, (H + 2 * G) * d + 16, generator=g)
    q_w, k_w = (1 + 0.2 * torch.randn(d, generator=g)).to(torch.bfloat16), (1 + 0.2 * torch.randn(d, generator=g)).to(torch.bfloat16)
    slots = [i % 2 for i in range(T)]
    where = [3 + i // 2 * 2 for i in range(T)]
    pages = max(where) // page + 1
    table = torch.arange(2 * pages - 1, -1, -1, dtype=torch.int32, device=DEV).reshape(2, pages).contiguous()
    pd = proj.to(DEV)
    q, k, v = pd[:, :H * d], pd[:, H * d:(H + G) * d], pd[:, (H + G) * d:(H + 2 * G) * d]
    made = []
    for cos, sin in ((None, None), (torch.ones(T, 2, device=DEV), torch.zeros(T, 2, device=DEV))):
        cache, out = torch.zeros(2 * pages, G * page * 2 * d, dtype=torch.bfloat16, device=DEV), torch.empty(T, H * d, dtype=torch.bfloat16, device=DEV)
        ops.norm_rope_store(q, k, v, q_w.to(DEV), k_w.to(DEV), 1e-5, cos, sin, 4 if cos is not None else 0, _ints(where), _ints(slots), table, out, cache, page, H, G, d, d,
                            v_scale=0.7, query_growth=(0.5, 4))
        made.append((out, cache))
    grow = torch.tensor([P.query_growth(p, 0.5, 4) for p in where], dtype=F64)[:, None, None]
    want = P.rms_norm(proj.double()[:, :H * d].reshape(T, H, d), q_w.double(), 1e-5) * grow
    assert relative_error(made[0][0], want.reshape(T, H * d)) < 5e-3
    assert relative_error(made[0][0], made[1][0]) < 5e-3 and relative_error(made[0][1], made[1][1]) < 5e-3
    for t in (0, T - 1):
        mine = made[0][1][int(table[slots[t], where[t] // page])].cpu().double()
        keys, values = mine[:G * page * d].reshape(G, page, d)[:, where[t] % page], mine[G * page * d:].reshape(G, d, page)[:, :, where[t] % page]
        assert relative_error(keys, P.rms_norm(proj.double()[t, H * d:(H + G) * d].reshape(G, d), k_w.double(), 1e-5)) < 5e-3
        assert relative_error(values, 0.7 * proj.double()[t, (H + G) * d:(H + 2 * G) * d].reshape(G, d)) < 5e-3


@pytest.mark.parametrize("rows, width, dim", [(1, 64, 10), (8, 2048, 256), (9, 128, 7), (16, 2056, 33), (3, 4096, 1)])
@pytest.mark.parametrize("activation", ["gelu_tanh", "silu"])
def test_the_gated_columns_of_a_few_rows(rows, width, dim, activation):
    """Rounding, product, activation and the token's columns in one kernel, from 32-bit rows and from rows already rounded: the same bits."""
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(rows + width)
    x, w = torch.randn(rows, width, generator=g), (torch.randn(dim, width, generator=g) * width ** -0.5).to(torch.bfloat16)
    table, tokens = torch.randn(20, dim + 5, generator=g).to(torch.bfloat16), torch.randint(0, 20, (rows,), generator=g)
    act = {"gelu_tanh": P.gelu_tanh, "silu": P.silu}[activation]
    want = act(x.to(torch.bfloat16).double() @ w.double().T) * table.double()[tokens][:, 3:3 + dim]
    outs = []
    for rows_in in (x, x.to(torch.bfloat16)):
        out = torch.empty(rows, dim, dtype=torch.bfloat16, device=DEV)
        ops.gate_token_columns_rows(rows_in.to(DEV), w.to(DEV), table.to(DEV), 3, tokens.to(torch.int32).to(DEV), out, activation)
        assert relative_error(out, want) < 5e-3
        outs.append(out)
    assert torch.equal(outs[0], outs[1])
    odd = torch.randn(rows, width + 1, generator=g).to(torch.bfloat16).to(DEV)[:, 1:]
    with pytest.raises(ops.KernelError):
        ops.gate_token_columns_rows(odd, w.to(DEV), table.to(DEV), 3, tokens.to(torch.int32).to(DEV), outs[0], activation)


def _pages(keys, values, page, hd, dtype, g):
    """Pages of several requests on scrambled numbers, between pages of NaN: (cache, table)."""
    per = [-(-k.shape[0] // page) for k in keys]
    n_pages, KV = sum(per) + 3, keys[0].shape[1]
    cache = torch.full((n_pages, 2, KV, page, hd), float("nan"), dtype=dtype)
    numbers = iter(torch.randperm(n_pages, generator=g)[:sum(per)].tolist())
    table = torch.full((len(keys), max(per)), -1, dtype=torch.int32)
    for s, (k, v) in enumerate(zip(keys, values)):
        for i in range(per[s]):
            n = table[s, i] = next(numbers)
            lo, hi = i * page, min(k.shape[0], (i + 1) * page)
            block = torch.zeros(2, page, KV, hd, dtype=dtype)
            block[0, :hi - lo], block[1, :hi - lo] = k[lo:hi], v[lo:hi]
            cache[n, 0] = block[0].permute(1, 0, 2)
            cache[n, 1] = block[1].permute(1, 2, 0).reshape(KV, page, hd)
    return cache.to(DEV), table.to(DEV)


@pytest.mark.parametrize("case", range(14))
def test_gates_per_channel_and_the_empty_seat_in_the_attention_kernels(case):
    """Steps drawn at random through the attention kernels (both prompt kernels, the decode kernel, keys shared out over workgroups, the
    exact kernel) with a gate per channel and a score of zero in the denominator, scores of which some rows' are all far below it:
    single rows, short portions and up to 700 rows on top of up to 1,500 cached positions; in every request one key, at a page's border or
    the sequence's first, points where the last row's query points."""
    from geneinfer_amd.kernels import ops
    from geneinfer_amd.parts import StepContext
    rng = random.Random(500 + case)
    g = torch.Generator().manual_seed(case)
    hd, dtype = [(64, torch.bfloat16), (128, torch.bfloat16), (32, torch.bfloat16), (96, torch.bfloat16), (48, torch.bfloat16), (40, torch.float32), (256, torch.bfloat16)][case % 7]
    KV, per = rng.choice([1, 2, 3]), rng.choice([1, 2, 6])
    H, page, scale = KV * per, rng.choice([16, 32]), rng.choice([0.125, 0.4])
    segs = []
    for s in range(rng.randrange(1, 5)):
        kind, start = rng.random(), rng.choice([0, 0, rng.randrange(1, 1500)])
        segs.append((s, start, 1 if kind < 0.35 else rng.randrange(2, 60) if kind < 0.6 or hd == 256 else rng.randrange(65, 700)))
    if hd == 256:          # (the decode kernel only: all rows of the step are its)
        segs = [(s, st, 1) for s, st, _ in segs]
    keys = [torch.randn(st + n, KV, hd, generator=g).to(dtype) for _, st, n in segs]
    values = [torch.randn(st + n, KV, hd, generator=g).to(dtype) for _, st, n in segs]
    T = sum(n for _, _, n in segs)
    q = torch.randn(T, H, hd, generator=g)
    at = 0
    for (s, st, n), k in zip(segs, keys):
        for a in range(KV):
            border = rng.choice([0, min(page, st + n - 1), max(0, (st + n - 1) // page * page - 1)])
            u = torch.randn(hd, generator=g)
            u /= u.norm()
            q[at + n - 1, a * per:(a + 1) * per] = 9.0 * u / scale ** 0.5
            k[border, a] = (1.5 * u / scale ** 0.5).to(dtype)
            if n > 2:                                    # a row whose scores all lie far below zero: nearly everything sits on the empty seat
                q[at, a * per:(a + 1) * per] = -8.0 * k[:st + 1, a].float().mean(0) * hd ** 0.5
        at += n
    q = q.to(dtype)
    gate_rows = torch.randn(T, H * hd + 16, generator=g) * 2
    cache, table = _pages(keys, values, page, hd, dtype, g)
    seg_start, rows = [], []
    for s, st, n in segs:
        seg_start.append(len(rows))
        rows += [(s, st + i) for i in range(n)]
    pos, slots = _ints([p for _, p in rows]), _ints([s for s, _ in rows])
    ctx = StepContext(n_rows=T, dtype=dtype, device=torch.device(DEV), tokens=pos, row_pos=pos, row_slot=slots, seg_slot=[s for s, _, _ in segs], seg_start=seg_start,
                      seg_len=[n for _, _, n in segs], seg_pos0=[st for _, st, _ in segs])
    gates = gate_rows.to(DEV)[:, 16:]
    sinks = torch.zeros(H, device=DEV)
    out = torch.full((T, H * hd), float("nan"), dtype=dtype, device=DEV)
    ops.attention_general(q.reshape(T, H * hd).to(DEV), cache, out, ctx, table, H, KV, hd, page_size=page, scale=scale, sinks=sinks, channel_gate=gates)
    want = torch.zeros(T, H, hd, dtype=F64)
    for (s, st, n), t0, k, v in zip(segs, seg_start, keys, values):
        for a in range(H):
            sc = (q[t0:t0 + n, a].double() @ k[:, a // per].double().T) * scale
            sc = sc.masked_fill(torch.arange(st + n)[None, :] > st + torch.arange(n)[:, None], float("-inf"))
            weights = torch.softmax(torch.cat([torch.zeros(n, 1, dtype=F64), sc], dim=1), dim=1)[:, 1:]
            want[t0:t0 + n, a] = weights @ v[:, a // per].double()
    want = want.reshape(T, H * hd) * torch.sigmoid(gate_rows[:, 16:].double())
    what = f"case {case}: hd {hd} heads {H}:{KV} page {page} scale {scale} segments {segs}"
    tol = 1e-5 if dtype == torch.float32 else 8e-3
    assert bool(torch.isfinite(out.float()).all()) and relative_error(out, want) < tol, what
    exact = torch.empty_like(out)
    ops.attention_exact(q.reshape(T, H * hd).to(DEV), cache.reshape(cache.shape[0], -1), exact, pos, slots, table, H, KV, hd, scale=scale, page_size=page, sinks=sinks, channel_gate=gates)
    assert relative_error(exact, want) < tol, what
    with pytest.raises(ops.KernelError):
        ops.attention_general(q.reshape(T, H * hd).to(DEV), cache, out, ctx, table, H, KV, hd, page_size=page, gate=gates[:, :H], channel_gate=gates)


# =============================================================================================== whole models
def _portions(n):
    sizes, out = (7, 2, 5, 3, 2, 11, 1, 4), []
    while sum(out) + sizes[len(out) % len(sizes)] <= n:
        out.append(sizes[len(out) % len(sizes)])
    return out


CUTS = {"whole": lambda n: [n], "singly": lambda n: [], "most then singly": lambda n: [n - 9], "portions": _portions, "twos": lambda n: [2] * (n // 2),
        "long portions": lambda n: [n // 2 + 3, 2, n - n // 2 - 5]}


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_residual_stream_after_every_layer(folders, name):
    """Layer by layer: the first difference names the layer."""
    tokens = _prompt(CONFIGS[name], 21, 3)
    want, _ = P.PlainVubenex(folders[name]).layer_runs(tokens)
    runner = make_runner(folders, name, "float32")
    runner.open("r")
    last = {}
    runner.model.set_trace(lambda tag, i, rows: last.__setitem__(i, rows.float().cpu()) if tag in ("embedding", "layer_out") else None)
    try:
        feed(runner, "r", tokens, [len(tokens)])
    finally:
        runner.model.set_trace(None)
    w = P.PlainVubenex(folders[name]).w
    assert relative_error(last.pop(-1), P.token_and_position_rows(tokens, w["embed"], CONFIGS[name]["embedding"]["scale"], w["pos"])) < 1e-6
    assert len(last) == len(want) == len(CONFIGS[name]["layers"])
    for i in sorted(last):
        assert relative_error(last[i], want[i]) < 2e-5, f"{name}: the stream differs behind layer {i}"


@pytest.mark.parametrize("name", list(CONFIGS))
def test_float32_logits_match_the_plain_model_and_do_not_depend_on_the_cut(folders, name):
    tokens = _prompt(CONFIGS[name], 75, 5)
    runner = make_runner(folders, name, "float32")
    got = {}
    for what, cuts in CUTS.items():
        runner.open(what)
        got[what] = feed(runner, what, tokens, cuts(len(tokens)))
        runner.close(what)
    check_against_plain(folders, name, "float32", tokens, got["whole"], f"{name} whole")
    for what in CUTS:
        assert torch.equal(got[what], got["whole"]), f"{name}: the logits of '{what}' differ from those of the whole prompt"


@pytest.mark.parametrize("name", list(CONFIGS))
def test_bfloat16_logits_lie_within_rounding_noise(folders, name):
    tokens = _prompt(CONFIGS[name], 150, 6)
    runner = make_runner(folders, name, "bfloat16")
    for what in ("whole", "portions", "most then singly", "twos", "long portions"):
        runner.open(what)
        got = feed(runner, what, tokens, CUTS[what](len(tokens)))
        runner.close(what)
        check_against_plain(folders, name, "bfloat16", tokens, got, f"{name} {what}")


@pytest.mark.parametrize("name, dtype", [("A", "float32"), ("B", "float32"), ("C", "float32"), ("D", "float32"), ("A", "bfloat16"), ("B", "bfloat16"), ("D", "bfloat16")])
def test_mixed_batches_on_a_pool_that_is_used_again(folders, name, dtype):
    """Up to four live requests, portions of some beside single tokens of others, through a pool that holds less than all requests
    together and four state slots: pages and slots are freed and used again.  Every request's logits against itself alone."""
    import traces
    from geneinfer_amd.engine import StepEntry
    cfg = CONFIGS[name]
    rng = random.Random(8)
    requests = {f"q{i}": [rng.randrange(cfg["vocab"]) for _ in range(n)] for i, n in enumerate([50, 1, 33, 77, 40, 9, 2, 61])}
    steps = traces.mixed(requests, seed=5)
    runner = make_runner(folders, name, dtype, max_tokens=traces.peak_tokens(steps, 64), max_requests=4)
    got = {}
    where = traces.wanted_positions(steps)
    for s in steps:
        for e in s["entries"]:
            if not runner.is_open(e["id"]):
                runner.open(e["id"])
        logits = runner.step([StepEntry(e["id"], e["tokens"], e["want"]) for e in s["entries"]])
        if logits is not None:
            for key, row in zip(where[s["step"]], logits.cpu()):
                got[key] = row.clone()
        for rid in s["end"]:
            runner.close(rid)
    runner.cache.check_consistency()
    alone = make_runner(folders, name, dtype)
    for rid, tokens in requests.items():
        mine = {p: row for (r, p), row in got.items() if r == rid}
        assert len(mine) == len(tokens)
        if dtype == "float32":
            alone.open(rid)
            ref = feed(alone, rid, tokens, [len(tokens)])
            alone.close(rid)
            assert all(torch.equal(mine[p], ref[p]) for p in mine), f"{name} {rid}: a mixed batch changed the logits"
        else:
            exact, rounded = plain_logits(folders, name, tokens), plain_logits(folders, name, tokens, rounded=True)
            assert_within_bfloat16_noise(mine, lambda p: exact[p], lambda p: rounded[p], f"{name} mixed {rid}")


@pytest.mark.parametrize("name, dtype", [("B", "bfloat16"), ("C", "float32"), ("B", "float32"), ("D", "bfloat16")])
def test_long_portions_beside_single_rows(folders, name, dtype):
    """Steps that hold portions of a hundred rows and more of some requests beside single rows and short portions of others, every
    request at another position; keys hundreds of positions back, across many pages; one request up to the last position there is in C."""
    from geneinfer_amd.engine import StepEntry
    cfg = CONFIGS[name]
    tokens = {r: _prompt(cfg, n, 70 + n) for r, n in (("a", 357), ("b", 150), ("c", 171), ("d", 40))}
    schedule = [[("a", 100), ("c", 70)], [("a", 130), ("b", 1), ("c", 1)], [("b", 140), ("a", 1), ("c", 99), ("d", 3)], [("a", 125), ("b", 2), ("c", 1), ("d", 37)], [("b", 7), ("a", 1)]]
    runner = make_runner(folders, name, dtype, max_tokens=1024, max_requests=4)
    at, got = {r: 0 for r in tokens}, {r: [] for r in tokens}
    for step in schedule:
        entries = []
        for r, n in step:
            if not runner.is_open(r):
                runner.open(r)
            entries.append(StepEntry(r, tokens[r][at[r]:at[r] + n], tuple(range(n))))
        logits = runner.step(entries).cpu()
        row = 0
        for r, n in step:
            got[r].append(logits[row:row + n])
            row += n
            at[r] += n
    assert all(at[r] == len(t) for r, t in tokens.items())
    alone = make_runner(folders, name, dtype)
    for r, t in tokens.items():
        mine = torch.cat(got[r])
        if dtype == "float32":
            alone.open(r)
            assert torch.equal(mine, feed(alone, r, t, [len(t)])), f"{name} {r}: a mixed step changed the logits"
            alone.close(r)
        check_against_plain(folders, name, dtype, t, mine, f"{name} {r} in mixed steps")


def test_long_decoding_through_the_captured_step(folders):
    """A short prompt and 300 tokens decoded one by one through the captured decode step: every layer's memories go from row to row in
    the request's slot, the positions' rows and the queries' growth follow the device's positions."""
    tokens = _prompt(CONFIGS["A"], 312, 9)
    for dtype in ("float32", "bfloat16"):
        runner = make_runner(folders, "A", dtype)
        runner.open("r")
        got = feed(runner, "r", tokens, [12])
        assert runner.steps_replayed > 250
        check_against_plain(folders, "A", dtype, tokens, got, f"A decoding ({dtype})")


def test_the_table_of_positions_ends_a_request(folders):
    """A runner made for longer requests than the table of positions has rows still refuses the row behind its last."""
    from geneinfer_amd.engine import StepEntry
    from geneinfer_amd.engine.runner import StepError
    n = CONFIGS["C"]["max_positions"]
    runner = make_runner(folders, "C", "float32", max_positions=4096)
    assert runner.max_positions == n
    runner.open("r")
    runner.step([StepEntry("r", [5] * (n - 1), ())])
    runner.step([StepEntry("r", [5], (0,))])
    for k in (1, 2):
        with pytest.raises(StepError):
            runner.step([StepEntry("r", [5] * k, (0,))])


def test_a_lost_memory_or_a_forgotten_position_shows(folders, tmp_path):
    """Weights made so that a fault shows: memories that never fade, so a state that is lost between steps or shared by two layers
    changes every later logit, and rows of positions ten times the tokens' rows."""
    cfg = copy.deepcopy(CONFIGS["A"])
    for layer in cfg["layers"]:
        if layer["type"] == "lightning":
            layer["mixer"]["decay"] = [1.0] * layer["mixer"]["heads"]
    w = random_weights(cfg, 77)
    w["pos"] = 10 * w["pos"]
    write_model(tmp_path / "m", cfg, weights=w)
    tokens = _prompt(cfg, 90, 12)
    own = {"A": tmp_path / "m"}
    for dtype in ("float32", "bfloat16"):
        runner = make_runner(own, "A", dtype, page_size=4)
        runner.open("r")
        got = feed(runner, "r", tokens, [5, 1, 1, 17, 2, 40])
        check_against_plain(own, "A", dtype, tokens, got, f"memories that never fade ({dtype})")
    # the same logits of a model that starts anew after half of the tokens, or whose positions do, differ by far more than any tolerance here
    plain = P.PlainVubenex(own["A"])
    assert relative_error(plain.logits(tokens)[45:], plain.logits(tokens[45:])) > 0.1
    forgot = copy.deepcopy(plain)
    for layer in forgot.cfg["layers"]:
        if layer["type"] == "lightning":
            layer["mixer"]["decay"] = [0.5] * layer["mixer"]["heads"]
    assert relative_error(plain.logits(tokens), forgot.logits(tokens)) > 0.1


def test_layers_in_another_order(folders, tmp_path):
    """Configuration A's layers backwards and one of them three times: order and number are the configuration's, nothing of them is fixed."""
    cfg = copy.deepcopy(CONFIGS["A"])
    cfg["layers"] = cfg["layers"][::-1] + [copy.deepcopy(cfg["layers"][1]), copy.deepcopy(cfg["layers"][1])]
    write_model(tmp_path / "m", cfg, seed=19)
    own = {"A": tmp_path / "m"}
    tokens = _prompt(cfg, 50, 14)
    for dtype in ("float32", "bfloat16"):
        runner = make_runner(own, "A", dtype)
        runner.open("r")
        got = feed(runner, "r", tokens, [13, 2, 20, 1])
        check_against_plain(own, "A", dtype, tokens, got, f"layers backwards ({dtype})")


def test_rows_handed_on_and_rows_made_anew_agree(folders):
    """The stream in bfloat16 as the kernel that wrote it left it for the next reader, and the stream read anew by every reader."""
    from geneinfer_amd.parts.block import SandwichBlock
    from geneinfer_amd.parts.stream import TokenSideInput
    tokens = _prompt(CONFIGS["B"], 120, 8)
    got = {}
    for hand in (True, False):
        SandwichBlock.hands_norm_on = TokenSideInput.hands_norm_on = hand
        try:
            runner = make_runner(folders, "B", "bfloat16", use_graphs=False)
            runner.open("r")
            got[hand] = feed(runner, "r", tokens, [90, 2, 18])
        finally:
            SandwichBlock.hands_norm_on = TokenSideInput.hands_norm_on = True
        check_against_plain(folders, "B", "bfloat16", tokens, got[hand], f"B, rows {'handed on' if hand else 'made anew'}")


@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation_through_the_entry_point_and_the_scheduler(folders, name):
    """Greedy tokens of several prompts, one by one through `LLM.generate` and together through the scheduler (more requests than
    it runs at once, prompts in portions), against the plain model's, as far as the plain model's two best logits are clearly apart."""
    import geneinfer_amd as gi
    from geneinfer_amd.engine import EngineConfig, EngineRequest
    from geneinfer_amd.sampling import SamplerConfig
    cfg = CONFIGS[name]
    plain = P.PlainVubenex(folders[name])
    prompts = [_prompt(cfg, n, 30 + n) for n in (5, 23, 1, 40)]
    want, sure = [], []
    for p in prompts:
        tokens = plain.greedy(p, 8)
        top2 = torch.topk(plain.logits(p + tokens)[len(p) - 1:-1], 2, dim=-1).values
        clear = [bool(c) for c in (top2[:, 0] - top2[:, 1] > 1e-3)]
        want.append(tokens)
        sure.append(clear.index(False) if False in clear else len(clear))
    assert sum(sure) >= 24
    llm = gi.LLM(str(folders[name]), dtype="float32", page_size=PAGE_SIZE[name], max_tokens=512, max_running=2)
    assert type(llm.model.config).__name__ == "VubenexConfig"
    for p, t, n in zip(prompts, want, sure):
        assert llm.generate(p, steps=len(p) + 7, temperature=0.0).generated_tokens[:n] == t[:n]
    eng = llm.engine(EngineConfig(max_running=2, step_rows=16, prefill_chunk=6))
    ids = [eng.submit(EngineRequest(p, len(p) + 7, SamplerConfig(0.0))) for p in prompts]
    eng.run_until_idle()
    for i, t, n in zip(ids, want, sure):
        assert eng.result(i).generated_tokens[:n] == t[:n]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_replay_through_the_command_line(folders, tmp_path, dtype):
    """bin/trace_run as a child process on a Vubenex folder: up to four live requests, portions beside single tokens, a pool that
    holds less than all requests together, so that pages and state slots are used again."""
    import json
    import subprocess
    from pathlib import Path
    import numpy as np
    import traces
    root = Path(__file__).resolve().parent.parent
    cfg = CONFIGS["B"]
    rng = random.Random(4)
    requests = {f"q{i}": [rng.randrange(cfg["vocab"]) for _ in range(n)] for i, n in enumerate([50, 1, 33, 77, 40, 9])}
    steps = traces.mixed(requests, seed=3)
    out = tmp_path / "out"
    cmd = [str(root / "bin" / "trace_run"), "--model", str(folders["B"]), "--dtype", dtype, "--out", str(out), "--max-tokens", str(traces.peak_tokens(steps, 64))]
    proc = subprocess.Popen(cmd, stdin=subprocess.PIPE, stdout=subprocess.PIPE, stderr=subprocess.PIPE, text=True)
    try:
        for s in steps:
            proc.stdin.write(json.dumps(s) + "\n")
            proc.stdin.flush()
            line = proc.stdout.readline().strip()
            assert line == f"done {s['step']}", (line, proc.stderr.read() if proc.poll() is not None else "")
        proc.stdin.close()
        assert proc.wait(timeout=60) == 0, proc.stderr.read()
    finally:
        if proc.poll() is None:
            proc.kill()
    got = {}
    for step, rows in traces.wanted_positions(steps).items():
        data = np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(rows), cfg["vocab"])
        for key, row in zip(rows, data):
            got[key] = torch.from_numpy(row.copy())
    for rid, tokens in requests.items():
        mine = {p: row for (r, p), row in got.items() if r == rid}
        assert len(mine) > 0
        exact = plain_logits(folders, "B", tokens)
        if dtype == "float32":
            single = plain_logits(folders, "B", tokens, dtype=torch.float32)
            noise = max(relative_error(single[p], exact[p]) for p in mine)
            assert max(relative_error(row, exact[p]) for p, row in mine.items()) < 4 * noise + 1e-5
        else:
            rounded = plain_logits(folders, "B", tokens, rounded=True)
            assert_within_bfloat16_noise(mine, lambda p: exact[p], lambda p: rounded[p], f"replay {rid}")


def test_generation_from_the_command_line_on_random_weights():
    """bin/gi_generate on the shipped example configuration, random weights, greedy: runs, and twice the same."""
    import subprocess
    from pathlib import Path
    root = Path(__file__).resolve().parent.parent
    cmd = [str(root / "bin" / "gi_generate"), "--config", str(root / "configs" / "vubenex-small.json"), "--random-seed", "3", "--prompt-ids", "5 17 3 999 4",
           "--steps", "24", "--temperature", "0"]
    runs = [subprocess.run(cmd, capture_output=True, text=True, timeout=280) for _ in range(2)]
    assert all(r.returncode == 0 for r in runs), runs[0].stderr[-2000:]
    assert runs[0].stdout == runs[1].stdout and len(runs[0].stdout.split()) >= 20


def test_the_new_parts_serve_other_designs():
    """The fading memories under the ordinary pre-norm block and beside an attention, whose keys serve as values behind a rotation and whose output is
    gated channel by channel, on token rows with learned positions and no scale: built from specs alone, run under two cuts with
    equal bits and against a statement in the plain implementation's functions."""
    from geneinfer_amd.config.spec import (AttentionSpec, LayerSpec, LearnedPositionsSpec, LightningSpec, ModelSpec, RmsNormSpec, RotarySpec, RunEntry, SideBySideSpec, SwiGluSpec)
    from geneinfer_amd.engine import Runner
    from geneinfer_amd.engine.model import DecoderModel
    from geneinfer_amd.parts import model_tensor_needs
    from geneinfer_amd.weights import random_tensors
    d, eps = 32, 1e-5
    norm = lambda name: RmsNormSpec(d, eps, name)
    memory = LightningSpec(hidden_size=d, n_heads=2, key_dim=8, value_dim=12, decay=(0.9, 0.99), norm_eps=eps, q_proj="mq", k_proj="mk", v_proj="mv", gate_proj="mg",
                           out_norm="mn", o_proj="mo")
    attention = AttentionSpec(hidden_size=d, n_heads=2, n_kv_heads=1, head_dim=16, q_proj="q", k_proj="k", v_proj="", o_proj="o", position=RotarySpec(16, 100.0),
                              values_are_keys=True, output_gate="g", sink_score=0.5)
    mlp = SwiGluSpec(d, 48, "gate", "up", "down")
    layers = (LayerSpec(mixer=memory, feed_forward=mlp, mixer_norm=norm("n1"), feed_forward_norm=norm("n2")),
              LayerSpec(mixer=SideBySideSpec(d, (attention, memory), (0.5, 2.0)), feed_forward=mlp, mixer_norm=norm("n3"), feed_forward_norm=norm("n4")))
    spec = ModelSpec(architecture="test", vocab_size=90, hidden_size=d, max_positions=256, embedding="embed", final_norm=norm("nf"), lm_head="embed", layers=layers,
                     run_order=(RunEntry(0), RunEntry(1)), after_embedding=(LearnedPositionsSpec(d, 80, "pos"),))
    tensors = {k: v.to(DEV) for k, v in random_tensors(model_tensor_needs(spec), 3, torch.float32, 0.2).items()}
    model = DecoderModel(spec, tensors, torch.float32, DEV)
    tokens = list(range(3, 40))
    got = []
    for cuts in ([len(tokens)], [5, 2, 9, 1, 1, 3]):
        runner = Runner(model, page_size=4, max_tokens=256, max_requests=2)
        assert runner.max_positions == 80
        runner.open("r")
        got.append(feed(runner, "r", tokens, cuts))
    assert torch.equal(got[0], got[1])
    w = {k: v.double().cpu() for k, v in tensors.items()}
    T = len(tokens)
    mem = lambda h: P.lightning_mixer(h, dict(q=w["mq"], k=w["mk"], v=w["mv"], g=w["mg"], norm=w["mn"], o=w["mo"]), dict(heads=2, dim=8, vdim=12, decay=(0.9, 0.99)), eps)

    def turned(x):
        a = torch.arange(T, dtype=F64)[:, None] * torch.tensor([100.0 ** (-2 * i / 16) for i in range(8)], dtype=F64)
        c, s, u, v = torch.cos(a)[:, None], torch.sin(a)[:, None], x[..., :8], x[..., 8:]
        return torch.cat([u * c - v * s, v * c + u * s], dim=-1)

    def att(h):
        q, k = (h @ w["q"].T).reshape(T, 2, 16), (h @ w["k"].T).reshape(T, 1, 16)
        sc = torch.einsum("iad,jd->aij", turned(q), turned(k)[:, 0]) * 0.25
        sc = sc.masked_fill(~torch.tril(torch.ones(T, T, dtype=torch.bool)), float("-inf"))
        p = torch.softmax(torch.cat([torch.full((2, T, 1), 0.5, dtype=F64), sc], dim=-1), dim=-1)[..., 1:]
        return (torch.einsum("aij,jd->iad", p, k[:, 0]).reshape(T, 32) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T

    x = w["embed"][torch.tensor(tokens)] + w["pos"][:T]
    for mixer, na, nb in ((mem, "n1", "n2"), (lambda h: 0.5 * att(h) + 2.0 * mem(h), "n3", "n4")):
        x = x + mixer(P.rms_norm(x, w[na], eps))
        x = x + P.gated_feed_forward(P.rms_norm(x, w[nb], eps), w["gate"], w["up"], w["down"])
    assert relative_error(got[0], P.rms_norm(x, w["nf"], eps) @ w["embed"].T) < 2e-5
