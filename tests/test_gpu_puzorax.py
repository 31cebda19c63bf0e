"""The Puzorax design in the engine against the plain implementation (`plain_puzorax.py`): each kernel alone, then whole models of five
small configurations under every way of cutting the work into steps, and generation through the entry point and the scheduler.  In
float32 the engine's logits must not depend on the cutting at all (equal bits); in bfloat16 they must lie as close to the exact model
as rounding alone explains."""
import pytest
import torch

import plain_puzorax as P
from model_folders import assert_within_bfloat16_noise, relative_error
from puzorax_folders import CONFIGS, PAGE_SIZE, RANKS, random_weights, stored_weights, write_model

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


def _prompt(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("puzorax")
    out = {}
    for name, cfg in CONFIGS.items():
        write_model(root / name, cfg, RANKS[name], seed=29 + ord(name))
        out[name] = root / name
    return out


_plain_cache = {}


def plain_logits(folders, name, tokens, rounded=False, dtype=torch.float64):
    key = (name, tuple(tokens), rounded, dtype)
    if key not in _plain_cache:
        _plain_cache[key] = P.forward(CONFIGS[name], stored_weights(folders[name]), tokens, dtype, store=P.to_bfloat16_and_back if rounded else P.same)
    return _plain_cache[key]


def make_runner(folders, name, dtype, **kw):
    from geneinfer_amd.engine import Runner, load_model
    model = load_model(folders[name], dtype, DEV)
    kw.setdefault("page_size", PAGE_SIZE[name])
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


def _segs(seg_lens, slots, pos0):
    starts = [sum(seg_lens[:i]) for i in range(len(seg_lens))]
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
    row_slot = i32([s for s, m in zip(slots, seg_lens) for _ in range(m)])
    row_pos = i32([p + i for p, m in zip(pos0, seg_lens) for i in range(m)])
    return i32(starts), i32(seg_lens), row_slot, row_pos


# =============================================================================================== kernels alone
@pytest.mark.parametrize("rows, dim", [(3, 50), (5, 64), (7, 1028), (2, 2048), (9, 3072), (4, 6000), (2, 9000), (1, 1)])
def test_layer_norm_alone_behind_sums_and_on_a_selection_of_rows(rows, dim):
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(dim)
    x, add = torch.randn(rows, dim, generator=g) + 3, torch.randn(rows, dim, generator=g)
    w, b, v = 1 + 0.1 * torch.randn(dim, generator=g), torch.randn(dim, generator=g), torch.randn(dim, generator=g)
    dev = lambda t: t.to(DEV)
    for store in (torch.float32, torch.bfloat16):
        lw, lb, lv = w.to(store), b.to(store), v.to(store)
        out = torch.empty(rows, dim, device=DEV)
        for what, kw, sum_ in (("alone", {}, x), ("rows", dict(add=dev(add)), x + add), ("vector", dict(vector=dev(lv)), x + lv.float()),
                               ("both", dict(add=dev(add), vector=dev(lv)), x + add + lv.float())):
            dx = dev(x)
            ops.layernorm(dx, dev(lw), dev(lb), 1e-3, out, **kw)
            assert relative_error(out, P.layer_norm(sum_.double(), lw.double(), lb.double(), 1e-3)) < 3e-6, what
            assert relative_error(dx, sum_.double()) < 1e-6
            low = torch.empty(rows, dim, device=DEV, dtype=torch.bfloat16)
            ops.layernorm(dev(x), dev(lw), dev(lb), 1e-3, low, **kw)
            assert torch.equal(low, out.to(torch.bfloat16))
        dx = dev(x)
        ops.layernorm(dx, None, None, 0.0, None, add=dev(add), vector=dev(lv))
        assert relative_error(dx, (x + add + lv.float()).double()) < 1e-6
        ops.layernorm(dev(x), dev(lw), dev(lb), 1e-3, out)
        some = torch.tensor([rows - 1, 0, rows // 2], dtype=torch.int32, device=DEV)
        picked = torch.empty(3, dim, device=DEV)
        ops.layernorm(dev(x), dev(lw), dev(lb), 1e-3, picked, rows=some)
        assert torch.equal(picked, out[some.long()])


@pytest.mark.parametrize("buckets, mul_prev, mul_cur, dim", [(97, 31, 5, 64), (1, 3, 4, 10), (50021, 2147483647, 2147483629, 300), (7, 0, 1, 12), (1000, 1000, 77, 33)])
def test_rows_of_pairs_under_every_cut_and_on_slots_used_again(buckets, mul_prev, mul_cur, dim):
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(buckets)
    vocab = 100000
    table, pairs = torch.randn(vocab, dim, generator=g).to(torch.bfloat16), torch.randn(buckets + 1, dim, generator=g).to(torch.bfloat16)
    d_table, d_pairs = table.to(DEV), pairs.to(DEV)
    seqs = [torch.randint(0, vocab, (n,), generator=g).tolist() for n in (1, 40, 23)]
    want = [P.embedding(s, table.float(), pairs.float(), mul_prev, mul_cur) for s in seqs]
    last = torch.zeros(5, 1, dtype=torch.int32, device=DEV)

    def run(parts):                                     # [(sequence, slot, from, to)]
        lens = [b - a for _, _, a, b in parts]
        seg_start, seg_len, slots, pos = _segs(lens, [s for _, s, _, _ in parts], [a for _, _, a, _ in parts])
        tokens = torch.tensor([t for q, _, a, b in parts for t in seqs[q][a:b]], dtype=torch.int32, device=DEV)
        x, keep = torch.empty(sum(lens), dim, device=DEV), torch.empty(sum(lens), dim, device=DEV)
        ops.embed_pairs(d_table, d_pairs, tokens, pos, slots, (seg_start, seg_len), last, mul_prev, mul_cur, x, keep)
        assert torch.equal(x, keep)
        assert torch.equal(x.cpu(), torch.cat([want[q][a:b] for q, _, a, b in parts]))

    run([(0, 3, 0, 1), (1, 1, 0, 40), (2, 0, 0, 23)])
    run([(1, 2, 0, 2), (2, 1, 0, 1)])                  # slot 1 again, from position 0: what it held is not read
    run([(2, 1, 1, 3), (1, 2, 2, 3)])
    run([(1, 2, 3, 4)])
    run([(1, 2, 4, 21), (2, 1, 3, 4), (0, 0, 0, 1)])
    run([(2, 1, 4, 6)])
    run([(2, 1, 6, 23), (1, 2, 21, 40)])


@pytest.mark.parametrize("heads, kv, dk, dv, taps", [(4, 2, 16, 24, 4), (3, 3, 64, 64, 2), (2, 1, 130, 10, 5), (1, 1, 7, 201, 1), (5, 5, 3, 5, 3), (2, 2, 300, 6, 8), (2, 1, 100, 33, 13)])
def test_delta_rule_with_a_decay_per_channel(heads, kv, dk, dv, taps):
    """Two requests of unequal length in one step; then the longer one again from a fresh slot in steps down to one and two rows (the
    steps of one row by the kernel without staging): the memories and the convolutions' tails carry, and the bits do not change.  The
    decays of some channels are close to one, so that what the first rows wrote is still there at the end; others forget at once."""
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(dk + taps)
    n_conv = 2 * kv * dk + heads * dv
    lens, cols = [29, 90], n_conv + heads + 3
    conv_off, b_off = 3, 3 + n_conv
    proj, pre = torch.randn(sum(lens), cols, generator=g), torch.randn(sum(lens), heads * dk, generator=g)
    w_taps = 0.6 * torch.randn(n_conv, taps, generator=g)
    a_log, dt_bias = -1.0 + 0.8 * torch.randn(heads, generator=g), 0.5 * torch.randn(heads * dk, generator=g)
    dt_bias[::3] = -9.0
    dt_bias[1::7] = 30.0

    def plain(rows):
        x = proj[rows].double()
        y = P.short_conv_silu(x[:, conv_off:conv_off + n_conv], w_taps.double())
        unit = lambda z: z / torch.sqrt((z * z).sum(-1, keepdim=True) + 1e-6)
        q, k = unit(y[:, :kv * dk].view(-1, kv, dk)) * dk ** -0.5, unit(y[:, kv * dk:2 * kv * dk].view(-1, kv, dk))
        v = y[:, 2 * kv * dk:].view(-1, heads, dv)
        decay = P.channel_decays(pre[rows].double(), a_log.double(), dt_bias.double(), heads, dk)
        beta = torch.sigmoid(x[:, b_off:b_off + heads])
        return torch.cat([P.channel_delta_rule(q[:, h // (heads // kv)], k[:, h // (heads // kv)], v[:, h], beta[:, h], decay[:, h]) for h in range(heads)], dim=-1)

    want = torch.cat([plain(slice(0, lens[0])), plain(slice(lens[0], None))])
    state = torch.zeros(5, ops.delta_state_floats(heads, kv, dk, dv, taps) + 3, device=DEV)
    dev = lambda t: t.to(DEV)

    def run(rows, pre_rows, seg_lens, slots, pos0):
        n = rows.shape[0]
        seg_start, seg_len, row_slot, row_pos = _segs(seg_lens, slots, pos0)
        qkv, gates, out = torch.empty(n, n_conv, device=DEV), torch.empty(n, heads * dk + heads, device=DEV), torch.empty(n, heads * dv, device=DEV)
        rows, single = dev(rows), max(seg_lens) == 1
        ops.delta_prepare(rows, conv_off, dev(pre_rows), b_off, dev(w_taps), dev(a_log), dev(dt_bias), row_slot, row_pos, state, qkv, gates, heads, kv, dk, dv, dk ** -0.5,
                          single_rows=single, channel=True)
        if not single:
            ops.delta_tail(rows, conv_off, taps, seg_start, seg_len, row_slot, state, heads, kv, dk, dv)
        ops.delta_scan(qkv, gates, seg_start, seg_len, row_slot, state, out, heads, kv, dk, dv, channel=True, single_rows=single)
        return out.cpu().double()

    got = run(proj, pre, lens, [2, 0], [0, 0])
    assert relative_error(got, want) < 3e-5
    assert relative_error(got[lens[0]:][-5:], want[lens[0]:][-5:]) < 3e-5
    second, second_pre = proj[lens[0]:], pre[lens[0]:]
    cuts, pieces, at = [2, 1, 1, 40, 1, 2, 3, 38, 2], [], 0
    for c in cuts:
        pieces.append(run(second[at:at + c], second_pre[at:at + c], [c], [4], [at]))
        at += c
    assert at == lens[1] and torch.equal(torch.cat(pieces), got[lens[0]:])
    state[1], state[3] = state[2], state[4]              # two requests that both go on, side by side in one step, each from its own slot
    more, more_pre = torch.randn(11, cols, generator=g), torch.randn(11, heads * dk, generator=g)
    both = run(more, more_pre, [4, 7], [1, 3], [lens[0], lens[1]])
    alone = torch.cat([run(more[:4], more_pre[:4], [4], [2], [lens[0]]), run(more[4:], more_pre[4:], [7], [4], [lens[1]])])
    assert torch.equal(both, alone)


@pytest.mark.parametrize("channel", [False, True])
def test_single_rows_take_the_memories_on_as_runs_of_rows_do(channel):
    """Both forms of the rule, several requests of one row each: the kernel without staging gives the bits of the one with it."""
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(7)
    heads, kv, dk, dv, n = 4, 2, 40, 30, 6
    n_gates = heads * (dk if channel else 1) + heads
    qkv, gates = torch.randn(n, 2 * kv * dk + heads * dv, generator=g).to(DEV), torch.rand(n, n_gates, generator=g).to(DEV)
    seg_start, seg_len, row_slot, _ = _segs([1] * n, [5, 0, 3, 1, 7, 2], [9] * n)
    first = torch.randn(8, ops.delta_memory_floats(heads, dk, dv), generator=g).to(DEV)
    states, outs = [first.clone(), first.clone()], [torch.empty(n, heads * dv, device=DEV) for _ in range(2)]
    for s, o, single in zip(states, outs, (False, True)):
        ops.delta_scan(qkv, gates, seg_start, seg_len, row_slot, s, o, heads, kv, dk, dv, channel=channel, single_rows=single)
    assert torch.equal(*outs) and torch.equal(*states)
    assert torch.equal(states[0][4], first[4]) and not torch.equal(states[0][5], first[5])


@pytest.mark.parametrize("ra, rg, heads, dk, dv", [(24, 40, 3, 20, 30), (1, 7, 2, 64, 8), (130, 64, 4, 100, 70)])
def test_products_behind_narrow_middles_made_inside_the_kernels_that_need_them(ra, rg, heads, dk, dv):
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(ra)
    n, kv = 5, heads
    n_conv = 2 * kv * dk + heads * dv
    proj = torch.randn(n, n_conv + ra + rg + heads, generator=g)
    wa, wg = (torch.randn(heads * dk, ra, generator=g) / ra ** 0.5).to(torch.bfloat16), (torch.randn(heads * dv, rg, generator=g) / rg ** 0.5).to(torch.bfloat16)
    a_log, dt_bias, taps = torch.randn(heads, generator=g), torch.randn(heads * dk, generator=g), torch.randn(n_conv, 1, generator=g)
    low_a, low_g = proj[:, n_conv:n_conv + ra], proj[:, n_conv + ra:n_conv + ra + rg]
    dev = lambda t: t.to(DEV)
    d_proj = dev(proj)
    seg_start, seg_len, row_slot, row_pos = _segs([1] * n, list(range(n)), [4] * n)
    state = torch.zeros(n, ops.delta_state_floats(heads, kv, dk, dv, 1), device=DEV)
    qkv, gates = torch.empty(n, n_conv, device=DEV), torch.empty(n, heads * dk + heads, device=DEV)
    ops.delta_prepare(d_proj, 0, None, n_conv + ra + rg, dev(taps), dev(a_log), dev(dt_bias), row_slot, row_pos, state, qkv, gates, heads, kv, dk, dv, 1.0, True, True,
                      (d_proj[:, n_conv:n_conv + ra], dev(wa)))
    pre = low_a.to(torch.bfloat16).double() @ wa.double().T
    want = P.channel_decays(pre, a_log.double(), dt_bias.double(), heads, dk).reshape(n, -1)
    assert relative_error(gates[:, :heads * dk], want) < 1e-5
    assert relative_error(gates[:, heads * dk:], torch.sigmoid(proj[:, n_conv + ra + rg:].double())) < 1e-6
    o, weight = torch.randn(n, heads * dv, generator=g), 1 + 0.1 * torch.randn(dv, generator=g)
    out = torch.empty(n, heads * dv, device=DEV)
    ops.head_norm_gate(dev(o), None, dev(weight), 1e-4, out, heads, dv, gate_activation="sigmoid", gate_up=(d_proj[:, n_conv + ra:n_conv + ra + rg], dev(wg)))
    gate = torch.sigmoid(low_g.to(torch.bfloat16).double() @ wg.double().T)
    want = P.rms_norm(o.double().view(n, heads, dv), weight.double(), 1e-4).reshape(n, -1) * gate
    assert relative_error(out, want) < 1e-5


def _paged(T, page, n_numbers, dtype, seed):
    """Pages for one request of T positions in slot 1, in a shuffled order, and its table."""
    n_pages = -(-T // page)
    order = torch.randperm(n_pages + 3, generator=torch.Generator().manual_seed(seed))[:n_pages]
    table = torch.full((3, n_pages + 2), -1, dtype=torch.int32)
    table[1, :n_pages] = order.to(torch.int32)
    cache = torch.zeros(n_pages + 3, page * n_numbers, dtype=dtype, device=DEV)
    return cache, table.to(DEV)


def _ctx(T, pos0=0, slot=1, dtype=torch.float32):
    from geneinfer_amd.parts import StepContext
    pos = torch.arange(pos0, pos0 + T, dtype=torch.int32, device=DEV)
    slots = torch.full((T,), slot, dtype=torch.int32, device=DEV)
    return StepContext(n_rows=T, dtype=dtype, device=torch.device(DEV), tokens=slots, row_pos=pos, row_slot=slots, seg_slot=[slot], seg_start=[0],
                       seg_len=[T], seg_pos0=[pos0])


LATENT = dict(heads=3, dim=12, rot_dim=6, vdim=7, kv_rank=18, scale=0.3)
LATENT_BIG = dict(heads=20, dim=16, rot_dim=32, vdim=24, kv_rank=64, scale=0.2)


@pytest.mark.parametrize("dtype, m, page", [("float32", LATENT, 4), ("bfloat16", LATENT_BIG, 16)])
@pytest.mark.parametrize("T, window, far, alone", [(200, 50, 149, 0), (200, 50, 150, 1), (45, 16, 29, 1), (45, 16, 28, 0), (300, 290, 11, 2), (300, 290, 10, 1), (70, 1, 69, 1), (70, 1, 68, 0),
                                                   (33, 64, 0, 1), (33, 64, 15, 0), (34, 64, 16, 1), (2, 5, 0, 1), (1, 5, 0, 0)])
def test_the_latent_attention_part_with_one_key_that_stands_out(T, window, far, alone, dtype, m, page):
    """The part itself on given rows (the last `alone` of them decoded one by one): the last row's query points at the key of position
    `far`, scaled up so that, if the window lets it be seen, it takes nearly all the weight: just inside, just outside, and far back.
    The other rows' weight is shared with a sink per head of which one is large."""
    from geneinfer_amd.config import LatentAttentionSpec, RotarySpec
    from geneinfer_amd.parts import LayerCache, mixer_class
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    hidden, eps = 64, 1e-5
    store = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    cfg = dict(m, rot=dict(dims=r, base=40.0), mask=dict(size=window))
    g = torch.Generator().manual_seed(T + far)
    rnd = lambda *s: (torch.randn(*s, generator=g) * 0.3).to(store).float()
    w = {"q": rnd(H * (d + r), hidden), "dkv": rnd(rank + r, hidden), "dkv.norm": 1 + rnd(rank), "uk": rnd(H * d, rank), "uv": rnd(H * dv, rank), "o": rnd(hidden, H * dv),
         "g": rnd(H * dv, hidden), "sink": torch.tensor([3.0, -1.0, 0.5] * H)[:H]}
    w["dkv.norm"] = w["dkv.norm"].to(store).float()
    h = torch.randn(T, hidden, generator=g).to(store).float()
    # input channel 0 speaks of nothing but latent channel 0, which only position `far` has; input channel 1 of every head's first query
    # channel, which only the last row has and which meets latent channel 0 alone
    h[:, :2] = 0.0
    for name in ("q", "dkv", "g"):
        w[name][:, :2] = 0.0
    q_heads, uk_heads = w["q"].view(H, d + r, hidden), w["uk"].view(H, d, rank)
    w["dkv"][0], q_heads[:, 0], uk_heads[:, 0] = 0.0, 0.0, 0.0
    w["dkv"][0, 0], uk_heads[:, 0, 0], q_heads[:, 0, 1] = 3.0, 1.0, 2.0 / m["scale"]
    if far < T - 1:
        h[far, 0], h[T - 1, 1] = 6.0, 10.0
    want = P.latent_attention(h.double(), {k: v.double() for k, v in w.items()}, cfg, eps)
    if far < T - 1:                                       # the premise: moving position `far` moves the last row exactly when it is seen
        other = h.double().clone()
        other[far] = -other[far]
        moved = P.latent_attention(other, {k: v.double() for k, v in w.items()}, cfg, eps)
        assert (relative_error(moved[T - 1], want[T - 1]) > 0.3) if T - 1 - far < window else torch.equal(moved[T - 1], want[T - 1])
    spec = LatentAttentionSpec(hidden_size=hidden, n_heads=H, head_dim=d, rotary_dim=r, value_dim=dv, q_rank=0, kv_rank=rank, scale=m["scale"], norm_eps=eps, dq_proj="", dq_norm="",
                               uq_proj="", q_proj="q", dkv_proj="dkv", dkv_norm="dkv.norm", uk_proj="uk", uv_proj="uv", o_proj="o", position=RotarySpec(r, 40.0), window=window,
                               sinks="sink", output_gate="g")
    part = mixer_class(spec)(spec, {k: v.to(store).to(DEV) for k, v in w.items()}, store, torch.device(DEV))
    kv, table = _paged(T, page, 2 * rank + r, store, seed=far)
    cache = LayerCache(kv=kv, table=table, page_size=page)
    out, at = torch.zeros(T, hidden, device=DEV), 0
    for n in ([T - alone] if T > alone else []) + [1] * min(alone, T):
        rows = out[at:at + n]
        part.forward(h[at:at + n].to(store).to(DEV), rows, _ctx(n, at, dtype=store), cache)
        at += n
    tol = 3e-5 if dtype == "float32" else 3e-2
    assert relative_error(out, want) < tol and relative_error(out[T - 1], want[T - 1]) < 2 * tol


@pytest.mark.parametrize("H, kd, vd, window, lens, pos0", [(20, 152, 136, 44, [1, 1, 1], [700, 43, 0]), (8, 80, 64, None, [130, 1], [0, 300]), (32, 288, 256, 100, [70], [50]),
                                                          (3, 24, 16, 17, [33, 2, 1], [15, 16, 17]), (16, 96, 64, 1, [20], [0]), (16, 576, 512, 48, [100, 1], [30, 200]),
                                                          (8, 288, 256, 300, [129, 200], [77, 0]), (130, 32, 16, 20, [80], [3])])
def test_matrix_core_attention_over_latent_pages_with_sinks(H, kd, vd, window, lens, pos0):
    """Single rows whose context is shared out over several waves, and portions of prompts, at other positions each.  One key just
    inside every row's window stands out for half of the heads; for others the sink takes nearly all the weight, or next to none."""
    from geneinfer_amd.kernels import ops
    from geneinfer_amd.parts import StepContext
    g = torch.Generator().manual_seed(H + kd)
    page, scale = 16, 0.2
    total = [p + n for p, n in zip(pos0, lens)]
    n_pages = sum(-(-t // page) for t in total)
    order = torch.randperm(n_pages + 2, generator=g).tolist()
    table = torch.full((len(lens) + 1, max(-(-t // page) for t in total) + 1), -1, dtype=torch.int32)
    cache = torch.zeros(n_pages + 2, page * (kd + vd), dtype=torch.bfloat16)
    keys = []
    for s, t in enumerate(total):
        k = torch.randn(t, kd, generator=g).to(torch.bfloat16)
        keys.append(k)
        for i in range(-(-t // page)):
            pg = order.pop()
            table[s, i] = pg
            block = k[i * page:(i + 1) * page]
            cache[pg, :block.shape[0] * kd] = block.reshape(-1)
            values = torch.zeros(vd, page, dtype=torch.bfloat16)
            values[:, :block.shape[0]] = block[:, :vd].T
            cache[pg, page * kd:] = values.reshape(-1)
    sinks = 2 * torch.randn(H, generator=g)
    sinks[1::3], sinks[2::5] = 12.0, -30.0
    q = torch.randn(sum(lens), H * kd, generator=g)
    row, want = 0, []
    for s, (p0, n) in enumerate(zip(pos0, lens)):
        kf = keys[s].double()
        for i in range(n):
            lo = 0 if window is None else max(0, p0 + i - window + 1)
            q.view(-1, H, kd)[row + i, ::2, :8] = 4.0 * kf[lo, :8] / kf[lo, :8].norm()
        qb = q[row:row + n].to(torch.bfloat16).double().view(n, H, kd)
        scores = torch.einsum("thd,sd->hts", qb, kf) * scale
        i_, j_ = torch.arange(p0, p0 + n)[:, None], torch.arange(total[s])[None, :]
        seen = (j_ <= i_) & ((i_ - j_ < window) if window is not None else True)
        more = torch.cat([scores.masked_fill(~seen[None], float("-inf")), sinks.double()[:, None, None].expand(H, n, 1)], -1)
        want.append(torch.einsum("hts,sd->thd", torch.softmax(more, -1)[..., :-1], kf[:, :vd]).reshape(n, H * vd))
        row += n
    want = torch.cat(want)
    T = sum(lens)
    starts = [sum(lens[:i]) for i in range(len(lens))]
    _, _, slots, pos = _segs(lens, list(range(len(lens))), pos0)
    ctx = StepContext(n_rows=T, dtype=torch.bfloat16, device=torch.device(DEV), tokens=slots, row_pos=pos, row_slot=slots, seg_slot=list(range(len(lens))),
                      seg_start=starts, seg_len=list(lens), seg_pos0=list(pos0))
    out, exact = torch.empty(T, H * vd, dtype=torch.bfloat16, device=DEV), torch.empty(T, H * vd, dtype=torch.bfloat16, device=DEV)
    ops.latent_attention_bf16(q.to(DEV, torch.bfloat16), cache.to(DEV), out, ctx, table.to(DEV), H, kd, vd, page, window, scale, sinks.to(DEV))
    assert relative_error(out, want) < 1.5e-2                                   # (probabilities and outputs are kept in bfloat16)
    ops.attention_general(q.to(DEV, torch.bfloat16), cache.to(DEV), exact, ctx, table.to(DEV), H, 1, kd, page_size=page, value_dim=vd, window=window, scale=scale, sinks=sinks.to(DEV))
    assert relative_error(exact, want) < 6e-3
    for h in range(min(H, 6)):                                                  # head by head: a sink that is left out shows
        a, b = out.view(T, H, vd)[:, h], want.view(T, H, vd)[:, h]
        assert relative_error(a, b) < 2.5e-2, f"head {h}"


@pytest.mark.parametrize("rows, H, k, n", [(1, 8, 32, 128), (37, 3, 72, 40), (300, 32, 64, 256), (5, 1, 8, 7)])
def test_every_head_s_product_with_a_gate_per_channel(rows, H, k, n):
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(rows + k)
    a, w = torch.randn(rows, H * k, generator=g).to(torch.bfloat16), torch.randn(H, n, k, generator=g).to(torch.bfloat16)
    wide = 2 * torch.randn(rows, H * n + 9, generator=g)
    gate = wide[:, 5:5 + H * n]
    want = torch.einsum("thk,hnk->thn", a.double().view(rows, H, k), w.double()).reshape(rows, -1) * torch.sigmoid(gate.double())
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 5e-3)):
        out = torch.empty(rows, H * n, dtype=dtype, device=DEV)
        assert ops.heads_product(a.to(DEV), w.to(DEV), out, H, channel_gate=wide.to(DEV)[:, 5:5 + H * n])
        assert relative_error(out, want) < tol


@pytest.mark.parametrize("experts, identity, top", [(5, 2, 2), (16, 0, 1), (3, 1, 4), (64, 8, 8), (130, 30, 4), (1, 1, 1), (12, 2, 3)])
def test_the_router_s_choice_with_a_correction(experts, identity, top):
    """The correction chooses and does not weigh: it is large enough to make experts of small scores chosen."""
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(experts)
    n = experts + identity
    logits, corr = 2 * torch.randn(50, n, generator=g), 0.5 * torch.randn(n, generator=g)
    for score, renorm, scale in (("softmax", True, 2.5), ("softmax", False, 0.7), ("sigmoid", True, 1.0)):
        z = logits.double()
        s = torch.softmax(z, -1) if score == "softmax" else torch.sigmoid(z)
        order = torch.sort(s + corr.double(), dim=-1, descending=True, stable=True).indices[:, :top]
        want = torch.gather(s, 1, order)
        if renorm:
            want = want / (want.sum(-1, keepdim=True) + 1e-20)
        ids, weights = torch.empty(50, top, dtype=torch.int32, device=DEV), torch.empty(50, top, device=DEV)
        ops.route_top(logits.to(DEV), top, ids, weights, score, renorm, floor=1e-20, correction=corr.to(DEV), scale=scale)
        assert torch.equal(ids.cpu().long(), order) and relative_error(weights, scale * want) < 2e-6
    h, router = torch.randn(50, 72, generator=g), torch.randn(n, 72, generator=g)
    ids2, weights2, kept = torch.empty_like(ids), torch.empty_like(weights), torch.empty(50, n, device=DEV)
    ops.route_rows(h.to(DEV), router.to(DEV), top, ids2, weights2, "softmax", True, logits=kept, correction=corr.to(DEV), scale=2.0)
    assert relative_error(kept, h.double() @ router.double().T) < 1e-6
    ops.route_top(kept, top, ids, weights, "softmax", True, correction=corr.to(DEV), scale=2.0)
    assert torch.equal(ids, ids2) and torch.equal(weights, weights2)


@pytest.mark.parametrize("rows, d, ff, E, identity, top, dtype", [(7, 50, 10, 3, 2, 3, "float32"), (1, 64, 24, 5, 1, 2, "float32"), (33, 128, 64, 8, 2, 3, "bfloat16"),
                                                                  (150, 256, 96, 4, 1, 2, "bfloat16"), (300, 128, 128, 16, 4, 4, "bfloat16"), (2, 128, 64, 4, 1, 2, "bfloat16"),
                                                                  (700, 192, 320, 5, 3, 1, "bfloat16"), (20, 128, 64, 1, 5, 2, "bfloat16"), (9, 2112, 64, 3, 1, 2, "bfloat16"),
                                                                  (3, 72, 48, 6, 1, 3, "bfloat16"), (30, 200, 80, 2, 1, 2, "bfloat16"), (1, 1000, 1040, 40, 0, 8, "bfloat16"),
                                                                  (21, 136, 16, 1, 1, 2, "bfloat16")])
def test_experts_that_return_their_input_and_the_norm_behind_them(rows, d, ff, E, identity, top, dtype):
    from geneinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(rows + d)
    store = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    r = lambda *s: (0.3 * torch.randn(*s, generator=g)).to(store)
    h, n = r(rows, d) * 3, E + identity
    w = {f"e{e}.{k}": r(*s) for e in range(E) for k, s in (("gate", (ff, d)), ("up", (ff, d)), ("down", (d, ff)))}
    w["router"], w["correction"] = (4.0 / d ** 0.5 * torch.randn(n, d, generator=g)).to(store), 0.1 * torch.randn(n, generator=g)
    m = dict(router=dict(experts=E, identity=identity, top=top, scale=1.7))
    rounding = P.to_bfloat16_and_back if dtype == "bfloat16" else P.same
    want = P.experts(h.double(), {k: v.double() for k, v in w.items()}, m, rounding)
    ids = P.route(h.double(), w["router"].double(), w["correction"].double(), top, 1.7)[0]
    assert rows < 5 or ((ids >= E).any() and (ids < E).any())
    dev = lambda t: t.to(DEV)
    stack = lambda k: dev(torch.stack([w[f"e{e}.{k}"] for e in range(E)])).contiguous()
    wg, wu, wd = stack("gate"), stack("up"), stack("down")
    if dtype == "bfloat16":
        wg, wu = torch.stack([ops.interleave_gate_up(wg[e], wu[e]) for e in range(E)]).contiguous(), None
    ids, weights = torch.empty(rows, top, dtype=torch.int32, device=DEV), torch.empty(rows, top, device=DEV)
    ops.route_rows(dev(h), dev(w["router"]), top, ids, weights, "softmax", True, floor=1e-20, correction=dev(w["correction"]), scale=1.7)
    tol = 2e-2 if dtype == "bfloat16" else 3e-5
    start = torch.randn(rows, d, generator=g)
    x = dev(start)
    assert ops.routed_experts(dev(h), wg, wu, wd, ids, weights, x, weigh="output") is None
    assert relative_error(x - dev(start), want) < tol
    y = torch.full((rows, d), 7.0, device=DEV)
    ops.routed_experts(dev(h), wg, wu, wd, ids, weights, y, accumulate=False, weigh="output")
    assert relative_error(y, want) < tol
    norm_w, norm_b = dev(1 + r(d)), dev(r(d))
    z = dev(start)
    ready = ops.routed_experts(dev(h), wg, wu, wd, ids, weights, z, weigh="output", then=(norm_w, norm_b, 1e-5))
    assert relative_error(z, x) < 1e-6
    many = rows * top >= ops.EXPERTS_GROUPED_FROM and ops.experts_grouped_supported(dev(h), wg, wu, wd)
    few = rows * top <= ops.EXPERTS_FEW_ITEMS and ops.experts_few_supported(dev(h), wg, wu, wd)
    assert (ready is not None) == (many or few)
    if ready is not None:
        ln = ops.layernorm(z.clone(), norm_w, norm_b, 1e-5, torch.empty(rows, d, device=DEV))
        assert relative_error(ready, ln) < 4e-3


# =============================================================================================== whole models
def _portions(n, sizes=(7, 2, 5, 3, 2, 11, 1, 4, 2, 19)):
    out, i = [], 0
    while sum(out) + sizes[i % len(sizes)] <= n:
        out.append(sizes[i % len(sizes)])
        i += 1
    return out


CUTS = {"whole": lambda n: [n], "singly": lambda n: [], "most then singly": lambda n: [n - 9], "portions": _portions, "twos": lambda n: [2] * (n // 2)}


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_residual_stream_after_every_layer_run(folders, name):
    """Layer by layer, walks included: the first difference names the layer."""
    cfg, tokens = CONFIGS[name], _prompt(CONFIGS[name], 21, 3)
    want = []
    P.forward(cfg, stored_weights(folders[name]), tokens, layer_outputs=want)
    runner = make_runner(folders, name, "float32")
    runner.open("r")
    last = {}
    runner.model.set_trace(lambda tag, i, rows: last.__setitem__(i, rows.float().cpu()) if tag == "ffn_out" else None)
    try:
        feed(runner, "r", tokens, [len(tokens)])
    finally:
        runner.model.set_trace(None)
    got = [last[i] for i in sorted(last)]
    assert len(got) == len(want) == len(P.layer_runs(cfg))
    for i, (g, w) in enumerate(zip(got, want)):
        assert relative_error(g, w) < 2e-5, f"{name}: the stream differs behind layer run {i} (layer {P.layer_runs(cfg)[i][0]})"


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
    tokens = _prompt(CONFIGS[name], 90, 6)
    runner = make_runner(folders, name, "bfloat16")
    for what in ("whole", "portions", "most then singly", "twos"):
        runner.open(what)
        got = feed(runner, what, tokens, CUTS[what](len(tokens)))
        runner.close(what)
        check_against_plain(folders, name, "bfloat16", tokens, got, f"{name} {what}")


@pytest.mark.parametrize("name, dtype", [("A", "float32"), ("B", "float32"), ("C", "float32"), ("D", "float32"), ("E", "float32"), ("A", "bfloat16"), ("B", "bfloat16"), ("E", "bfloat16")])
def test_mixed_batches_on_a_pool_that_is_used_again(folders, name, dtype):
    """Up to four live requests, portions of some beside single tokens of others, through a pool that holds less than all requests
    together and four state slots: pages and slots are freed and used again.  Every request's logits against itself alone."""
    import random
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


@pytest.mark.parametrize("name, dtype", [("B", "bfloat16"), ("C", "float32"), ("B", "float32"), ("A", "float32")])
def test_long_portions_beside_single_rows(folders, name, dtype):
    """Steps that hold portions of a hundred rows and more of some requests (the kernels that take the rows of prompts tile by tile)
    beside single rows and short portions of others, every request at another position."""
    from geneinfer_amd.engine import StepEntry
    cfg = CONFIGS[name]
    tokens = {r: _prompt(cfg, n, 70 + n) for r, n in (("a", 330), ("b", 150), ("c", 171), ("d", 40))}
    schedule = [[("a", 100), ("c", 70)], [("a", 130), ("b", 1), ("c", 1)], [("b", 140), ("a", 1), ("c", 99), ("d", 3)], [("a", 99), ("b", 2), ("c", 1), ("d", 37)], [("b", 7)]]
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


def test_long_decoding_carries_state_and_passes_windows(folders):
    """A short prompt and 300 tokens decoded one by one through the captured decode step: the memories, the convolutions' tails and the
    last token carry in every walk's own slot, and every window passes over decoded tokens only."""
    tokens = _prompt(CONFIGS["A"], 312, 9)
    for dtype in ("float32", "bfloat16"):
        runner = make_runner(folders, "A", dtype)
        runner.open("r")
        got = feed(runner, "r", tokens, [12])
        assert runner.steps_replayed > 250
        check_against_plain(folders, "A", dtype, tokens, got, f"A decoding ({dtype})")


def test_a_state_that_is_lost_or_a_walk_that_shares_one_shows(folders, tmp_path):
    """Weights made so that a fault shows: the memories hardly decay, so the last logits rest on what the first tokens left in every
    walk's state."""
    cfg, w = CONFIGS["D"], random_weights(CONFIGS["D"], RANKS["D"], 77)
    for i in range(len(cfg["layers"])):
        w[f"l{i}.mix.A_log"] = torch.full_like(w[f"l{i}.mix.A_log"], -8.0)
        w[f"l{i}.mix.b"] = 0.5 * w[f"l{i}.mix.b"]
    write_model(tmp_path / "m", cfg, weights=w)
    from geneinfer_amd.engine import Runner, load_model
    tokens = _prompt(cfg, 150, 4)
    stored = stored_weights(tmp_path / "m")
    want = P.forward(cfg, stored, tokens)
    without = P.forward(cfg, stored, tokens[60:])                            # the premise: the first tokens matter at the end
    assert relative_error(without[-1], want[-1]) > 0.01
    runner = Runner(load_model(tmp_path / "m", "float32", DEV), page_size=4, max_tokens=512, max_requests=2)
    for what, cuts in (("whole", [150]), ("cut", [40, 2, 70]), ("singly", [3])):
        runner.open(what)
        got = feed(runner, what, tokens, cuts)
        runner.close(what)
        assert relative_error(got, want) < 5e-5, what


def test_layers_in_another_order_and_a_walk_elsewhere(folders, tmp_path):
    import copy
    cfg = copy.deepcopy(CONFIGS["A"])
    cfg["layers"] = [cfg["layers"][i] for i in (2, 0, 3, 1)]
    cfg["loop"] = dict(start=2, stop=4, times=3)
    write_model(tmp_path / "m", cfg, (9, 2), seed=4)
    from geneinfer_amd.engine import Runner, load_model
    tokens = _prompt(cfg, 40, 2)
    want = P.forward(cfg, stored_weights(tmp_path / "m"), tokens)
    runner = Runner(load_model(tmp_path / "m", "float32", DEV), page_size=8, max_tokens=256, max_requests=2)
    runner.open("r")
    got = feed(runner, "r", tokens, [13, 2])
    assert relative_error(got, want) < 5e-5


def test_a_pass_that_fails_leaves_the_last_token_and_the_memories_as_they_were(folders, monkeypatch):
    from geneinfer_amd.engine import StepEntry
    runner = make_runner(folders, "A", "float32", use_graphs=False)
    tokens = _prompt(CONFIGS["A"], 30, 1)
    runner.open("r")
    want = feed(runner, "r", tokens, [20])
    runner.close("r")
    runner.open("r")
    got = [runner.step([StepEntry("r", tokens[:20], tuple(range(20)))]).cpu()]
    block = runner.model.layers[3]

    def fails(*a, **k):
        raise RuntimeError("on purpose")
    with monkeypatch.context() as patch:
        patch.setattr(block, "forward", fails)
        with pytest.raises(RuntimeError):
            runner.step([StepEntry("r", tokens[20:25], (4,))])
    got.append(runner.step([StepEntry("r", tokens[20:], tuple(range(10)))]).cpu())
    assert torch.equal(torch.cat(got), want)


# =============================================================================================== entry points
@pytest.mark.parametrize("name", ["A", "D"])
def test_greedy_generation_through_the_entry_point_and_the_scheduler(folders, name):
    """Greedy tokens of several prompts, one by one through `LLM.generate` and together through the scheduler (more requests than
    it runs at once, prompts in portions), against the plain model's, as far as the plain model's two best logits are clearly apart."""
    import geneinfer_amd as gi
    from geneinfer_amd.engine import EngineConfig, EngineRequest
    from geneinfer_amd.sampling import SamplerConfig
    cfg, w = CONFIGS[name], stored_weights(folders[name])
    prompts = [_prompt(cfg, n, 30 + n) for n in (5, 23, 1, 40)]
    want, sure = [], []
    for p in prompts:
        tokens = P.greedy(cfg, w, p, 8)
        top2 = torch.topk(P.forward(cfg, w, p + tokens)[len(p) - 1:-1], 2, dim=-1).values
        clear = [bool(c) for c in (top2[:, 0] - top2[:, 1] > 1e-3)]
        want.append(tokens)
        sure.append(clear.index(False) if False in clear else len(clear))
    assert sum(sure) >= 24
    llm = gi.LLM(str(folders[name]), dtype="float32", page_size=PAGE_SIZE[name], max_tokens=512, max_running=2)
    assert type(llm.model.config).__name__ == "PuzoraxConfig"
    for p, t, n in zip(prompts, want, sure):
        assert llm.generate(p, steps=len(p) + 7, temperature=0.0).generated_tokens[:n] == t[:n]
    eng = llm.engine(EngineConfig(max_running=2, step_rows=16, prefill_chunk=6))
    ids = [eng.submit(EngineRequest(p, len(p) + 7, SamplerConfig(0.0))) for p in prompts]
    eng.run_until_idle()
    for i, t, n in zip(ids, want, sure):
        assert eng.result(i).generated_tokens[:n] == t[:n]


@pytest.mark.parametrize("dtype, mode", [("float32", "mixed"), ("bfloat16", "mixed"), ("float32", "portions")])
def test_replay_through_the_command_line(folders, tmp_path, dtype, mode):
    """bin/trace_run as a child process on a Puzorax folder: up to four live requests, portions beside single tokens, a pool that
    holds less than all requests together, so that pages and state slots are used again."""
    import json
    import random
    import subprocess
    from pathlib import Path
    import numpy as np
    import traces
    root = Path(__file__).resolve().parent.parent
    cfg = CONFIGS["B"]
    rng = random.Random(4)
    requests = {f"q{i}": [rng.randrange(cfg["vocab"]) for _ in range(n)] for i, n in enumerate([50, 1, 33, 77, 40, 9])}
    steps = traces.mixed(requests, seed=3) if mode == "mixed" else traces.portions(requests)
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
            assert_within_bfloat16_noise(mine, lambda p: exact[p], lambda p: rounded[p], f"replay {mode} {rid}")


def test_generation_from_the_command_line_on_random_weights():
    """bin/gi_generate on the shipped example configuration, random weights, greedy: runs, and twice the same."""
    import subprocess
    from pathlib import Path
    root = Path(__file__).resolve().parent.parent
    cmd = [str(root / "bin" / "gi_generate"), "--config", str(root / "configs" / "puzorax-small.json"), "--random-seed", "3", "--prompt-ids", "5 17 3 999 4",
           "--steps", "24", "--temperature", "0"]
    runs = [subprocess.run(cmd, capture_output=True, text=True, timeout=280) for _ in range(2)]
    assert all(r.returncode == 0 for r in runs), runs[0].stderr[-2000:]
    assert runs[0].stdout == runs[1].stdout and len(runs[0].stdout.split()) >= 20


def test_the_new_parts_serve_other_designs():
    """The parts are not Puzorax's own: a model put together by hand, a pre-norm layer (RMS norms) around latent attention with a query
    latent, neighbouring pairs and sinks, without gates, and a SiLU-gated feed-forward; then a layer with layer norms before both halves
    around the delta rule with one decay a head that comes through a narrow middle and a SiLU gate that does not, and experts with a
    correction beside a shared one, entered through a vector alone; against a plain computation from the plain functions."""
    from geneinfer_amd.config import (AddRowsSpec, GatedDeltaSpec, InterleavedRotarySpec, LatentAttentionSpec, LayerNormSpec, LayerSpec, ModelSpec, RmsNormSpec, RoutedExpertsSpec,
                                      RunEntry, SwiGluSpec, TokenPairSpec)
    from geneinfer_amd.engine import Runner
    from geneinfer_amd.engine.model import DecoderModel
    from geneinfer_amd.parts import model_tensor_needs
    from geneinfer_amd.weights import random_tensors
    from plain_llama import rms_norm, swiglu
    from plain_rigalorn import delta_rule, rotary_frequencies, rotate_interleaved
    d, vocab, eps, E = 64, 100, 1e-5, 4
    ln = lambda name: LayerNormSpec(d, eps, name, name + ".b")
    latent = LatentAttentionSpec(hidden_size=d, n_heads=3, head_dim=8, rotary_dim=4, value_dim=6, q_rank=10, kv_rank=12, scale=0.3, norm_eps=eps, dq_proj="t.dq", dq_norm="t.qn", uq_proj="t.uq",
                                 dkv_proj="t.dkv", dkv_norm="t.kn", uk_proj="t.uk", uv_proj="t.uv", o_proj="t.o", position=InterleavedRotarySpec(4, 30.0), window=9, sinks="t.s")
    delta = GatedDeltaSpec(hidden_size=d, n_heads=2, n_kv_heads=1, key_dim=8, value_dim=24, conv_taps=3, norm_eps=eps, q_proj="m.q", k_proj="m.k", v_proj="m.v", q_conv="m.qc", k_conv="m.kc",
                           v_conv="m.vc", a_proj="m.a2", a_log="m.al", dt_bias="m.dt", b_proj="m.b", gate_proj="m.g", out_norm="m.n", o_proj="m.o", a_down="m.a1", a_rank=5)
    moe = RoutedExpertsSpec(hidden_size=d, intermediate_size=24, n_experts=E, top=2, router="r", gate_projs=tuple(f"e{j}.g" for j in range(E)), up_projs=tuple(f"e{j}.u" for j in range(E)),
                            down_projs=tuple(f"e{j}.d" for j in range(E)), score="sigmoid", weigh="output", correction="c", weight_scale=0.5, n_identity=1,
                            shared=SwiGluSpec(d, 32, "s.g", "s.u", "s.d"))
    spec = ModelSpec(architecture="by hand", vocab_size=vocab, hidden_size=d, max_positions=256, embedding="emb", final_norm=ln("fn"), lm_head="head", layers=(
        LayerSpec(mixer=latent, feed_forward=SwiGluSpec(d, 80, "g.g", "g.u", "g.d"), mixer_norm=RmsNormSpec(d, eps, "p1"), feed_forward_norm=RmsNormSpec(d, eps, "p2"), block="prenorm"),
        LayerSpec(mixer=delta, feed_forward=moe, mixer_norm=ln("n1"), feed_forward_norm=ln("n2"), block="prenorm")),
        run_order=(RunEntry(0), RunEntry(1, before=AddRowsSpec(d, "steps", 3, 2))), after_embedding=(TokenPairSpec(d, 11, 3, 7, "pairs"),))
    host = random_tensors(model_tensor_needs(spec), seed=5, dtype="float32", std=0.2)
    model = DecoderModel(spec, {k: v.to(DEV) for k, v in host.items()}, torch.float32, DEV)
    runner = Runner(model, page_size=4, max_tokens=256, max_requests=2)
    tokens = _prompt(dict(vocab=vocab), 45, 2)
    got = {}
    for what, cuts in (("whole", [45]), ("cut", [3, 20, 2])):
        runner.open(what)
        got[what] = feed(runner, what, tokens, cuts)
        runner.close(what)
    assert torch.equal(got["whole"], got["cut"])

    w = {k: v.double() for k, v in host.items()}
    T = len(tokens)
    x = P.embedding(tokens, w["emb"], w["pairs"], 3, 7)
    h = rms_norm(x, w["p1"], eps)
    q = (rms_norm(h @ w["t.dq"].T, w["t.qn"], eps) @ w["t.uq"].T).view(T, 3, 12)
    down = h @ w["t.dkv"].T
    c, f = rms_norm(down[:, :12], w["t.kn"], eps), rotary_frequencies(4, 30.0)[0]
    k_rot, q_rot = rotate_interleaved(down[:, None, 12:], f)[:, 0], rotate_interleaved(q[..., 8:], f)
    scores = (torch.einsum("thd,shd->hts", q[..., :8], (c @ w["t.uk"].T).view(T, 3, 8)) + torch.einsum("thr,sr->hts", q_rot, k_rot)) * 0.3
    p = P.sink_softmax(scores, P.window_mask(T, 9), w["t.s"])
    x = x + torch.einsum("hts,shd->thd", p, (c @ w["t.uv"].T).view(T, 3, 6)).reshape(T, 18) @ w["t.o"].T
    x = x + swiglu(rms_norm(x, w["p2"], eps), w["g.g"], w["g.u"], w["g.d"]) + w["steps"][2]
    h = P.layer_norm(x, w["n1"], w["n1.b"], eps)
    conv = lambda n: P.short_conv_silu(h @ w[f"m.{n}"].T, w[f"m.{n}c"])
    unit = lambda z: z / torch.sqrt((z * z).sum(dim=-1, keepdim=True) + 1e-6)
    q, k, v = unit(conv("q")) * 8 ** -0.5, unit(conv("k")), conv("v").view(T, 2, 24)
    beta = torch.sigmoid(h @ w["m.b"].T)
    decay = torch.exp(-torch.exp(w["m.al"]) * P.softplus((h @ w["m.a1"].T) @ w["m.a2"].T + w["m.dt"]))
    heads = [rms_norm(delta_rule(q, k, v[:, i], beta[:, i], decay[:, i]), w["m.n"], eps) for i in range(2)]
    x = x + (torch.cat(heads, -1) * P.silu(h @ w["m.g"].T)) @ w["m.o"].T
    h = P.layer_norm(x, w["n2"], w["n2.b"], eps)
    s = torch.sigmoid(h @ w["r"].T)
    ids = torch.topk(s + w["c"], 2, dim=-1).indices
    y = torch.stack([sum(0.5 * s[t, e] * (h[t] if e == E else swiglu(h[t][None], w[f"e{e}.g"], w[f"e{e}.u"], w[f"e{e}.d"])[0]) for e in ids[t].tolist()) for t in range(T)])
    x = x + y + swiglu(h, w["s.g"], w["s.u"], w["s.d"])
    want = P.layer_norm(x, w["fn"], w["fn.b"], eps) @ w["head"].T
    assert relative_error(got["whole"], want) < 5e-5
