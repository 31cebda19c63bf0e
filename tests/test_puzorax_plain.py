"""What pins the plain Puzorax implementation (`plain_puzorax.py`) beside a reading of its equations, and what the configuration
class accepts and refuses.  All on the CPU."""
import copy
import math

import pytest
import torch

import plain_puzorax as P
from puzorax_folders import CONFIGS, RANKS, random_weights, tensor_layout

D = torch.float64


def test_layer_norm_against_the_library_routine_and_eps_inside_the_root():
    g = torch.Generator().manual_seed(0)
    x, w, b = torch.randn(5, 9, generator=g, dtype=D), torch.randn(9, generator=g, dtype=D), torch.randn(9, generator=g, dtype=D)
    assert torch.allclose(P.layer_norm(x, w, b, 0.3), torch.nn.functional.layer_norm(x, (9,), w, b, eps=0.3))
    one = torch.tensor([[1.0, -1.0]], dtype=D)
    assert torch.allclose(P.layer_norm(one, torch.ones(2, dtype=D), torch.zeros(2, dtype=D), 3.0), one / 2)          # variance 1, eps 3


def test_rows_of_pairs_by_hand():
    assert P.pair_rows([4, 9, 9, 0], 3, 5, 7) == [7, (12 + 45) % 7, (27 + 45) % 7, 27 % 7]
    table, pairs = torch.arange(10, dtype=D)[:, None], 100 * torch.arange(8, dtype=D)[:, None]
    assert P.embedding([4, 9], table, pairs, 3, 5)[:, 0].tolist() == [4 + 700, 9 + 100 * (57 % 7)]


def test_rotation_keeps_lengths_depends_on_distance_only_and_pairs_halves():
    g = torch.Generator().manual_seed(1)
    a, b = torch.randn(8, generator=g, dtype=D), torch.randn(8, generator=g, dtype=D)
    at = lambda v, p: P.rotate_half_split(torch.stack([v] * 12)[:, None, :], 50.0)[p, 0]
    assert torch.allclose(at(a, 7).norm(), a.norm()) and torch.equal(at(a, 0), a)
    assert torch.allclose(at(a, 3) @ at(b, 1), at(a, 9) @ at(b, 7))
    e = torch.zeros(8, dtype=D)
    e[1] = 1.0                                                            # pair (1, 5), frequency 50^(-1/4)
    t = at(e, 2)
    angle = 2 * 50.0 ** -0.25
    assert math.isclose(float(t[1]), math.cos(angle)) and math.isclose(float(t[5]), math.sin(angle)) and t.abs().sum() == t[1].abs() + t[5].abs()


def test_softmax_with_a_sink_is_a_softmax_with_one_more_key_of_no_value():
    g = torch.Generator().manual_seed(2)
    H, T = 3, 6
    scores, sinks = torch.randn(H, T, T, generator=g, dtype=D), torch.tensor([-2.0, 0.5, 40.0], dtype=D)
    for window in (None, 1, 3):
        seen = P.window_mask(T, window)
        p = P.sink_softmax(scores, seen, sinks)
        more = torch.cat([scores.masked_fill(~seen[None], float("-inf")), sinks[:, None, None].expand(H, T, 1)], dim=-1)
        assert torch.allclose(p, torch.softmax(more, -1)[..., :T])
    assert P.window_mask(6, 2).tolist()[4] == [False, False, False, True, True, False]


def test_latents_folded_into_query_and_output_give_the_same_layer():
    """score = (W_uk^T q) . c + q_rot . k_rot and o = W_uv (sum p c): what an engine that caches only c and k_rot computes."""
    g = torch.Generator().manual_seed(3)
    H, d, r, dv, rank, hidden, T, eps = 2, 6, 4, 5, 7, 10, 17, 1e-5
    m = dict(heads=H, dim=d, rot_dim=r, vdim=dv, kv_rank=rank, scale=0.37, rot=dict(dims=r, base=25.0), mask=dict(size=6))
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=D) * 0.4
    w = {"q": rnd(H * (d + r), hidden), "dkv": rnd(rank + r, hidden), "dkv.norm": 1 + rnd(rank), "uk": rnd(H * d, rank), "uv": rnd(H * dv, rank), "o": rnd(hidden, H * dv),
         "g": rnd(H * dv, hidden), "sink": rnd(H)}
    h = rnd(T, hidden)
    q, down = (h @ w["q"].T).view(T, H, d + r), h @ w["dkv"].T
    c, k_rot = P.rms_norm(down[:, :rank], w["dkv.norm"], eps), P.rotate_half_split(down[:, None, rank:], 25.0)[:, 0]
    folded = torch.einsum("thd,hdr->thr", q[..., :d], w["uk"].view(H, d, rank))
    scores = (torch.einsum("thr,sr->hts", folded, c) + torch.einsum("thr,sr->hts", P.rotate_half_split(q[..., d:], 25.0), k_rot)) * 0.37
    p = P.sink_softmax(scores, P.window_mask(T, 6), w["sink"])
    o = torch.einsum("thr,hvr->thv", torch.einsum("hts,sr->thr", p, c), w["uv"].view(H, dv, rank)).reshape(T, H * dv)
    assert torch.allclose((o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T, P.latent_attention(h, w, m, eps))


def test_delta_rule_in_closed_form_for_two_tokens_and_decays_act_on_the_key_s_rows():
    g = torch.Generator().manual_seed(4)
    q, k, v = torch.randn(2, 5, generator=g, dtype=D), torch.randn(2, 5, generator=g, dtype=D), torch.randn(2, 3, generator=g, dtype=D)
    beta, decay = torch.tensor([0.7, 0.4], dtype=D), torch.rand(2, 5, generator=g, dtype=D)
    out = P.channel_delta_rule(q, k, v, beta, decay)
    S0 = beta[0] * torch.outer(k[0], v[0])
    assert torch.allclose(out[0], S0.T @ q[0])
    S1 = decay[1][:, None] * S0
    S1 = S1 + torch.outer(k[1], beta[1] * (v[1] - S1.T @ k[1]))
    assert torch.allclose(out[1], S1.T @ q[1])
    # a row whose decay is zero forgets; with equal decays it is the rule with one decay a head
    zero = decay.clone()
    zero[1] = torch.tensor([0.0, 1.0, 1.0, 1.0, 1.0], dtype=D)
    only = torch.zeros(5, dtype=D)
    only[0] = 1.0
    none = P.channel_delta_rule(torch.stack([q[0], only]), torch.stack([only, torch.zeros(5, dtype=D)]), v, beta, zero)
    assert torch.equal(none[1], torch.zeros(3, dtype=D))
    from plain_rigalorn import delta_rule
    one = torch.tensor([0.9, 0.6], dtype=D)
    assert torch.allclose(P.channel_delta_rule(q, k, v, beta, one[:, None].expand(2, 5)), delta_rule(q, k, v, beta, one))


def test_decays_and_softplus_by_hand():
    got = P.channel_decays(torch.tensor([[0.2, -1.0, 3.0, 0.0]], dtype=D), torch.tensor([0.5, -1.0], dtype=D), torch.tensor([0.1, 0.0, -3.0, 50.0], dtype=D), 2, 2)
    sp = lambda z: math.log1p(math.exp(z))
    want = [math.exp(-math.exp(0.5) * sp(0.3)), math.exp(-math.exp(0.5) * sp(-1.0)), math.exp(-math.exp(-1.0) * sp(0.0)), math.exp(-math.exp(-1.0) * 50.0)]
    assert torch.allclose(got.reshape(-1), torch.tensor(want, dtype=D))


def test_short_convolution_is_causal_and_ends_on_the_token_s_own_tap():
    x = torch.zeros(6, 2, dtype=D)
    x[2] = torch.tensor([1.0, 2.0])
    taps = torch.tensor([[0.1, 0.2, 0.3], [1.0, 0.0, -1.0]], dtype=D)
    want = torch.zeros(6, 2, dtype=D)
    want[2], want[3], want[4] = P.silu(torch.tensor([0.3, -2.0], dtype=D)), P.silu(torch.tensor([0.2, 0.0], dtype=D)), P.silu(torch.tensor([0.1, 2.0], dtype=D))
    assert torch.allclose(P.short_conv_silu(x, taps), want)


def test_routing_by_hand_the_correction_chooses_and_does_not_weigh():
    h = torch.eye(4, dtype=D)[:1]
    router = torch.zeros(4, 4, dtype=D)
    router[:, 0] = torch.log(torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=D))          # scores 0.1 0.2 0.3 0.4
    ids, weights = P.route(h, router, torch.tensor([0.35, 0.0, 0.0, -0.2], dtype=D), 2, 3.0)
    assert sorted(ids[0].tolist()) == [0, 2]                                        # choice scores 0.45 0.2 0.3 0.2
    by_id = dict(zip(ids[0].tolist(), weights[0].tolist()))
    assert math.isclose(by_id[0], 3.0 * 0.1 / 0.4) and math.isclose(by_id[2], 3.0 * 0.3 / 0.4)
    # expert numbers from `experts` on return their input
    w = dict(router=router, correction=torch.tensor([0.35, 0.0, 0.0, -0.2], dtype=D))
    g = torch.Generator().manual_seed(5)
    for e in range(2):
        w.update({f"e{e}.gate": torch.randn(3, 4, generator=g, dtype=D), f"e{e}.up": torch.randn(3, 4, generator=g, dtype=D), f"e{e}.down": torch.randn(4, 3, generator=g, dtype=D)})
    m = dict(router=dict(experts=2, identity=2, top=2, scale=3.0), expert=dict(ff=3))
    want = by_id[0] * P.expert(h, w["e0.gate"], w["e0.up"], w["e0.down"]) + by_id[2] * h
    assert torch.allclose(P.experts(h, w, m), want)


def test_order_of_layer_runs_and_what_joins_before_a_walk():
    assert P.layer_runs(CONFIGS["A"]) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert P.layer_runs(CONFIGS["C"]) == [(0, None), (1, None), (2, None)]
    # without output products a layer adds nothing (its experts aside): the stream is the token rows and what joins before the walks
    cfg = copy.deepcopy(CONFIGS["A"])
    for layer in cfg["layers"]:
        layer["mlp"] = None
    w = {n: (torch.zeros_like(t) if n.endswith(".mix.o") else t) for n, t in random_weights(cfg, RANKS["A"], 3).items()}
    outs, tokens = [], [3, 9, 27, 81]
    P.forward(cfg, w, tokens, layer_outputs=outs)
    b = cfg["embedding"]["bigram"]
    x0 = P.embedding(tokens, w["embed"].double(), w["bigram"].double(), b["mul_prev"], b["mul_cur"])
    step = w["loop.step"].double()
    assert torch.allclose(outs[0], x0) and torch.allclose(outs[2], x0 + step[0]) and torch.allclose(outs[5], 2 * x0 + step[0] + step[1])


# ------------------------------------------------------------------------------------------------- the configuration
def test_configurations_read_back_equal_and_name_every_tensor():
    from geneinfer_amd.config import parse_config
    from geneinfer_amd.parts import model_tensor_needs
    for name, cfg in CONFIGS.items():
        have = dict(tensor_layout(cfg, RANKS[name]))
        config = parse_config(cfg).fit_to_tensors(have)
        assert type(config).__name__ == "PuzoraxConfig" and type(config).from_dict(config.to_dict()) == config
        spec = config.model_spec()
        assert {n.name: tuple(n.shape) for n in model_tensor_needs(spec)} == have
        assert [e.layer for e in spec.run_order] == [i for i, _ in P.layer_runs(cfg)] and all(l.block == "parallel" for l in spec.layers)


def test_configuration_refusals():
    from geneinfer_amd.config import ConfigError, parse_config
    def broken(change):
        cfg = copy.deepcopy(CONFIGS["A"])
        change(cfg)
        with pytest.raises(ConfigError):
            parse_config(cfg)
    broken(lambda c: c["layers"][0].update(type="delta"))
    broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3))
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=6))
    broken(lambda c: c["layers"][1]["mixer"].update(rot_dim=7, rot=dict(base=10.0, dims=7)))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=8))
    broken(lambda c: c["layers"][0]["mixer"].pop("conv"))
    broken(lambda c: c["loop"].update(stop=9))
    broken(lambda c: c["embedding"]["bigram"].pop("buckets"))
    broken(lambda c: c.update(layers=[]))


def test_cache_needs_and_the_last_token_s_place():
    from geneinfer_amd.cache import CacheManager, PagedKvNeed, StateNeed
    from geneinfer_amd.config import TokenPairSpec, parse_config
    from geneinfer_amd.parts import block_class, row_transform_class
    spec = parse_config(CONFIGS["A"]).model_spec()
    needs = [block_class(spec.layers[e.layer].block).cache_need(spec.layers[e.layer]) for e in spec.run_order]
    assert isinstance(needs[0], StateNeed) and needs[0].shape == (4 * 6 * 16 * 4 + 3 * (2 * 2 * 16 + 4 * 24),)
    assert needs[1] == needs[3] == PagedKvNeed(1, 40, 20, 32, None) and needs[5] == PagedKvNeed(1, 24, 9, 20, None)
    assert needs[5].first_visible(8) == 0 and needs[5].first_visible(9) == 1
    (pairs,) = spec.after_embedding
    assert isinstance(pairs, TokenPairSpec) and row_transform_class(pairs).cache_need(pairs) == StateNeed((1,), torch.int32)
    # a request that opens finds its slot of every state zeroed, the integer one too; nothing with a state is shared or rewound
    cache = CacheManager([*needs, StateNeed((1,), torch.int32)], [None] * 7, page_size=4, n_pages=8, max_requests=2, max_positions=64)
    assert cache.states[6].dtype == torch.int32 and not cache.enable_prefix_sharing()
    slot = cache.open("a")
    cache.states[6][slot] = 17
    cache.close("a")
    assert cache.open("b") == slot and int(cache.states[6][slot, 0]) == 0
