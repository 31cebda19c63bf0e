"""What fixes the plain Vubenex implementation (`plain_vubenex.py`) and the configuration class, on the CPU: each mechanism against a
second formulation or a case worked by hand, the configuration's reading, its refusals and what it writes back, and the list of tensors a
configuration asks for against the folders the tests write."""
import copy
import math

import pytest
import torch

import plain_vubenex as P
from vubenex_folders import CONFIGS, random_weights, tensor_layout, write_model

torch.manual_seed(0)
F64 = torch.float64


# ------------------------------------------------------------------------------------------------ the plain mechanisms
def test_the_fading_memory_token_by_token_is_a_weighted_sum_over_the_rows_so_far():
    T, H, d, e = 17, 4, 5, 3
    q, k, v = torch.randn(T, H, d, dtype=F64), torch.randn(T, H, d, dtype=F64), torch.randn(T, H, e, dtype=F64)
    decay = [0.9, 0.5, 1.0, 0.0]
    a, b = P.fading_memory(q, k, v, decay), P.fading_memory_as_weights(q, k, v, decay)
    assert torch.allclose(a, b, atol=1e-12)
    assert torch.allclose(a[:, 3], (q[:, 3] * k[:, 3]).sum(-1, keepdim=True) * v[:, 3])          # what fades at once holds the row itself only
    whole = torch.cumsum(torch.einsum("td,te->tde", k[:, 2], v[:, 2]), dim=0)                    # what never fades holds all
    assert torch.allclose(a[:, 2], torch.einsum("td,tde->te", q[:, 2], whole))


def test_the_fading_memory_by_hand():
    one = lambda *values: torch.tensor(values, dtype=F64).reshape(-1, 1, 1)
    out = P.fading_memory(one(1, 10, 100), one(2, 3, 4), one(5, 6, 7), [0.5])[:, 0, 0]
    assert out.tolist() == [10.0, 10 * (5 + 18), 100 * (2.5 + 9 + 28)]


def test_the_empty_seat_is_a_key_of_score_zero_without_a_value():
    T, H, G, d = 9, 4, 2, 6
    q, k, v = torch.randn(T, H, d, dtype=F64), torch.randn(T, G, d, dtype=F64), torch.randn(T, G, d, dtype=F64)
    got = P.attention_with_an_empty_seat(q, k, v, 0.7)
    seat = lambda x: torch.cat([torch.zeros(1, G, d, dtype=F64), x]).transpose(0, 1).repeat_interleave(H // G, 0)[None]
    mask = torch.cat([torch.ones(T, 1, dtype=torch.bool), torch.tril(torch.ones(T, T, dtype=torch.bool))], dim=1)
    want = torch.nn.functional.scaled_dot_product_attention(q.transpose(0, 1)[None], seat(k), seat(v), attn_mask=mask, scale=0.7)[0].transpose(0, 1)
    assert torch.allclose(got, want, atol=1e-12)
    far = P.attention_with_an_empty_seat(torch.ones(2, 1, 1, dtype=F64), torch.full((2, 1, 1), -900.0, dtype=F64), torch.ones(2, 1, 1, dtype=F64), 1.0)
    near = P.attention_with_an_empty_seat(torch.ones(2, 1, 1, dtype=F64), torch.full((2, 1, 1), 900.0, dtype=F64), torch.ones(2, 1, 1, dtype=F64), 1.0)
    assert far.abs().max() < 1e-300 and torch.allclose(near, torch.ones_like(near))


def test_query_growth_at_its_steps():
    assert [P.query_growth(p, 0.3, 4) for p in (0, 1, 2)] == [1.0] * 3
    assert P.query_growth(3, 0.3, 4) == P.query_growth(6, 0.3, 4) == 1 + 0.3 * math.log(2)
    assert P.query_growth(7, 0.3, 4) == 1 + 0.3 * math.log(3)
    assert P.query_growth(0, 2.0, 1) == 1 + 2 * math.log(2)
    assert P.query_growth(1, 0.5, 2.5) == 1.0 and P.query_growth(2, 0.5, 2.5) == 1 + 0.5 * math.log(2) and P.query_growth(4, 0.5, 2.5) == 1 + 0.5 * math.log(3)


def test_the_values_are_the_keys_before_their_norm():
    cfg = CONFIGS["A"]
    m, w = cfg["layers"][1]["mixer"], {n[len("l1.mix."):]: t.double() for n, t in random_weights(cfg, 3).items() if n.startswith("l1.mix.")}
    h = torch.randn(1, cfg["width"], dtype=F64)
    # a single row sees itself: its output is its value times its weight 1 / (1 + e^-s), gated
    k = (h @ w["k"].T).reshape(m["kv_heads"], m["dim"])
    q, kn = P.rms_norm((h @ w["q"].T).reshape(m["heads"], m["dim"]), w["q.norm"], 1e-5), P.rms_norm(k, w["k.norm"], 1e-5)
    per = m["heads"] // m["kv_heads"]
    s = torch.stack([q[a] @ kn[a // per] for a in range(m["heads"])]) * m["scale"]
    y = torch.stack([k[a // per] * torch.sigmoid(s[a]) for a in range(m["heads"])]).reshape(1, -1) * torch.sigmoid(h @ w["g"].T)
    assert torch.allclose(P.attention_mixer(h, w, m, 1e-5), y @ w["o"].T)


def test_the_start_of_the_stream():
    table, where = torch.tensor([[1.0, 2.0], [3.0, 4.0]]), torch.tensor([[10.0, 0.0], [20.0, 0.0], [30.0, 1.0]])
    assert P.token_and_position_rows([1, 1, 0], table, 2.0, where).tolist() == [[16.0, 8.0], [26.0, 8.0], [32.0, 5.0]]


def test_activations_and_the_feed_forward_against_the_library_s():
    z = torch.randn(50, dtype=F64) * 3
    assert torch.allclose(P.silu(z), torch.nn.functional.silu(z)) and torch.allclose(P.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    h, g, u, d = torch.randn(3, 4, dtype=F64), torch.randn(6, 4, dtype=F64), torch.randn(6, 4, dtype=F64), torch.randn(4, 6, dtype=F64)
    F = torch.nn.functional
    assert torch.allclose(P.gated_feed_forward(h, g, u, d), F.linear(F.silu(F.linear(h, g)) * F.linear(h, u), d))
    assert torch.allclose(P.rms_norm(h, torch.ones(4, dtype=F64), 1e-6), F.rms_norm(h, (4,), eps=1e-6))


def test_the_second_input_takes_the_layer_s_own_columns():
    table = torch.arange(24, dtype=F64).reshape(4, 6)                      # three layers of two columns
    gate, proj = torch.zeros(2, 5, dtype=F64), torch.eye(5, 2, dtype=F64)
    gate[:, 0] = 100.0                                                     # gelu(100 x) = 100 x for a clearly positive x
    x = torch.zeros(2, 5, dtype=F64)
    x[:, 0] = 1.0
    got = P.token_side_input(x, [3, 1], table, 1, 2, gate, proj, torch.ones(5, dtype=F64), 0.0)
    want = torch.zeros(2, 5, dtype=F64)
    want[0, :2], want[1, :2] = torch.tensor([20.0, 21.0]), torch.tensor([8.0, 9.0])
    assert torch.allclose(got, want / want.pow(2).mean(-1, keepdim=True).sqrt())


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_plain_model_is_causal(name):
    m = P.PlainVubenex(config=CONFIGS[name], tensors=random_weights(CONFIGS[name], 4))
    tokens = torch.randint(0, CONFIGS[name]["vocab"], (14,), generator=torch.Generator().manual_seed(1)).tolist()
    runs, logits = m.layer_runs(tokens)
    assert len(runs) == len(CONFIGS[name]["layers"]) and torch.allclose(logits[:9], m.logits(tokens[:9]), atol=1e-10)


def test_without_its_output_products_the_model_is_the_head_of_the_normed_first_rows():
    cfg = CONFIGS["D"]
    w = random_weights(cfg, 2)
    for name in w:
        if name.endswith("mix.o") or name.endswith(".down") or name.endswith("side.proj"):
            w[name] = torch.zeros_like(w[name])
    tokens = [3, 17, 149, 0]
    x = w["embed"].double()[torch.tensor(tokens)] * cfg["embedding"]["scale"] + w["pos"].double()[:4]
    want = P.rms_norm(x, w["final.norm"].double(), cfg["norm"]["eps"]) @ w["embed"].double().T
    assert torch.allclose(P.PlainVubenex(config=cfg, tensors=w).logits(tokens), want)


# ------------------------------------------------------------------------------------------------ configuration
@pytest.mark.parametrize("name", list(CONFIGS))
def test_reading_writing_back_and_the_list_of_tensors(name, tmp_path):
    from geneinfer_amd.config import VubenexConfig, parse_config, read_config
    from geneinfer_amd.parts import model_tensor_needs
    config = parse_config(CONFIGS[name])
    assert type(config) is VubenexConfig and VubenexConfig.from_dict(config.to_dict()) == config
    needs = {n.name: n.shape for n in model_tensor_needs(config.model_spec())}
    assert needs == dict(tensor_layout(CONFIGS[name]))
    write_model(tmp_path / name, CONFIGS[name])
    assert read_config(tmp_path / name) == config
    spec = config.model_spec()
    assert len(spec.run_order) == len(CONFIGS[name]["layers"]) and spec.lm_head == spec.embedding == "embed"


def test_the_table_of_positions_says_how_many_there_are():
    from geneinfer_amd.config import parse_config
    config = parse_config(CONFIGS["A"])
    assert config.fit_to_tensors({"pos": (123, 64), "embed": (300, 64)}).max_positions == 123
    assert config.fit_to_tensors({"embed": (300, 64)}) == config


def test_refusals():
    from geneinfer_amd.config import ConfigError, parse_config

    def broken(change):
        cfg = copy.deepcopy(CONFIGS["A"])
        change(cfg)
        with pytest.raises(ConfigError):
            parse_config(cfg)

    broken(lambda c: c["layers"].clear())
    broken(lambda c: c["layers"][0].update(type="mlstm"))
    broken(lambda c: c["layers"][0]["mixer"]["decay"].pop())
    broken(lambda c: c["layers"][0]["mixer"].update(decay=[0.9, 0.5, 1.5]))
    broken(lambda c: c["layers"][0]["mixer"].update(decay="slow"))
    broken(lambda c: c["layers"][1]["mixer"].update(vdim=8))
    broken(lambda c: c["layers"][1]["mixer"].update(kv_heads=3))
    broken(lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0))
    broken(lambda c: c["layers"][1]["mixer"]["q_temp"].pop("coef"))
    broken(lambda c: c["layers"][1]["mixer"].pop("scale"))
    broken(lambda c: c["layers"][3].update(mlp=dict(kind="moe", ff=8)))
    broken(lambda c: c.pop("token_side"))
    broken(lambda c: c.pop("max_positions"))
    broken(lambda c: c.update(embedding={}))
    broken(lambda c: c["norm"].update(eps=0))


def test_parts_refuse_combinations_that_mean_nothing():
    from geneinfer_amd.config.spec import AttentionSpec, LightningSpec
    from geneinfer_amd.parts import mixer_class
    with pytest.raises(ValueError):
        LightningSpec(hidden_size=8, n_heads=2, key_dim=4, value_dim=4, decay=(0.5,), norm_eps=1e-5, q_proj="q", k_proj="k", v_proj="v", gate_proj="g", out_norm="n", o_proj="o")
    base = dict(hidden_size=8, n_heads=2, n_kv_heads=1, head_dim=4, q_proj="q", k_proj="k", v_proj="", o_proj="o", values_are_keys=True)
    needs = [n.name for n in mixer_class(AttentionSpec(**base)).tensor_needs(AttentionSpec(**base, output_gate="g"))]
    assert needs == ["q", "k", "o", "g"]


def test_a_request_cannot_be_longer_than_the_table_of_positions():
    """The step function's limit, whatever a caller asks for: positions behind the table's last row do not exist."""
    from geneinfer_amd.config.spec import LearnedPositionsSpec
    from geneinfer_amd.parts import row_transform_class
    spec = LearnedPositionsSpec(4, 7, "pos")
    part = row_transform_class(spec)(spec, {"pos": torch.zeros(7, 4)}, torch.float32, "cpu")
    assert part.position_limit == 7 and [n.shape for n in type(part).tensor_needs(spec)] == [(7, 4)]


def test_the_decays_powers():
    from geneinfer_amd.kernels import ops
    table = ops.lightning_powers((0.5, 1.0, 0.0, 0.999), "cpu")
    assert table.shape == (4, 65) and table.dtype == torch.float32
    assert table[0, :4].tolist() == [1.0, 0.5, 0.25, 0.125] and bool((table[1] == 1).all()) and table[2].tolist() == [1.0] + [0.0] * 64
    assert float(table[3, 64]) == pytest.approx(0.999 ** 64, rel=1e-7)
