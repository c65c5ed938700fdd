"""The plain Mitunex implementation (tests/plain_mitunex.py) against closed forms and cases worked out by hand, mistakes planted in
it that must show, and the configuration class. No GPU."""
import copy
import math

import pytest
import torch

import plain_mitunex as P
from helpers import token_ids
from mitunex_models import CONFIGS, make_mitunex_folder

F = torch.float64


def rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F)


# ---- the stream's ends -----------------------------------------------------------------------------------------------------

def test_a_tokens_row_and_its_positions_are_added_before_the_norm():
    table, positions, gain = rand(5, 6), rand(9, 6, seed=1), rand(6, seed=2)
    x = P.embedding([3, 0, 3], table, positions, gain, 0.01)
    for t, token in enumerate((3, 0, 3)):
        s = table[token] + positions[t]
        assert torch.allclose(x[t], s / math.sqrt(float((s * s).mean()) + 0.01) * gain)
    assert not torch.allclose(x[0], x[2])


def test_logits_are_scaled_before_the_cap():
    x, gain, head = rand(2, 4), torch.ones(4, dtype=F), rand(3, 4, seed=1)
    normed = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + 1e-6)
    got = P.output_logits(x, gain, head, 1e-6, 2.0, 3.0)
    assert torch.allclose(got, 3.0 * torch.tanh(2.0 * (normed @ head.T) / 3.0)) and float(got.abs().max()) < 3.0


def test_gelu_by_hand():
    z = torch.tensor([0.0, 1.0, -1.0, 3.0], dtype=F)
    assert torch.allclose(P.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"), atol=1e-12)
    assert abs(float(P.gelu_tanh(z)[1]) - 0.8411919906) < 1e-9


# ---- attention ---------------------------------------------------------------------------------------------------------------

def test_the_window_holds_the_query_itself_and_what_is_just_before_it():
    mask = P.window_mask(6, 3)
    assert mask[5].tolist() == [False, False, False, True, True, True] and mask[0].tolist() == [True] + [False] * 5
    assert torch.equal(P.window_mask(6, 1), torch.eye(6, dtype=torch.bool)) and torch.equal(P.window_mask(6, None), torch.ones(6, 6, dtype=torch.bool).tril())


def test_neighbours_turn_together_and_scores_depend_on_the_distance_alone():
    base, dims = 100.0, 6
    part = rand(8, 8)
    turned = P.turn_neighbours(part, dims, base)
    assert torch.equal(turned[0], part[0]) and torch.equal(turned[:, 6:], part[:, 6:])
    a = 3 * base ** (-2.0 / dims)
    assert abs(float(turned[3, 2]) - float(part[3, 2] * math.cos(a) - part[3, 3] * math.sin(a))) < 1e-12
    assert abs(float(turned[3, 3]) - float(part[3, 3] * math.cos(a) + part[3, 2] * math.sin(a))) < 1e-12
    same = part[:1].repeat(8, 1)
    again = P.turn_neighbours(same, 8, base)
    assert abs(float(again[2] @ again[5]) - float(again[4] @ again[7])) < 1e-12


def test_latent_attention_by_hand():
    """Against the same sums written out key by key, with the keys folded into the latent (how a cache of latents is read)."""
    tokens, width, eps = 7, 5, 1e-4
    m = {"heads": 2, "dim": 3, "rot_dim": 4, "vdim": 6, "kv_rank": 8, "scale": 0.7, "mask": {"size": 3}, "rot": {"dims": 4, "base": 20.0}}
    p = {"q": rand(14, width, seed=1), "dkv": rand(12, width, seed=2), "dkv.norm": rand(8, seed=3), "uk": rand(6, 8, seed=4), "uv": rand(12, 8, seed=5),
         "g": rand(2, width, seed=6), "o": torch.eye(12, dtype=F)}
    h = rand(tokens, width, seed=7)
    got = P.latent_attention(h, p, m, eps)
    latent, turned = P.latent_rows(h, p, m, eps)
    for i in range(tokens):
        for head in range(2):
            q = p["q"][head * 7:(head + 1) * 7] @ h[i]
            folded = p["uk"][head * 3:(head + 1) * 3].T @ q[:3]
            part = q[3:].clone()
            for pair in range(2):
                a = i * 20.0 ** (-2.0 * pair / 4)
                u, v = float(q[3 + 2 * pair]), float(q[4 + 2 * pair])
                part[2 * pair], part[2 * pair + 1] = u * math.cos(a) - v * math.sin(a), v * math.cos(a) + u * math.sin(a)
            keys = range(max(0, i - 2), i + 1)
            weights = torch.softmax(torch.stack([(folded @ latent[j] + part @ turned[j]) * 0.7 for j in keys]), dim=0)
            summed = sum(w * latent[j] for w, j in zip(weights, keys))
            want = p["uv"][head * 6:(head + 1) * 6] @ summed / (1.0 + math.exp(-float(p["g"][head] @ h[i])))
            assert torch.allclose(got[i, head * 6:(head + 1) * 6], want, atol=1e-10)


# ---- experts -----------------------------------------------------------------------------------------------------------------

def test_weights_are_the_scores_themselves_and_multiply_what_the_expert_reads():
    chosen, weights = P.choose(torch.tensor([0.5, 2.0, -1.0, 2.0], dtype=F), 2)
    assert chosen == [1, 3] and weights == pytest.approx([1 / (1 + math.exp(-2.0))] * 2)
    width, ff = 4, 3
    mlp = {"router": {"experts": 2, "top": 1}, "shared": {"ff": 5}}
    p = {"router": rand(2, width, seed=1)}
    for n in ("e0", "e1"):
        p.update({f"{n}.gate": rand(ff, width, seed=2), f"{n}.up": rand(ff, width, seed=3), f"{n}.down": rand(width, ff, seed=4)})
    p.update({"shared.gate": rand(5, width, seed=5), "shared.up": rand(5, width, seed=6), "shared.down": rand(width, 5, seed=7), "shared.sg": rand(1, width, seed=8)})
    h = rand(1, width, seed=9)
    w = float(torch.sigmoid((h @ p["router"].T).max()))
    gate, up = w * (p["e0.gate"] @ h[0]), w * (p["e0.up"] @ h[0])
    of_expert = p["e0.down"] @ (gate * torch.sigmoid(gate) * up)
    gate, up = p["shared.gate"] @ h[0], p["shared.up"] @ h[0]
    of_shared = torch.sigmoid(p["shared.sg"] @ h[0]) * (p["shared.down"] @ (gate * torch.sigmoid(gate) * up))
    assert torch.allclose(P.experts(h, p, mlp)[0], of_expert + of_shared)
    assert not torch.allclose(of_expert, w * P.expert(h, p["e0.gate"], p["e0.up"], p["e0.down"])[0])
    assert torch.allclose(P.experts(h, p, {"router": mlp["router"]})[0], of_expert)


# ---- the model -----------------------------------------------------------------------------------------------------------------

@pytest.fixture(scope="module")
def mixed(tmp_path_factory):
    folder = make_mitunex_folder(CONFIGS["mixed"], tmp_path_factory.mktemp("mixed"), seed=3)
    ids = token_ids(CONFIGS["mixed"]["vocab"], 90, seed=4)
    model = P.PlainModel(folder)
    return folder, model, ids, model.logits(ids)


def test_a_longer_sequence_has_the_same_first_logits(mixed):
    _, model, ids, want = mixed
    for length in (1, 2, 25, 66):
        assert torch.allclose(model.logits(ids[:length]), want[:length], atol=1e-5)


def _window(model):
    for layer in model.config["layers"]:
        if layer["mixer"]["mask"]["size"] == 24:
            layer["mixer"]["mask"]["size"] = 25


def _far_window(model):
    for layer in model.config["layers"]:
        if layer["mixer"]["mask"]["size"] == 65:
            layer["mixer"]["mask"]["size"] = 64


def _own_weights(model):
    model.config["layers"][2]["weights_of"] = 0
    model.config["layers"][2].update({key: copy.deepcopy(model.config["layers"][0][key]) for key in ("mixer", "mlp")})


def _gate(model):
    model.tensors["l1.mix.g"] = torch.zeros_like(model.tensors["l1.mix.g"])


def _position(model):
    model.tensors["pos"] = model.tensors["pos"].roll(1, dims=0)


def _shared(model):
    for layer in model.config["layers"]:
        if layer["mlp"] is not None:
            layer["mlp"].pop("shared", None)


def _post_norm(model):
    model.tensors["l1.norm2"] = torch.ones_like(model.tensors["l1.norm2"])


def _rotation(model):
    for layer in model.config["layers"]:
        layer["mixer"]["rot"]["base"] *= 2.0


def _cap(model):
    model.config["logit_softcap"] *= 2.0


def _scale(model):
    model.config["logit_scale"] *= 1.01


@pytest.mark.parametrize("mistake", [_window, _far_window, _own_weights, _gate, _position, _shared, _post_norm, _rotation, _cap, _scale])
def test_a_mistake_planted_in_the_plain_model_shows_in_the_logits(mistake, mixed):
    """What the comparisons on the GPU rest on: with these weights each of these is far above the limit that 32-bit is held to."""
    folder, _, ids, want = mixed
    model = P.PlainModel(folder)
    mistake(model)
    assert float((model.logits(ids) - want).abs().max()) > 1e-3 * float(want.abs().max())


# ---- configuration, registry, tensors ----------------------------------------------------------------------------------------

@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_configuration_survives_its_dictionary_and_names_the_checkpoints_tensors(name, tmp_path):
    from xeno_rt_amd.config import architecture, load_config, parse_config
    raw = CONFIGS[name]
    config = parse_config(raw)
    assert config.architecture == "Mitunex" and parse_config(config.to_dict()) == config
    assert config.vocab_size == raw["vocab"] and config.hidden_size == raw["width"] and config.max_position_embeddings == raw["max_positions"]
    folder = make_mitunex_folder(raw, tmp_path, seed=1)
    assert load_config(folder) == config
    _, tensors = P.load_folder(folder)
    specs = architecture("Mitunex").build(config).weight_specs()
    assert {n: tuple(t.shape) for n, t in tensors.items()} == {n: s.shape for n, s in specs.items()}
    for index, layer in enumerate(raw["layers"]):
        assert any(n.startswith(f"l{index}.") for n in tensors) == (layer.get("weights_of") is None)


def test_a_layer_that_runs_anothers_weights_has_a_cache_of_its_own():
    from xeno_rt_amd.config import architecture, parse_config
    spec = architecture("Mitunex").build(parse_config(CONFIGS["mixed"]))
    assert len(spec.layers) == 3 and [call.layer for call in spec.schedule] == [0, 1, 1, 2, 0]
    assert all(call.reads_cache_of is None for call in spec.schedule) and len(spec.cache_needs()) == 5 and spec.capturable()
    assert [need.kv.window for need in spec.cache_needs()] == [24, 65, 65, 7, 24]
    edges = architecture("Mitunex").build(parse_config(CONFIGS["edges"]))
    assert [call.layer for call in edges.schedule] == [1, 0, 1, 1]


@pytest.mark.parametrize("change", [
    lambda c: c.pop("layers"), lambda c: c.update(layers=[]), lambda c: c.pop("norm"), lambda c: c.pop("logit_scale"), lambda c: c.update(logit_softcap=0),
    lambda c: c.pop("max_positions"), lambda c: c["layers"][0].update(type="attention"), lambda c: c["layers"][0]["mixer"].pop("kv_rank"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10), lambda c: c["layers"][0]["mixer"].pop("rot"),
    lambda c: c["layers"][0]["mixer"].update(mask={"size": 0}), lambda c: c["layers"][0]["mlp"].update(kind="gated"), lambda c: c["layers"][1]["mlp"].pop("expert"),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=7), lambda c: c["layers"][1]["mlp"].update(shared={}), lambda c: c["layers"][2].update(weights_of=9),
    lambda c: c["layers"][2].update(weights_of=2), lambda c: c["layers"][2].update(weights_of=0), lambda c: c["layers"][2].update(weights_of=True),
])
def test_what_config_json_must_not_say(change):
    from xeno_rt_amd.config import ConfigError, parse_config
    raw = copy.deepcopy(CONFIGS["mixed"])
    change(raw)
    with pytest.raises(ConfigError):
        parse_config(raw)


def test_layers_that_run_each_others_weights_are_refused():
    from xeno_rt_amd.config import ConfigError, parse_config
    raw = copy.deepcopy(CONFIGS["mixed"])
    raw["layers"][1]["weights_of"] = 2
    with pytest.raises(ConfigError):
        parse_config(raw)


def test_a_checkpoint_may_carry_a_second_norm_for_a_layer_without_a_feed_forward(tmp_path):
    from xeno_rt_amd.config import architecture, parse_config
    spec = architecture("Mitunex").build(parse_config(CONFIGS["mixed"]))
    assert spec.ignored_names() == ["l3.norm2"] and "l3.norm2" not in spec.weight_specs()


@pytest.mark.parametrize("options", [dict(clamp=(1.0, 1.7), shared=8), dict(clamp=(1.0, 1.7), weigh_input=True), dict(shared=0)])
def test_experts_that_do_not_go_together_are_refused(options):
    from xeno_rt_amd.parts import ExpertsMLP
    with pytest.raises(ValueError):
        ExpertsMLP("mlp.", 8, 4, 2, 1, **options)


@pytest.mark.parametrize("options", [dict(window=0), dict(q_rank=0), dict(kv_rank=0)])
def test_a_latent_attention_without_size_is_refused(options):
    from xeno_rt_amd.parts import LatentAttention
    arguments = dict(n_heads=2, dim=4, rot_dim=2, value_dim=4, kv_rank=8, q_rank=None, scale=1.0, eps=1e-5, rot_dims=2, rot_base=10.0)
    with pytest.raises(ValueError):
        LatentAttention("mix.", 8, **{**arguments, **options})
