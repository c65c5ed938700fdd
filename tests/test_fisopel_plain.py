"""The plain Fisopel implementation (tests/plain_fisopel.py) against closed forms and cases worked out by hand, mistakes planted in
it that must show, and the configuration class. No GPU."""
import copy
import math

import pytest
import torch

import plain_fisopel as P
from fisopel_models import CONFIGS, make_fisopel_folder
from helpers import token_ids

F = torch.float64


def rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F)


# ---- the stream's ends, and what comes before a pass ------------------------------------------------------------------------

def test_the_table_is_scaled_on_the_way_in_and_not_on_the_way_out():
    table, gain = rand(5, 6), rand(6, seed=1)
    x = P.embedding([3, 0, 3], table, 2.5)
    assert torch.allclose(x[0], 2.5 * table[3]) and torch.equal(x[0], x[2])
    got = P.output_logits(x, gain, table, 0.01)
    assert torch.allclose(got[0], table @ (x[0] / math.sqrt(float((x[0] ** 2).mean()) + 0.01) * gain))


def test_a_pass_begins_with_the_stream_before_what_it_began_with():
    x, first, w = rand(4, 3), rand(4, 3, seed=1), rand(3, 6, seed=2)
    got = P.enter_pass(x, first, w)
    for t in range(4):
        for n in range(3):
            assert abs(float(got[t, n]) - float(sum(w[n, k] * x[t, k] + w[n, 3 + k] * first[t, k] for k in range(3)))) < 1e-12


def test_the_order_of_layers_and_passes():
    layers = [None] * 5
    assert P.order({"layers": layers}) == [(i, False) for i in range(5)]
    assert P.order({"layers": layers, "loop": {"start": 1, "stop": 3, "times": 2}}) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False), (4, False)]
    assert P.order({"layers": layers[:2], "loop": {"start": 0, "stop": 2, "times": 1}}) == [(0, True), (1, False)]


# ---- rotation -------------------------------------------------------------------------------------------------------------------

def test_halves_turn_together_and_scores_depend_on_the_distance_alone():
    rot = {"dims": 6, "base": 100.0}
    part = rand(8, 8)
    turned = P.turn_halves(part, rot)
    assert torch.equal(turned[0], part[0]) and torch.equal(turned[:, 6:], part[:, 6:])
    a = 3 * 100.0 ** (-2.0 / 6)
    assert abs(float(turned[3, 1]) - float(part[3, 1] * math.cos(a) - part[3, 4] * math.sin(a))) < 1e-12
    assert abs(float(turned[3, 4]) - float(part[3, 4] * math.cos(a) + part[3, 1] * math.sin(a))) < 1e-12
    again = P.turn_halves(part[:1].repeat(8, 1), rot)
    assert abs(float(again[2] @ again[5]) - float(again[4] @ again[7])) < 1e-12


def test_slow_waves_are_stretched_and_fast_ones_stay():
    dims, base, scaling = 16, 10000.0, {"factor": 8.0, "original": 256, "fast": 16.0, "slow": 1.0}
    plain, one = P.frequencies(dims, base, None)
    got, magnitude = P.frequencies(dims, base, scaling)
    assert one == 1.0 and magnitude == pytest.approx(0.1 * math.log(8.0) + 1.0)
    turns = [256 * f / (2 * math.pi) for f in plain]            # of a wave over the original length
    for f, g, n in zip(plain, got, turns):
        if n > 16.0 * base ** (2 / dims):
            assert g == pytest.approx(f)
        if n < 1.0 / base ** (2 / dims):
            assert g == pytest.approx(f / 8.0)
        assert f / 8.0 - 1e-12 <= g <= f + 1e-12
    assert got[0] == plain[0] and got[-1] == pytest.approx(plain[-1] / 8.0)
    # the pair at which a wave makes one turn, worked out from the frequencies themselves: f = 2 pi / original
    exact = dims * math.log(256 / (2 * math.pi)) / (2 * math.log(base))
    assert base ** (-2 * exact / dims) == pytest.approx(2 * math.pi / 256)
    part = rand(3, dims)
    assert torch.allclose(P.turn_halves(part, {"dims": dims, "base": base, "scaling": scaling})[0], magnitude * part[0])


# ---- attention -------------------------------------------------------------------------------------------------------------------

def test_a_query_sees_its_window_and_the_first_tokens():
    mask = P.seen(8, 3, 2)
    assert mask[7].tolist() == [True, True, False, False, False, True, True, True] and mask[0].tolist() == [True] + [False] * 7
    assert mask[2].tolist() == [True] * 3 + [False] * 5 and mask[3].tolist() == [True] * 4 + [False] * 4
    assert mask[4].tolist() == [True, True, True, True, True, False, False, False] and not bool(mask[5][2])
    assert torch.equal(P.seen(6, 1), torch.eye(6, dtype=torch.bool)) and torch.equal(P.seen(6), torch.ones(6, 6, dtype=torch.bool).tril())
    assert torch.equal(P.seen(6, 2, 100), P.seen(6)) and torch.equal(P.seen(6, 6, 0), P.seen(6))


def test_attention_by_hand():
    """Against the same sums written out key by key: head norms, the cap before the mask, a sink that is neither scaled nor capped."""
    tokens, width, eps = 7, 5, 1e-3
    m = {"heads": 4, "kv_heads": 2, "dim": 3, "vdim": 2, "scale": 0.7, "softcap": 0.4, "mask": {"size": 2, "keep_first": 1}}
    p = {"q": rand(12, width, seed=1), "k": rand(6, width, seed=2), "v": rand(4, width, seed=3), "q.norm": rand(3, seed=4), "k.norm": rand(3, seed=5),
         "sink": rand(4, seed=6), "o": torch.eye(8, dtype=F)}
    h = rand(tokens, width, seed=7)
    got = P.attention(h, p, m, eps)
    norm = lambda v, w: v / math.sqrt(float((v * v).mean()) + eps) * w
    for i in range(tokens):
        for head in range(4):
            q = norm(p["q"][head * 3:(head + 1) * 3] @ h[i], p["q.norm"])
            kv = head // 2
            top, bottom = torch.zeros(2, dtype=F), math.exp(float(p["sink"][head]))
            for j in sorted({j for j in (0, i - 1, i) if 0 <= j <= i}):
                k = norm(p["k"][kv * 3:(kv + 1) * 3] @ h[j], p["k.norm"])
                weight = math.exp(0.4 * math.tanh(0.7 * float(q @ k) / 0.4))
                top, bottom = top + weight * (p["v"][kv * 2:(kv + 1) * 2] @ h[j]), bottom + weight
            assert torch.allclose(got[i, head * 2:(head + 1) * 2], top / bottom, atol=1e-10)


def test_latent_attention_by_hand():
    """Against the same sums written out key by key, with the keys folded into the latent (how a cache of latents is read)."""
    tokens, width, eps = 6, 5, 1e-4
    m = {"heads": 2, "dim": 3, "rot_dim": 4, "vdim": 6, "kv_rank": 8, "scale": 0.7,
         "rot": {"dims": 4, "base": 20.0, "scaling": {"factor": 3.0, "original": 40, "fast": 4.0, "slow": 0.5}}}
    p = {"q": rand(14, width, seed=1), "dkv": rand(12, width, seed=2), "dkv.norm": rand(8, seed=3), "uk": rand(6, 8, seed=4), "uv": rand(12, 8, seed=5),
         "g": rand(12, width, seed=6), "o": torch.eye(12, dtype=F)}
    h = rand(tokens, width, seed=7)
    got = P.latent_attention(h, p, m, eps)
    latent, turned = P.latent_rows(h, p, m, eps)
    for i in range(tokens):
        for head in range(2):
            q = p["q"][head * 7:(head + 1) * 7] @ h[i]
            folded = p["uk"][head * 3:(head + 1) * 3].T @ q[:3]
            part = P.turn_halves(q[3:].repeat(i + 1, 1), m["rot"])[i]
            weights = torch.softmax(torch.stack([(folded @ latent[j] + part @ turned[j]) * 0.7 for j in range(i + 1)]), dim=0)
            of_head = p["uv"][head * 6:(head + 1) * 6] @ sum(w * latent[j] for j, w in enumerate(weights))
            want = of_head / (1.0 + torch.exp(-p["g"][head * 6:(head + 1) * 6] @ h[i]))
            assert torch.allclose(got[i, head * 6:(head + 1) * 6], want, atol=1e-10)


# ---- experts -----------------------------------------------------------------------------------------------------------------------

def test_weights_are_a_softmax_over_the_chosen_logits_alone():
    chosen, weights = P.choose(torch.tensor([0.5, 2.0, -1.0, 1.0, 2.0], dtype=F), 3)
    assert chosen == [1, 4, 3]
    assert weights == pytest.approx([math.exp(2.0) / (2 * math.exp(2.0) + math.exp(1.0))] * 2 + [math.exp(1.0) / (2 * math.exp(2.0) + math.exp(1.0))])
    assert P.choose(torch.tensor([3.0, -2.0], dtype=F), 1) == ([0], [1.0])
    width = 4
    mlp = {"router": {"experts": 3, "top": 2}, "shared": {"ff": 5}}
    p = {"router": rand(3, width, seed=1), "shared.gate": rand(5, width, seed=5), "shared.up": rand(5, width, seed=6), "shared.down": rand(width, 5, seed=7)}
    for n in range(3):
        p.update({f"e{n}.gate": rand(3, width, seed=10 + n), f"e{n}.up": rand(3, width, seed=20 + n), f"e{n}.down": rand(width, 3, seed=30 + n)})
    h = rand(1, width, seed=9)
    def by_hand(name):
        gate, up = p[name + ".gate"] @ h[0], p[name + ".up"] @ h[0]
        return p[name + ".down"] @ (gate / (1.0 + torch.exp(-gate)) * up)
    chosen, weights = P.choose(h[0] @ p["router"].T, 2)
    routed = sum(w * by_hand(f"e{e}") for e, w in zip(chosen, weights))
    assert torch.allclose(P.experts(h, p, mlp)[0], routed + by_hand("shared")) and torch.allclose(P.experts(h, p, {"router": mlp["router"]})[0], routed)


def test_both_sublayers_of_a_layer_read_the_same_stream():
    raw = CONFIGS["odd"]
    layer = raw["layers"][0]
    generator = torch.Generator().manual_seed(1)
    from xeno_rt_amd.config import architecture, parse_config
    tensors = {n: torch.randn(s.shape, generator=generator, dtype=F) * 0.3 for n, s in architecture("Fisopel").build(parse_config(raw)).weight_specs().items()}
    x = rand(5, raw["width"])
    got = P.add_layer(x, tensors, 0, layer, 1e-4)
    mixer = P.attention(P.rms_norm(x, tensors["l0.norm1"], 1e-4), P.part(tensors, "l0.mix."), layer["mixer"], 1e-4)
    other = P.experts(P.rms_norm(x, tensors["l0.norm2"], 1e-4), P.part(tensors, "l0.mlp."), layer["mlp"])
    assert torch.allclose(got, x + mixer + other)


# ---- the model -----------------------------------------------------------------------------------------------------------------------

@pytest.fixture(scope="module")
def mixed(tmp_path_factory):
    folder = make_fisopel_folder(CONFIGS["mixed"], tmp_path_factory.mktemp("mixed"), seed=3)
    ids = token_ids(CONFIGS["mixed"]["vocab"], 160, seed=4)
    model = P.PlainModel(folder)
    return folder, model, ids, model.logits(ids)


def test_a_longer_sequence_has_the_same_first_logits(mixed):
    _, model, ids, want = mixed
    for length in (1, 2, 25, 66):
        assert torch.allclose(model.logits(ids[:length]), want[:length], atol=1e-5)


def _mixer(index, key, value):
    def change(model):
        at = model.config["layers"][index]["mixer"]
        for name in key[:-1]:
            at = at[name]
        at[key[-1]] = value(at[key[-1]])
    return change


def _tensor(name, value):
    def change(model):
        model.tensors[name] = value(model.tensors[name].to(F))
    return change


def _config(*path, value):
    def change(model):
        at = model.config
        for name in path[:-1]:
            at = at[name]
        at[path[-1]] = value
    return change


MISTAKES = {
    "window": _mixer(1, ("mask", "size"), lambda n: n + 1),
    "wide window": _mixer(2, ("mask", "size"), lambda n: n - 1),
    "kept": _mixer(1, ("mask", "keep_first"), lambda n: n + 1),
    "kept short": _mixer(1, ("mask", "keep_first"), lambda n: n - 1),
    "kept beyond a block": _mixer(2, ("mask", "keep_first"), lambda n: n - 1),
    "softcap": _mixer(1, ("softcap",), lambda c: c * 1.05),
    "scale": _mixer(0, ("scale",), lambda s: s * 1.02),
    "no stretching": _mixer(0, ("rot", "scaling"), lambda s: None),
    "stretching": _mixer(0, ("rot", "scaling", "factor"), lambda f: f * 1.3),
    "base": _mixer(3, ("rot", "base"), lambda b: b * 1.5),
    "sink": _tensor("l1.mix.sink", lambda t: t - 100.0),
    "gate": _tensor("l0.mix.g", lambda t: t * 0.0),
    "gate order": _tensor("l0.mix.g", lambda t: t.roll(1, dims=0)),
    "q norm": _tensor("l1.mix.q.norm", lambda t: t + 1.0),
    "k norm": _tensor("l2.mix.k.norm", lambda t: t * 0.0 + 1.0),
    "norm2": _tensor("l0.norm2", lambda t: t * 0.0 + 1.0),
    "second norm": lambda model: model.tensors.update({"l0.norm2": model.tensors["l0.norm1"]}),
    "entry": _tensor("loop.in", lambda t: t.roll(t.shape[1] // 2, dims=1)),
    "passes": _config("loop", "times", value=3),
    "no passes": _config("loop", value=None),
    "embedding scale": _config("embedding", "scale", value=2.0),
    "top": _config("layers", 1, "mlp", "router", "top", value=2),
    "shared": _config("layers", 3, "mlp", "shared", value=None),
    "eps": _config("norm", "eps", value=1e-2),
}


@pytest.mark.parametrize("mistake", sorted(MISTAKES))
def test_a_mistake_planted_in_the_plain_model_shows_in_the_logits(mistake, mixed):
    """What the comparisons on the GPU rest on: with these weights each of these is far above the limit that 32-bit is held to."""
    folder, _, ids, want = mixed
    model = P.PlainModel(folder)
    MISTAKES[mistake](model)
    assert float((model.logits(ids) - want).abs().max()) > 1e-3 * float(want.abs().max())


# ---- configuration, registry, tensors, cache -------------------------------------------------------------------------------------

@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_configuration_survives_its_dictionary_and_names_the_checkpoints_tensors(name, tmp_path):
    from xeno_rt_amd.config import architecture, load_config, parse_config
    raw = CONFIGS[name]
    config = parse_config(raw)
    assert config.architecture == "Fisopel" and parse_config(config.to_dict()) == config
    assert config.vocab_size == raw["vocab"] and config.hidden_size == raw["width"] and config.max_position_embeddings is None
    assert config.order() == P.order(raw)
    folder = make_fisopel_folder(raw, tmp_path, seed=1)
    assert load_config(folder) == config
    _, tensors = P.load_folder(folder)
    specs = architecture("Fisopel").build(config).weight_specs()
    assert {n: tuple(t.shape) for n, t in tensors.items()} == {n: s.shape for n, s in specs.items()}
    assert ("loop.in" in tensors) == ("loop" in raw) and "head" not in tensors


def test_every_pass_has_cache_entries_of_its_own():
    from xeno_rt_amd.config import architecture, parse_config
    spec = architecture("Fisopel").build(parse_config(CONFIGS["mixed"]))
    assert len(spec.layers) == 4 and [call.layer for call in spec.schedule] == [0, 1, 2, 1, 2, 3]
    assert [call.enters for call in spec.schedule] == [False, True, False, True, False, False]
    assert all(call.reads_cache_of is None for call in spec.schedule) and len(spec.cache_needs()) == 6 and spec.capturable()
    assert [(need.kv.window, need.kv.keep_first) for need in spec.cache_needs()] == [(None, 0), (24, 3), (65, 70), (24, 3), (65, 70), (None, 0)]
    assert spec.cache_needs()[0].kv.head_dim == 24 + 8 and spec.cache_needs()[0].kv.value_width == 24


@pytest.mark.parametrize("change", [
    lambda c: c.pop("layers"), lambda c: c.update(layers=[]), lambda c: c.pop("norm"), lambda c: c.update(embedding={"scale": "big"}), lambda c: c.update(embedding=3),
    lambda c: c["layers"][0].update(type="lightning"), lambda c: c["layers"][0]["mixer"].pop("kv_rank"), lambda c: c["layers"][0]["mixer"].pop("scale"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10), lambda c: c["layers"][0]["mixer"].pop("rot"),
    lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"), lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0),
    lambda c: c["layers"][0]["mixer"]["rot"].update(base=1), lambda c: c["layers"][1]["mixer"].update(kv_heads=3), lambda c: c["layers"][1]["mixer"].pop("vdim"),
    lambda c: c["layers"][1]["mixer"].update(mask={"size": 0}), lambda c: c["layers"][1]["mixer"].update(mask={"keep_first": 2}),
    lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1), lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=True),
    lambda c: c["layers"][1]["mixer"].update(softcap=0), lambda c: c["layers"][0]["mlp"].update(kind="dense"), lambda c: c["layers"][0]["mlp"].pop("expert"),
    lambda c: c["layers"][0]["mlp"]["router"].update(top=7), lambda c: c["layers"][0]["mlp"].update(shared={}), lambda c: c.update(loop={"start": 1, "stop": 3}),
    lambda c: c.update(loop={"start": 2, "stop": 2, "times": 1}), lambda c: c.update(loop={"start": 0, "stop": 5, "times": 1}),
    lambda c: c.update(loop={"start": 0, "stop": 2, "times": 0}), lambda c: c.update(loop={"start": -1, "stop": 2, "times": 1}), lambda c: c.update(loop=[0, 2, 1]),
])
def test_what_config_json_must_not_say(change):
    from xeno_rt_amd.config import ConfigError, parse_config
    raw = copy.deepcopy(CONFIGS["mixed"])
    change(raw)
    with pytest.raises(ConfigError):
        parse_config(raw)


def test_what_config_json_may_leave_out():
    from xeno_rt_amd.config import parse_config
    raw = copy.deepcopy(CONFIGS["mixed"])
    raw["loop"] = None
    raw.pop("embedding")
    raw["layers"][1]["mixer"]["mask"].pop("keep_first")
    raw["layers"][0]["mlp"]["shared"] = None
    config = parse_config(raw)
    assert config.loop is None and config.embedding_scale == 1.0 and [layer for layer, _ in config.order()] == [0, 1, 2, 3]


def test_a_checkpoint_may_carry_a_second_norm_for_a_layer_without_experts():
    from xeno_rt_amd.config import architecture, parse_config
    spec = architecture("Fisopel").build(parse_config(CONFIGS["mixed"]))
    assert "l2.norm2" in spec.ignored_names() and "l2.norm2" not in spec.weight_specs() and "l1.norm2" in spec.weight_specs()


@pytest.mark.parametrize("options", [dict(softcap=0.0), dict(softcap=-1.0), dict(window=4, keep_first=-1), dict(weights="sigmoid", softcap=1.0),
                                     dict(weights="sigmoid", window=4, keep_first=1)])
def test_an_attention_that_makes_no_sense_is_refused(options):
    from xeno_rt_amd.parts import Attention
    with pytest.raises(ValueError):
        Attention("mix.", 8, 2, 1, 4, **options)


def test_passes_need_an_entry_and_a_feed_forwards_norm_a_feed_forward():
    from xeno_rt_amd.config import architecture, parse_config
    from xeno_rt_amd.models import LayerCall, ModelSpec
    from xeno_rt_amd.parts import LatentAttention, PairRotation, ParallelBlock, RMSNorm
    spec = architecture("Fisopel").build(parse_config(CONFIGS["odd"]))
    with pytest.raises(ValueError):
        ModelSpec(config=spec.config, embedding=spec.embedding, layers=spec.layers, final_norm=spec.final_norm, head=spec.head, schedule=[LayerCall(0, enters=True)])
    with pytest.raises(ValueError):
        ParallelBlock(RMSNorm("a.", 8, 1e-5), spec.layers[0].mixer, feed_forward_norm=RMSNorm("b.", 8, 1e-5))
    arguments = dict(n_heads=2, dim=4, rot_dim=4, value_dim=4, kv_rank=8, q_rank=None, scale=1.0, eps=1e-5, rot_dims=4, rot_base=10.0)
    for options in (dict(gate_per="token"), dict(position=PairRotation(2, 10.0))):
        with pytest.raises(ValueError):
            LatentAttention("mix.", 8, **arguments, **options)
