"""The Mitunex decoder on the GPU against the plain implementation (tests/plain_mitunex.py), for four small configurations that
differ in every size and option: whole prompts, token-by-token decoding from the first token, portions of several sizes, unequal
batches through reused slots, greedy generation through the library's loop and programs; and every mechanism alone against
plain arithmetic, with inputs made so that a far key, a window's edge, a block's border or a weight on the wrong side of an expert shows."""
import math
import types

import pytest
import torch

from helpers import errors, run_batched, run_whole, token_ids
from mitunex_models import CONFIGS, _layer, _model, _moe, _dense, make_mitunex_folder
from test_renapel_gpu import Step, in_portions, layer_cache, run_mixer, runtime, same_but_for_rounding, schedules, short, tensors_for
import plain_mitunex as P

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
NAMES = sorted(CONFIGS)
LENGTH = {"mixed": 150, "tiles": 170, "edges": 140, "odd": 135}
F = torch.float64

# Largest difference from the plain implementation (float64), relative to the largest logit. In bfloat16 the router reads rounded rows,
# and with random weights a token now and then has two experts whose scores lie closer than that rounding: the engine then takes another
# expert than the float64 model, the norm behind the experts makes of that a row of its own, and tokens whose attention rests on it
# follow. (The plain model with its sublayers' inputs rounded to bfloat16 loses the same rows.) So in bfloat16 a share of a request's
# rows (OUTLIER_ROWS, two at least, one of a short request's) may exceed the limit on single logits, and both limits are then held
# over the other rows; 32-bit has no such allowance, and it runs the same code around its kernels.
LIMITS = {"float32": dict(max=6e-5, rms=5e-6), "bfloat16": dict(max=1e-1, rms=2.5e-2)}
OUTLIER_ROWS = 0.1
WORST = {}


def assert_logits(got, want, dtype, what):
    assert torch.isfinite(got).all(), f"{what}: logits are not finite"
    worst, rms = errors(got, want)
    if dtype == "bfloat16" and (worst > LIMITS[dtype]["max"] or rms > LIMITS[dtype]["rms"]):
        diff = (got.double().cpu() - want.double()) / float(want.abs().max())
        per_row = diff.abs().max(dim=1).values
        allowed = 1 if want.shape[0] < 20 else max(2, int(OUTLIER_ROWS * want.shape[0]))
        kept = per_row.argsort()[:want.shape[0] - allowed]
        assert int((per_row > LIMITS[dtype]["max"]).sum()) <= allowed, \
            f"{what} [{dtype}]: rows {(per_row > LIMITS[dtype]['max']).nonzero().flatten().tolist()} of {want.shape[0]} exceed {LIMITS[dtype]['max']:.1e}"
        worst, rms = float(per_row[kept].max()), float(diff[kept].pow(2).mean().sqrt())
    seen = WORST.setdefault(dtype, [0.0, 0.0])
    seen[0], seen[1] = max(seen[0], worst), max(seen[1], rms)
    assert worst <= LIMITS[dtype]["max"] and rms <= LIMITS[dtype]["rms"], \
        f"{what} [{dtype}]: max error {worst:.3e} (limit {LIMITS[dtype]['max']:.1e}), rms {rms:.3e} (limit {LIMITS[dtype]['rms']:.1e})"


def first_bad_position(got, want, dtype):
    scale = float(want.abs().max())
    for t in range(want.shape[0]):
        if float((got[t].double().cpu() - want[t].double()).abs().max()) / scale > LIMITS[dtype]["max"]:
            return t
    return None


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (folder, plain model, ids, plain logits)"""
    out = {}
    for index, name in enumerate(NAMES):
        folder = make_mitunex_folder(CONFIGS[name], tmp_path_factory.mktemp(name), seed=31 + index)
        plain = P.PlainModel(folder)
        ids = token_ids(CONFIGS[name]["vocab"], LENGTH[name], seed=700 + index)
        out[name] = (folder, plain, ids, plain.logits(ids))
    return out


@pytest.fixture(scope="module")
def engines(models):
    from xeno_rt_amd.engine import Engine
    cache = {}

    def get(name, dtype):
        if (name, dtype) not in cache:
            cache[(name, dtype)] = Engine.load(models[name][0], dtype=dtype, max_tokens=64 * 9, max_slots=3)
        return cache[(name, dtype)]
    return get


@pytest.fixture(scope="module")
def ops():
    from xeno_rt_amd.ops import load_ops
    return load_ops()


# ---- the model under every schedule ----------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts(name, dtype, models, engines):
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    got = run_whole(engine, ids)
    assert_logits(got, want, dtype, f"mitunex {name} whole, first bad row {first_bad_position(got, want, dtype)}")
    for length in (1, 2, 3, 66):                                    # the first tokens of a sequence, and just past a block
        got = run_whole(engine, ids[:length])
        assert_logits(got, want[:length], dtype, f"mitunex {name} whole, {length} tokens")
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_token_by_token_from_the_first(name, dtype, models, engines):
    """Every token in a step of its own: long decoding through recorded steps, across cache blocks and windows' edges."""
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    got = in_portions(engine, ids, [1])
    assert_logits(got, want, dtype, f"mitunex {name} token by token, first bad row {first_bad_position(got, want, dtype)}")
    if dtype == "float32":
        assert same_but_for_rounding(got, run_whole(engine, ids)), "a decoded token differs from the same token in a prompt"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [[2], [3, 7], [64, 1], [65, 2, 2, 1, 30], [33], [1, 1, 2, 61, 5]])
@pytest.mark.parametrize("name", NAMES)
def test_portions(name, sizes, dtype, models, engines):
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    got = in_portions(engine, ids, sizes)
    assert_logits(got, want, dtype, f"mitunex {name} portions {sizes}, first bad row {first_bad_position(got, want, dtype)}")
    if dtype == "float32":
        assert same_but_for_rounding(got, run_whole(engine, ids)), f"portions {sizes} change more than the rounding"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_unequal_batches_through_reused_slots(name, dtype, models, engines):
    """Three requests of different lengths start together and end one after the other, twice over, so that the second round runs
    in slots and blocks that the first has used."""
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    vocab = CONFIGS[name]["vocab"]
    requests = [ids, token_ids(vocab, 37, seed=900), token_ids(vocab, 71, seed=901)]
    wants = [want, plain.logits(requests[1]), plain.logits(requests[2])]
    for prompts in ([len(ids) - 40, 5, 66], [3, 36, 1]):
        got = run_batched(engine, requests, prompts)
        for index, (g, w) in enumerate(zip(got, wants)):
            assert_logits(g, w, dtype, f"mitunex {name} batch {prompts} request {index}, first bad row {first_bad_position(g, w, dtype)}")
            if dtype == "float32":
                assert same_but_for_rounding(g, run_whole(engine, requests[index])), "a request depends on its batch"
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_step_that_mixes_prompts_portions_and_decoded_tokens(dtype, models, engines):
    engine = engines("tiles", dtype)
    _, plain, ids, want = models["tiles"]
    other = token_ids(CONFIGS["tiles"]["vocab"], 90, seed=5)
    want_other = plain.logits(other)
    a, b, c = (engine.alloc_slot() for _ in range(3))
    try:
        engine.step([(a, ids[:100], []), (b, other[:89], [])])
        logits = engine.step([(b, other[89:], [0]), (c, ids[:50], [49]), (a, ids[100:140], [0, 39])])
        rows = torch.cat([want_other[89:], want[49:50], want[100:101], want[139:140]])
        assert_logits(logits, rows, dtype, "mitunex tiles, a mixed step")
    finally:
        for slot in (a, b, c):
            engine.free_slot(slot)
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_loop(dtype, models, engines):
    from xeno_rt_amd.engine import GenerateRequest, generate
    name = "mixed"
    engine = engines(name, dtype)
    _, plain, ids, _ = models[name]
    prompts = [ids[:9], ids[20:21], ids[40:75]]
    requests = [GenerateRequest(p, max_tokens=8, temperature=0.0, repetition_penalty=1.0, stop_ids=[]) for p in prompts]
    got = [r.tokens for r in generate(engine, requests)]
    for prompt, tokens in zip(prompts, got):
        assert len(tokens) == 8
        history = list(prompt)
        for index, token in enumerate(tokens):
            row = plain.logits(history)[-1]
            if dtype == "float32":
                assert token == int(row.argmax()), f"token {index} is {token}, the plain loop chooses {int(row.argmax())}"
            else:
                assert float(row.max() - row[token]) <= 0.1 * float(row.abs().max()), f"token {index} ({token}) is not among the best"
            history.append(token)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_request_decoded_far_past_its_prompt_keeps_only_its_windows(dtype, models, engines):
    """500 tokens, the last 300 of them decoded one by one: the windows' blocks are let go of and used again on the way."""
    engine = engines("mixed", dtype)
    _, plain, _, _ = models["mixed"]
    ids = token_ids(CONFIGS["mixed"]["vocab"], 500, seed=77)
    want = plain.logits(ids)
    slot = engine.alloc_slot()
    try:
        rows = [engine.step([(slot, ids[:200], list(range(200)))])]
        for token in ids[200:]:
            rows.append(engine.step([(slot, [token], [0])]))
            assert engine.cache.held_blocks() <= 3, "a window of 65 tokens needs three blocks at most"
    finally:
        engine.free_slot(slot)
    got = torch.cat(rows)
    assert_logits(got, want, dtype, f"mitunex mixed long decoding, first bad row {first_bad_position(got, want, dtype)}")
    engine.cache.check()


def test_a_sequence_ends_where_the_table_of_positions_does(models, engines):
    from xeno_rt_amd.engine import Engine, StepError
    folder, plain, _, _ = models["odd"]
    engine = Engine.load(folder, dtype="float32", max_tokens=1024, max_slots=2)
    assert engine.max_context == CONFIGS["odd"]["max_positions"]
    ids = token_ids(CONFIGS["odd"]["vocab"], engine.max_context + 1, seed=3)
    slot = engine.alloc_slot()
    engine.step([(slot, ids[:-2], [])])
    got = engine.step([(slot, [ids[-2]], [0])])
    assert_logits(got, plain.logits(ids[:-1])[-1:], "float32", "the last position")
    with pytest.raises(StepError):
        engine.step([(slot, [ids[-1]], [0])])
    engine.free_slot(slot)


# ---- what enters the stream, what is added to it, what leaves it --------------------------------------------------------------

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [50, 72, 256, 1000, 4096])
def test_the_embedding_with_positions_and_norm(width, dtype, ops):
    vocab, rows = 40, 30
    generator = torch.Generator().manual_seed(width)
    table, positions, gain = (torch.randn(*shape, generator=generator).to(dtype) for shape in ((vocab, width), (rows, width), (width,)))
    ids = torch.randint(0, vocab, (33,), generator=generator, dtype=torch.int32)
    at = torch.randint(0, rows, (33,), generator=generator, dtype=torch.int32)
    at[0], at[1] = rows - 1, 0
    want = P.rms_norm(table[ids.long()].double() + positions[at.long()].double(), gain, 1e-3)
    out, copy = torch.empty(33, width, device="cuda"), torch.empty(33, width, dtype=dtype, device="cuda")
    ops.embed_normed(table.cuda(), ids.cuda(), gain.cuda(), 1e-3, out, positions_table=positions.cuda(), positions=at.cuda(), copy=copy)
    assert float((out.double().cpu() - want).abs().max()) <= 2e-6 * float(want.abs().max())
    assert torch.equal(copy, out.to(dtype)), "the copy is the row, rounded once"
    ops.embed_normed(table.cuda(), ids.cuda(), gain.cuda(), 1e-3, out)
    want = P.rms_norm(table[ids.long()].double(), gain, 1e-3)
    assert float((out.double().cpu() - want).abs().max()) <= 2e-6 * float(want.abs().max())


@pytest.mark.parametrize("gain_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [50, 64, 256, 1000, 4096, 20000])
def test_a_normed_output_is_added_to_the_stream_and_the_stream_copied(width, gain_dtype, ops):
    generator = torch.Generator().manual_seed(width)
    x, y, gain = torch.randn(7, width, generator=generator), 3.0 * torch.randn(7, width, generator=generator), torch.randn(width, generator=generator).to(gain_dtype)
    want = x.double() + 0.5 * P.rms_norm(y.double(), gain, 1e-2)
    for copy_dtype in (None, torch.float32, torch.bfloat16):
        stream = x.cuda()
        copy = None if copy_dtype is None else torch.empty(7, width, dtype=copy_dtype, device="cuda")
        ops.add_normed(stream, [(y.cuda(), gain.cuda())], 1e-2, 0.5, copy=copy)
        assert float((stream.double().cpu() - want).abs().max()) <= 2e-6 * float(want.abs().max())
        assert copy is None or torch.equal(copy, stream.to(copy_dtype))
    stream, copy = x.cuda(), torch.empty(7, width, dtype=torch.bfloat16, device="cuda")
    ops.add_normed(stream, [(y.cuda(), gain.cuda()), (y.cuda(), gain.cuda())], 1e-2, 0.25, copy=copy)
    assert float((stream.double().cpu() - want).abs().max()) <= 2e-6 * float(want.abs().max()) and torch.equal(copy, stream.bfloat16())


def test_the_cap_follows_the_scale(ops):
    z = 20.0 * torch.randn(5, 33, generator=torch.Generator().manual_seed(0))
    for cap, scale in ((30.0, 1.0), (7.0, 2.5), (None, 0.5)):
        x = z.cuda()
        ops.softcap(x, cap, scale=scale)
        want = z.double() * scale
        want = want if cap is None else cap * torch.tanh(want / cap)
        assert float((x.double().cpu() - want).abs().max()) <= 2e-6 * float(want.abs().max())


@pytest.mark.parametrize("count", [(3, 7), (5, 64), (9, 1000)])
def test_gelus_tanh_form(count, ops):
    z = 3.0 * torch.randn(*count, generator=torch.Generator().manual_seed(1))
    z[0, :4] = torch.tensor([0.0, -12.0, 12.0, 1e-3])
    want = P.gelu_tanh(z.double())
    for x_dtype, out_dtype in ((torch.float32, torch.float32), (torch.float32, torch.bfloat16), (torch.bfloat16, torch.bfloat16)):
        out = torch.empty(*count, dtype=out_dtype, device="cuda")
        ops.activation(z.to(x_dtype).cuda(), out, "gelu_tanh")
        limit = 1e-6 if out_dtype == torch.float32 else 5e-3 if x_dtype == torch.float32 else 2e-2
        assert float((out.double().cpu() - want).abs().max()) <= limit * float(want.abs().max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_dense_feed_forward_alone(dtype, ops):
    from xeno_rt_amd.parts import DenseMLP
    width, ff = 56, 90
    part = DenseMLP("mlp.", width, ff, "gelu_tanh")
    tensors = tensors_for(part, seed=1, std=0.3)
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(21, width, generator=torch.Generator().manual_seed(2)).to(dtype)
    want = P.dense(h.double(), short(tensors, "mlp."))
    out, residual = torch.empty(21, width, device="cuda"), torch.ones(21, width, device="cuda")
    part.forward_into(h.cuda(), None, out)
    part.forward(h.cuda(), None, residual)
    limit = (1e-5 if dtype == torch.float32 else 2e-2) * float(want.abs().max())
    assert float((out.double().cpu() - want).abs().max()) <= limit and float((residual.double().cpu() - 1.0 - want).abs().max()) <= limit


# ---- attention through a latent under a window ----------------------------------------------------------------------------------

def plain_windowed(q, k, v, n_heads, scale, window, sink=None):
    """One key/value head: q [tokens, n_heads * dim], k [tokens, dim], v [tokens, vdim]."""
    length = q.shape[0]
    q = q.double().reshape(length, n_heads, -1)
    scores = torch.einsum("ihd,jd->hij", q, k.double()) * scale
    scores = scores.masked_fill(~P.window_mask(length, window), -math.inf)
    if sink is not None:
        scores = torch.cat([scores, sink.double()[:, None, None].expand(n_heads, length, 1)], dim=-1)
    weights = torch.softmax(scores, dim=-1)[..., :length]
    return torch.einsum("hij,je->ihe", weights, v.double()).reshape(length, -1)


def attend(ops, q, k, v, cuts, dtype, n_heads, dim, vdim, ahead=0, **options):
    """Keys and values through `kv_store` into a paged cache, then the attention on the queries alone, step by step. Every step may
    bring `ahead` tokens of a sequence of no slot before the sequence's own."""
    from xeno_rt_amd.parts.base import CacheNeeds, KVSpec
    cache = layer_cache(CacheNeeds(kv=KVSpec(1, dim, None, vdim)), dtype, q.shape[0])
    rows, at = [], 0
    for count in cuts:
        if count == 0:
            continue
        step = Step([-1, 1], [ahead, count], [0, at]) if ahead else Step([1], [count], [at])
        cut = lambda t: torch.cat([torch.ones(ahead, t.shape[1]), t[at:at + count].float()]).to(dtype).cuda()
        ops.kv_store(cut(k), cut(v), 1, dim, vdim, cache.kv, step)
        out = torch.full((ahead + count, n_heads * vdim), float("nan"), dtype=dtype, device="cuda")
        ops.attention(cut(q), n_heads, 1, dim, cache.kv, step, out, value_dim=vdim, queries_alone=True, **options)
        assert not ahead or float(out[:ahead].float().abs().max()) == 0.0, "rows of no sequence are zeros"
        rows.append(out[ahead:])
        at += count
    return torch.cat(rows).double().cpu()


MATRIX_CORE_SIZES = [(16, 128, 96), (9, 224, 160), (20, 64, 32), (5, 448, 384), (33, 96, 64), (1, 32, 32), (3, 192, 192), (7, 320, 256), (2, 576, 512), (4, 640, 512)]


@pytest.mark.parametrize("n_heads,dim,vdim", MATRIX_CORE_SIZES)
@pytest.mark.parametrize("window", [None, 1, 31, 32, 33, 64, 90])
def test_windows_on_the_matrix_cores(window, n_heads, dim, vdim, ops):
    """bfloat16, key and value sizes in whole tiles: prompts and portions through one kernel, steps of few tokens through the other,
    against plain arithmetic, with windows smaller and larger than the kernels' groups of 32 keys and than a cache block."""
    length = 150
    generator = torch.Generator().manual_seed(dim + vdim + n_heads)
    q, k, v = (torch.randn(length, width, generator=generator).bfloat16().float() for width in (n_heads * dim, dim, vdim))
    scale = 0.6 / math.sqrt(dim)
    want = plain_windowed(q, k, v, n_heads, scale, window)
    for cuts in schedules(length) + [[40, 40, 40, 30]]:
        got = attend(ops, q, k, v, cuts, torch.bfloat16, n_heads, dim, vdim, scale=scale, window=window, ahead=3 if cuts[0] == 40 else 0)
        assert float((got - want).abs().max()) <= 2e-2 * float(want.abs().max()), f"window {window}, cuts {cuts[:4]}"


@pytest.mark.parametrize("window", [None, 33])
def test_a_sink_on_the_kernel_for_prompts(window, ops):
    n_heads, dim, vdim, length = 6, 96, 64, 150
    generator = torch.Generator().manual_seed(9)
    q, k, v = (torch.randn(length, width, generator=generator).bfloat16().float() for width in (n_heads * dim, dim, vdim))
    sink = torch.tensor([2.0, -40.0, 40.0, 0.0, 6.0, -3.0])
    want = plain_windowed(q, k, v, n_heads, 0.1, window, sink)
    for cuts in ([length], [70, 80], [length - 3, 1, 2]):
        got = attend(ops, q, k, v, cuts, torch.bfloat16, n_heads, dim, vdim, scale=0.1, window=window, sink=sink.cuda())
        assert float((got - want).abs().max()) <= 2e-2 * float(want.abs().max()), f"cuts {cuts}"


def test_a_prompts_scores_that_grow_along_the_keys_move_the_exponent(ops):
    """Scores that rise by far more than 2^8 from one group of keys to the next, fall again, and differ from row to row."""
    n_heads, dim, vdim, length = 3, 64, 32, 200
    generator = torch.Generator().manual_seed(4)
    q, k, v = (torch.randn(length, width, generator=generator) for width in (n_heads * dim, dim, vdim))
    k[:, 0] = torch.linspace(0.0, 60.0, length)
    k[100:, 1] = 80.0
    q[:, 0::dim] = torch.randn(length, n_heads, generator=generator)
    q, k, v = q.bfloat16().float(), k.bfloat16().float(), v.bfloat16().float()
    for window in (None, 70):
        want = plain_windowed(q, k, v, n_heads, 1.0, window)
        got = attend(ops, q, k, v, [length], torch.bfloat16, n_heads, dim, vdim, scale=1.0, window=window)
        assert float((got - want).abs().max()) <= 2e-2 * float(want.abs().max())


@pytest.mark.parametrize("dtype,n_heads,dim,vdim", [(torch.float32, 2, 32, 16), (torch.bfloat16, 2, 128, 96), (torch.bfloat16, 18, 96, 64), (torch.bfloat16, 3, 40, 24)])
@pytest.mark.parametrize("window", [41, 64, 65, 300])
def test_a_key_just_inside_a_window_is_found_and_one_just_outside_is_not(window, dtype, n_heads, dim, vdim, ops):
    """One key towers over all others: the query for which it is the window's last key reads its value, the next query does not, wherever
    the key lies in its block, in a prompt, in a portion and decoded."""
    length = 660
    generator = torch.Generator().manual_seed(window)
    for key in (0, 1, 31, 32, 63, 64, 65, 127, 200, 300):
        q, k, v = (0.05 * torch.randn(length, width, generator=generator) for width in (n_heads * dim, dim, vdim))
        last = key + window - 1
        q[key:] = 3.0
        k[key], v[key] = 3.0, 7.0
        for cuts in ([length], [last - 5] + [1] * 12 + [length - last - 7], [key + 1, last - key - 1, 40, length - last - 40]):
            got = attend(ops, q, k, v, cuts, dtype, n_heads, dim, vdim, scale=3.2 / dim, window=window)
            inside, outside = got[key:last + 1], got[last + 1:last + 9]
            assert float((inside - 7.0).abs().max()) < 0.1, f"key {key} is not seen at {int((inside - 7.0).abs().max(dim=1).values.argmax()) + key}, cuts {cuts[:3]}"
            assert float(outside.abs().max()) < 0.5, f"key {key} is seen beyond a window of {window}, cuts {cuts[:3]}"


@pytest.mark.parametrize("key", [0, 1, 63, 64, 65, 511, 512, 700, 1500])
def test_one_key_far_back_is_found_by_the_kernel_for_prompts(key, ops):
    n_heads, dim, vdim, length = 5, 96, 64, 1700
    generator = torch.Generator().manual_seed(key)
    q, k, v = (0.1 * torch.randn(length, width, generator=generator) for width in (n_heads * dim, dim, vdim))
    q[-20:], k[key] = 3.0, 3.0
    v[key] = 7.0
    for cuts in ([length], [length - 40, 40], [length - 20] + [1] * 20):
        got = attend(ops, q, k, v, cuts, torch.bfloat16, n_heads, dim, vdim, scale=0.1 * 32 / dim)
        assert float((got[-20:] - 7.0).abs().max()) < 0.1, f"key {key}, cuts {cuts[:2]}"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("dim,vdim", [(700, 516), (1024, 768), (600, 40)])
def test_heads_larger_than_the_matrix_core_kernels_take(dim, vdim, dtype, ops):
    n_heads, length = 3, 130
    generator = torch.Generator().manual_seed(dim)
    q, k, v = (torch.randn(length, width, generator=generator).to(dtype).float() for width in (n_heads * dim, dim, vdim))
    for window in (None, 70):
        want = plain_windowed(q, k, v, n_heads, 0.03, window)
        for cuts in ([length], [length - 4] + [1] * 4):
            got = attend(ops, q, k, v, cuts, dtype, n_heads, dim, vdim, scale=0.03, window=window)
            assert float((got - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 2e-2) * float(want.abs().max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,dim,rot_dim,rank", [(3, 16, 8, 24), (7, 32, 32, 96), (5, 7, 2, 9), (1, 40, 64, 96)])
def test_one_launch_prepares_what_two_would(heads, dim, rot_dim, rank, dtype, ops):
    from xeno_rt_amd.parts.base import CacheNeeds, KVSpec
    tokens, q_width = 70, heads * (dim + rot_dim)
    generator = torch.Generator().manual_seed(rank)
    sums = torch.randn(tokens + 2, q_width + rank + rot_dim + 3, generator=generator).cuda()
    gain = (1 + 0.3 * torch.randn(rank, generator=generator)).to(dtype).cuda()
    frequencies = torch.tensor([50.0 ** (-2.0 * i / rot_dim) for i in range(rot_dim // 2)], device="cuda")
    step = Step([-1, 1], [2, tokens], [0, 0])
    q, down = sums[:, :q_width], sums[:, q_width:q_width + rank + rot_dim]
    made = []
    for together in (True, False):
        cache = layer_cache(CacheNeeds(kv=KVSpec(1, rank + rot_dim, None, rank)), dtype, tokens)
        plain, full = (torch.zeros(tokens + 2, heads * width, dtype=dtype, device="cuda") for width in (dim, rank + rot_dim))
        if together:
            ops.latent_prepare(q, down, heads, dim, rank, rot_dim, gain, 1e-5, frequencies, rot_dim, cache.kv, step, plain, full)
        else:
            ops.latent_complete(down, rank, rot_dim, gain, 1e-5, frequencies, rot_dim, cache.kv, step, like=plain)
            ops.latent_queries(q, heads, dim, rot_dim, frequencies, rot_dim, step, plain, full, rank)
        made.append((plain, full, cache.kv.k, cache.kv.v))
    assert all(torch.equal(a, b) for a, b in zip(*made)) and float(made[0][2].float().abs().max()) > 0
    # one token alone, whose row lies nowhere apart from others
    cache = layer_cache(CacheNeeds(kv=KVSpec(1, rank + rot_dim, None, rank)), dtype, tokens)
    one, rest = torch.zeros(1, heads * dim, dtype=dtype, device="cuda"), torch.zeros(1, heads * (rank + rot_dim), dtype=dtype, device="cuda")
    ops.latent_prepare(q[2:3], down[2:3], heads, dim, rank, rot_dim, gain, 1e-5, frequencies, rot_dim, cache.kv, Step([1], [1], [0]), one, rest)
    assert torch.equal(one, made[0][0][2:3]) and torch.equal(rest, made[0][1][2:3])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("tokens,heads,n,k", [(1, 3, 24, 16), (5, 7, 72, 96), (16, 2, 33, 64), (17, 2, 33, 64), (70, 5, 40, 8), (200, 1, 80, 72), (600, 3, 70, 96), (512, 2, 64, 32)])
def test_a_heads_outputs_times_the_sigmoid_of_its_gate(tokens, heads, n, k, dtype, ops):
    generator = torch.Generator().manual_seed(n + k)
    a, w = torch.randn(tokens, heads * k, generator=generator).to(dtype), torch.randn(heads, n, k, generator=generator).to(dtype)
    sums = 2.0 * torch.randn(tokens, heads + 5, generator=generator)
    gates = torch.sigmoid(sums[:, 3:3 + heads].double())
    want = torch.einsum("thk,hnk->thn", a.double().reshape(tokens, heads, k), w.double()) * gates[..., None]
    out = torch.zeros(tokens, heads * (n + 3), dtype=dtype, device="cuda")
    ops.linear_heads(a.cuda(), w.cuda(), out, out_head=n + 3, gate_logits=sums.cuda()[:, 3:3 + heads])
    got = out.double().cpu().reshape(tokens, heads, n + 3)
    assert float((got[..., :n] - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())
    assert float(got[..., n:].abs().max()) == 0.0, "what lies behind a head's outputs was touched"
    if dtype == torch.bfloat16 and k % 32 == 0:                 # on the matrix cores a row has the same bits in any company
        for some in (1, 7, 30):
            if some < tokens:
                fewer = torch.zeros(some, heads * (n + 3), dtype=dtype, device="cuda")
                ops.linear_heads(a[tokens - some:].cuda(), w.cuda(), fewer, out_head=n + 3, gate_logits=sums.cuda()[tokens - some:, 3:3 + heads])
                assert torch.equal(fewer, out[tokens - some:])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m", [layer["mixer"] for name in sorted(CONFIGS) for layer in CONFIGS[name]["layers"] if "weights_of" not in layer]
                         + [_layer(3, 128, 64, 96, 448, 0.08, 5e5, 77, None)["mixer"], _layer(2, 24, 16, 40, 620, 0.1, 100.0, 30, None)["mixer"]])
def test_latent_attention_alone(m, dtype, ops):
    from xeno_rt_amd.models.mitunex import _mixer
    width, length = 48, 150
    part = _mixer(m, "mix.", types.SimpleNamespace(width=width, norm_eps=1e-5))
    tensors = tensors_for(part, seed=m["kv_rank"], std=0.25, norm=(1.0, 0.3), g=(0.0, 0.5))
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(length, width, generator=torch.Generator().manual_seed(1)).to(dtype)
    want = P.latent_attention(h.double(), short(tensors), m, 1e-5)
    limit = 3e-5 if dtype == torch.float32 else 5e-2
    for padding, cuts in ((2, [length]), (0, [length]), (2, [1] * length), (0, [length - 20] + [1] * 20), (2, [3, 64, 2, length - 69])):
        cache = layer_cache(part.cache_needs(), dtype, length)
        got = run_mixer(part, h, cuts, cache, dtype, padding=padding)
        assert float((got - want).abs().max()) <= limit * float(want.abs().max()), f"cuts {cuts[:3]}"
    assert part.cache_needs().kv.window == (m.get("mask") or {}).get("size") and part.cache_needs().kv.head_dim == m["kv_rank"] + m["rot_dim"]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("window,sink,gate,q_rank", [(44, "sink", None, None), (None, "sink", "g", 24), (33, None, "g", 20), (None, None, None, 16), (20, "sink", "g", 12)])
def test_the_latent_attentions_options_in_other_combinations(window, sink, gate, q_rank, dtype, ops):
    """A low rank for the queries with a window and a gate, a sink under a window, neither: the part serves other designs too."""
    from xeno_rt_amd.parts import LatentAttention
    width, length, m = 40, 130, dict(heads=3, dim=16, rot_dim=32, vdim=20, kv_rank=64, scale=0.2, rot={"dims": 16, "base": 100.0})
    part = LatentAttention("mix.", width, 3, 16, 32, 20, 64, q_rank, 0.2, 1e-5, 16, 100.0, sink=sink, window=window, output_gate=gate)
    tensors = tensors_for(part, seed=3, std=0.25, norm=(1.0, 0.3), sink=(0.5, 1.0), g=(0.0, 0.5))
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(length, width, generator=torch.Generator().manual_seed(1)).to(dtype)
    p, x = short(tensors), h.double()
    low = x if q_rank is None else P.rms_norm(x @ p["dq"].T, p["dq.norm"], 1e-5)
    q = (low @ p["q" if q_rank is None else "uq"].T).reshape(length, 3, 48)
    latent, turned = P.latent_rows(x, p, m, 1e-5)
    scores = (torch.einsum("ihd,jhd->hij", q[..., :16], (latent @ p["uk"].T).reshape(length, 3, 16))
              + torch.einsum("ihr,jr->hij", P.turn_neighbours(q[..., 16:], 16, 100.0), turned)) * 0.2
    scores = scores.masked_fill(~P.window_mask(length, window), -math.inf)
    weights = scores.exp() / (scores.exp().sum(dim=-1, keepdim=True) + (p["sink"].exp()[:, None, None] if sink else 0.0))
    o = torch.einsum("hij,jhe->ihe", weights, (latent @ p["uv"].T).reshape(length, 3, 20))
    o = o if gate is None else o * P.head_gate(x, p["g"])[..., None]
    want = o.reshape(length, -1) @ p["o"].T
    for padding, cuts in ((0, [length]), (2, [length - 20] + [1] * 20), (0, [3, 64, 2, length - 69])):
        got = run_mixer(part, h, cuts, layer_cache(part.cache_needs(), dtype, length), dtype, padding=padding)
        assert float((got - want).abs().max()) <= (3e-5 if dtype == torch.float32 else 5e-2) * float(want.abs().max()), f"cuts {cuts[:3]}"


# ---- experts ---------------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("normalized", [True, False])
@pytest.mark.parametrize("experts,top", [(8, 1), (6, 3), (5, 5), (64, 8), (65, 2), (256, 7)])
def test_sigmoid_scores_choose_without_groups(experts, top, normalized, ops):
    tokens = 301
    logits = 2.0 * torch.randn(tokens, experts + 3, generator=torch.Generator().manual_seed(experts))
    weights, chosen = torch.full((tokens, experts), float("nan"), device="cuda"), torch.full((tokens, top), -1, dtype=torch.int32, device="cuda")
    ops.route_experts(logits.cuda()[:, 1:1 + experts], weights, top, chosen=chosen, scale=1.5, normalized=normalized)
    for t in range(tokens):
        picked, scores = P.choose(logits[t, 1:1 + experts].double(), top)
        total = sum(scores) if normalized else 1.0
        assert chosen[t].tolist() == picked
        assert weights[t].nonzero().flatten().tolist() == sorted(picked)
        assert weights[t, picked].tolist() == pytest.approx([1.5 * s / total for s in scores], rel=1e-5)


def test_among_equal_logits_the_lower_expert_wins_and_scores_of_one_are_still_told_apart(ops):
    logits = torch.zeros(3, 130)
    logits[1, [7, 70, 129]] = 1.0
    logits[2, 128], logits[2, 3] = 100.0, 40.0                   # (in float32 sigmoid(100) and sigmoid(40) are both one)
    weights, chosen = torch.empty(3, 130, device="cuda"), torch.empty(3, 4, dtype=torch.int32, device="cuda")
    ops.route_experts(logits.cuda(), weights, 4, chosen=chosen, normalized=False)
    assert chosen.tolist() == [[0, 1, 2, 3], [7, 70, 129, 0], [128, 3, 0, 1]]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("weigh_input", [True, False])
@pytest.mark.parametrize("experts,width,shared", [(4, 24, 40), (3, 9, 5), (6, 64, 0), (2, 4, 8), (5, 8, 16)])
def test_the_experts_activations_from_their_sums(experts, width, shared, weigh_input, dtype, ops):
    tokens, total = 23, experts * width + shared
    generator = torch.Generator().manual_seed(total)
    gate, up = torch.randn(tokens, total, generator=generator), torch.randn(tokens, total, generator=generator)
    weights = torch.rand(tokens, experts, generator=generator) * (torch.rand(tokens, experts, generator=generator) < 0.5)
    logits = torch.randn(tokens, 4, generator=generator)
    w = weights.double().repeat_interleave(width, dim=1)
    g, u = gate[:, :experts * width].double(), up[:, :experts * width].double()
    want = P.silu(w * g) * (w * u) if weigh_input else P.silu(g) * u * w
    want = torch.cat([want, P.silu(gate[:, experts * width:].double()) * up[:, experts * width:].double() * torch.sigmoid(logits[:, 2:3].double())], dim=1)
    layouts = {False: torch.cat([gate, up], dim=1)}
    if total % 8 == 0:
        layouts[True] = torch.stack([gate.reshape(tokens, -1, 8), up.reshape(tokens, -1, 8)], dim=2).reshape(tokens, -1)
    for interleaved, sums in layouts.items():
        out = torch.full((tokens, total), float("nan"), dtype=dtype, device="cuda")
        ops.glu_experts(sums.contiguous().cuda(), out, weights.cuda(), width, shared_width=shared, shared_logits=logits.cuda()[:, 2] if shared else None,
                        weigh_input=weigh_input, interleaved=interleaved)
        assert float((out.double().cpu() - want).abs().max()) <= (1e-6 if dtype == torch.float32 else 1e-2) * float(want.abs().max())
        assert float(out[:, :experts * width].double().cpu()[w == 0].abs().sum()) == 0.0


def experts_part(raw, width, seed, ops, dtype, pack="auto", weigh_input=True):
    from xeno_rt_amd.parts import ExpertsMLP
    from xeno_rt_amd.parts.base import Runtime
    part = ExpertsMLP("mlp.", width, raw["expert"]["ff"], raw["router"]["experts"], raw["router"]["top"], normalized=False, weigh_input=weigh_input,
                      shared=None if "shared" not in raw else raw["shared"]["ff"])
    tensors = tensors_for(part, seed=seed, std=0.3, router=(0.0, 0.7), sg=(0.0, 0.5))
    part.bind(tensors, Runtime(ops, dtype, "cuda", pack_weights=pack))
    return part, tensors


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("raw", [_moe(24, 6, 2, 40), _moe(9, 3, 2, 5), _moe(64, 4, 1, 128), _moe(16, 5, 5), _moe(40, 7, 3, 8)])
def test_experts_alone(raw, dtype, ops):
    width, tokens = 48, 61
    part, tensors = experts_part(raw, width, 7, ops, dtype)
    h = torch.randn(tokens, width, generator=torch.Generator().manual_seed(5)).to(dtype)
    want = P.experts(h.double(), short(tensors, "mlp."), raw)
    out, residual = torch.empty(tokens, width, device="cuda"), torch.ones(tokens, width, device="cuda")
    part.forward_into(h.cuda(), None, out)
    part.forward(h.cuda(), None, residual)
    limit = 2e-5 if dtype == torch.float32 else 3e-2
    for got in (out.double().cpu(), residual.double().cpu() - 1.0):
        per_row = (got - want).abs().max(dim=1).values / float(want.abs().max())
        assert int((per_row > limit).sum()) <= (0 if dtype == torch.float32 else 2), f"rows {(per_row > limit).nonzero().flatten().tolist()} differ"


@pytest.mark.parametrize("weigh_input", [True, False])
@pytest.mark.parametrize("pack", ["auto", "always"])
@pytest.mark.parametrize("raw,tokens", [(_moe(64, 8, 2, 128), 300), (_moe(128, 16, 4, 64), 1000), (_moe(192, 4, 1), 600), (_moe(64, 3, 1, 320), 401)])
def test_experts_multiply_only_the_tokens_that_chose_them(raw, tokens, pack, weigh_input, ops):
    """A step of many tokens sorts its picks by expert, the shared expert beside them: against the plain sum, and against the same part
    with every token through every expert."""
    width = 64
    part, tensors = experts_part(raw, width, 8, ops, torch.bfloat16, pack, weigh_input)
    options = {} if part.shared is None else {"shared_width": part.shared}
    takes = ops.experts_sorted_takes
    h = torch.randn(tokens, width, generator=torch.Generator().manual_seed(6)).bfloat16()
    assert takes(h.cuda(), part.w_gate_up, part.w_down, part.experts, part.intermediate, part.top, **options)
    assert not takes(h[:8].cuda(), part.w_gate_up, part.w_down, part.experts, part.intermediate, part.top, **options)
    out = torch.full((tokens, width), float("nan"), device="cuda")
    part.forward_into(h.cuda(), None, out)
    ops.experts_sorted_takes = lambda *operands, **named: False
    try:
        dense = torch.empty(tokens, width, device="cuda")
        part.forward_into(h.cuda(), None, dense)
    finally:
        ops.experts_sorted_takes = takes
    p = short(tensors, "mlp.")
    if weigh_input:
        want = P.experts(h.double(), p, raw)
    else:
        want = torch.zeros(tokens, width, dtype=F)
        for t in range(tokens):
            for e, w in zip(*P.choose(h[t].double() @ p["router"].T, part.top)):
                want[t] += w * P.expert(h[t:t + 1].double(), p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])[0]
        if part.shared is not None:
            want += torch.sigmoid(h.double() @ p["shared.sg"].T) * P.expert(h.double(), p["shared.gate"], p["shared.up"], p["shared.down"])
    scale = float(want.abs().max())
    assert float((out - dense).abs().max()) <= 2e-2 * scale
    per_row = (out.double().cpu() - want).abs().max(dim=1).values / scale
    assert int((per_row > 3e-2).sum()) <= max(2, tokens // 50), f"rows {(per_row > 3e-2).nonzero().flatten().tolist()} differ from the plain sum"
    some = torch.arange(tokens - 1, -1, -1)[:max(80, tokens // 3)]
    fewer = torch.empty(len(some), width, device="cuda")
    part.forward_into(h[some].cuda(), None, fewer)
    assert float((fewer - out[some.cuda()]).abs().max()) <= 2e-2 * scale


# ---- through the programs a user runs ----------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay_of_whole_requests_decoded_tails_and_batches(dtype, models, tmp_path):
    from test_trace_run_gpu import collect, replay, trace_batches, trace_tail, trace_whole
    folder, plain, _, _ = models["tiles"]
    vocab = CONFIGS["tiles"]["vocab"]
    lengths = {"a": 40, "b": 7, "c": 140, "d": 65, "e": 1, "f": 90}
    requests = {n: token_ids(vocab, length, seed=length) for n, length in lengths.items()}
    want = {n: plain.logits(ids) for n, ids in requests.items()}
    whole = trace_whole(requests)
    got_whole = collect(whole, replay(folder, dtype, tmp_path / "whole", whole, 256))
    tail = trace_tail(requests)
    got_tail = collect(tail, replay(folder, dtype, tmp_path / "tail", tail, 256))
    names = list(requests)
    batches = [{n: requests[n] for n in names[:3]}, {n: requests[n] for n in names[3:]}]
    batched = trace_batches(batches, lambda n, ids: max(1, len(ids) - 5 - ord(n) % 3))
    got_batched = collect(batched, replay(folder, dtype, tmp_path / "batched", batched, 384))
    for n in names:
        assert_logits(got_whole[n], want[n], dtype, f"trace whole {n}")
        assert_logits(got_tail[n], want[n], dtype, f"trace tail {n}")
        assert_logits(got_batched[n], want[n], dtype, f"trace batched {n}")


def test_the_command_line_generates_what_the_plain_loop_does(models):
    import os
    import subprocess
    import sys
    folder, plain, ids, _ = models["mixed"]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompts = [ids[:5], ids[30:31]]
    done = subprocess.run([sys.executable, os.path.join(root, "bin", "xrt"), "generate", "--model", folder, "--dtype", "float32",
                           "--prompt-ids", ";".join(",".join(map(str, p)) for p in prompts), "--max-tokens", "6",
                           "--temperature", "0", "--repetition-penalty", "1.0", "--stop-ids", ""],
                          capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr
    lines = [line for line in done.stdout.splitlines() if line.strip()]
    assert [[int(t) for t in line.split()] for line in lines] == [P.generate_greedy(plain, p, 6) for p in prompts]


# ---- configurations drawn at random: other sizes, orders and constants than any above -----------------------------------

def random_configuration(seed):
    import random
    r = random.Random(seed)
    layers = []
    for index in range(r.randint(2, 5)):
        if layers and r.random() < 0.35:
            source = r.randrange(len(layers))
            layers.append(dict(layers[source], weights_of=source))
            continue
        mlp = None
        if r.random() < 0.4:
            mlp = _dense(r.choice([8, 33, 96, 130]))
        elif r.random() < 0.85:
            experts = r.randint(1, 9)
            mlp = _moe(r.choice([6, 20, 64, 128]), experts, r.randint(1, experts), r.choice([None, 7, 32, 64, 192]))
        layers.append(_layer(r.randint(1, 20), r.choice([4, 12, 32]), r.choice([2, 16, 32, 64]), r.choice([6, 16, 36, 72]), r.choice([8, 30, 64, 96, 160]),
                             r.choice([0.1, 0.25]), r.choice([10.0, 1e4, 3e5]), r.choice([None, 1, 5, 32, 50, 64, 90]), mlp))
    return _model(r.choice([50, 97, 200]), r.choice([24, 40, 64, 96, 128]), r.choice([100, 512]), r.choice([1e-6, 1e-4]), r.choice([0.5, 1.0, 3.0]),
                  r.choice([5.0, 20.0]), layers)


@pytest.mark.parametrize("seed", range(12))
def test_configurations_drawn_at_random(seed, tmp_path):
    from xeno_rt_amd.engine import Engine
    raw = random_configuration(seed)
    folder = make_mitunex_folder(raw, tmp_path, seed=seed, std=0.1)
    plain = P.PlainModel(folder)
    ids = [token_ids(raw["vocab"], 100, seed=seed), token_ids(raw["vocab"], 31, seed=seed + 50)]
    wants = [plain.logits(i) for i in ids]
    for dtype in DTYPES:
        engine = Engine.load(folder, dtype=dtype, max_tokens=64 * 5, max_slots=2)
        assert_logits(run_whole(engine, ids[0]), wants[0], dtype, f"random configuration {seed} whole: {raw}")
        assert_logits(in_portions(engine, ids[0], [40, 2, 1]), wants[0], dtype, f"random configuration {seed} in portions: {raw}")
        for got, want in zip(run_batched(engine, ids, [80, 9]), wants):
            assert_logits(got, want, dtype, f"random configuration {seed} in a batch: {raw}")
        engine.cache.check()


def test_zz_the_largest_errors_seen_are_reported():
    for dtype, (worst, rms) in WORST.items():
        print(f"mitunex, largest errors against the plain model [{dtype}]: max {worst:.2e} (limit {LIMITS[dtype]['max']:.0e}), "
              f"rms {rms:.2e} (limit {LIMITS[dtype]['rms']:.0e})")
