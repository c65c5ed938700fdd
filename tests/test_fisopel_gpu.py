"""The Fisopel decoder on the GPU against the plain implementation (tests/plain_fisopel.py), for four small configurations that
differ in every size and option: whole prompts, token-by-token decoding from the first token, portions of several sizes, unequal
batches through reused slots, greedy generation through the library's loop and programs; and every mechanism alone against
plain arithmetic, with inputs made so that a far key, a window's edge, a kept token, a block's border or a sink shows."""
import math
import types

import pytest
import torch

from fisopel_models import CONFIGS, _attention, _latent, _moe, _model, make_fisopel_folder
from helpers import errors, run_batched, run_whole, token_ids
from test_renapel_gpu import Step, in_portions, layer_cache, run_mixer, runtime, same_but_for_rounding, schedules, short, tensors_for
import plain_fisopel as P

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
NAMES = sorted(CONFIGS)
LENGTH = {"mixed": 160, "tiles": 170, "edges": 150, "odd": 135}
F = torch.float64

# Largest difference from the plain implementation (float64), relative to the largest logit. In bfloat16 the router reads rounded rows,
# and with random weights a token now and then has two experts whose logits lie closer than that rounding: the engine then takes another
# expert than the float64 model, and that row, and a little of those whose attention rests on it, follow. So in bfloat16 a share of a
# request's rows (OUTLIER_ROWS, two at least, one of a short request's) may exceed the limit on single logits, and both limits are
# then held over the other rows; 32-bit has no such allowance, and it runs the same code around its kernels.
LIMITS = {"float32": dict(max=6e-6, rms=1e-6), "bfloat16": dict(max=1e-1, rms=2.5e-2)}
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
        folder = make_fisopel_folder(CONFIGS[name], tmp_path_factory.mktemp(name), seed=31 + index)
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
    assert_logits(got, want, dtype, f"fisopel {name} whole, first bad row {first_bad_position(got, want, dtype)}")
    for length in (1, 2, 3, 66):                                    # the first tokens of a sequence, and just past a block
        got = run_whole(engine, ids[:length])
        assert_logits(got, want[:length], dtype, f"fisopel {name} whole, {length} tokens")
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_token_by_token_from_the_first(name, dtype, models, engines):
    """Every token in a step of its own: long decoding through recorded steps, across cache blocks and windows' edges."""
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    got = in_portions(engine, ids, [1])
    assert_logits(got, want, dtype, f"fisopel {name} token by token, first bad row {first_bad_position(got, want, dtype)}")
    if dtype == "float32":
        assert same_but_for_rounding(got, run_whole(engine, ids)), "a decoded token differs from the same token in a prompt"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [[2], [3, 7], [64, 1], [65, 2, 2, 1, 30], [33], [1, 1, 2, 61, 5]])
@pytest.mark.parametrize("name", NAMES)
def test_portions(name, sizes, dtype, models, engines):
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    got = in_portions(engine, ids, sizes)
    assert_logits(got, want, dtype, f"fisopel {name} portions {sizes}, first bad row {first_bad_position(got, want, dtype)}")
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
            assert_logits(g, w, dtype, f"fisopel {name} batch {prompts} request {index}, first bad row {first_bad_position(g, w, dtype)}")
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
        assert_logits(logits, rows, dtype, "fisopel tiles, a mixed step")
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
@pytest.mark.parametrize("name", ["mixed", "tiles"])
def test_a_long_request_decoded_far_past_its_prompt_keeps_its_windows_and_its_first_tokens(name, dtype, models, engines):
    """500 tokens, the last 300 of them decoded one by one: the windows' blocks are let go of and used again on the way, those of the
    first tokens stay."""
    engine = engines(name, dtype)
    _, plain, _, _ = models[name]
    ids = token_ids(CONFIGS[name]["vocab"], 500, seed=77)
    want = plain.logits(ids)
    slot = engine.alloc_slot()
    windowed = [group for group in engine.cache.groups if group.spec.window is not None]
    try:
        rows = [engine.step([(slot, ids[:200], list(range(200)))])]
        for token in ids[200:]:
            rows.append(engine.step([(slot, [token], [0])]))
            for group in windowed:
                kept = (group.spec.keep_first + 63) // 64
                assert group.pool.n_held <= kept + (group.spec.window + 62) // 64 + 1
                assert all(block >= 0 for block in group.table[slot][:kept].tolist())
    finally:
        engine.free_slot(slot)
    assert windowed
    got = torch.cat(rows)
    assert_logits(got, want, dtype, f"fisopel {name} long decoding, first bad row {first_bad_position(got, want, dtype)}")
    engine.cache.check()


# ---- what enters the stream, what enters it again, what a layer reads of it ----------------------------------------------------

@pytest.mark.parametrize("width", [50, 64, 256, 1000])
@pytest.mark.parametrize("scale", [1.0, 3.5])
def test_the_embeddings_scale(scale, width, ops):
    table = torch.randn(40, width, generator=torch.Generator().manual_seed(width))
    ids = torch.tensor([3, 39, 0, 3, 17], dtype=torch.int32)
    tables = [table.cuda(), table.bfloat16().cuda()] + ([ops.pack(table.bfloat16().cuda(), "tiles")] if width % 32 == 0 else [])
    for kept in tables:
        out = torch.empty(5, width, device="cuda")
        ops.embed(kept, ids.cuda(), out, scale=scale)
        want = (table if kept.dtype == torch.float32 else table.bfloat16()).float()[ids.long()] * scale
        assert torch.equal(out.cpu(), want)


@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("gain_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [50, 64, 256, 1000, 4096, 12000])
def test_two_norms_of_the_same_rows_in_one_pass(width, gain_dtype, out_dtype, ops):
    generator = torch.Generator().manual_seed(width)
    x, a, b = 3.0 * torch.randn(7, width, generator=generator), torch.randn(width, generator=generator).to(gain_dtype), torch.randn(width, generator=generator).to(gain_dtype)
    outs = [torch.full((7, width), float("nan"), dtype=out_dtype, device="cuda") for _ in range(2)]
    ops.rmsnorm_two(x.cuda(), [a.cuda(), b.cuda()], 1e-2, outs)
    for out, gain in zip(outs, (a, b)):
        want = P.rms_norm(x.double(), gain, 1e-2)
        assert float((out.double().cpu() - want).abs().max()) <= (2e-6 if out_dtype == torch.float32 else 5e-3) * float(want.abs().max())
        alone = torch.empty(7, width, dtype=out_dtype, device="cuda")
        ops.rmsnorm(x.cuda(), gain.cuda(), 1e-2, alone)
        assert torch.equal(alone, out), "the norm alone gives other bits"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", [(3, 7), (5, 64), (1, 1), (9, 1000)])
def test_rows_are_copied_out_and_replaced(shape, dtype, ops):
    x, base = torch.randn(*shape), torch.randn(*shape)
    stream, copy = x.cuda(), torch.empty(*shape, dtype=dtype, device="cuda")
    ops.replace_rows(stream, base.cuda(), copy)
    assert torch.equal(stream.cpu(), base) and torch.equal(copy.cpu(), x.to(dtype))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,tokens", [(50, 3), (64, 1), (64, 70), (256, 16), (192, 300)])
def test_what_comes_before_a_pass(width, tokens, dtype, ops):
    from xeno_rt_amd.parts import PassEntry
    part = PassEntry("loop.in", width)
    tensors = tensors_for(part, seed=width, std=0.1)
    part.bind(tensors, runtime(ops, dtype))
    first, later = (torch.randn(tokens, width, generator=torch.Generator().manual_seed(n)) for n in (1, 2))
    opened = part.open(first.cuda())
    for x in (first, later):                                        # two passes: what the stream began with is the same for both
        stream = x.cuda()
        part.forward(stream, opened)
        want = P.enter_pass(x.double(), first.double(), tensors["loop.in"])
        assert float((stream.double().cpu() - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())


def test_a_layers_sublayers_read_the_same_stream_in_any_form_of_the_block(ops):
    """Each sublayer adding its own output in turn, and the sum of weighted terms (with a vector of ones) as the block's other form."""
    from xeno_rt_amd.models.fisopel import _feed_forward, _mixer
    from xeno_rt_amd.parts import ParallelBlock, RMSNorm
    c, layer = types.SimpleNamespace(width=48, norm_eps=1e-5), CONFIGS["mixed"]["layers"][1]
    x = torch.randn(40, 48, generator=torch.Generator().manual_seed(3))
    results = []
    for scales in ({}, {"mixer_scale": "ls1", "feed_forward_scale": "ls2"}):
        block = ParallelBlock(RMSNorm("", 48, 1e-5, name="norm1"), _mixer("attention", layer["mixer"], "mix.", c), _feed_forward(layer["mlp"], "mlp.", c), hidden=48,
                              feed_forward_norm=RMSNorm("", 48, 1e-5, name="norm2"), **scales)
        tensors = tensors_for(block, seed=5, std=0.2, norm1=(1.0, 0.3), norm2=(1.0, 0.3), norm=(1.0, 0.3), ls1=(1.0, 0.0), ls2=(1.0, 0.0))
        if results:
            tensors.update({name: t for name, t in results[0][1].items()})
        block.bind(tensors, runtime(ops, torch.float32))
        stream = x.cuda()
        block.forward(stream, Step([1], [40], [0]), layer_cache(block.cache_needs(), torch.float32, 40))
        results.append((stream.double().cpu(), tensors))
    want = P.add_layer(x.double(), {"l0." + n: t for n, t in results[0][1].items()}, 0, layer, 1e-5)
    for got, _ in results:
        assert float((got - want).abs().max()) <= 2e-5 * float(want.abs().max())


# ---- attention under a window that keeps a sequence's first tokens --------------------------------------------------------------

def plain_attention(q, k, v, n_heads, n_kv_heads, scale, window=None, keep_first=0, softcap=None, sink=None):
    """q [tokens, n_heads * dim], k [tokens, n_kv_heads * dim], v [tokens, n_kv_heads * vdim]."""
    length, group = q.shape[0], n_heads // n_kv_heads
    q = q.double().reshape(length, n_heads, -1)
    k, v = (t.double().reshape(length, n_kv_heads, -1).repeat_interleave(group, dim=1) for t in (k, v))
    scores = P.cap(torch.einsum("ihd,jhd->hij", q, k) * scale, softcap)
    weights = P.weights_with_sink(scores, P.seen(length, window, keep_first), sink)
    return torch.einsum("hij,jhe->ihe", weights, v).reshape(length, -1)


def forget(cache, at, window, keep_first):
    """What a window lets go of when a sequence has `at` tokens: the blocks leave the table, and what they held becomes no numbers."""
    first = max(0, at - window + 1) // 64
    for block in range((keep_first + 63) // 64, first):
        physical = int(cache.kv.block_table[1, block])
        if physical >= 0:
            cache.kv.k[physical], cache.kv.v[physical] = float("nan"), float("nan")
            cache.kv.block_table[1, block] = -1


def attend(ops, q, k, v, cuts, dtype, n_heads, n_kv_heads, dim, vdim, ahead=0, window=None, keep_first=0, **options):
    """Keys and values through `kv_store` into a paged cache, then the attention on the queries alone, step by step, the cache letting go
    of blocks between the steps. Every step may bring `ahead` tokens of a sequence of no slot before the sequence's own."""
    from xeno_rt_amd.parts.base import CacheNeeds, KVSpec
    cache = layer_cache(CacheNeeds(kv=KVSpec(n_kv_heads, dim, None, vdim)), dtype, q.shape[0])
    rows, at = [], 0
    for count in cuts:
        if count == 0:
            continue
        step = Step([-1, 1], [ahead, count], [0, at]) if ahead else Step([1], [count], [at])
        cut = lambda t: torch.cat([torch.ones(ahead, t.shape[1]), t[at:at + count].float()]).to(dtype).cuda()
        ops.kv_store(cut(k), cut(v), n_kv_heads, dim, vdim, cache.kv, step)
        out = torch.full((ahead + count, n_heads * vdim), float("nan"), dtype=dtype, device="cuda")
        ops.attention(cut(q), n_heads, n_kv_heads, dim, cache.kv, step, out, value_dim=vdim, queries_alone=True, window=window, keep_first=keep_first, **options)
        assert not ahead or float(out[:ahead].float().abs().max()) == 0.0, "rows of no sequence are zeros"
        rows.append(out[ahead:])
        at += count
        if window is not None:
            forget(cache, at, window, keep_first)
    return torch.cat(rows).double().cpu()


# heads, key/value heads, key size, value size: in whole tiles (the matrix-core kernels in bfloat16), and not
TILES = [(8, 2, 64, 96), (16, 16, 32, 32), (20, 1, 128, 64), (4, 2, 128, 128), (34, 2, 64, 64), (6, 3, 192, 160), (2, 1, 448, 384), (3, 1, 576, 512), (5, 5, 64, 128)]
OTHERS = [(9, 3, 64, 72), (4, 1, 40, 24), (5, 5, 7, 3), (12, 2, 100, 130), (2, 2, 33, 32)]


@pytest.mark.parametrize("dtype,sizes", [(torch.bfloat16, s) for s in TILES + OTHERS] + [(torch.float32, s) for s in OTHERS + TILES[:2] + TILES[6:7]])
@pytest.mark.parametrize("window,keep_first,softcap", [(None, 0, 1.5), (40, 4, None), (40, 0, 1.5), (33, 1, 0.7), (1, 65, 2.0), (64, 64, None), (90, 100, 3.0), (31, 33, None)])
def test_windows_kept_tokens_and_caps(window, keep_first, softcap, dtype, sizes, ops):
    n_heads, n_kv_heads, dim, vdim = sizes
    length = 230
    generator = torch.Generator().manual_seed(dim + vdim + n_heads)
    q, k, v = (torch.randn(length, width, generator=generator).bfloat16().float() for width in (n_heads * dim, n_kv_heads * dim, n_kv_heads * vdim))
    sink = torch.randn(n_heads, generator=generator) + 1.0
    scale = 1.5 / math.sqrt(dim)
    want = plain_attention(q, k, v, n_heads, n_kv_heads, scale, window, keep_first, softcap, sink)
    limit = (1e-5 if dtype == torch.float32 else 1.5e-2) * float(want.abs().max())
    for cuts in schedules(length) + [[40, 40, 40, 110], [100, 2, 1, 1, 16, 110]]:
        got = attend(ops, q, k, v, cuts, dtype, n_heads, n_kv_heads, dim, vdim, ahead=3 if cuts[0] == 40 else 0, scale=scale, window=window, keep_first=keep_first,
                     softcap=softcap, sink=sink.cuda())
        worst = (got - want).abs().max(dim=1).values
        assert float(worst.max()) <= limit, f"cuts {cuts[:4]}, row {int(worst.argmax())}: {float(worst.max()):.3e}"


@pytest.mark.parametrize("dtype,n_heads,n_kv_heads,dim,vdim", [(torch.float32, 2, 1, 32, 16), (torch.bfloat16, 4, 2, 64, 96), (torch.bfloat16, 18, 1, 128, 64), (torch.bfloat16, 6, 3, 40, 24)])
@pytest.mark.parametrize("window,keep_first", [(41, 4), (64, 1), (65, 64), (100, 65), (300, 2)])
def test_a_key_inside_a_window_or_kept_is_found_and_one_outside_is_not(window, keep_first, dtype, n_heads, n_kv_heads, dim, vdim, ops):
    """One key towers over all others: queries for which it lies in the window read its value, later ones only if it is one of the
    first that are kept, wherever it lies in its block, in a prompt, in a portion and decoded."""
    length = 660
    generator = torch.Generator().manual_seed(window)
    for key in sorted({0, keep_first - 1, keep_first, keep_first + 1, 31, 32, 63, 64, 127, 200, 300}):
        q, k, v = (0.05 * torch.randn(length, width, generator=generator) for width in (n_heads * dim, n_kv_heads * dim, n_kv_heads * vdim))
        last = key + window - 1
        q[key:] = 3.0
        k[key], v[key] = 3.0, 7.0
        for cuts in ([length], [last - 5] + [1] * 12 + [length - last - 7], [key + 1, last - key - 1, 40, length - last - 40]):
            got = attend(ops, q, k, v, cuts, dtype, n_heads, n_kv_heads, dim, vdim, scale=3.2 / dim, window=window, keep_first=keep_first, softcap=60.0)
            inside, outside = got[key:last + 1], got[last + 1:]
            assert float((inside - 7.0).abs().max()) < 0.1, f"key {key} is not seen at {int((inside - 7.0).abs().max(dim=1).values.argmax()) + key}, cuts {cuts[:3]}"
            if key < keep_first:
                assert float((outside - 7.0).abs().max()) < 0.1, f"key {key} is kept and not seen, cuts {cuts[:3]}"
            else:
                assert float(outside.abs().max()) < 0.5, f"key {key} is seen beyond a window of {window}, cuts {cuts[:3]}"


@pytest.mark.parametrize("key", [0, 1, 63, 64, 65, 511, 512, 700, 1500])
@pytest.mark.parametrize("dtype,n_heads,n_kv_heads,dim,vdim", [(torch.float32, 2, 1, 16, 24), (torch.bfloat16, 4, 2, 64, 64), (torch.bfloat16, 6, 2, 96, 128), (torch.bfloat16, 3, 1, 20, 12)])
def test_one_key_far_back_is_found_under_a_cap(dtype, n_heads, n_kv_heads, dim, vdim, key, ops):
    length = 1700
    generator = torch.Generator().manual_seed(key)
    q, k, v = (0.1 * torch.randn(length, width, generator=generator) for width in (n_heads * dim, n_kv_heads * dim, n_kv_heads * vdim))
    q[-20:], k[key], v[key] = 3.0, 3.0, 7.0
    for cuts in ([length], [length - 40, 40], [length - 20] + [1] * 20):
        got = attend(ops, q, k, v, cuts, dtype, n_heads, n_kv_heads, dim, vdim, scale=3.2 / dim, softcap=40.0)
        assert float((got[-20:] - 7.0).abs().max()) < 0.1, f"key {key}, cuts {cuts[:2]}"


@pytest.mark.parametrize("dtype,dim,vdim", [(torch.float32, 24, 16), (torch.bfloat16, 64, 64), (torch.bfloat16, 64, 72)])
def test_a_cap_flattens_scores_far_above_it_and_leaves_small_ones(dtype, dim, vdim, ops):
    """Scores of some hundreds under a cap of two: all that are large have nearly the same weight; and scores of thousandths, which the
    cap must leave as they are."""
    n_heads, length = 4, 140
    generator = torch.Generator().manual_seed(2)
    q, k, v = (torch.randn(length, width, generator=generator).bfloat16().float() for width in (n_heads * dim, 2 * dim, 2 * vdim))
    for scale, cap in ((40.0, 2.0), (1e-3, 60.0), (3.0, 30.0), (500.0, 0.01)):
        want = plain_attention(q, k, v, n_heads, 2, scale, 50, 3, cap, torch.full((n_heads,), -1.0))
        for cuts in ([length], [length - 6] + [1] * 6):
            got = attend(ops, q, k, v, cuts, dtype, n_heads, 2, dim, vdim, scale=scale, window=50, keep_first=3, softcap=cap, sink=torch.full((n_heads,), -1.0).cuda())
            assert float((got - want).abs().max()) <= (2e-5 if dtype == torch.float32 else 1.5e-2) * float(want.abs().max()), f"scale {scale}, cap {cap}"


@pytest.mark.parametrize("dtype,dim,vdim", [(torch.float32, 24, 16), (torch.bfloat16, 64, 96), (torch.bfloat16, 40, 24)])
def test_a_sink_joins_the_denominator_once_and_uncapped(dtype, dim, vdim, ops):
    n_heads, length = 6, 150
    generator = torch.Generator().manual_seed(9)
    q, k, v = (torch.randn(length, width, generator=generator).bfloat16().float() for width in (n_heads * dim, 3 * dim, 3 * vdim))
    sink = torch.tensor([2.0, -40.0, 40.0, 0.0, 6.0, -3.0])
    want = plain_attention(q, k, v, n_heads, 3, 0.3, 33, 2, 1.0, sink)
    assert float(want.reshape(length, n_heads, -1)[:, 2].abs().max()) < 1e-10      # (a sink of forty under scores of at most one)
    for cuts in ([length], [70, 80], [length - 3, 1, 2]):
        got = attend(ops, q, k, v, cuts, dtype, n_heads, 3, dim, vdim, scale=0.3, window=33, keep_first=2, softcap=1.0, sink=sink.cuda())
        assert float((got - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 1.5e-2) * float(want.abs().max()), f"cuts {cuts}"


def test_32_bit_attention_gives_the_same_bits_however_a_request_is_cut(ops):
    n_heads, n_kv_heads, dim, vdim, length = 4, 2, 24, 40, 400
    generator = torch.Generator().manual_seed(5)
    q, k, v = (torch.randn(length, width, generator=generator) for width in (n_heads * dim, n_kv_heads * dim, n_kv_heads * vdim))
    for window, keep_first in ((70, 5), (70, 130), (None, 0)):
        options = dict(scale=0.3, window=window, keep_first=keep_first, softcap=2.0, sink=torch.zeros(n_heads).cuda())
        whole = attend(ops, q, k, v, [length], torch.float32, n_heads, n_kv_heads, dim, vdim, **options)
        for cuts in ([1] * length, [130, 2, 1, 67, 200]):
            assert torch.equal(attend(ops, q, k, v, cuts, torch.float32, n_heads, n_kv_heads, dim, vdim, **options), whole)


def test_what_attention_refuses(ops):
    from xeno_rt_amd.ops.hip import KernelError
    q, k, v = (torch.randn(10, 32) for _ in range(3))
    for options in (dict(softcap=0.0), dict(softcap=-1.0), dict(window=4, keep_first=-1)):
        with pytest.raises(KernelError):
            attend(ops, q, k, v, [10], torch.float32, 1, 1, 32, 32, scale=1.0, **options)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m", [layer["mixer"] for name in NAMES for layer in CONFIGS[name]["layers"] if layer["type"] == "attention"])
def test_attention_alone(m, dtype, ops):
    from xeno_rt_amd.models.fisopel import _mixer
    width, length = 48, 150
    part = _mixer("attention", m, "mix.", types.SimpleNamespace(width=width, norm_eps=1e-5))
    tensors = tensors_for(part, seed=m["dim"], std=0.25, norm=(1.0, 0.3), sink=(0.5, 1.0))
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(length, width, generator=torch.Generator().manual_seed(1)).to(dtype)
    want = P.attention(h.double(), short(tensors), m, 1e-5)
    limit = 3e-5 if dtype == torch.float32 else 5e-2
    for padding, cuts in ((2, [length]), (0, [length]), (2, [1] * length), (0, [length - 20] + [1] * 20), (2, [3, 64, 2, length - 69])):
        cache = layer_cache(part.cache_needs(), dtype, length)
        got = run_mixer(part, h, cuts, cache, dtype, padding=padding)
        assert float((got - want).abs().max()) <= limit * float(want.abs().max()), f"cuts {cuts[:3]}"
    mask = m.get("mask") or {}
    assert part.cache_needs().kv.window == mask.get("size") and part.cache_needs().kv.keep_first == (mask.get("keep_first") or 0)


# ---- attention through a latent ---------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("neighbours,magnitude", [(False, 1.0), (False, 1.3), (True, 0.7)])
@pytest.mark.parametrize("heads,dim,rot_dim,rot_dims,rank", [(3, 16, 8, 8, 24), (7, 32, 32, 32, 96), (5, 7, 6, 4, 9), (1, 40, 64, 64, 96)])
def test_queries_and_latents_turn_in_halves_with_a_magnitude(heads, dim, rot_dim, rot_dims, rank, neighbours, magnitude, dtype, ops):
    from xeno_rt_amd.parts.base import CacheNeeds, KVSpec
    tokens, q_width, eps = 70, heads * (dim + rot_dim), 1e-5
    generator = torch.Generator().manual_seed(rank)
    sums = torch.randn(tokens, q_width + rank + rot_dim + 3, generator=generator)
    gain = (1 + 0.3 * torch.randn(rank, generator=generator)).to(dtype)
    frequencies = torch.tensor([50.0 ** (-2.0 * i / rot_dims) for i in range(rot_dims // 2)])
    q, down = sums[:, :q_width], sums[:, q_width:q_width + rank + rot_dim]

    def turned(part):                                               # [tokens, ..., rot_dim]
        out = part.double().clone()
        for i, f in enumerate(frequencies.double()):
            a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + rot_dims // 2)
            angle = torch.arange(tokens, dtype=F).reshape(-1, *[1] * (part.dim() - 2)) * f
            out[..., a] = magnitude * (part[..., a].double() * angle.cos() - part[..., b].double() * angle.sin())
            out[..., b] = magnitude * (part[..., b].double() * angle.cos() + part[..., a].double() * angle.sin())
        return out

    step, turn = Step([1], [tokens], [0]), dict(neighbours=neighbours, magnitude=magnitude)
    for together in (True, False):
        cache = layer_cache(CacheNeeds(kv=KVSpec(1, rank + rot_dim, None, rank)), dtype, tokens)
        plain, full = (torch.zeros(tokens, heads * width, dtype=dtype, device="cuda") for width in (dim, rank + rot_dim))
        rows = torch.zeros(tokens, rank + rot_dim, dtype=dtype, device="cuda")
        on_gpu = sums.cuda()
        q_gpu, down_gpu = on_gpu[:, :q_width], on_gpu[:, q_width:q_width + rank + rot_dim]
        if together:
            ops.latent_prepare(q_gpu, down_gpu, heads, dim, rank, rot_dim, gain.cuda(), eps, frequencies.cuda(), rot_dims, cache.kv, step, plain, full, **turn)
        else:
            ops.latent_complete(down_gpu, rank, rot_dim, gain.cuda(), eps, frequencies.cuda(), rot_dims, cache.kv, step, like=plain, rows_out=rows, **turn)
            ops.latent_queries(q_gpu, heads, dim, rot_dim, frequencies.cuda(), rot_dims, step, plain, full, rank, **turn)
            want = torch.cat([P.rms_norm(down[:, :rank].double(), gain, eps), turned(down[:, rank:])], dim=1)
            assert float((rows.double().cpu() - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())
            assert torch.equal(cache.kv.k, before.kv.k) and torch.equal(cache.kv.v, before.kv.v) and float(before.kv.k.float().abs().max()) > 0
        before = cache
        of_heads = q.reshape(tokens, heads, dim + rot_dim)
        got = full.reshape(tokens, heads, -1)[..., rank:].double().cpu()
        want = turned(of_heads[..., dim:])
        assert float((got - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())
        assert torch.equal(plain.cpu(), of_heads[..., :dim].reshape(tokens, -1).to(dtype))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("tokens,heads,n,k", [(1, 3, 24, 16), (5, 7, 72, 96), (16, 2, 33, 64), (17, 2, 33, 64), (70, 5, 40, 8), (200, 1, 80, 72), (600, 3, 70, 96), (512, 2, 64, 32), (9, 4, 1, 32)])
def test_every_output_times_the_sigmoid_of_a_gate_of_its_own(tokens, heads, n, k, dtype, ops):
    generator = torch.Generator().manual_seed(n + k)
    a, w = torch.randn(tokens, heads * k, generator=generator).to(dtype), torch.randn(heads, n, k, generator=generator).to(dtype)
    sums = 2.0 * torch.randn(tokens, heads * n + 5, generator=generator)
    gates = torch.sigmoid(sums[:, 3:3 + heads * n].double()).reshape(tokens, heads, n)
    want = torch.einsum("thk,hnk->thn", a.double().reshape(tokens, heads, k), w.double()) * gates
    out = torch.zeros(tokens, heads * (n + 3), dtype=dtype, device="cuda")
    ops.linear_heads(a.cuda(), w.cuda(), out, out_head=n + 3, gate_logits=sums.cuda()[:, 3:3 + heads * n])
    got = out.double().cpu().reshape(tokens, heads, n + 3)
    assert float((got[..., :n] - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())
    assert float(got[..., n:].abs().max()) == 0.0, "what lies behind a head's outputs was touched"


LARGE_LATENTS = [_latent(3, 128, 64, 96, 448, 0.08, 5e5, None, (4.0, 128, 8.0, 1.0))["mixer"], _latent(2, 24, 16, 40, 620, 0.1, 100.0, None)["mixer"],
                 _latent(4, 16, 64, 24, 512, 0.1, 1000.0, None, (2.0, 64, 4.0, 0.5))["mixer"]]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m", [layer["mixer"] for name in NAMES for layer in CONFIGS[name]["layers"] if layer["type"] == "latent_attention"] + LARGE_LATENTS)
def test_latent_attention_alone(m, dtype, ops):
    from xeno_rt_amd.models.fisopel import _mixer
    width, length = 48, 150
    part = _mixer("latent_attention", m, "mix.", types.SimpleNamespace(width=width, norm_eps=1e-5))
    tensors = tensors_for(part, seed=m["kv_rank"], std=0.25, norm=(1.0, 0.3), g=(0.0, 0.5))
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(length, width, generator=torch.Generator().manual_seed(1)).to(dtype)
    want = P.latent_attention(h.double(), short(tensors), m, 1e-5)
    limit = 3e-5 if dtype == torch.float32 else 5e-2
    for padding, cuts in ((2, [length]), (0, [length]), (2, [1] * length), (0, [length - 20] + [1] * 20), (2, [3, 64, 2, length - 69])):
        cache = layer_cache(part.cache_needs(), dtype, length)
        got = run_mixer(part, h, cuts, cache, dtype, padding=padding)
        assert float((got - want).abs().max()) <= limit * float(want.abs().max()), f"cuts {cuts[:3]}"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_gate_for_each_output_beside_a_low_rank_for_the_queries(dtype, ops):
    """The part serves other designs too: a gate per output where the queries come through a rank of their own, under a window."""
    from xeno_rt_amd.parts import LatentAttention, PairRotation
    width, length = 40, 130
    m = dict(heads=3, dim=16, rot_dim=32, vdim=20, kv_rank=64, scale=0.2, rot={"dims": 16, "base": 100.0, "scaling": {"factor": 2.0, "original": 30, "fast": 4.0, "slow": 0.5}})
    part = LatentAttention("mix.", width, 3, 16, 32, 20, 64, 24, 0.2, 1e-5, 16, 100.0, sink=None, window=33, output_gate="g", gate_per="output",
                           position=PairRotation(16, 100.0, neighbours=False, scaling=m["rot"]["scaling"]))
    tensors = tensors_for(part, seed=3, std=0.25, norm=(1.0, 0.3), g=(0.0, 0.5))
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(length, width, generator=torch.Generator().manual_seed(1)).to(dtype)
    p, x = short(tensors), h.double()
    q = (P.rms_norm(x @ p["dq"].T, p["dq.norm"], 1e-5) @ p["uq"].T).reshape(length, 3, 48)
    latent, turned = P.latent_rows(x, p, m, 1e-5)
    scores = (torch.einsum("ihd,jhd->hij", q[..., :16], (latent @ p["uk"].T).reshape(length, 3, 16))
              + torch.einsum("ihr,jr->hij", P.turn_halves(q[..., 16:], m["rot"]), turned)) * 0.2
    weights = torch.softmax(scores.masked_fill(~P.seen(length, 33), -math.inf), dim=-1)
    o = torch.einsum("hij,jhe->ihe", weights, (latent @ p["uv"].T).reshape(length, 3, 20)).reshape(length, -1)
    want = (o * torch.sigmoid(x @ p["g"].T)) @ p["o"].T
    for padding, cuts in ((0, [length]), (2, [length - 20] + [1] * 20), (0, [3, 64, 2, length - 69])):
        got = run_mixer(part, h, cuts, layer_cache(part.cache_needs(), dtype, length), dtype, padding=padding)
        assert float((got - want).abs().max()) <= (3e-5 if dtype == torch.float32 else 5e-2) * float(want.abs().max()), f"cuts {cuts[:3]}"


# ---- experts ---------------------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("experts,top", [(8, 1), (6, 3), (5, 5), (64, 8), (65, 2), (256, 7), (1, 1)])
def test_a_softmax_over_the_chosen_logits(experts, top, ops):
    tokens = 301
    logits = 3.0 * torch.randn(tokens, experts + 3, generator=torch.Generator().manual_seed(experts))
    logits[0] += 200.0                                              # (exponentials of these would be no numbers)
    logits[1] -= 200.0
    weights, chosen = torch.full((tokens, experts), float("nan"), device="cuda"), torch.full((tokens, top), -1, dtype=torch.int32, device="cuda")
    ops.route_experts(logits.cuda()[:, 1:1 + experts], weights, top, chosen=chosen, scores="softmax")
    for t in range(tokens):
        picked, scores = P.choose(logits[t, 1:1 + experts].double(), top)
        assert chosen[t].tolist() == picked
        assert weights[t].nonzero().flatten().tolist() == sorted(picked)
        assert weights[t, picked].tolist() == pytest.approx(scores, rel=1e-5)
    ops.route_experts(logits.cuda()[:, 1:1 + experts], weights, top, scores="softmax", normalized=False, scale=2.0)
    want = 2.0 * torch.softmax(logits[:, 1:1 + experts].double(), dim=1)
    picked = weights.cpu() != 0
    assert float((weights.double().cpu() - want)[picked].abs().max()) < 1e-5 and int(picked.sum()) == tokens * top


def experts_part(raw, width, seed, ops, dtype, pack="auto"):
    from xeno_rt_amd.models.fisopel import _feed_forward
    from xeno_rt_amd.parts.base import Runtime
    part = _feed_forward(raw, "mlp.", types.SimpleNamespace(width=width))
    tensors = tensors_for(part, seed=seed, std=0.3, router=(0.0, 0.7))
    part.bind(tensors, Runtime(ops, dtype, "cuda", pack_weights=pack))
    return part, tensors


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("raw", [_moe(24, 6, 2, 40), _moe(9, 3, 2, 5), _moe(64, 4, 1, 128), _moe(16, 5, 5), _moe(40, 7, 3, 8), _moe(8, 1, 1, 8)])
@pytest.mark.parametrize("tokens", [1, 7, 61])
def test_experts_alone(tokens, raw, dtype, ops):
    width = 48
    part, tensors = experts_part(raw, width, 7, ops, dtype)
    assert not any(name.endswith("sg") for name in tensors)
    h = torch.randn(tokens, width, generator=torch.Generator().manual_seed(5)).to(dtype)
    want = P.experts(h.double(), short(tensors, "mlp."), raw)
    out, residual = torch.empty(tokens, width, device="cuda"), torch.ones(tokens, width, device="cuda")
    part.forward_into(h.cuda(), None, out)
    part.forward(h.cuda(), None, residual)
    limit = 2e-5 if dtype == torch.float32 else 3e-2
    for got in (out.double().cpu(), residual.double().cpu() - 1.0):
        per_row = (got - want).abs().max(dim=1).values / float(want.abs().max())
        assert int((per_row > limit).sum()) <= (0 if dtype == torch.float32 else 2), f"rows {(per_row > limit).nonzero().flatten().tolist()} differ"


@pytest.mark.parametrize("pack", ["auto", "always"])
@pytest.mark.parametrize("raw,tokens", [(_moe(64, 8, 2, 128), 300), (_moe(128, 16, 4, 64), 1000), (_moe(192, 4, 1), 600), (_moe(64, 3, 1, 320), 401)])
def test_experts_multiply_only_the_tokens_that_chose_them(raw, tokens, pack, ops):
    """A step of many tokens sorts its picks by expert, the shared expert beside them: against the plain sum, against the same part with
    every token through every expert, and onto a stream instead of aside."""
    width = 64
    part, tensors = experts_part(raw, width, 8, ops, torch.bfloat16, pack)
    options = {} if part.shared is None else {"shared_width": part.shared}
    takes = ops.experts_sorted_takes
    h = torch.randn(tokens, width, generator=torch.Generator().manual_seed(6)).bfloat16()
    assert takes(h.cuda(), part.w_gate_up, part.w_down, part.experts, part.intermediate, part.top, **options)
    out, residual = torch.full((tokens, width), float("nan"), device="cuda"), torch.ones(tokens, width, device="cuda")
    part.forward_into(h.cuda(), None, out)
    part.forward(h.cuda(), None, residual)
    ops.experts_sorted_takes = lambda *operands, **named: False
    try:
        dense = torch.empty(tokens, width, device="cuda")
        part.forward_into(h.cuda(), None, dense)
    finally:
        ops.experts_sorted_takes = takes
    want = P.experts(h.double(), short(tensors, "mlp."), raw)
    scale = float(want.abs().max())
    assert float((out - dense).abs().max()) <= 2e-2 * scale and float((residual - 1.0 - out).abs().max()) <= 1e-5 * (1.0 + scale)
    per_row = (out.double().cpu() - want).abs().max(dim=1).values / scale
    assert int((per_row > 3e-2).sum()) <= max(2, tokens // 50), f"rows {(per_row > 3e-2).nonzero().flatten().tolist()} differ from the plain sum"


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
        mlp = None
        if r.random() < 0.85:
            experts = r.randint(1, 9)
            mlp = _moe(r.choice([6, 20, 64, 128]), experts, r.randint(1, experts), r.choice([None, 7, 32, 64, 192]))
        if r.random() < 0.5:
            kv_heads = r.choice([1, 2, 3])
            layers.append(_attention(kv_heads * r.choice([1, 2, 5]), kv_heads, r.choice([4, 11, 32, 64, 96]), r.choice([6, 32, 40, 64, 128]), r.choice([0.1, 0.4]), mlp,
                                     r.choice([None, 1, 5, 32, 50, 64, 90]), r.choice([0, 1, 4, 31, 64, 80]), r.choice([None, 0.5, 3.0, 20.0])))
        else:
            scaling = (r.choice([1.5, 4.0, 16.0]), r.choice([16, 64, 500]), r.choice([4.0, 16.0]), r.choice([0.5, 1.0, 2.0])) if r.random() < 0.7 else None
            layers.append(_latent(r.randint(1, 20), r.choice([4, 12, 32]), r.choice([2, 16, 32, 64]), r.choice([6, 16, 36, 72]), r.choice([8, 30, 64, 96, 160]),
                                  r.choice([0.1, 0.25]), r.choice([10.0, 1e4, 3e5]), mlp, scaling))
    loop = None
    if r.random() < 0.8:
        start = r.randrange(len(layers))
        loop = (start, r.randint(start + 1, len(layers)), r.randint(1, 3))
    return _model(r.choice([50, 97, 200]), r.choice([24, 40, 64, 96, 128]), r.choice([1e-6, 1e-4]), r.choice([0.5, 1.0, 4.0]), layers, loop)


@pytest.mark.parametrize("seed", range(14))
def test_configurations_drawn_at_random(seed, tmp_path):
    from xeno_rt_amd.engine import Engine
    raw = random_configuration(seed)
    folder = make_fisopel_folder(raw, tmp_path, seed=seed, std=0.1)
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
        print(f"fisopel, largest errors against the plain model [{dtype}]: max {worst:.2e} (limit {LIMITS[dtype]['max']:.0e}), "
              f"rms {rms:.2e} (limit {LIMITS[dtype]['rms']:.0e})")
