"""The Renapel decoder on the GPU against the plain implementation (tests/plain_renapel.py), for four small configurations
that differ in every size and option: whole prompts, token-by-token decoding from the first token, portions of several sizes,
unequal batches through reused slots, greedy generation through the library's loop and programs; and every new mechanism
alone against plain arithmetic, with inputs made so that a far key, a sink, a block's border or a closed group of experts
shows."""
import math
import types

import pytest
import torch

from helpers import errors, run_batched, run_whole, token_ids
from renapel_models import CONFIGS, make_renapel_folder
import plain_renapel as P

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
NAMES = sorted(CONFIGS)
LENGTH = {"mixed": 150, "wide": 160, "edges": 140, "plain": 135}
F = torch.float64

# Largest difference from the plain implementation (float64), relative to the largest logit. The experts' weights divide by
# a sum of a few scores and the copies of the stream are mixed again and again, so float32 sums in another order show up a
# little above their own rounding. In bfloat16 the router reads rounded rows, and with random weights a token now and then has
# two experts (or two groups) whose scores lie closer than that rounding: the engine then takes another expert than the
# float64 model and that one row is off by what the two experts differ in (with one expert of three chosen, by all of the
# feed-forward's output). So in bfloat16 a few of a request's rows (OUTLIER_ROWS of them, two at least, one of a short request's)
# may exceed the limit on single logits, and both limits are then held over the other rows; 32-bit has no such allowance, and it
# runs the same kernels.
LIMITS = {"float32": dict(max=2e-5, rms=3e-6), "bfloat16": dict(max=1e-1, rms=2.5e-2)}
OUTLIER_ROWS = 0.03
WORST = {}


def assert_logits(got, want, dtype, what, outlier_rows=None):
    assert torch.isfinite(got).all(), f"{what}: logits are not finite"
    worst, rms = errors(got, want)
    if dtype == "bfloat16" and (worst > LIMITS[dtype]["max"] or rms > LIMITS[dtype]["rms"]):
        # the rows that took another expert: a few are allowed, and both measures are taken over the others
        diff = (got.double().cpu() - want.double()) / float(want.abs().max())
        per_row = diff.abs().max(dim=1).values
        allowed = 1 if want.shape[0] < 20 else max(2, int((outlier_rows or OUTLIER_ROWS) * want.shape[0]))
        kept = per_row.argsort()[:want.shape[0] - allowed]
        assert int((per_row > LIMITS[dtype]["max"]).sum()) <= allowed, \
            f"{what} [{dtype}]: {int((per_row > LIMITS[dtype]['max']).sum())} of {want.shape[0]} rows exceed {LIMITS[dtype]['max']:.1e}"
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
    """name -> (folder, plain model, ids, plain logits); every other folder's config.json leaves the tables' rows to the checkpoint"""
    out = {}
    for index, name in enumerate(NAMES):
        folder = make_renapel_folder(CONFIGS[name], tmp_path_factory.mktemp(name), seed=31 + index, name_the_rows=index % 2 == 0)
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


def same_but_for_rounding(got, want):
    return float((got - want).abs().max()) <= 3e-5 * float(want.abs().max())


def in_portions(engine, ids, sizes):
    """The request alone, cut into steps of the given sizes (the last size repeats); logits of every token."""
    slot = engine.alloc_slot()
    rows, at, index = [], 0, 0
    try:
        while at < len(ids):
            size = min(sizes[min(index, len(sizes) - 1)], len(ids) - at)
            rows.append(engine.step([(slot, ids[at:at + size], list(range(size)))]))
            at, index = at + size, index + 1
        return torch.cat(rows)
    finally:
        engine.free_slot(slot)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts(name, dtype, models, engines):
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    got = run_whole(engine, ids)
    assert_logits(got, want, dtype, f"renapel {name} whole, first bad row {first_bad_position(got, want, dtype)}")
    for length in (1, 2, 3, 66):                                    # the first tokens of a sequence, and just past a block
        got = run_whole(engine, ids[:length])
        assert_logits(got, want[:length], dtype, f"renapel {name} whole, {length} tokens")
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_token_by_token_from_the_first(name, dtype, models, engines):
    """Every token in a step of its own: long decoding through recorded steps, across cache blocks."""
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    got = in_portions(engine, ids, [1])
    assert_logits(got, want, dtype, f"renapel {name} token by token, first bad row {first_bad_position(got, want, dtype)}")
    if dtype == "float32":
        assert same_but_for_rounding(got, run_whole(engine, ids)), "a decoded token differs from the same token in a prompt"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [[2], [3, 7], [64, 1], [65, 2, 2, 1, 30], [33], [1, 1, 2, 61, 5]])
@pytest.mark.parametrize("name", NAMES)
def test_portions(name, sizes, dtype, models, engines):
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    got = in_portions(engine, ids, sizes)
    assert_logits(got, want, dtype, f"renapel {name} portions {sizes}, first bad row {first_bad_position(got, want, dtype)}")
    if dtype == "float32":
        assert same_but_for_rounding(got, run_whole(engine, ids)), f"portions {sizes} change more than the rounding"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_unequal_batches_through_reused_slots(name, dtype, models, engines):
    """Three requests of different lengths start together and end one after the other, twice over, so that the second
    round runs in slots, blocks and states that the first has used."""
    engine = engines(name, dtype)
    _, plain, ids, want = models[name]
    vocab = CONFIGS[name]["vocab"]
    requests = [ids, token_ids(vocab, 37, seed=900), token_ids(vocab, 71, seed=901)]
    wants = [want, plain.logits(requests[1]), plain.logits(requests[2])]
    for prompts in ([len(ids) - 40, 5, 66], [3, 36, 1]):
        got = run_batched(engine, requests, prompts)
        for index, (g, w) in enumerate(zip(got, wants)):
            assert_logits(g, w, dtype, f"renapel {name} batch {prompts} request {index}, first bad row {first_bad_position(g, w, dtype)}")
            if dtype == "float32":
                assert same_but_for_rounding(g, run_whole(engine, requests[index])), "a request depends on its batch"
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


def test_a_long_request_decoded_far_past_its_prompt(models, engines):
    """500 tokens, the last 300 of them decoded one by one: states, the latent's cache and the tables of biases far beyond their last row."""
    engine = engines("mixed", "float32")
    _, plain, _, _ = models["mixed"]
    ids = token_ids(CONFIGS["mixed"]["vocab"], 500, seed=77)
    want = plain.logits(ids)
    got = in_portions(engine, ids, [200, 1])
    assert_logits(got, want, "float32", f"renapel mixed long decoding, first bad row {first_bad_position(got, want, 'float32')}")


# ---- every mechanism alone -------------------------------------------------------------------------------------

class Step:
    """A step's sequences as the kernels want them described: `counts[i]` new tokens of the sequence in `slots[i]`."""

    def __init__(self, slots, counts, starts, device="cuda"):
        ints = lambda values: torch.tensor(values, dtype=torch.int32, device=device)
        offsets = [0]
        for count in counts:
            offsets.append(offsets[-1] + count)
        self.n_tokens, self.n_sequences, self.max_count = offsets[-1], len(slots), max(counts)
        self.sequence_offsets, self.sequence_slots, self.sequence_starts = ints(offsets), ints(slots), ints(starts)
        self.positions = ints([start + t for start, count in zip(starts, counts) for t in range(count)])
        self.slots = ints([slot for slot, count in zip(slots, counts) for _ in range(count)])
        self.max_context = max(start + count for start, count in zip(starts, counts))
        self.host_slots, self.host_counts, self.host_starts = list(slots), list(counts), list(starts)


def schedules(length):
    """Ways to cut a sequence of `length` tokens into steps."""
    return [[length], [1] * length, [2] * (length // 2) + [length % 2] * (length % 2), [length - 3, 1, 2], [70, length - 70]]


@pytest.fixture(scope="module")
def ops():
    from xeno_rt_amd.ops import load_ops
    return load_ops()


def runtime(ops, dtype):
    from xeno_rt_amd.parts.base import Runtime
    return Runtime(ops, dtype, "cuda")


def layer_cache(needs, dtype, length, slots=3):
    """What a layer call finds in the cache, for a part run by hand: keys and values in blocks that lie in another order than the
    sequence's (slot 1 is the sequence's), states that hold sevens in the other slots."""
    from xeno_rt_amd.cache import BLOCK_TOKENS
    from xeno_rt_amd.cache.sequence_cache import KVView
    cache = types.SimpleNamespace(kv=None, state=None, states={}, writable=True)
    if needs.kv is not None:
        spec = needs.kv
        blocks = (length + BLOCK_TOKENS - 1) // BLOCK_TOKENS
        table = torch.full((slots, blocks), -1, dtype=torch.int32)
        table[1] = torch.arange(blocks - 1, -1, -1, dtype=torch.int32) + 1
        cache.kv = KVView(spec, torch.zeros(blocks + 1, spec.n_kv_heads, BLOCK_TOKENS, spec.head_dim, dtype=dtype, device="cuda"),
                          torch.zeros(blocks + 1, spec.n_kv_heads, spec.value_width, BLOCK_TOKENS, dtype=dtype, device="cuda"), table.cuda())
    for name, spec in needs.states:
        state = torch.full((slots, *spec.shape), 7.0, dtype=spec.dtype, device="cuda")
        state[1].zero_()
        cache.states[name] = state
    return cache


def run_mixer(part, h, cuts, cache, dtype, padding=2):
    """The mixer's float32 output for the rows h of the sequence in slot 1, cut into steps; every step also brings `padding`
    rows that belong to no sequence, ahead of the sequence's."""
    rows, at = [], 0
    width = h.shape[1]
    for count in cuts:
        if count == 0:
            continue
        step = Step([-1, 1], [padding, count], [0, at]) if padding else Step([1], [count], [at])
        x = torch.cat([torch.ones(padding, width), h[at:at + count].float()]).to(dtype).cuda()
        out = torch.full((padding + count, part.hidden), float("nan"), device="cuda")
        part.forward_into(x, step, cache, out)
        rows.append(out[padding:])
        at += count
    return torch.cat(rows).double().cpu()


def tensors_for(part, seed, std=0.3, **special):
    """Random tensors for a part's declared weights (as the compute dtype rounds them); `special` gives means and deviations
    for tensors by the last piece of their names."""
    generator = torch.Generator().manual_seed(seed)
    out = {}
    for name, spec in part.weight_specs().items():
        mean, deviation = special.get(name.split(".")[-1], (0.0, std))
        out[name] = (mean + deviation * torch.randn(spec.shape, generator=generator)).bfloat16()
    return out


def short(tensors, prefix="mix."):
    return {name[len(prefix):]: t.double() for name, t in tensors.items()}


@pytest.mark.parametrize("copies", [1, 2, 3, 8])
def test_the_copies_of_the_stream_are_read_and_written_as_the_plain_sums_say(copies, ops):
    tokens, width = 37, 72
    generator = torch.Generator().manual_seed(copies)
    x = torch.randn(tokens, width, generator=generator)
    streams = torch.empty(tokens, copies, width, device="cuda")
    ops.streams_open(x.cuda(), streams)
    assert torch.equal(streams.cpu(), x[:, None, :].expand(tokens, copies, width))
    X = torch.randn(copies, tokens, width, generator=generator, dtype=F)
    streams = X.permute(1, 0, 2).float().contiguous().cuda()
    X = streams.double().cpu().permute(1, 0, 2)
    weights, out_weights, mix = (torch.randn(shape, generator=generator) for shape in ((copies,), (copies,), (copies, copies)))
    gain, next_weights = 1 + 0.3 * torch.randn(width, generator=generator), torch.randn(copies, generator=generator)
    for dtype in (torch.float32, torch.bfloat16):
        got = torch.empty(tokens, width, dtype=dtype, device="cuda")
        ops.streams_read(streams, weights.cuda(), gain.to(dtype).cuda(), 1e-5, got)
        want = P.rms_norm(P.copies_read(X, weights), gain.to(dtype), 1e-5)
        assert float((got.double().cpu() - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())
    rows = torch.tensor([5, 0, 36, 5], dtype=torch.int32)
    some = torch.empty(4, width, device="cuda")
    ops.streams_read(streams, weights.cuda(), gain.cuda(), 1e-5, some, rows=rows.cuda())
    assert torch.equal(some, got_all(ops, streams, weights, gain)[rows.long().cuda()])
    y = torch.randn(tokens, width, generator=generator)
    want = P.copies_write(X, y.double(), mix, out_weights)
    normed = torch.empty(tokens, width, device="cuda")
    ops.streams_write(streams, mix.cuda(), out_weights.cuda(), y.cuda(), then=(next_weights.cuda(), gain.cuda(), 1e-5, normed))
    assert float((streams.double().cpu().permute(1, 0, 2) - want).abs().max()) <= 1e-5 * float(want.abs().max())
    assert torch.equal(normed, got_all(ops, streams, next_weights, gain)), "the read in the write's pass is the read alone, to the bit"


def got_all(ops, streams, weights, gain):
    out = torch.empty(streams.shape[0], streams.shape[2], device="cuda")
    ops.streams_read(streams, weights.cuda(), gain.cuda(), 1e-5, out)
    return out


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,dim,vdim,decay", [(3, 20, 12, [0.5, 0.9, 1.0]), (1, 72, 136, [0.99]), (4, 8, 8, [0.6, 0.8, 0.9, 0.999]),
                                                   (2, 64, 40, [0.97, 0.75]), (2, 128, 64, [1.0, 0.3]), (5, 200, 24, [0.9] * 5)])
def test_lightning_attention_alone(heads, dim, vdim, decay, dtype, ops):
    from xeno_rt_amd.parts import LightningAttention
    width, length = 40, 150
    part = LightningAttention("mix.", width, heads, dim, vdim, decay, 1e-5)
    tensors = tensors_for(part, seed=dim + vdim, std=0.3, norm=(1.0, 0.3))
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(length, width, generator=torch.Generator().manual_seed(1)).to(dtype)
    want = P.lightning(h.double(), short(tensors), {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, 1e-5)
    limit = 2e-5 if dtype == torch.float32 else 4e-2
    for cuts in schedules(length):
        cache = layer_cache(part.cache_needs(), dtype, length)
        got = run_mixer(part, h, cuts, cache, dtype)
        assert float((got - want).abs().max()) <= limit * float(want.abs().max()), f"cuts {cuts[:4]}"
        state = cache.states["lightning"]
        assert float(state[0].min()) == 7.0 and float(state[2].max()) == 7.0, "another sequence's state was touched"


def test_a_state_without_decay_keeps_the_first_token_for_good(ops):
    """With a decay of one, keys that are equal and a value that only the first token has, the last query reads that value
    back in full 300 tokens later, in a prompt and decoded."""
    heads, dim, vdim, length = 1, 16, 8, 300
    zeros = lambda width: torch.zeros(length, width)
    q, k, v = zeros(dim), zeros(dim), zeros(vdim)
    k[0, 3], q[-1, 3], v[0] = 2.0, 2.0, 5.0
    k[1:, 5] = 1.0                                              # the later keys point elsewhere, and their values are nothing
    for cuts in ([length], [length - 40] + [1] * 40):
        state = torch.zeros(2, heads, dim, vdim, device="cuda")
        rows, at = [], 0
        for count in cuts:
            out = torch.empty(count, vdim, device="cuda")
            ops.linear_recurrence(q[at:at + count].cuda(), k[at:at + count].cuda(), v[at:at + count].cuda(), state, Step([1], [count], [at]), out,
                                  heads, dim, vdim, torch.ones(1, device="cuda"), "per_head", input_activation="silu")
            rows.append(out)
            at += count
        silu = lambda z: z / (1 + math.exp(-z))
        assert abs(float(torch.cat(rows)[-1, 0]) - silu(2.0) * silu(2.0) * silu(5.0)) < 1e-4


def plain_attention_with_sink(q, k, v, n_heads, n_kv_heads, dim, vdim, scale, sink, table=None):
    length = q.shape[0]
    q, k, v = q.double().reshape(length, n_heads, dim), k.double().reshape(length, n_kv_heads, dim), v.double().reshape(length, n_kv_heads, vdim)
    share = n_heads // n_kv_heads
    scores = torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(share, dim=1)) * scale
    if table is not None:
        span = table.shape[1]
        distance = (torch.arange(length)[:, None] - torch.arange(length)[None, :]).clamp(min=0, max=span - 1)
        scores = scores + table.double()[:, distance]
    scores = scores.masked_fill(~P.causal_mask(length), -math.inf)
    weights = P.softmax_with_sink(scores, sink.double())
    return torch.einsum("hij,jhe->ihe", weights, v.repeat_interleave(share, dim=1)).reshape(length, n_heads * vdim)


def attend(ops, q, k, v, cuts, dtype, n_heads, n_kv_heads, dim, vdim, **options):
    """Keys and values through `kv_store` into a paged cache whose blocks lie in another order than the sequence's, then
    the general attention kernel on the queries alone, step by step."""
    from xeno_rt_amd.parts.base import CacheNeeds, KVSpec
    cache = layer_cache(CacheNeeds(kv=KVSpec(n_kv_heads, dim, None, vdim)), dtype, q.shape[0])
    rows, at = [], 0
    for count in cuts:
        if count == 0:
            continue
        step = Step([1], [count], [at])
        cut = lambda t: t[at:at + count].to(dtype).cuda().contiguous()
        ops.kv_store(cut(k), cut(v), n_kv_heads, dim, vdim, cache.kv, step)
        out = torch.empty(count, n_heads * vdim, dtype=dtype, device="cuda")
        ops.attention(cut(q), n_heads, n_kv_heads, dim, cache.kv, step, out, value_dim=vdim, queries_alone=True, **options)
        rows.append(out)
        at += count
    return torch.cat(rows).double().cpu()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n_heads,n_kv_heads,dim,vdim", [(4, 2, 24, 16), (2, 2, 32, 48), (6, 1, 10, 6), (5, 1, 46, 40), (1, 1, 96, 80), (8, 2, 64, 64),
                                                        (3, 1, 144, 128)])
def test_attention_with_a_learnt_sink_and_a_bias_by_distance(n_heads, n_kv_heads, dim, vdim, dtype, ops):
    length = 150
    generator = torch.Generator().manual_seed(dim + vdim)
    q, k, v = (torch.randn(length, width, generator=generator).to(dtype).float() for width in (n_heads * dim, n_kv_heads * dim, n_kv_heads * vdim))
    sink, table = 2.0 * torch.randn(n_heads, generator=generator), torch.randn(n_heads, 19, generator=generator)
    scale = 0.6 / math.sqrt(dim)
    want = plain_attention_with_sink(q, k, v, n_heads, n_kv_heads, dim, vdim, scale, sink, table)
    first = None
    for cuts in schedules(length):
        got = attend(ops, q, k, v, cuts, dtype, n_heads, n_kv_heads, dim, vdim, scale=scale, sink=sink.cuda(), distance_bias=table.cuda())
        assert float((got - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 2e-2) * float(want.abs().max()), f"cuts {cuts[:4]}"
        first = got if first is None else first
        # (bfloat16 heads of 64 or 128 dims: steps of several tokens go to the matrix cores, steps of one token do not, and the
        # two agree but for rounding)
        if not (dtype == torch.bfloat16 and dim == vdim and dim in (64, 128)):
            assert torch.equal(got, first), f"cuts {cuts[:4]} change the bits"


def test_the_sink_takes_its_share_and_nothing_else(ops):
    """Equal scores: every key's weight is 1 / (keys + exp(sink - score)), so values of one sum to keys / (keys + exp(sink - score));
    a sink far below the scores changes nothing, one far above leaves nothing; the scale does not touch it."""
    n_heads, dim, vdim, length = 3, 16, 8, 70
    q, k, v = torch.zeros(length, n_heads * dim), torch.zeros(length, dim), torch.ones(length, vdim)
    q[:, 0::dim], k[:, 0] = 1.0, 4.0                               # every score is 4 * scale = 2
    sink = torch.tensor([2.0 + math.log(3.0), -40.0, 40.0])
    for cuts in ([length], [length - 7] + [1] * 7):
        got = attend(ops, q, k, v, cuts, torch.float32, n_heads, 1, dim, vdim, scale=0.5, sink=sink.cuda())
        for i in (0, 1, 63, 64, 69):
            assert abs(float(got[i, 0]) - (i + 1) / (i + 1 + 3.0)) < 1e-5 and abs(float(got[i, vdim]) - 1.0) < 1e-5 and float(got[i, 2 * vdim]) < 1e-12


@pytest.mark.parametrize("key", [0, 1, 62, 63, 64, 65, 127, 128, 500, 511, 512, 513])
def test_one_key_far_back_or_at_a_blocks_border_is_found(key, ops):
    """One key whose score towers over hundreds of others, at the first places of a sequence, on either side of a cache block's
    border and of the border between the kernel's chunks of blocks: the last query, in a prompt and decoded, returns its value
    whatever the sink and the bias by distance say of the others."""
    n_heads, n_kv_heads, dim, vdim, length = 2, 1, 32, 16, 900
    generator = torch.Generator().manual_seed(key)
    q, k, v = (0.1 * torch.randn(length, width, generator=generator) for width in (n_heads * dim, dim, vdim))
    q[-1], k[key] = 3.0, 3.0
    v[key] = 7.0
    sink, table = torch.tensor([1.0, -1.0]), 0.5 * torch.randn(n_heads, 40, generator=generator)
    for cuts in ([length], [length - 33] + [1] * 33, [key + 1, length - key - 2, 1]):
        got = attend(ops, q, k, v, cuts, torch.float32, n_heads, n_kv_heads, dim, vdim, scale=0.1, sink=sink.cuda(), distance_bias=table.cuda())
        assert abs(float(got[-1, 0]) - 7.0) < 2e-2 and abs(float(got[-1, vdim]) - 7.0) < 2e-2, f"key {key}, cuts {cuts[:2]}"


@pytest.mark.parametrize("n_heads,dim,vdim", [(16, 128, 96), (6, 128, 96), (20, 64, 32), (5, 448, 384), (33, 96, 64), (1, 32, 32)])
def test_many_heads_on_one_key_value_head_on_the_matrix_cores(n_heads, dim, vdim, ops):
    """bfloat16, one key/value head, key and value sizes in whole tiles: the kernel that takes sixteen heads of a token as the
    columns of its score tiles, against plain arithmetic, for every way to cut the sequence; then one key far back or at a
    block's border whose score towers over the others."""
    length = 150
    generator = torch.Generator().manual_seed(dim + vdim + n_heads)
    q, k, v = (torch.randn(length, width, generator=generator).bfloat16().float() for width in (n_heads * dim, dim, vdim))
    sink = 2.0 * torch.randn(n_heads, generator=generator)
    scale = 0.6 / math.sqrt(dim)
    want = plain_attention_with_sink(q, k, v, n_heads, 1, dim, vdim, scale, sink)
    for cuts in schedules(length):
        got = attend(ops, q, k, v, cuts, torch.bfloat16, n_heads, 1, dim, vdim, scale=scale, sink=sink.cuda())
        assert float((got - want).abs().max()) <= 2e-2 * float(want.abs().max()), f"cuts {cuts[:4]}"
    want = plain_attention_with_sink(q, k, v, n_heads, 1, dim, vdim, scale, torch.full((n_heads,), -math.inf))
    got = attend(ops, q, k, v, [length - 9] + [1] * 9, torch.bfloat16, n_heads, 1, dim, vdim, scale=scale)
    assert float((got - want).abs().max()) <= 2e-2 * float(want.abs().max()), "without a sink"
    length = 900
    for key in (0, 1, 63, 64, 65, 511, 512, 700):
        q, k, v = (0.1 * torch.randn(length, width, generator=generator) for width in (n_heads * dim, dim, vdim))
        q[-1], k[key] = 3.0, 3.0
        v[key] = 7.0
        for cuts in ([length - 33] + [1] * 33, [key + 1, length - key - 2, 1]):
            got = attend(ops, q, k, v, cuts, torch.bfloat16, n_heads, 1, dim, vdim, scale=0.1 * 32 / dim, sink=sink.cuda())
            assert abs(float(got[-1, 0]) - 7.0) < 5e-2 and abs(float(got[-1, -1]) - 7.0) < 5e-2, f"key {key}, cuts {cuts[:2]}"


def test_queries_are_completed_with_plain_norms_and_a_temperature(ops):
    """What lies between the projection and the scores: biases, every head divided by its root mean square, and the queries
    times a temperature that steps up with the position, in prompts and decoded, also for a layer that projects queries only."""
    n_heads, n_kv_heads, dim, vdim, length, coef, every = 3, 1, 20, 12, 90, 0.4, 16
    generator = torch.Generator().manual_seed(3)
    proj = torch.randn(length, (n_heads + n_kv_heads) * dim + n_kv_heads * vdim, generator=generator)
    bias = torch.randn(n_heads * dim, generator=generator)
    want = P.rms_divided((proj[:, :n_heads * dim].double() + bias.double()).reshape(length, n_heads, dim), 1e-4)
    want = (want * P.query_temperature(length, coef, every)[:, None, None]).reshape(length, -1)
    zeros = lambda n: torch.zeros(n, device="cuda")
    for only in (False, True):
        for cuts in ([length], [50] + [1] * 40):
            rows, at = [], 0
            for count in cuts:
                q = torch.empty(count, n_heads * dim, device="cuda")
                rows_in = proj[at:at + count, :n_heads * dim + 3] if only else proj[at:at + count]
                ops.qkv_complete(rows_in.contiguous().cuda(), n_heads, n_kv_heads, dim, vdim, Step([0], [count], [at]), q, norm_eps=1e-4, plain_norm=True,
                                 biases=(bias.cuda(), None if only else zeros(n_kv_heads * dim), None if only else zeros(n_kv_heads * vdim)),
                                 query_temperature=(coef, every), queries_only=only)
                rows.append(q)
                at += count
            assert torch.allclose(torch.cat(rows).double().cpu(), want, atol=2e-5), (only, cuts[:2])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m", [dict(heads=4, kv_heads=2, dim=24, vdim=16, scale=0.3, bias_max=40, bias_rows=12, q_temp={"coef": 0.4, "every": 16}),
                               dict(heads=6, kv_heads=1, dim=10, vdim=6, scale=0.5, bias_max=1000, bias_rows=6),
                               dict(heads=2, kv_heads=2, dim=64, vdim=64, scale=0.1, bias_max=9, bias_rows=4, q_temp={"coef": 1.0, "every": 1})])
def test_the_softmax_attention_layer_alone_and_a_layer_that_reads_its_keys(m, dtype, ops):
    from xeno_rt_amd.models.renapel import _mixer
    width, length = 40, 150
    config = types.SimpleNamespace(width=width, norm_eps=1e-5)
    owner, reader = _mixer("attention", m, "mix.", config), _mixer("attention", dict(m, kv_from=0, scale=m["scale"] * 0.7), "other.", config)
    special = dict(b=(0.0, 0.5), rel=(0.0, 0.5), sink=(0.5, 1.0))
    tensors, others = tensors_for(owner, seed=m["dim"], **special), tensors_for(reader, seed=m["dim"] + 1, **special)
    assert not any(name.startswith(("other.k", "other.v")) for name in others)
    owner.bind(tensors, runtime(ops, dtype))
    reader.bind(others, runtime(ops, dtype))
    h = torch.randn(length, width, generator=torch.Generator().manual_seed(1)).to(dtype)
    h2 = torch.randn(length, width, generator=torch.Generator().manual_seed(2)).to(dtype)
    want = P.attention(h.double(), short(tensors), m, 1e-5)
    kept = P.attention_keys_values(h.double(), short(tensors), m, 1e-5)
    want_reader = P.attention(h2.double(), short(others, "other."), dict(m, scale=m["scale"] * 0.7), 1e-5, kept)
    limit = 2e-5 if dtype == torch.float32 else 4e-2
    for cuts in ([length], [length - 20] + [1] * 20, [3, 64, 2, length - 69]):
        cache = layer_cache(owner.cache_needs(), dtype, length)
        reading = types.SimpleNamespace(kv=cache.kv, state=None, states={}, writable=False)
        rows, rows_reader, at = [], [], 0
        for count in cuts:
            rows.append(run_step(owner, h[at:at + count], at, cache, dtype))
            rows_reader.append(run_step(reader, h2[at:at + count], at, reading, dtype))
            at += count
        for got, wanted, what in ((torch.cat(rows), want, "owner"), (torch.cat(rows_reader), want_reader, "reader")):
            assert float((got - wanted).abs().max()) <= limit * float(wanted.abs().max()), f"{what}, cuts {cuts[:3]}"


def run_step(part, h, at, cache, dtype):
    out = torch.full((h.shape[0], part.hidden), float("nan"), device="cuda")
    part.forward_into(h.to(dtype).cuda(), Step([1], [h.shape[0]], [at]), cache, out)
    return out.double().cpu()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m", [dict(heads=3, dim=16, rot_dim=8, vdim=12, kv_rank=24, q_rank=20, scale=0.2, rot={"dims": 8, "base": 1000.0}),
                               dict(heads=1, dim=40, rot_dim=16, vdim=72, kv_rank=80, q_rank=12, scale=0.15, rot={"dims": 8, "base": 10000.0}),
                               dict(heads=5, dim=8, rot_dim=6, vdim=4, kv_rank=40, q_rank=48, scale=0.3, rot={"dims": 2, "base": 10.0}),
                               dict(heads=8, dim=64, rot_dim=32, vdim=64, kv_rank=160, q_rank=96, scale=0.1, rot={"dims": 32, "base": 250.0}),
                               dict(heads=18, dim=24, rot_dim=32, vdim=16, kv_rank=96, q_rank=40, scale=0.2, rot={"dims": 16, "base": 5000.0})])
def test_latent_attention_alone(m, dtype, ops):
    from xeno_rt_amd.models.renapel import _mixer
    width, length = 48, 150
    part = _mixer("latent_attention", m, "mix.", types.SimpleNamespace(width=width, norm_eps=1e-5))
    tensors = tensors_for(part, seed=m["kv_rank"], std=0.25, norm=(1.0, 0.3), sink=(0.5, 1.0))
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(length, width, generator=torch.Generator().manual_seed(1)).to(dtype)
    want = P.latent_attention(h.double(), short(tensors), m, 1e-5)
    limit = 3e-5 if dtype == torch.float32 else 5e-2
    for cuts in ([length], [1] * length, [length - 20] + [1] * 20, [3, 64, 2, length - 69]):
        cache = layer_cache(part.cache_needs(), dtype, length)
        got = run_mixer(part, h, cuts, cache, dtype)
        assert float((got - want).abs().max()) <= limit * float(want.abs().max()), f"cuts {cuts[:3]}"
    assert cache.kv.k.shape[1] == 1 and cache.kv.k.shape[3] == m["kv_rank"] + m["rot_dim"] and cache.kv.v.shape[2] == m["kv_rank"]
    # prompts that start their sequences, nothing else in the step: in bfloat16 the matrix-core kernel takes sizes in whole tiles, and for
    # others the scores are a matrix product of the step's own rows
    dense = dtype == torch.bfloat16 and not ops.attention_takes_latent(dtype, m["kv_rank"] + m["rot_dim"], m["kv_rank"])
    if dtype == torch.bfloat16:
        part.DENSE_SCORES = 70 * m["heads"] * length                 # (the prompt's queries in three stretches)
    cache = layer_cache(part.cache_needs(), dtype, length)
    assert part._prompts_alone(h.cuda(), Step([1], [length], [0]), cache) == dense
    for cuts in ([length], [length - 20] + [1] * 20):
        cache = layer_cache(part.cache_needs(), dtype, length)
        got = run_mixer(part, h, cuts, cache, dtype, padding=0)
        assert float((got - want).abs().max()) <= limit * float(want.abs().max()), f"prompts alone, cuts {cuts[:3]}"
    # two prompts of unequal length in one step, against each alone
    if dtype == torch.bfloat16:
        cache = layer_cache(part.cache_needs(), dtype, length + 128)
        cache.kv.block_table[0, :2] = torch.tensor([0, 1], dtype=torch.int32)      # (two blocks that the sequence in slot 1 does not reach)
        both = torch.full((length + 70, part.hidden), float("nan"), device="cuda")
        part.forward_into(torch.cat([h[:70], h]).to(dtype).cuda(), Step([0, 1], [70, length], [0, 0]), cache, both)
        assert float((both[70:].double().cpu() - want).abs().max()) <= limit * float(want.abs().max())
        assert float((both[:70].double().cpu() - want[:70]).abs().max()) <= limit * float(want.abs().max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("tokens,heads,n,k", [(1, 3, 24, 16), (70, 5, 40, 8), (200, 1, 80, 72), (65, 8, 160, 64), (9, 2, 3, 130), (300, 16, 384, 128),
                                              (100, 4, 96, 96), (17, 3, 50, 32)])
def test_products_with_a_matrix_per_head(tokens, heads, n, k, dtype, ops):
    generator = torch.Generator().manual_seed(n + k)
    a, w = torch.randn(tokens, heads * k, generator=generator).to(dtype), torch.randn(heads, n, k, generator=generator).to(dtype)
    want = torch.einsum("thk,hnk->thn", a.double().reshape(tokens, heads, k), w.double())
    out = torch.zeros(tokens, heads * (n + 5), dtype=dtype, device="cuda")
    ops.linear_heads(a.cuda(), w.cuda(), out, out_head=n + 5)
    got = out.double().cpu().reshape(tokens, heads, n + 5)
    assert float((got[..., :n] - want).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())
    assert float(got[..., n:].abs().max()) == 0.0, "what lies behind a head's outputs was touched"
    # a row's bits do not depend on its company (steps of up to 16 rows add up in another order than longer ones: rounding apart)
    some = min(tokens, 3 if tokens <= 16 else 40)
    fewer = torch.zeros(some, heads * n, dtype=dtype, device="cuda")
    ops.linear_heads(a[tokens - some:].cuda(), w.cuda(), fewer)
    assert torch.equal(fewer.reshape(some, heads, n), out[tokens - some:].reshape(some, heads, n + 5)[..., :n]), "a row's bits depend on its company"
    alone = torch.zeros(1, heads * n, dtype=dtype, device="cuda")
    ops.linear_heads(a[tokens - 1:].cuda(), w.cuda(), alone)
    assert float((alone.double().cpu().reshape(heads, n) - want[tokens - 1]).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())


@pytest.mark.parametrize("experts,top,groups,keep,scale", [(8, 2, 4, 2, 1.7), (6, 3, None, None, 1.0), (12, 4, 3, 3, 0.5), (4, 1, 2, 1, 1.0), (5, 5, None, None, 1.0),
                                                         (16, 3, 8, 2, 2.5), (256, 8, None, None, 1.0), (64, 6, 8, 3, 1.0)])
def test_experts_are_chosen_by_softmax_scores_inside_the_groups_with_the_best_expert(experts, top, groups, keep, scale, ops):
    tokens = 300
    logits = 2.0 * torch.randn(tokens, experts, generator=torch.Generator().manual_seed(experts))
    router = {"experts": experts, "top": top, "scale": scale}
    if groups is not None:
        router["groups"] = {"count": groups, "keep": keep}
    want = P.route(logits.double(), torch.eye(experts, dtype=F), router)                # (a router that passes its input on)
    got = torch.empty(tokens, experts, device="cuda")
    ops.route_experts(logits.cuda(), got, top, groups or 1, keep or 1, group_top=1, scores="softmax", scale=scale)
    assert torch.equal(got.cpu() > 0, want > 0)
    assert torch.allclose(got.double().cpu(), want, atol=1e-6) and torch.allclose(got.sum(dim=1).cpu(), torch.full((tokens,), scale), atol=1e-5)


def test_an_expert_outside_the_kept_groups_is_never_chosen_however_large_its_score(ops):
    # groups {0,1} {2,3} {4,5} score 5, 4 and 3 by their best expert; the second best expert of all (3.9) is in a kept group, 3.0 is not
    logits = torch.tensor([[5.0, 0.0, 4.0, 3.9, 3.0, 2.9], [0.0, 0.1, 0.2, 3.0, 2.9, 2.95]]).cuda()
    weights = torch.empty(2, 6, device="cuda")
    ops.route_experts(logits, weights, 3, 3, 2, group_top=1, scores="softmax", scale=1.0)
    assert weights[0].nonzero().flatten().tolist() == [0, 2, 3] and weights[1].nonzero().flatten().tolist() == [3, 4, 5]
    scores = torch.softmax(logits[0].double().cpu(), dim=0)
    assert weights[0, 3].item() == pytest.approx(float(scores[3] / (scores[0] + scores[2] + scores[3])), rel=1e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("mlp", [dict(ff=24, limit=1.5, experts=8, top=2, groups=(4, 2), scale=1.7), dict(ff=8, limit=0.25, experts=5, top=5),
                                 dict(ff=40, limit=4.0, experts=12, top=4, groups=(3, 2), scale=2.5), dict(ff=64, limit=1.0, experts=3, top=1)])
def test_clamped_experts_alone(mlp, dtype, ops):
    from renapel_models import _moe
    from xeno_rt_amd.models.renapel import _feed_forward
    width, tokens = 48, 90
    raw = _moe(mlp["ff"], mlp["limit"], mlp["experts"], mlp["top"], mlp.get("groups"), mlp.get("scale"))
    part = _feed_forward(raw, "mlp.", types.SimpleNamespace(width=width))
    tensors = tensors_for(part, seed=mlp["ff"], std=0.4, router=(0.0, 0.7))
    part.bind(tensors, runtime(ops, dtype))
    h = torch.randn(tokens, width, generator=torch.Generator().manual_seed(5)).to(dtype)
    want = P.experts_ff(h.double(), short(tensors, "mlp."), raw)
    out = torch.empty(tokens, width, device="cuda")
    part.forward_into(h.cuda(), None, out)
    got = out.double().cpu()
    per_row = (got - want).abs().max(dim=1).values / float(want.abs().max())
    limit = 2e-5 if dtype == torch.float32 else 3e-2
    assert int((per_row > limit).sum()) <= (0 if dtype == torch.float32 else 2), f"rows {(per_row > limit).nonzero().flatten().tolist()} differ"
    alone = torch.empty(1, width, device="cuda")
    part.forward_into(h[17:18].cuda(), None, alone)
    assert float((alone[0] - out[17]).abs().max()) <= 1e-5 * float(want.abs().max()) if dtype == torch.float32 else True


@pytest.mark.parametrize("pack", ["auto", "always", False])
@pytest.mark.parametrize("ff,experts,top,groups,tokens", [(64, 8, 2, (4, 2), 300), (128, 16, 4, None, 1000), (192, 4, 1, (2, 1), 600)])
def test_clamped_experts_multiply_only_the_tokens_that_chose_them(ff, experts, top, groups, tokens, pack, ops):
    """A step of many tokens sorts its picks by expert: against the plain sum, and against the same part with every token
    through every expert (the same choices, so rounding alone differs)."""
    from renapel_models import _moe
    from xeno_rt_amd.models.renapel import _feed_forward
    width = 64
    raw = _moe(ff, 1.5, experts, top, groups, 2.0)
    part = _feed_forward(raw, "mlp.", types.SimpleNamespace(width=width))
    tensors = tensors_for(part, seed=ff, std=0.3, router=(0.0, 0.7))
    from xeno_rt_amd.parts.base import Runtime
    part.bind(tensors, Runtime(ops, torch.bfloat16, "cuda", pack_weights=pack))       # (the stacked gate/up matrix plain, and in tiles)
    assert pack != "always" or hasattr(part.w_gate_up, "unpacked")
    h = torch.randn(tokens, width, generator=torch.Generator().manual_seed(6)).bfloat16()
    assert ops.experts_sorted_takes(h.cuda(), part.w_gate_up, part.w_down, experts, ff, top, stacked=True)
    assert not ops.experts_sorted_takes(h[:8].cuda(), part.w_gate_up, part.w_down, experts, ff, top, stacked=True)
    out = torch.full((tokens, width), float("nan"), device="cuda")
    part.forward_into(h.cuda(), None, out)
    takes = ops.experts_sorted_takes
    ops.experts_sorted_takes = lambda *operands, **options: False
    try:
        dense = torch.empty(tokens, width, device="cuda")
        part.forward_into(h.cuda(), None, dense)
    finally:
        ops.experts_sorted_takes = takes
    want = P.experts_ff(h.double(), short(tensors, "mlp."), raw)
    scale = float(want.abs().max())
    assert float((out - dense).abs().max()) <= 1e-2 * scale
    per_row = (out.double().cpu() - want).abs().max(dim=1).values / scale
    assert int((per_row > 3e-2).sum()) <= max(2, tokens // 50), f"rows {(per_row > 3e-2).nonzero().flatten().tolist()} differ from the plain sum"
    some = torch.arange(tokens - 1, -1, -3)
    fewer = torch.empty(len(some), width, device="cuda")
    part.forward_into(h[some].cuda(), None, fewer)
    if ops.experts_sorted_takes(h[some].cuda(), part.w_gate_up, part.w_down, experts, ff, top, stacked=True):
        assert torch.equal(fewer, out[some.cuda()]), "a token's bits depend on its company"


# ---- through the programs a user runs ----------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay_of_whole_requests_decoded_tails_and_batches(dtype, models, tmp_path):
    from test_trace_run_gpu import collect, replay, trace_batches, trace_tail, trace_whole
    folder, plain, _, _ = models["wide"]
    vocab = CONFIGS["wide"]["vocab"]
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
    folder, plain, ids, _ = models["plain"]
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
    from renapel_models import _moe
    r = random.Random(seed)
    width = r.choice([24, 40, 72, 96, 136])
    layers, owners = [], []
    for index in range(r.randint(2, 6)):
        kind = r.choice(["lightning", "attention", "latent_attention"])
        if kind == "lightning":
            heads = r.randint(1, 4)
            mixer = {"heads": heads, "dim": r.choice([4, 12, 20, 64, 72]), "vdim": r.choice([6, 16, 40, 68]), "decay": [r.choice([0.5, 0.9, 0.99, 1.0]) for _ in range(heads)]}
        elif kind == "attention":
            if owners and r.random() < 0.5:
                source = r.choice(owners)
                mixer = dict(layers[source]["mixer"], kv_from=source, scale=r.choice([0.1, 0.3]), bias_rows=r.choice([2, 6, 16]), bias_max=r.choice([20, 300]))
                mixer.pop("q_temp", None)
            else:
                kv_heads = r.randint(1, 3)
                mixer = {"heads": kv_heads * r.randint(1, 3), "kv_heads": kv_heads, "dim": r.choice([6, 16, 20, 64]), "vdim": r.choice([4, 16, 24, 64]),
                         "scale": r.choice([0.1, 0.3]), "bias_rows": r.choice([2, 5, 12, 40]), "bias_max": r.choice([30, 100, 1000])}
                owners.append(index)
            if r.random() < 0.6:
                mixer["q_temp"] = {"coef": r.choice([0.1, 0.5]), "every": r.choice([1, 7, 64, 100])}
        else:
            rot_dim = r.choice([2, 4, 8, 16])
            mixer = {"heads": r.randint(1, 5), "dim": r.choice([4, 12, 32]), "rot_dim": rot_dim, "vdim": r.choice([6, 16, 36]), "kv_rank": r.choice([8, 30, 56, 96]),
                     "q_rank": r.choice([6, 24, 50]), "scale": r.choice([0.1, 0.25]), "rot": {"dims": r.choice([d for d in (2, 4, 8, 16) if d <= rot_dim]), "base": r.choice([10.0, 1e4])}}
        mlp = None
        if r.random() < 0.75:
            groups = r.choice([None, (2, 1), (3, 2), (4, 4)])
            per_group = r.randint(1, 3)
            experts = per_group * groups[0] if groups else r.randint(1, 9)
            top = r.randint(1, groups[1] * per_group if groups else experts)
            mlp = _moe(r.choice([8, 20, 48]), r.choice([0.3, 1.0, 5.0]), experts, top, groups, r.choice([None, 0.5, 2.0]))
        layers.append({"type": kind, "mixer": mixer, "mlp": mlp})
    config = {"architecture": "Renapel", "vocab": r.choice([50, 97, 200]), "width": width, "norm": {"eps": r.choice([1e-6, 1e-4])}, "layers": layers}
    if r.random() < 0.8:
        config["streams"] = r.randint(1, 5)
    return config


ODD = {          # sizes that are multiples of nothing: no kernel may lean on an alignment that a model need not have
    "architecture": "Renapel", "vocab": 33, "width": 50, "norm": {"eps": 1e-5}, "streams": 3,
    "layers": [
        {"type": "latent_attention", "mixer": {"heads": 3, "dim": 5, "rot_dim": 2, "vdim": 3, "kv_rank": 7, "q_rank": 5, "scale": 0.3,
                                               "rot": {"dims": 2, "base": 100.0}},
         "mlp": {"kind": "moe", "expert": {"ff": 9, "limit": 1.0}, "router": {"experts": 3, "top": 2}}},
        {"type": "attention", "mixer": {"heads": 3, "kv_heads": 1, "dim": 7, "vdim": 5, "scale": 0.4, "bias_max": 50, "bias_rows": 7,
                                        "q_temp": {"coef": 0.2, "every": 3}}, "mlp": None},
        {"type": "lightning", "mixer": {"heads": 3, "dim": 5, "vdim": 7, "decay": [0.9, 0.95, 0.8]},
         "mlp": {"kind": "moe", "expert": {"ff": 11, "limit": 2.0}, "router": {"experts": 6, "top": 3, "groups": {"count": 2, "keep": 1}, "scale": 1.5}}},
        {"type": "attention", "mixer": {"heads": 3, "kv_heads": 1, "dim": 7, "vdim": 5, "scale": 0.4, "bias_max": 13, "bias_rows": 3, "kv_from": 1},
         "mlp": None},
    ],
}


@pytest.mark.parametrize("dtype", DTYPES)
def test_sizes_that_are_multiples_of_nothing(dtype, tmp_path):
    from xeno_rt_amd.engine import Engine
    folder = make_renapel_folder(ODD, tmp_path, seed=5, name_the_rows=False)
    plain = P.PlainModel(folder)
    ids = [token_ids(ODD["vocab"], 131, seed=1), token_ids(ODD["vocab"], 67, seed=2)]
    wants = [plain.logits(i) for i in ids]
    engine = Engine.load(folder, dtype=dtype, max_tokens=64 * 5, max_slots=2)
    assert_logits(run_whole(engine, ids[0]), wants[0], dtype, "odd sizes whole", 0.1)
    assert_logits(in_portions(engine, ids[0], [70, 3, 1]), wants[0], dtype, "odd sizes in portions", 0.1)
    for got, want in zip(run_batched(engine, ids, [100, 65]), wants):
        assert_logits(got, want, dtype, "odd sizes in a batch", 0.1)
    engine.cache.check()


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(seed, tmp_path):
    from xeno_rt_amd.engine import Engine
    raw = random_configuration(seed)
    folder = make_renapel_folder(raw, tmp_path, seed=seed, std=0.15, name_the_rows=seed % 2 == 1)
    plain = P.PlainModel(folder)
    ids = [token_ids(raw["vocab"], 100, seed=seed), token_ids(raw["vocab"], 31, seed=seed + 50)]
    wants = [plain.logits(i) for i in ids]
    # Weights drawn at random make layers that no trained model has: a lightning layer of one small head, whose first tokens'
    # outputs are a vector times a sum that nearly cancels and are then divided by their own size, turns the sign of its whole
    # output on a rounding of bfloat16. So bfloat16 may miss a tenth of a request's rows here (and holds both limits over the
    # others); float32, through the same kernels, may miss none.
    for dtype in DTYPES:
        engine = Engine.load(folder, dtype=dtype, max_tokens=64 * 5, max_slots=2)
        assert_logits(run_whole(engine, ids[0]), wants[0], dtype, f"random configuration {seed} whole: {raw}", 0.1)
        assert_logits(in_portions(engine, ids[0], [40, 2, 1]), wants[0], dtype, f"random configuration {seed} in portions: {raw}", 0.1)
        for got, want in zip(run_batched(engine, ids, [80, 9]), wants):
            assert_logits(got, want, dtype, f"random configuration {seed} in a batch: {raw}", 0.1)
        engine.cache.check()


def test_zz_the_largest_errors_seen_are_reported():
    for dtype, (worst, rms) in WORST.items():
        print(f"renapel, largest errors against the plain model [{dtype}]: max {worst:.2e} (limit {LIMITS[dtype]['max']:.0e}), "
              f"rms {rms:.2e} (limit {LIMITS[dtype]['rms']:.0e})")
