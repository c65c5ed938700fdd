// Attention of query heads that share key/value heads, on the matrix cores, for keys and values of any sizes in whole tiles. It was made
// for attention through a cached latent (parts/latent.py), where all heads of a token read the same row [latent | turned key part]
// and the values are the latents, and serves grouped heads as well. bfloat16, the queries alone in q; key size a multiple of 32 up
// to 640, value size a multiple of 32 up to 512 (the sizes at which cache blocks lie in the tiles of cache_layout.h). A query sees all
// keys at or before it, or with a window the `window` newest of them and the sequence's first keep_first ones. With a softcap c
// a scaled score s becomes c * tanh(s / c).
//
// Steps of few tokens (xrt_attention_latent).
// A wavefront takes a token, up to sixteen heads of one key/value head and a chunk of the keys that the token sees, in groups of 32. The
// heads are columns of v_mfma_f32_16x16x32_bf16: S^T[key][head] = K Q^T with a tile of the cache (16 keys x 32 dims, in the
// order of the A operand: one load instruction takes a contiguous kilobyte) as A and the heads' queries, kept in registers,
// as B; after the two tiles of a group of 32 keys a lane holds the scores of eight consecutive keys of one head, which is the
// B operand of O^T[dim][head] += V^T P^T, whose A operand is a tile of the value block (16 dims x 32 tokens) as it lies.
// The softmax's weights are float32 and enter that product as two bfloat16 numbers each, the rounded weight and what the
// rounding left. Every chunk is worked off from empty hands; a second kernel merges a token's chunks in their order, adds the
// head's sink to the denominator (a learnt score without a value, or none) and writes the result.
//
// Steps that bring sequences many tokens (xrt_attention_latent_prompts). The heads of a key/value head read the same keys in all
// tokens, so its (token, head) pairs of a sequence are simply rows, one after another, and a wavefront takes sixteen of them as the columns of
// its products: with many heads its rows are one token's or a few tokens', with few heads many tokens'. A workgroup of eight
// wavefronts (or four) walks the groups of 32 keys that some row of it sees; a group's tiles of keys and values (a contiguous
// stretch each) travel straight into LDS while the group before it is multiplied. The softmax keeps its exponent until a score
// exceeds it by 8 (in log2), so that the sums are rarely rescaled.
#include "cache_layout.h"
#include "xrt_hip.h"

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float floatx4 __attribute__((ext_vector_type(4)));

constexpr int KEYS_MOST = 640, LATENT_MOST = 512;       // largest key and value size
constexpr int KEY_STEPS = KEYS_MOST / 32;        // steps of 32 dims of a score product
constexpr int VALUE_TILES = LATENT_MOST / 16;    // tiles of 16 dims of the value product
constexpr int HEADS_A_WAVE = 16;
constexpr int GROUP = 32;                        // keys that are multiplied together (half a cache block)
constexpr int BATCH = 8;                         // tiles (or pairs of them) that a decode step's wavefront asks for at a time
static_assert(VALUE_TILES % BATCH == 0, "values come in whole batches");
constexpr float LOG2E = 1.4426950408889634f;
constexpr int MOST_CHUNKS = XRT_WAVE;            // chunks of groups that a query's keys are cut into at most (a lane each in the merge)

// What a query sees: keys from `first` on up to its own, and those before `kept`, which end before `first`. In groups of 32
// keys, counted through: first the groups of kept keys that lie wholly before the window's first group, then the window's. Every
// group that is counted holds a key that is seen.
struct Seen {
    int first, kept, low, kept_groups;
    __host__ __device__ __forceinline__ Seen(int pos, int window, int keep_first) {
        first = window > 0 && pos >= window ? pos - window + 1 : 0;
        kept = keep_first < first ? keep_first : first;
        low = first / GROUP;
        kept_groups = (kept + GROUP - 1) / GROUP;
        kept_groups = kept_groups < low ? kept_groups : low;
    }
    __host__ __device__ __forceinline__ int groups(int last) const { return kept_groups + last / GROUP - low + 1; }
    __device__ __forceinline__ int group_at(int counted) const { return counted < kept_groups ? counted : low + counted - kept_groups; }
    __device__ __forceinline__ bool sees(int key, int pos) const { return key <= pos && (key >= first || key < kept); }
};

// cap * tanh(score * scale / cap) with the score's scale and the factor of the result's unit folded into two constants: to_power turns
// a raw score into the power of two that tanh is made from, cap is in the result's unit.
__device__ __forceinline__ float capped(float raw, float to_power, float cap) {
    return cap * (1.0f - 2.0f * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(raw * to_power) + 1.0f));
}

// Heads, sizes and which keys are seen.
struct Shape {
    int n_heads, n_kv_heads, head_dim, value_dim, window, keep_first;
    __host__ __device__ __forceinline__ int group() const { return n_heads / n_kv_heads; }                                    // heads that share a key/value head
    __host__ __device__ __forceinline__ int head_tiles() const { return (group() + HEADS_A_WAVE - 1) / HEADS_A_WAVE; }       // sixteens of them
};

// floats a (token, head group, chunk) leaves for the merge: for each of 16 heads the weighted values, the largest score, the sum
__host__ __device__ inline int head_floats(int value_dim) { return value_dim + 4; }     // (a multiple of four: a lane stores four at a time)
__host__ __device__ inline long partial_floats(int value_dim) { return (long)HEADS_A_WAVE * head_floats(value_dim); }

// KEY_STEPS_, VALUE_TILES_: the steps of 32 key dims and tiles of 16 value dims that this instantiation has registers for. CAP: with a softcap.
template <int KEY_STEPS_, int VALUE_TILES_, bool CAP>
__global__ void __launch_bounds__(XRT_WAVE) latent_chunks_kernel(const bf16* __restrict__ q, long q_stride, const Shape shape,
                                                                const bf16* __restrict__ k_cache, const bf16* __restrict__ v_cache,
                                                                const int* __restrict__ block_table, int table_stride, int n_blocks,
                                                                const int* __restrict__ positions, const int* __restrict__ slots, float scale, float softcap,
                                                                int chunk_groups, int chunks, float* __restrict__ partial) {
    const int lane = threadIdx.x, column = lane % 16, quarter = lane / 16;
    const int head_dim = shape.head_dim, value_dim = shape.value_dim;
    const int chunk = blockIdx.x, groups = gridDim.z, kv_head = (int)blockIdx.z / shape.head_tiles(), head_tile = (int)blockIdx.z % shape.head_tiles();
    const long token = blockIdx.y;
    const int slot = slots[token], pos = positions[token];
    if (slot < 0) return;                                      // (the merge writes zeros)
    const Seen seen(pos, shape.window, shape.keep_first);
    const int first_group = chunk * chunk_groups, last_group = min(seen.groups(pos), first_group + chunk_groups) - 1;
    if (first_group > last_group) return;                      // (the merge knows from the position which chunks exist)
    const int in_group = head_tile * HEADS_A_WAVE + column, group_size = shape.group();
    const bool wanted = in_group < group_size;
    const int head = kv_head * group_size + min(in_group, group_size - 1);
    const float to_power = CAP ? 2.0f * LOG2E * scale / softcap : 0.f;
    const int key_steps = head_dim / 32, value_tiles = value_dim / 16;

    // the heads' queries: lane (column, quarter) holds dims 32 s + 8 quarter .. + 7 of head `column`, for every step s
    bf16x8 queries[KEY_STEPS_];
    const bf16* mine = q + token * q_stride + (long)head * head_dim + quarter * 8;
#pragma unroll
    for (int s = 0; s < KEY_STEPS_; ++s) {
#pragma unroll
        for (int e = 0; e < 8; ++e) queries[s][e] = (bf16)0.f;
        if (s < key_steps && wanted) queries[s] = *reinterpret_cast<const bf16x8*>(mine + s * 32);
    }
    floatx4 o[VALUE_TILES_];
#pragma unroll
    for (int u = 0; u < VALUE_TILES_; ++u) o[u] = floatx4{0.f, 0.f, 0.f, 0.f};
    float top = -INFINITY, sum = 0.f;                          // of this lane's head: top is shared by the head's four lanes, sum is this lane's share

    const int* table = block_table + (long)slot * table_stride;
    for (int counted = first_group; counted <= last_group; ++counted) {
        const int g = seen.group_at(counted);
        const int k0 = g * GROUP, half = g % 2;                // the first or second half of the cache block g / 2
        const int block = min(max(table[g / 2], 0), n_blocks - 1);     // the host never hands out anything else
        const bf16* keys = k_cache + ((long)block * shape.n_kv_heads + kv_head) * XRT_BLOCK_TOKENS * head_dim;
        const bf16* values = v_cache + ((long)block * shape.n_kv_heads + kv_head) * XRT_BLOCK_TOKENS * value_dim;
        // The tiles are asked for BATCH steps at a time, both tiles of a step, before the products that use them (a branch per step
        // would have every load awaited alone; a decode step's wavefronts are few, and what they wait for is memory); steps
        // beyond the key's size read the last tile again and multiply it with queries that are zeros.
        floatx4 s[2] = {floatx4{0.f, 0.f, 0.f, 0.f}, floatx4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int step0 = 0; step0 < KEY_STEPS_; step0 += BATCH) {
            if (step0 < key_steps) {
                bf16x8 tiles[2][BATCH];
#pragma unroll
                for (int t = 0; t < 2; ++t)
#pragma unroll
                    for (int i = 0; i < BATCH; ++i)
                        if (step0 + i < KEY_STEPS_)
                            tiles[t][i] = *reinterpret_cast<const bf16x8*>(keys + ((long)((half * 2 + t) * key_steps + min(step0 + i, key_steps - 1)) * XRT_WAVE + lane) * 8);
#pragma unroll
                for (int i = 0; i < BATCH; ++i)
#pragma unroll
                    for (int t = 0; t < 2; ++t)
                        if (step0 + i < KEY_STEPS_) s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tiles[t][i], queries[step0 + i], s[t], 0, 0, 0);
            }
        }
        // the first values are on their way while the softmax is done, and later ones while those before them are multiplied
        // (tiles beyond the value's size: the last one again, into sums that nobody reads)
        auto value_at = [&](int u) { return *reinterpret_cast<const bf16x8*>(values + ((long)(half * value_tiles + min(u, value_tiles - 1)) * XRT_WAVE + lane) * 8); };
        bf16x8 coming[BATCH];
#pragma unroll
        for (int i = 0; i < BATCH; ++i) coming[i] = value_at(i);
        // register i of tile t is the key k0 + 8 quarter + 4 t + i, for this lane's head
        float scores[8];
        float here = -INFINITY;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float raw = s[e / 4][e % 4];
            scores[e] = seen.sees(k0 + quarter * 8 + e, pos) ? (CAP ? capped(raw, to_power, softcap) : raw * scale) : -INFINITY;
            here = fmaxf(here, scores[e]);
        }
        here = fmaxf(here, __shfl_xor(here, 16, XRT_WAVE));
        here = fmaxf(here, __shfl_xor(here, 32, XRT_WAVE));
        const float top_new = fmaxf(top, here);            // (finite: every group of the chunk has a key that the query sees)
        const float correction = expf(top - top_new);      // 0 for empty hands
        top = top_new;
        sum *= correction;
        bf16x8 rounded, rest;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float weight = expf(scores[e] - top);     // 0 for a key that is not seen
            sum += weight;
            rounded[e] = (bf16)weight;
            rest[e] = (bf16)(weight - (float)rounded[e]);
        }
        const bool edge = k0 + 31 > pos;                    // what lies behind the sequence's last key is not ours: kept away from the zeros
#pragma unroll
        for (int u0 = 0; u0 < VALUE_TILES_; u0 += BATCH) {
            if (u0 < value_tiles) {
                bf16x8 tiles[BATCH];
#pragma unroll
                for (int i = 0; i < BATCH; ++i) {
                    tiles[i] = coming[i];
                    if (u0 + BATCH < VALUE_TILES_) coming[i] = value_at(u0 + BATCH + i);
                }
#pragma unroll
                for (int i = 0; i < BATCH; ++i) {
                    if (edge) {
#pragma unroll
                        for (int e = 0; e < 8; ++e)
                            if (k0 + quarter * 8 + e > pos) tiles[i][e] = (bf16)0.f;
                    }
#pragma unroll
                    for (int j = 0; j < 4; ++j) o[u0 + i][j] *= correction;
                    o[u0 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tiles[i], rounded, o[u0 + i], 0, 0, 0);
                    o[u0 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tiles[i], rest, o[u0 + i], 0, 0, 0);
                }
            }
        }
    }
    sum += __shfl_xor(sum, 16, XRT_WAVE);
    sum += __shfl_xor(sum, 32, XRT_WAVE);
    // register i of tile u is dim 16 u + 4 quarter + i of head `column`
    float* out = partial + ((token * groups + blockIdx.z) * chunks + chunk) * partial_floats(value_dim) + (long)column * head_floats(value_dim);
#pragma unroll
    for (int u = 0; u < VALUE_TILES_; ++u) {
        if (u < value_tiles && wanted) *reinterpret_cast<floatx4*>(out + u * 16 + quarter * 4) = o[u];
    }
    if (quarter == 0 && wanted) {
        out[value_dim] = top;
        out[value_dim + 1] = sum;
    }
}

// A workgroup a (token, head): the chunks' parts in their order, the sink, the quotient. OWNED: value dims a lane has (value size / 64 at least).
template <int OWNED>
__global__ void __launch_bounds__(XRT_WAVE) latent_merge_kernel(const float* __restrict__ partial, const Shape shape, int chunk_groups, int chunks, const int* __restrict__ positions,
                                                               const int* __restrict__ slots, const float* __restrict__ sinks, bf16* __restrict__ out) {
    const long token = blockIdx.x;
    const int head = blockIdx.y, lane = threadIdx.x, value_dim = shape.value_dim, groups = shape.n_kv_heads * shape.head_tiles();
    const int in_group = head % shape.group(), group = head / shape.group() * shape.head_tiles() + in_group / HEADS_A_WAVE;
    bf16* dst = out + (token * shape.n_heads + head) * value_dim;
    if (slots[token] < 0) {
        for (int d = lane; d < value_dim; d += XRT_WAVE) dst[d] = (bf16)0.f;
        return;
    }
    const int pos = positions[token];
    const int mine = (Seen(pos, shape.window, shape.keep_first).groups(pos) - 1) / chunk_groups + 1;      // this query's chunks
    const float* parts = partial + ((token * groups + group) * chunks) * partial_floats(value_dim) + (long)(in_group % HEADS_A_WAVE) * head_floats(value_dim);
    constexpr int MERGED = 8;
    float acc[OWNED], top = -INFINITY, sum = 0.f;
#pragma unroll
    for (int i = 0; i < OWNED; ++i) acc[i] = 0.f;
    // First the largest score of all chunks (lane c reads chunk c's), then every chunk's share relative to it, in the chunks'
    // order, MERGED chunks' loads on their way at a time (chunks beyond the sequence's read the last one again with a share of nothing).
    const long stride = partial_floats(value_dim);
    const float my_top = lane < mine ? parts[(long)lane * stride + value_dim] : -INFINITY;
    top = wave_max(my_top);
    const float my_take = lane < mine ? expf(my_top - top) : 0.f;
    sum = wave_sum(lane < mine ? parts[(long)lane * stride + value_dim + 1] * my_take : 0.f);
#pragma unroll
    for (int c0 = 0; c0 < MOST_CHUNKS; c0 += MERGED) {
        if (c0 < mine) {
            float loaded[MERGED][OWNED], take[MERGED];
#pragma unroll
            for (int j = 0; j < MERGED; ++j) {
                const float* part = parts + (long)min(c0 + j, mine - 1) * stride;
                take[j] = __shfl(my_take, c0 + j, XRT_WAVE);       // (0 from a lane beyond the sequence's chunks)
#pragma unroll
                for (int i = 0; i < OWNED; ++i) loaded[j][i] = lane + i * XRT_WAVE < value_dim ? part[lane + i * XRT_WAVE] : 0.f;
            }
#pragma unroll
            for (int j = 0; j < MERGED; ++j)
#pragma unroll
                for (int i = 0; i < OWNED; ++i) acc[i] = fmaf(loaded[j][i], take[j], acc[i]);
        }
    }
    if (sinks != nullptr) {                                    // one more term of the denominator, without a value
        const float sink = sinks[head], top_new = fmaxf(top, sink);
        const float keep = expf(top - top_new);
        sum = fmaf(sum, keep, expf(sink - top_new));
#pragma unroll
        for (int i = 0; i < OWNED; ++i) acc[i] *= keep;
    }
    const float inv = sum > 0.f ? 1.0f / sum : 0.f;
#pragma unroll
    for (int i = 0; i < OWNED; ++i) {
        const int d = lane + i * XRT_WAVE;
        if (d < value_dim) dst[d] = (bf16)(acc[i] * inv);
    }
}

// Groups of keys that a query sees at most (a window's keys may begin and end inside a group, and kept ones lie in groups of their own
// before it), and how many of them a chunk has.
int most_groups(int max_context, int window, int keep_first) {
    const int all = (max(max_context, 1) + GROUP - 1) / GROUP;
    if (window <= 0) return all;
    const long some = ((long)window + GROUP - 2) / GROUP + 1 + ((long)keep_first + GROUP - 1) / GROUP;
    return (int)min((long)all, some);
}
int chunk_groups_for(int max_context, int window, int keep_first) { return (most_groups(max_context, window, keep_first) + MOST_CHUNKS - 1) / MOST_CHUNKS; }
int chunks_for(int max_context, int window, int keep_first) {
    const int groups = chunk_groups_for(max_context, window, keep_first);
    return (most_groups(max_context, window, keep_first) + groups - 1) / groups;
}

// ---- steps that bring sequences many tokens -------------------------------------------------------------------------------

constexpr int WAVE_ROWS = 16;                    // rows of a wavefront: the columns of its products
constexpr int AHEAD = 2;                         // pairs of tiles that are read from LDS ahead of their products
constexpr int TILE_BYTES = 1024;                 // an operand tile of the cache, in the order of the lanes

// KS, VT: the steps of 32 key dims and tiles of 16 value dims that this instantiation multiplies, whatever the sizes leave of them.
// WAVES: wavefronts of a workgroup. CAP: with a softcap. (Tried and no faster: two sets of sixteen rows a wavefront, which share the tiles
// read from LDS, and three groups of keys in LDS instead of two.)
template <int KS, int VT, int WAVES, bool CAP>
__global__ void __launch_bounds__(WAVES * XRT_WAVE) latent_prompts_kernel(
    const bf16* __restrict__ q, const Shape shape, const bf16* __restrict__ k_cache, const bf16* __restrict__ v_cache,
    const int* __restrict__ block_table, int table_stride, int n_blocks, const int* __restrict__ seq_offsets, const int* __restrict__ seq_slots,
    const int* __restrict__ seq_starts, int n_seqs, float scale, float softcap, const float* __restrict__ sinks, bf16* __restrict__ out) {
    constexpr int TILE_ROWS = WAVES * WAVE_ROWS;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
    const int lane = threadIdx.x % XRT_WAVE, column = lane % 16, quarter = lane / 16;
    const int wave = __builtin_amdgcn_readfirstlane((int)threadIdx.x / XRT_WAVE);
    const int head_dim = shape.head_dim, value_dim = shape.value_dim, window = shape.window, keep_first = shape.keep_first;
    const int key_steps = head_dim / 32, value_tiles = value_dim / 16;
    const int kv_head = blockIdx.y, group_size = shape.group();

    // which sequence, and which of its tiles of rows (the last ones, which see most keys, first)
    int tile = blockIdx.x, seq = 0, count = 0;
    bool found = false;
    for (; seq < n_seqs; ++seq) {
        count = seq_offsets[seq + 1] - seq_offsets[seq];
        const int tiles = (int)(((long)count * group_size + TILE_ROWS - 1) / TILE_ROWS);
        if (tile < tiles) {
            tile = tiles - 1 - tile;
            found = true;
            break;
        }
        tile -= tiles;
    }
    if (!found) return;                                        // the whole workgroup leaves
    const int slot = seq_slots[seq], start = seq_starts[seq];
    const long first_token = seq_offsets[seq];
    const int rows = count * group_size;                       // (below 2^31: checked on the host)
    // row r of a sequence is head r % group_size of the key/value head, of token r / group_size
    auto at = [&](int r) { return (first_token + r / group_size) * shape.n_heads + (long)kv_head * group_size + r % group_size; };
    if (slot < 0) {                                            // a sequence of padding: zeros, which nobody reads
        for (int r = tile * TILE_ROWS; r < min(rows, (tile + 1) * TILE_ROWS); ++r)
            for (int d = threadIdx.x; d < value_dim; d += blockDim.x) out[at(r) * value_dim + d] = (bf16)0.f;
        return;
    }
    // the groups of keys that some row of the workgroup sees: kept ones, then those of the windows
    const int pos_low = start + tile * TILE_ROWS / group_size, pos_high = start + (min(rows, (tile + 1) * TILE_ROWS) - 1) / group_size;
    const int group_low = Seen(pos_low, window, keep_first).low, group_high = pos_high / GROUP;
    const int kept_groups = min((Seen(pos_high, window, keep_first).kept + GROUP - 1) / GROUP, group_low);
    const int groups = kept_groups + group_high - group_low + 1;
    auto group_at = [&](int counted) { return counted < kept_groups ? counted : group_low + counted - kept_groups; };

    // this wavefront's rows, a column each
    const int wave_row = tile * TILE_ROWS + wave * WAVE_ROWS;
    const bool awake = wave_row < rows;
    const int wave_low = start + min(wave_row, rows - 1) / group_size, wave_high = start + min(wave_row + WAVE_ROWS - 1, rows - 1) / group_size;
    const int wave_all = Seen(wave_high, window, keep_first).first;      // the first key that the windows of all rows of the wavefront hold
    const int row = wave_row + column, clamped = min(row, rows - 1);
    const int pos = start + clamped / group_size, head = kv_head * group_size + clamped % group_size;
    const bf16* of_row = q + at(clamped) * head_dim + quarter * 8;
    bf16x8 queries[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
#pragma unroll
        for (int e = 0; e < 8; ++e) queries[s][e] = (bf16)0.f;
        if (s < key_steps) queries[s] = *reinterpret_cast<const bf16x8*>(of_row + s * 32);
    }
    // (awaited here: left to their first use the wait would stand inside the loop and hold up the tiles on their way to LDS)
#pragma unroll
    for (int s = 0; s < KS; ++s) asm volatile("" : "+v"(queries[s]));
    floatx4 o[VT];
#pragma unroll
    for (int u = 0; u < VT; ++u) o[u] = floatx4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;                              // m is shared by the row's four lanes, l is this lane's share

    // scores are kept in units of log2: scaled as they are used, or, with a softcap, scaled and capped at once
    const float scale2 = CAP ? 1.0f : scale * LOG2E;
    const float to_power = CAP ? 2.0f * LOG2E * scale / softcap : 0.f, cap2 = CAP ? softcap * LOG2E : 0.f;
    // A buffer has a place for every tile that this instantiation may have: keys' first tiles, their second ones, values. (The places
    // are the same whatever the sizes, so that the reads have their offsets in the instructions.)
    constexpr int PLACES = 2 * KS + VT;
    const int key_tiles = 2 * key_steps, tiles_a_group = key_tiles + value_tiles;
    const unsigned lds0 = lds_address(lds_raw);
    constexpr unsigned buffer_bytes = (unsigned)PLACES * TILE_BYTES;
    const int* table = block_table + (long)slot * table_stride;
    // a group's tiles into buffer `buffer`: keys, then values, dealt to the wavefronts in turn
    auto fetch = [&](int g, int buffer) {
        const int block = __builtin_amdgcn_readfirstlane(min(max(table[g / 2], 0), n_blocks - 1));       // the host never hands out anything else
        const long of_head = ((long)block * shape.n_kv_heads + kv_head) * XRT_BLOCK_TOKENS;
        const char* keys = reinterpret_cast<const char*>(k_cache + of_head * head_dim) + (long)(g % 2) * key_tiles * TILE_BYTES;
        const char* values = reinterpret_cast<const char*>(v_cache + of_head * value_dim) + (long)(g % 2) * value_tiles * TILE_BYTES;
        for (int t = wave; t < tiles_a_group; t += WAVES) {
            const bool is_key = t < key_tiles;
            const int place = !is_key ? 2 * KS + t - key_tiles : t < key_steps ? t : KS + t - key_steps;
            load_to_lds(is_key ? keys : values, (unsigned)((is_key ? t : t - key_tiles) * TILE_BYTES + lane * 16),
                        lds0 + (unsigned)buffer * buffer_bytes + (unsigned)place * TILE_BYTES);
        }
    };

    // places that the sizes at hand leave empty hold zeros (the code multiplies them all, without a branch)
    for (int t = wave; t < 2 * PLACES; t += WAVES) {
        const int place = t % PLACES;
        if (place < 2 * KS ? place % KS >= key_steps : place - 2 * KS >= value_tiles)
            *reinterpret_cast<uint4*>(lds_raw + (size_t)t * TILE_BYTES + lane * 16) = make_uint4(0u, 0u, 0u, 0u);
    }
    fetch(group_at(0), 0);
    for (int counted = 0; counted < groups; ++counted) {
        // this group has arrived from every wavefront, and the one before it has been read by all: its buffer takes the next one
        wait_loads_and_barrier<0>();
        const int buffer = counted & 1;
        if (counted + 1 < groups) fetch(group_at(counted + 1), buffer ^ 1);
        const int k0 = group_at(counted) * GROUP;
        const unsigned char* tiles = lds_raw + (size_t)buffer * buffer_bytes + lane * 16;
        auto tile_at = [&](int t) { return *reinterpret_cast<const bf16x8*>(tiles + (size_t)t * TILE_BYTES); };
        floatx4 s[2] = {floatx4{0.f, 0.f, 0.f, 0.f}, floatx4{0.f, 0.f, 0.f, 0.f}};
        // A tile is read AHEAD steps before it is multiplied. (The fences between the steps keep the compiler from reading
        // all of them at once.)
        bf16x8 ahead[AHEAD][2];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) { ahead[i][0] = tile_at(i); ahead[i][1] = tile_at(KS + i); }
#pragma unroll
        for (int step = 0; step < KS; ++step) {
            __builtin_amdgcn_sched_barrier(0);
            const bf16x8 first = ahead[step % AHEAD][0], second = ahead[step % AHEAD][1];
            if (step + AHEAD < KS) { ahead[step % AHEAD][0] = tile_at(step + AHEAD); ahead[step % AHEAD][1] = tile_at(KS + step + AHEAD); }
            s[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(first, queries[step], s[0], 0, 0, 0);
            s[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(second, queries[step], s[1], 0, 0, 0);
        }
        // the first values are on their way while the softmax is done
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) { ahead[i][0] = tile_at(2 * KS + 2 * i); ahead[i][1] = tile_at(2 * KS + 2 * i + 1); }
        __builtin_amdgcn_sched_barrier(0);
        // register i of tile t is the key k0 + 8 quarter + 4 t + i, for the row of this lane's column
        const bool masked = k0 + GROUP - 1 > wave_low || k0 < wave_all;
        if constexpr (CAP) {
#pragma unroll
            for (int e = 0; e < 8; ++e) s[e / 4][e % 4] = capped(s[e / 4][e % 4], to_power, cap2);
        }
        if (masked) {
            const Seen seen(pos, window, keep_first);
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (!seen.sees(k0 + quarter * 8 + e, pos)) s[e / 4][e % 4] = -INFINITY;
        }
        float top = s[0][0];
#pragma unroll
        for (int e = 1; e < 8; ++e) top = fmaxf(top, s[e / 4][e % 4]);
        top *= scale2;                                     // (the scale is positive: checked on the host)
        // m is the exponent that the sums are relative to; it moves only when some row meets a score more than 8 above it (in
        // log2), until when the weights stay below 2^8 and the quotient in the end is the same.
        if (__builtin_amdgcn_ballot_w64(top > m + 8.0f) != 0) {
            float here = fmaxf(top, __shfl_xor(top, 16, XRT_WAVE));
            here = fmaxf(here, __shfl_xor(here, 32, XRT_WAVE));
            const float m_new = fmaxf(m, here);
            const float correction = __builtin_amdgcn_exp2f(m - (m_new == -INFINITY ? 0.f : m_new));
            m = m_new;
            l *= correction;
#pragma unroll
            for (int u = 0; u < VT; ++u)
#pragma unroll
                for (int j = 0; j < 4; ++j) o[u][j] *= correction;
        }
        bf16x8 rounded, rest;
        const float m_safe = m == -INFINITY ? 0.f : m;       // a row that has seen no key yet
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float weight = __builtin_amdgcn_exp2f(fmaf(s[e / 4][e % 4], scale2, -m_safe));
            l += weight;
            rounded[e] = (bf16)weight;
            rest[e] = (bf16)(weight - (float)rounded[e]);
        }
        const bool edge = k0 + GROUP - 1 > pos_high;       // what lies behind the last key may be anything: kept away from the weights' zeros
#pragma unroll
        for (int u0 = 0; u0 < VT; u0 += 2) {
            __builtin_amdgcn_sched_barrier(0);
            bf16x8 value[2] = {ahead[u0 / 2 % AHEAD][0], ahead[u0 / 2 % AHEAD][1]};
            if (u0 + 2 * AHEAD < VT) {
                ahead[u0 / 2 % AHEAD][0] = tile_at(2 * KS + u0 + 2 * AHEAD);
                ahead[u0 / 2 % AHEAD][1] = tile_at(2 * KS + u0 + 2 * AHEAD + 1);
            }
            if (edge) {
#pragma unroll
                for (int i = 0; i < 2; ++i)
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (k0 + quarter * 8 + e > pos_high) value[i][e] = (bf16)0.f;
            }
#pragma unroll
            for (int i = 0; i < 2; ++i)
                o[u0 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(value[i], rounded, o[u0 + i], 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 2; ++i)
                o[u0 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(value[i], rest, o[u0 + i], 0, 0, 0);
        }
    }
    if (!awake) return;
    float sum = l;
    sum += __shfl_xor(sum, 16, XRT_WAVE);
    sum += __shfl_xor(sum, 32, XRT_WAVE);
    if (sinks != nullptr) sum += __builtin_amdgcn_exp2f(fmaf(sinks[head], LOG2E, -(m == -INFINITY ? 0.f : m)));    // (relative to the same exponent)
    const float inv = sum > 0.f ? 1.0f / sum : 0.f;
    if (row < rows) {
        // register i of tile u is dim 16 u + 4 quarter + i of this lane's row
        bf16* dst = out + at(row) * value_dim + quarter * 4;
#pragma unroll
        for (int u = 0; u < VT; ++u) {
            if (u < value_tiles) {
                struct alignas(8) Four { bf16 e[4]; } four;
#pragma unroll
                for (int i = 0; i < 4; ++i) four.e[i] = (bf16)(o[u][i] * inv);
                *reinterpret_cast<Four*>(dst + u * 16) = four;
            }
        }
    }
}

template <int KS, int VT, int WAVES, bool CAP>
int launch_prompts(const bf16* q, long tokens, const Shape& shape, const bf16* k_cache, const bf16* v_cache, const int* block_table, int table_stride,
                   int n_blocks, const int* seq_offsets, const int* seq_slots, const int* seq_starts, int n_seqs, float scale, float softcap,
                   const float* sinks, bf16* out, hipStream_t s) {
    constexpr int TILE_ROWS = WAVES * WAVE_ROWS;
    const long tiles = tokens * shape.group() / TILE_ROWS + n_seqs;     // every sequence's last tile may be partly filled
    XRT_REQUIRE(tiles < (1L << 31), "attention (latent, prompts): too many rows");
    constexpr size_t lds = (size_t)2 * (2 * KS + VT) * TILE_BYTES;
    static bool configured = false;                            // per instantiation
    if (!configured) {
        hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(latent_prompts_kernel<KS, VT, WAVES, CAP>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        XRT_REQUIRE(e == hipSuccess, "attention (latent, prompts): cannot reserve %zu bytes of LDS: %s", lds, hipGetErrorString(e));
        configured = true;
    }
    latent_prompts_kernel<KS, VT, WAVES, CAP><<<dim3((unsigned)tiles, shape.n_kv_heads), WAVES * XRT_WAVE, lds, s>>>(
        q, shape, k_cache, v_cache, block_table, table_stride, n_blocks, seq_offsets, seq_slots, seq_starts, n_seqs, scale, softcap, sinks, out);
    XRT_LAUNCH_CHECK("attention (latent, prompts)");
    return 0;
}

bool shape_is_sound(const Shape& shape) {
    return shape.n_heads > 0 && shape.n_kv_heads > 0 && shape.n_heads % shape.n_kv_heads == 0 && shape.window >= 0 && shape.keep_first >= 0 &&
           (shape.window > 0 || shape.keep_first == 0);
}

}  // namespace

extern "C" int xrt_attention_latent_accepts(int dtype, int head_dim, int value_dim) {
    return dtype == XRT_BF16 && head_dim % 32 == 0 && value_dim % 32 == 0 && head_dim > 0 && value_dim > 0 && head_dim <= KEYS_MOST && value_dim <= LATENT_MOST;
}

extern "C" long xrt_attention_latent_workspace(long tokens, int n_heads, int n_kv_heads, int value_dim, int max_context, int window, int keep_first) {
    if (n_kv_heads <= 0 || n_heads % n_kv_heads != 0) return 0;
    const Shape shape{n_heads, n_kv_heads, 0, value_dim, window, keep_first};
    return tokens * n_kv_heads * shape.head_tiles() * chunks_for(max_context, window, keep_first) * partial_floats(value_dim);
}

extern "C" int xrt_attention_latent(const void* q, long q_stride, long tokens, int n_heads, int n_kv_heads, int head_dim, int value_dim, const void* k_cache,
                                    const void* v_cache, const int* block_table, int table_stride, int n_blocks, const int* positions,
                                    const int* slots, void* out, float scale, float softcap, int window, int keep_first, const float* sink_scores,
                                    int max_context, float* workspace, long workspace_floats, void* stream) {
    XRT_REQUIRE(xrt_attention_latent_accepts(XRT_BF16, head_dim, value_dim), "attention (latent): key and value sizes %d and %d: multiples of 32 up to %d and %d",
                head_dim, value_dim, KEYS_MOST, LATENT_MOST);
    XRT_REQUIRE(q && k_cache && v_cache && block_table && positions && slots && out, "attention (latent): null operand");
    const Shape shape{n_heads, n_kv_heads, head_dim, value_dim, window, keep_first};
    XRT_REQUIRE(shape_is_sound(shape) && tokens >= 0 && tokens <= 65535 && n_heads <= 65535 && (long)n_kv_heads * shape.head_tiles() <= 65535 && table_stride > 0 &&
                n_blocks > 0 && max_context > 0 && softcap >= 0.f, "attention (latent): bad sizes (%ld tokens, %d heads on %d)", tokens, n_heads, n_kv_heads);
    XRT_REQUIRE(q_stride >= (long)n_heads * head_dim && q_stride % 8 == 0 && (uintptr_t)q % 16 == 0 && (uintptr_t)k_cache % 16 == 0 && (uintptr_t)v_cache % 16 == 0,
                "attention (latent): rows of q %ld apart, or operands off their sixteen bytes", q_stride);
    XRT_REQUIRE(max_context <= table_stride * XRT_BLOCK_TOKENS, "attention (latent): a sequence of %d tokens exceeds the block table", max_context);
    if (tokens == 0) return 0;
    const int chunk_groups = chunk_groups_for(max_context, window, keep_first), chunks = chunks_for(max_context, window, keep_first);
    const int groups = n_kv_heads * shape.head_tiles();
    XRT_REQUIRE(workspace != nullptr && workspace_floats >= tokens * groups * chunks * partial_floats(value_dim) && (uintptr_t)workspace % 16 == 0,
                "attention (latent): the workspace needs %ld floats", tokens * groups * chunks * partial_floats(value_dim));
    const dim3 grid(chunks, (unsigned)tokens, groups);
#define XRT_CHUNKS(KS_, VT_, CAP_)                                                                                                                     \
    latent_chunks_kernel<KS_, VT_, CAP_><<<grid, XRT_WAVE, 0, (hipStream_t)stream>>>((const bf16*)q, q_stride, shape, (const bf16*)k_cache,            \
        (const bf16*)v_cache, block_table, table_stride, n_blocks, positions, slots, scale, softcap, chunk_groups, chunks, workspace)
    if (head_dim <= 128 && value_dim <= 128) { if (softcap > 0.f) XRT_CHUNKS(4, 8, true); else XRT_CHUNKS(4, 8, false); }
    else if (softcap > 0.f) XRT_CHUNKS(KEY_STEPS, VALUE_TILES, true);
    else XRT_CHUNKS(KEY_STEPS, VALUE_TILES, false);
#undef XRT_CHUNKS
    XRT_LAUNCH_CHECK("attention (latent, chunks)");
#define XRT_MERGE(OWNED_)                                                                                                                               \
    latent_merge_kernel<OWNED_><<<dim3((unsigned)tokens, n_heads), XRT_WAVE, 0, (hipStream_t)stream>>>(workspace, shape, chunk_groups, chunks, positions, \
                                                                                                      slots, sink_scores, (bf16*)out)
    if (value_dim <= 2 * XRT_WAVE) XRT_MERGE(2); else XRT_MERGE(LATENT_MOST / XRT_WAVE);
#undef XRT_MERGE
    XRT_LAUNCH_CHECK("attention (latent, merge)");
    return 0;
}

extern "C" int xrt_attention_latent_prompts(const void* q, long tokens, int n_heads, int n_kv_heads, int head_dim, int value_dim, const void* k_cache,
                                            const void* v_cache, const int* block_table, int table_stride, int n_blocks, const int* seq_offsets,
                                            const int* seq_slots, const int* seq_starts, int n_seqs, void* out, float scale, float softcap, int window,
                                            int keep_first, const float* sink_scores, int max_context, void* stream) {
    XRT_REQUIRE(xrt_attention_latent_accepts(XRT_BF16, head_dim, value_dim), "attention (latent, prompts): key and value sizes %d and %d: multiples of 32 up to %d and %d",
                head_dim, value_dim, KEYS_MOST, LATENT_MOST);
    XRT_REQUIRE(q && k_cache && v_cache && block_table && seq_offsets && seq_slots && seq_starts && out, "attention (latent, prompts): null operand");
    const Shape shape{n_heads, n_kv_heads, head_dim, value_dim, window, keep_first};
    XRT_REQUIRE(shape_is_sound(shape) && tokens >= 0 && tokens * n_heads < (1L << 31) - 512 && n_kv_heads <= 65535 && n_seqs > 0 && n_seqs <= tokens && table_stride > 0 &&
                n_blocks > 0 && scale > 0.f && softcap >= 0.f, "attention (latent, prompts): bad sizes (%ld tokens, %d heads on %d, %d sequences)", tokens, n_heads, n_kv_heads, n_seqs);
    XRT_REQUIRE(((uintptr_t)q | (uintptr_t)k_cache | (uintptr_t)v_cache) % 16 == 0 && (uintptr_t)out % 8 == 0, "attention (latent, prompts): operands off their sixteen bytes");
    XRT_REQUIRE(max_context > 0 && max_context <= table_stride * XRT_BLOCK_TOKENS, "attention (latent, prompts): a sequence of %d tokens exceeds the block table", max_context);
    if (tokens == 0) return 0;
    auto run = [&](auto launcher) {
        return launcher((const bf16*)q, tokens, shape, (const bf16*)k_cache, (const bf16*)v_cache, block_table, table_stride, n_blocks, seq_offsets, seq_slots,
                        seq_starts, n_seqs, scale, softcap, sink_scores, (bf16*)out, (hipStream_t)stream);
    };
    // the instantiation that holds the sizes with the least to spare (the largest ones in workgroups of four wavefronts, which may have
    // twice the registers each)
#define XRT_PROMPTS(KS_, VT_, WAVES_) (softcap > 0.f ? run(launch_prompts<KS_, VT_, WAVES_, true>) : run(launch_prompts<KS_, VT_, WAVES_, false>))
    if (head_dim <= 64 && value_dim <= 64) return XRT_PROMPTS(2, 4, 8);
    if (head_dim <= 128 && value_dim <= 128) return XRT_PROMPTS(4, 8, 8);
    if (head_dim <= 192 && value_dim <= 128) return XRT_PROMPTS(6, 8, 8);
    if (head_dim <= 256 && value_dim <= 192) return XRT_PROMPTS(8, 12, 8);
    if (head_dim <= 320 && value_dim <= 256) return XRT_PROMPTS(10, 16, 8);
    if (head_dim <= 448 && value_dim <= 384) return XRT_PROMPTS(14, 24, 8);
    if (head_dim <= 576) return XRT_PROMPTS(18, 32, 4);
    return XRT_PROMPTS(20, 32, 4);
#undef XRT_PROMPTS
}
