// Attention whose keys and values are made from a latent: the cache keeps, for every token, one row [latent | turned key part]
// as the key of a single key/value head and the latent once more as its value. The scores against such a key are those of the
// design's per-head keys when the query's plain part has first been multiplied by the head's key matrix, transposed
// (q_h . (W_h c) = (W_h^T q_h) . c); the sum of the latents under the softmax's weights is turned into the head's output by
// the head's value matrix afterwards. Both are products with a matrix per head (xrt_linear_heads).
//   xrt_latent_complete  from the down projection's float32 sums [latent | key part]: the latent divided by its root mean
//                        square, times a gain; the first rot_dims of the key part turned in pairs of neighbours (2i, 2i + 1) or of
//                        halves (i, i + rot_dims / 2) by position * frequencies[i], cosines and sines times a magnitude; both into the cache
//   xrt_latent_queries   from the queries' float32 sums, head by head [plain | part to turn]: the plain parts to rows of
//                        their own, the turned parts to the tail of the rows that the attention kernel reads
//   xrt_latent_prepare   both of them in one launch, for layers whose queries come straight from the layer's input
//   xrt_linear_heads     out[t][h][n] = sum over k of a[t][h][k] * w[h][n][k], float32 sums (bfloat16 with k in whole steps of 32: on the
//                        matrix cores; else steps of many rows in the order of k, steps of few with the lanes of a wavefront along k);
//                        with gates (float32 [t][h] or [t][h][n], any stride) times sigmoid(gates[t][h]) or sigmoid(gates[t][h][n]) before
//                        it is rounded
// A prompt that starts a sequence can have its scores as a matrix product of its own rows (all heads' queries of a stretch of
// tokens against the prompt's cached rows, which the step has at hand): then
//   xrt_causal_softmax   turns the float32 scores [queries x heads][keys] into the softmax's weights over the keys at or before
//                        each query, with the heads' sinks in the denominators, as two bfloat16 numbers each (the rounded weight
//                        and what the rounding left) for the product with the latents
//   xrt_transpose        dst[c][r] = src[r][c]: the latents with the tokens along the rows, as that product wants them
#include "cache_layout.h"
#include "xrt_hip.h"

namespace {

__device__ __forceinline__ float small_at(const void* p, int dtype, int i) {
    return dtype == XRT_F32 ? ((const float*)p)[i] : to_float(((const bf16*)p)[i]);
}

// How the first `dims` numbers of a part turn: in pairs of neighbours (2i, 2i + 1) or of halves (i, i + dims / 2), by position *
// frequencies[i], cosines and sines times `magnitude`.
struct Turn {
    int dims, neighbours; float magnitude; const float* frequencies;
    bool is_sound(int part) const { return dims >= 0 && dims % 2 == 0 && dims <= part && (dims == 0 || frequencies != nullptr); }
    // the element e of a part, turned
    __device__ __forceinline__ float operator()(const float* part, int e, int pos) const {
        if (e >= dims) return part[e];
        const int half = dims / 2;
        const bool is_first = neighbours ? e % 2 == 0 : e < half;
        float sine, cosine;
        sincosf((float)pos * frequencies[neighbours ? e / 2 : is_first ? e : e - half], &sine, &cosine);
        sine *= magnitude;
        cosine *= magnitude;
        const float mine = part[e], other = part[neighbours ? e ^ 1 : is_first ? e + half : e - half];
        return is_first ? mine * cosine - other * sine : mine * cosine + other * sine;
    }
};

// What becomes of a token's float32 row [latent | key part], by the whole workgroup.
template <typename T>
__device__ __forceinline__ void complete_row(long t, const float* __restrict__ down, long down_stride, int rank, int rot_dim, const Turn turn,
                                             const void* __restrict__ gain, int gain_dtype, float eps,
                                             const int* __restrict__ positions, const int* __restrict__ slots, T* __restrict__ k_cache,
                                             T* __restrict__ v_cache, const int* __restrict__ block_table, int table_stride, int n_blocks,
                                             T* __restrict__ rows_out) {
    __shared__ float scratch[32];
    const int slot = slots[t], pos = positions[t];
    if (slot < 0) {                                            // (the whole workgroup)
        if (rows_out != nullptr) for (int e = threadIdx.x; e < rank + rot_dim; e += blockDim.x) rows_out[t * (rank + rot_dim) + e] = from_float<T>(0.f);
        return;
    }
    const int block = block_table[(long)slot * table_stride + pos / XRT_BLOCK_TOKENS];
    if (block < 0 || block >= n_blocks) return;
    const float* row = down + t * down_stride;
    float squares = 0.f;
    for (int e = threadIdx.x; e < rank; e += blockDim.x) squares = fmaf(row[e], row[e], squares);
    const float inv = 1.0f / sqrtf(block_sum(squares, scratch) / (float)rank + eps);
    const int head_dim = rank + rot_dim, place = pos % XRT_BLOCK_TOKENS;
    T* keys = k_cache + (long)block * XRT_BLOCK_TOKENS * head_dim;
    T* values = v_cache + (long)block * XRT_BLOCK_TOKENS * rank;
    for (int e = threadIdx.x; e < head_dim; e += blockDim.x) {
        if (e < rank) {
            const T c = from_float<T>(row[e] * inv * small_at(gain, gain_dtype, e));
            keys[cache_key_offset(place, e, head_dim)] = c;
            values[cache_value_offset(e, place, rank)] = c;
            if (rows_out != nullptr) rows_out[t * head_dim + e] = c;
        } else {
            const T k = from_float<T>(turn(row + rank, e - rank, pos));
            keys[cache_key_offset(place, e, head_dim)] = k;
            if (rows_out != nullptr) rows_out[t * head_dim + e] = k;
        }
    }
}

template <typename T>
__global__ void __launch_bounds__(256) latent_complete_kernel(const float* __restrict__ down, long down_stride, int rank, int rot_dim, const Turn turn,
                                                             const void* __restrict__ gain, int gain_dtype, float eps, const int* __restrict__ positions,
                                                             const int* __restrict__ slots, T* __restrict__ k_cache, T* __restrict__ v_cache,
                                                             const int* __restrict__ block_table, int table_stride, int n_blocks,
                                                             T* __restrict__ rows_out) {
    complete_row(blockIdx.x, down, down_stride, rank, rot_dim, turn, gain, gain_dtype, eps, positions, slots, k_cache, v_cache,
                 block_table, table_stride, n_blocks, rows_out);
}

// A head's query of a token, by one wavefront.
template <typename T>
__device__ __forceinline__ void query_row(long t, int head, int lane, const float* __restrict__ q, long q_stride, int heads, int dim, int rot_dim,
                                          const Turn turn, const int* __restrict__ positions,
                                          T* __restrict__ plain, T* __restrict__ full, long full_stride, int rank) {
    const int pos = positions[t];
    const float* mine = q + t * q_stride + (long)head * (dim + rot_dim);
    for (int e = lane; e < dim; e += XRT_WAVE) plain[(t * heads + head) * dim + e] = from_float<T>(mine[e]);
    T* tail = full + t * full_stride + (long)head * (rank + rot_dim) + rank;
    for (int e = lane; e < rot_dim; e += XRT_WAVE) tail[e] = from_float<T>(turn(mine + dim, e, pos));
}

template <typename T>
__global__ void __launch_bounds__(XRT_WAVE) latent_queries_kernel(const float* __restrict__ q, long q_stride, int heads, int dim, int rot_dim,
                                                                 const Turn turn, const int* __restrict__ positions, T* __restrict__ plain, T* __restrict__ full,
                                                                 long full_stride, int rank) {
    query_row((long)blockIdx.x / heads, (int)(blockIdx.x % heads), (int)threadIdx.x, q, q_stride, heads, dim, rot_dim, turn,
              positions, plain, full, full_stride, rank);
}

// Workgroup (token, 0) completes the token's row; workgroup (token, 1 + i) makes the queries of heads PREPARE_HEADS i .. + PREPARE_HEADS - 1.
constexpr int PREPARE_HEADS = 256 / XRT_WAVE;

template <typename T>
__global__ void __launch_bounds__(256) latent_prepare_kernel(const float* __restrict__ q, const float* __restrict__ down, long stride, int heads,
                                                            int dim, int rank, int rot_dim, const Turn turn, const void* __restrict__ gain,
                                                            int gain_dtype, float eps,
                                                            const int* __restrict__ positions, const int* __restrict__ slots,
                                                            T* __restrict__ k_cache, T* __restrict__ v_cache, const int* __restrict__ block_table,
                                                            int table_stride, int n_blocks, T* __restrict__ plain, T* __restrict__ full,
                                                            long full_stride) {
    if (blockIdx.y == 0) {
        complete_row<T>(blockIdx.x, down, stride, rank, rot_dim, turn, gain, gain_dtype, eps, positions, slots, k_cache, v_cache,
                        block_table, table_stride, n_blocks, nullptr);
        return;
    }
    const int head = ((int)blockIdx.y - 1) * PREPARE_HEADS + (int)threadIdx.x / XRT_WAVE;
    if (head < heads)
        query_row((long)blockIdx.x, head, (int)threadIdx.x % XRT_WAVE, q, stride, heads, dim, rot_dim, turn, positions, plain, full,
                  full_stride, rank);
}

// What a head's outputs are multiplied by: the sigmoid of the head's gate (width 1), or of a gate for each of its outputs (width: as
// many as a head has outputs), or one.
struct HeadGates {
    const float* logits; long stride; int width;
    __device__ __forceinline__ float operator()(long row, int head, int output) const {
        return logits == nullptr ? 1.0f : 1.0f / (1.0f + expf(-logits[row * stride + (width == 1 ? (long)head : (long)head * width + output)]));
    }
};

// A tile of 64 rows x 64 outputs of one head a workgroup, k in steps of 16 through LDS, 4 x 4 outputs a thread; every
// output's sum runs over k in order, whatever the tile it falls into.
constexpr int HEADS_TILE = 64, HEADS_K = 16;

template <typename T>
__global__ void __launch_bounds__(256) linear_heads_kernel(const T* __restrict__ a, long a_stride, long a_head, const T* __restrict__ w,
                                                          T* __restrict__ out, long out_stride, long out_head, long rows, int n, int k, const HeadGates gates) {
    __shared__ float as[HEADS_K][HEADS_TILE + 1], ws[HEADS_K][HEADS_TILE + 1];
    const int head = blockIdx.z;
    const long row0 = (long)blockIdx.x * HEADS_TILE;
    const int n0 = blockIdx.y * HEADS_TILE;
    const int tr = threadIdx.x / 16, tc = threadIdx.x % 16;
    const T* a_base = a + (long)head * a_head;
    const T* w_base = w + (long)head * n * k;
    float acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = 0.f;
    for (int k0 = 0; k0 < k; k0 += HEADS_K) {
        for (int e = threadIdx.x; e < HEADS_TILE * HEADS_K; e += 256) {
            const int r = e / HEADS_K, kk = e % HEADS_K;
            as[kk][r] = row0 + r < rows && k0 + kk < k ? to_float(a_base[(row0 + r) * a_stride + k0 + kk]) : 0.f;
            ws[kk][r] = n0 + r < n && k0 + kk < k ? to_float(w_base[(long)(n0 + r) * k + k0 + kk]) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int kk = 0; kk < HEADS_K; ++kk) {
            float av[4], wv[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) { av[i] = as[kk][tr * 4 + i]; wv[i] = ws[kk][tc * 4 + i]; }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(av[i], wv[j], acc[i][j]);
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const long r = row0 + tr * 4 + i;
            const int c = n0 + tc * 4 + j;
            if (r < rows && c < n) out[r * out_stride + (long)head * out_head + c] = from_float<T>(acc[i][j] * gates(r, head, c));
        }
}

// A workgroup a row: row m is the query at position first_position + m / heads of head m % heads. Three passes over the row
// (largest visible score, sum, weights); keys behind the query's position get a weight of nothing.
__global__ void __launch_bounds__(256) causal_softmax_kernel(const float* __restrict__ scores, long keys, int heads, int first_position, float scale,
                                                            const float* __restrict__ sinks, bf16* __restrict__ rounded, bf16* __restrict__ rest) {
    __shared__ float scratch[32];
    const long row = blockIdx.x;
    const int head = (int)(row % heads), visible = min((long)first_position + row / heads + 1, keys);
    const float* mine = scores + row * keys;
    const float sink = sinks != nullptr ? sinks[head] : -INFINITY;
    float top = sink;
    for (int j = threadIdx.x; j < visible; j += 256) top = fmaxf(top, mine[j] * scale);
    top = wave_max(top);
    __syncthreads();
    if (threadIdx.x % XRT_WAVE == 0) scratch[threadIdx.x / XRT_WAVE] = top;
    __syncthreads();
    for (int w = 0; w < 256 / XRT_WAVE; ++w) top = fmaxf(top, scratch[w]);
    float sum = 0.f;
    for (int j = threadIdx.x; j < visible; j += 256) sum += expf(mine[j] * scale - top);
    sum = block_sum(sum, scratch);
    if (sinks != nullptr) sum += expf(sink - top);
    const float inv = 1.0f / sum;
    for (long j = threadIdx.x; j < keys; j += 256) {
        const float weight = j < visible ? expf(mine[j] * scale - top) * inv : 0.f;
        const bf16 first = from_float<bf16>(weight);
        rounded[row * keys + j] = first;
        rest[row * keys + j] = from_float<bf16>(weight - to_float(first));
    }
}

template <typename T>
__global__ void __launch_bounds__(256) transpose_kernel(const T* __restrict__ src, long src_stride, long rows, int cols, T* __restrict__ dst) {
    __shared__ T tile[32][33];
    const long r0 = (long)blockIdx.x * 32;
    const int c0 = blockIdx.y * 32, tx = threadIdx.x % 32, ty = threadIdx.x / 32;
    for (int i = ty; i < 32; i += 8)
        if (r0 + i < rows && c0 + tx < cols) tile[i][tx] = src[(r0 + i) * src_stride + c0 + tx];
    __syncthreads();
    for (int i = ty; i < 32; i += 8)
        if (c0 + i < cols && r0 + tx < rows) dst[(long)(c0 + i) * rows + r0 + tx] = tile[tx][i];
}

// The same product on the matrix cores, for bfloat16 with k in whole steps of 32: a wavefront takes RT x 16 rows and NT x 16
// outputs of one head; both operands of v_mfma_f32_16x16x32_bf16 come straight from memory, sixteen bytes a lane (a row of w:
// 8 consecutive k of one output; a row of a: 8 consecutive k of one token), nothing passes LDS. The outputs are the rows of
// the products, dealt to the tiles such that a lane ends up with 4 NT consecutive outputs of one token. A token's sums run
// over k in one order whatever RT and NT are.
typedef __bf16 heads_bf16x8 __attribute__((ext_vector_type(8)));
typedef float heads_floatx4 __attribute__((ext_vector_type(4)));
constexpr int MFMA_WAVES = 4;

template <int RT, int NT>
__global__ void __launch_bounds__(MFMA_WAVES * XRT_WAVE) linear_heads_mfma_kernel(const bf16* __restrict__ a, long a_stride, long a_head,
                                                                                 const bf16* __restrict__ w, bf16* __restrict__ out, long out_stride,
                                                                                 long out_head, long rows, int n, int k, long row_blocks, int n_blocks,
                                                                                 bool fours, const HeadGates gates) {
    const int head = blockIdx.y, lane = threadIdx.x % XRT_WAVE, r = lane % 16, c = lane / 16;
    const long unit = (long)blockIdx.x * MFMA_WAVES + threadIdx.x / XRT_WAVE;
    if (unit >= row_blocks * n_blocks) return;                 // (the whole wavefront)
    const long row0 = unit % row_blocks * (16 * RT);           // (a workgroup's wavefronts share their outputs' rows of w)
    const int n0 = (int)(unit / row_blocks) * (16 * NT);
    const bf16* of_a[RT];
    const bf16* of_w[NT];
#pragma unroll
    for (int t = 0; t < RT; ++t) of_a[t] = a + min(row0 + 16 * t + r, rows - 1) * a_stride + (long)head * a_head + c * 8;
#pragma unroll
    for (int j = 0; j < NT; ++j) of_w[j] = w + ((long)head * n + min(n0 + r / 4 * (4 * NT) + 4 * j + r % 4, n - 1)) * k + c * 8;
    heads_floatx4 acc[RT][NT];
#pragma unroll
    for (int t = 0; t < RT; ++t)
#pragma unroll
        for (int j = 0; j < NT; ++j) acc[t][j] = heads_floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll(RT * NT == 1 ? 4 : 2)
    for (int k0 = 0; k0 < k; k0 += 32) {
        heads_bf16x8 of_rows[RT], of_outputs[NT];
#pragma unroll
        for (int t = 0; t < RT; ++t) of_rows[t] = *reinterpret_cast<const heads_bf16x8*>(of_a[t] + k0);
#pragma unroll
        for (int j = 0; j < NT; ++j) of_outputs[j] = *reinterpret_cast<const heads_bf16x8*>(of_w[j] + k0);
#pragma unroll
        for (int t = 0; t < RT; ++t)
#pragma unroll
            for (int j = 0; j < NT; ++j) acc[t][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(of_outputs[j], of_rows[t], acc[t][j], 0, 0, 0);
    }
    // register i of tile (t, j) is output n0 + 4 NT c + 4 j + i of row row0 + 16 t + r
#pragma unroll
    for (int t = 0; t < RT; ++t) {
        const long row = row0 + 16 * t + r;
        if (row >= rows) continue;
        const bool same = gates.width == 1;                    // (one gate for all outputs of the head: worked out once)
        const float gate = same ? gates(row, head, 0) : 1.f;
        bf16* dst = out + row * out_stride + (long)head * out_head;
#pragma unroll
        for (int j = 0; j < NT; ++j) {
            const int column = n0 + c * (4 * NT) + 4 * j;
            if (fours && column + 3 < n) {
                struct alignas(8) Four { bf16 e[4]; } four;
#pragma unroll
                for (int i = 0; i < 4; ++i) four.e[i] = (bf16)(acc[t][j][i] * (same ? gate : gates(row, head, column + i)));
                *reinterpret_cast<Four*>(dst + column) = four;
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (column + i < n) dst[column + i] = (bf16)(acc[t][j][i] * (same ? gate : gates(row, head, column + i)));
            }
        }
    }
}

// The same product for a step of few rows (a decode step) in float32 or with other sizes: a wavefront an output column of one head, its lanes along k (a lane
// takes sixteen bytes of the column's row of w at a time, and the same stretch of every row of a), the lanes' sums added in
// the fixed order of the wavefront's butterfly. A row's result does not depend on the rows around it.
constexpr int HEADS_FEW = 16, FEW_WAVES = 4;
constexpr int HEADS_MANY = 512;                  // rows from which a wavefront takes 64 of them

template <typename T>
__global__ void __launch_bounds__(FEW_WAVES * XRT_WAVE) linear_heads_few_kernel(const T* __restrict__ a, long a_stride, long a_head,
                                                                               const T* __restrict__ w, T* __restrict__ out, long out_stride,
                                                                               long out_head, int rows, int n, int k, const HeadGates gates) {
    const int head = blockIdx.y, lane = threadIdx.x % XRT_WAVE, column = blockIdx.x * FEW_WAVES + threadIdx.x / XRT_WAVE;
    if (column >= n) return;                                   // (the whole wavefront)
    const T* of_w = w + ((long)head * n + column) * k;
    const T* of_a = a + (long)head * a_head;
    constexpr int PIECE = 16 / sizeof(T);
    struct alignas(16) Piece { T e[PIECE]; };
    const bool whole = k % PIECE == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)a % 16 == 0 && a_stride % PIECE == 0 && a_head % PIECE == 0;
    float acc[HEADS_FEW];
#pragma unroll
    for (int r = 0; r < HEADS_FEW; ++r) acc[r] = 0.f;
    for (int k0 = lane * PIECE; k0 < k; k0 += XRT_WAVE * PIECE) {
        float piece[PIECE];
        if (whole) {
            const Piece loaded = *reinterpret_cast<const Piece*>(of_w + k0);
#pragma unroll
            for (int e = 0; e < PIECE; ++e) piece[e] = to_float(loaded.e[e]);
        } else {
#pragma unroll
            for (int e = 0; e < PIECE; ++e) piece[e] = k0 + e < k ? to_float(of_w[k0 + e]) : 0.f;
        }
#pragma unroll
        for (int r = 0; r < HEADS_FEW; ++r) {
            if (r < rows) {
                const T* of_row = of_a + (long)r * a_stride + k0;
                if (whole) {
                    const Piece loaded = *reinterpret_cast<const Piece*>(of_row);
#pragma unroll
                    for (int e = 0; e < PIECE; ++e) acc[r] = fmaf(to_float(loaded.e[e]), piece[e], acc[r]);
                } else {
#pragma unroll
                    for (int e = 0; e < PIECE; ++e)
                        if (k0 + e < k) acc[r] = fmaf(to_float(of_row[e]), piece[e], acc[r]);
                }
            }
        }
    }
#pragma unroll
    for (int r = 0; r < HEADS_FEW; ++r) {
        if (r < rows) {
            const float sum = wave_sum(acc[r]);
            if (lane == 0) out[(long)r * out_stride + (long)head * out_head + column] = from_float<T>(sum * gates(r, head, column));
        }
    }
}

}  // namespace

extern "C" int xrt_causal_softmax(const float* scores, long rows, long keys, int heads, int first_position, float scale, const float* sinks,
                                  void* rounded, void* rest, void* stream) {
    XRT_REQUIRE(scores && rounded && rest && rows >= 0 && rows < (1L << 31) && keys > 0 && keys < (1L << 31) && heads > 0 && first_position >= 0,
                "causal_softmax: bad operands");
    if (rows == 0) return 0;
    causal_softmax_kernel<<<(unsigned)rows, 256, 0, (hipStream_t)stream>>>(scores, keys, heads, first_position, scale, sinks, (bf16*)rounded, (bf16*)rest);
    XRT_LAUNCH_CHECK("causal_softmax");
    return 0;
}

extern "C" int xrt_transpose(const void* src, long src_stride, int dtype, long rows, int cols, void* dst, void* stream) {
    XRT_REQUIRE(dtype == XRT_F32 || dtype == XRT_BF16, "transpose: unknown dtype %d", dtype);
    XRT_REQUIRE(src && dst && rows >= 0 && cols > 0 && src_stride >= cols && (rows + 31) / 32 < (1L << 31) && (cols + 31) / 32 <= 65535, "transpose: bad operands");
    if (rows == 0) return 0;
    const dim3 grid((unsigned)((rows + 31) / 32), (cols + 31) / 32);
    if (dtype == XRT_F32) transpose_kernel<float><<<grid, 256, 0, (hipStream_t)stream>>>((const float*)src, src_stride, rows, cols, (float*)dst);
    else transpose_kernel<bf16><<<grid, 256, 0, (hipStream_t)stream>>>((const bf16*)src, src_stride, rows, cols, (bf16*)dst);
    XRT_LAUNCH_CHECK("transpose");
    return 0;
}

extern "C" int xrt_latent_complete(const float* down, long down_stride, int dtype, long tokens, int rank, int rot_dim, int rot_dims,
                                   const void* gain, int gain_dtype, float eps, const float* frequencies, int neighbours, float magnitude,
                                   const int* positions, const int* slots, void* k_cache, void* v_cache, const int* block_table, int table_stride, int n_blocks, void* rows_out,
                                   void* stream) {
    XRT_REQUIRE(dtype == XRT_F32 || dtype == XRT_BF16, "latent_complete: unknown dtype %d", dtype);
    XRT_REQUIRE(gain_dtype == XRT_F32 || gain_dtype == XRT_BF16, "latent_complete: unknown dtype %d of the gain", gain_dtype);
    XRT_REQUIRE(down && gain && positions && slots && k_cache && v_cache && block_table, "latent_complete: null operand");
    XRT_REQUIRE(tokens >= 0 && tokens < (1L << 31) && rank > 0 && rot_dim >= 0 && down_stride >= rank + rot_dim && table_stride > 0 && n_blocks > 0,
                "latent_complete: bad sizes");
    const Turn turn{rot_dims, neighbours, magnitude, frequencies};
    XRT_REQUIRE(turn.is_sound(rot_dim),
                "latent_complete: %d dims turn in pairs inside a part of %d", rot_dims, rot_dim);
    if (tokens == 0) return 0;
    if (dtype == XRT_F32)
        latent_complete_kernel<float><<<(unsigned)tokens, 256, 0, (hipStream_t)stream>>>(down, down_stride, rank, rot_dim, turn, gain, gain_dtype, eps,
                                                                                      positions, slots, (float*)k_cache, (float*)v_cache,
                                                                                      block_table, table_stride, n_blocks, (float*)rows_out);
    else
        latent_complete_kernel<bf16><<<(unsigned)tokens, 256, 0, (hipStream_t)stream>>>(down, down_stride, rank, rot_dim, turn, gain, gain_dtype, eps,
                                                                                     positions, slots, (bf16*)k_cache, (bf16*)v_cache,
                                                                                     block_table, table_stride, n_blocks, (bf16*)rows_out);
    XRT_LAUNCH_CHECK("latent_complete");
    return 0;
}

extern "C" int xrt_latent_queries(const float* q, long q_stride, int dtype, long tokens, int heads, int dim, int rot_dim, int rot_dims,
                                  const float* frequencies, int neighbours, float magnitude, const int* positions, void* plain, void* full,
                                  long full_stride, int rank, void* stream) {
    XRT_REQUIRE(dtype == XRT_F32 || dtype == XRT_BF16, "latent_queries: unknown dtype %d", dtype);
    XRT_REQUIRE(q && positions && plain && full, "latent_queries: null operand");
    XRT_REQUIRE(tokens >= 0 && heads > 0 && tokens * heads < (1L << 31) && dim > 0 && rot_dim >= 0 && rank > 0 &&
                q_stride >= (long)heads * (dim + rot_dim) && full_stride >= (long)heads * (rank + rot_dim), "latent_queries: bad sizes");
    const Turn turn{rot_dims, neighbours, magnitude, frequencies};
    XRT_REQUIRE(turn.is_sound(rot_dim),
                "latent_queries: %d dims turn in pairs inside a part of %d", rot_dims, rot_dim);
    if (tokens == 0) return 0;
    if (dtype == XRT_F32)
        latent_queries_kernel<float><<<(unsigned)(tokens * heads), XRT_WAVE, 0, (hipStream_t)stream>>>(q, q_stride, heads, dim, rot_dim, turn,
                                                                                                    positions, (float*)plain, (float*)full, full_stride, rank);
    else
        latent_queries_kernel<bf16><<<(unsigned)(tokens * heads), XRT_WAVE, 0, (hipStream_t)stream>>>(q, q_stride, heads, dim, rot_dim, turn,
                                                                                                   positions, (bf16*)plain, (bf16*)full, full_stride, rank);
    XRT_LAUNCH_CHECK("latent_queries");
    return 0;
}

extern "C" int xrt_latent_prepare(const float* q, const float* down, long stride, int dtype, long tokens, int heads, int dim, int rank, int rot_dim,
                                  int rot_dims, const void* gain, int gain_dtype, float eps, const float* frequencies, int neighbours,
                                  float magnitude, const int* positions, const int* slots, void* k_cache, void* v_cache, const int* block_table, int table_stride, int n_blocks,
                                  void* plain, void* full, long full_stride, void* stream) {
    XRT_REQUIRE(dtype == XRT_F32 || dtype == XRT_BF16, "latent_prepare: unknown dtype %d", dtype);
    XRT_REQUIRE(gain_dtype == XRT_F32 || gain_dtype == XRT_BF16, "latent_prepare: unknown dtype %d of the gain", gain_dtype);
    XRT_REQUIRE(q && down && gain && positions && slots && k_cache && v_cache && block_table && plain && full, "latent_prepare: null operand");
    XRT_REQUIRE(tokens >= 0 && tokens < (1L << 31) && heads > 0 && heads <= 65534 && dim > 0 && rank > 0 && rot_dim >= 0 &&
                stride >= (long)heads * (dim + rot_dim) && stride >= rank + rot_dim && full_stride >= (long)heads * (rank + rot_dim) &&
                table_stride > 0 && n_blocks > 0, "latent_prepare: bad sizes");
    const Turn turn{rot_dims, neighbours, magnitude, frequencies};
    XRT_REQUIRE(turn.is_sound(rot_dim),
                "latent_prepare: %d dims turn in pairs inside a part of %d", rot_dims, rot_dim);
    if (tokens == 0) return 0;
    const dim3 grid((unsigned)tokens, 1 + (heads + PREPARE_HEADS - 1) / PREPARE_HEADS);
    if (dtype == XRT_F32)
        latent_prepare_kernel<float><<<grid, 256, 0, (hipStream_t)stream>>>(q, down, stride, heads, dim, rank, rot_dim, turn, gain, gain_dtype, eps,
                                                                            positions, slots, (float*)k_cache, (float*)v_cache, block_table, table_stride,
                                                                            n_blocks, (float*)plain, (float*)full, full_stride);
    else
        latent_prepare_kernel<bf16><<<grid, 256, 0, (hipStream_t)stream>>>(q, down, stride, heads, dim, rank, rot_dim, turn, gain, gain_dtype, eps,
                                                                           positions, slots, (bf16*)k_cache, (bf16*)v_cache, block_table, table_stride,
                                                                           n_blocks, (bf16*)plain, (bf16*)full, full_stride);
    XRT_LAUNCH_CHECK("latent_prepare");
    return 0;
}

extern "C" int xrt_linear_heads(const void* a, long a_stride, long a_head, const void* w, int dtype, void* out, long out_stride, long out_head,
                                long rows, int heads, int n, int k, const float* gate_logits, long gate_stride, int gate_width, void* stream) {
    XRT_REQUIRE(gate_logits == nullptr || ((gate_width == 1 || gate_width == n) && gate_stride >= (long)heads * gate_width),
                "linear_heads: rows of gates %ld apart, %d a head, for %d heads of %d outputs", gate_stride, gate_width, heads, n);
    const HeadGates gates{gate_logits, gate_stride, gate_logits == nullptr ? 1 : gate_width};
    XRT_REQUIRE(dtype == XRT_F32 || dtype == XRT_BF16, "linear_heads: unknown dtype %d", dtype);
    XRT_REQUIRE(a && w && out && rows >= 0 && heads > 0 && heads <= 65535 && n > 0 && k > 0, "linear_heads: bad operands");
    XRT_REQUIRE(a_head >= k && a_stride >= (heads - 1) * a_head + k && out_head >= n && out_stride >= (heads - 1) * out_head + n,
                "linear_heads: rows %ld and %ld apart do not hold %d heads %ld and %ld apart", a_stride, out_stride, heads, a_head, out_head);
    if (rows == 0) return 0;
    if (dtype == XRT_BF16 && k % 32 == 0 && a_stride % 8 == 0 && a_head % 8 == 0 && (uintptr_t)a % 16 == 0 && (uintptr_t)w % 16 == 0) {
        const bool fours = out_stride % 4 == 0 && out_head % 4 == 0 && (uintptr_t)out % 8 == 0;
        // a tile a wavefront for a step of few rows, whose wavefronts would else be few; more as the rows are more
        const int rt = rows >= HEADS_MANY ? 4 : 1, nt = rows > HEADS_FEW ? 4 : 1;
        const long row_blocks = (rows + 16 * rt - 1) / (16 * rt);
        const int n_blocks = (n + 16 * nt - 1) / (16 * nt);
        const long groups = (row_blocks * n_blocks + MFMA_WAVES - 1) / MFMA_WAVES;
        XRT_REQUIRE(groups < (1L << 31), "linear_heads: too many tiles");
        const dim3 grid((unsigned)groups, heads);
#define XRT_HEADS_MFMA(RT_, NT_)                                                                                                                          \
    linear_heads_mfma_kernel<RT_, NT_><<<grid, MFMA_WAVES * XRT_WAVE, 0, (hipStream_t)stream>>>((const bf16*)a, a_stride, a_head, (const bf16*)w, (bf16*)out, \
                                                                                              out_stride, out_head, rows, n, k, row_blocks, n_blocks, fours, gates)
        if (rt == 4) XRT_HEADS_MFMA(4, 4);
        else if (nt == 4) XRT_HEADS_MFMA(1, 4);
        else XRT_HEADS_MFMA(1, 1);
#undef XRT_HEADS_MFMA
        XRT_LAUNCH_CHECK("linear_heads");
        return 0;
    }
    if (rows <= HEADS_FEW) {
        const dim3 few((n + FEW_WAVES - 1) / FEW_WAVES, heads);
        if (dtype == XRT_F32)
            linear_heads_few_kernel<float><<<few, FEW_WAVES * XRT_WAVE, 0, (hipStream_t)stream>>>((const float*)a, a_stride, a_head, (const float*)w,
                                                                                               (float*)out, out_stride, out_head, (int)rows, n, k, gates);
        else
            linear_heads_few_kernel<bf16><<<few, FEW_WAVES * XRT_WAVE, 0, (hipStream_t)stream>>>((const bf16*)a, a_stride, a_head, (const bf16*)w,
                                                                                              (bf16*)out, out_stride, out_head, (int)rows, n, k, gates);
        XRT_LAUNCH_CHECK("linear_heads");
        return 0;
    }
    const long row_tiles = (rows + HEADS_TILE - 1) / HEADS_TILE;
    XRT_REQUIRE(row_tiles < (1L << 31) && (n + HEADS_TILE - 1) / HEADS_TILE <= 65535, "linear_heads: too many tiles");
    const dim3 grid((unsigned)row_tiles, (n + HEADS_TILE - 1) / HEADS_TILE, heads);
    if (dtype == XRT_F32)
        linear_heads_kernel<float><<<grid, 256, 0, (hipStream_t)stream>>>((const float*)a, a_stride, a_head, (const float*)w, (float*)out, out_stride,
                                                                       out_head, rows, n, k, gates);
    else
        linear_heads_kernel<bf16><<<grid, 256, 0, (hipStream_t)stream>>>((const bf16*)a, a_stride, a_head, (const bf16*)w, (bf16*)out, out_stride,
                                                                      out_head, rows, n, k, gates);
    XRT_LAUNCH_CHECK("linear_heads");
    return 0;
}
