// Embedding gather, residual add and RMSNorm.
//
// RMSNorm: y = (x * r) * w, r = 1/sqrt(mean(x^2) + eps), all in float32
// (reference: crates/xrt-kernels/src/cpu/rmsnorm.rs:26-43). One workgroup per row;
// the order of the sum depends only on the row length, so a row's result is the
// same in any batch.
#include "common.h"
#include "xrt_hip.h"
#include "packing.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

template <typename T>
__global__ void embed_kernel(const T* __restrict__ table, const int* __restrict__ ids,
                             float* __restrict__ out, int hidden, float scale) {
    const long token = blockIdx.x;
    const T* row = table + (long)ids[token] * hidden;
    float* dst = out + token * hidden;
    if constexpr (sizeof(T) == 2) {
        if (hidden % 8 == 0) {              // 16 bytes of the row a lane and step (a row then starts at a multiple of 16 bytes)
            for (int i = threadIdx.x * 8; i < hidden; i += blockDim.x * 8) {
                const bf16x8 eight = *reinterpret_cast<const bf16x8*>(row + i);
                float4 low, high;
                low.x = (float)eight[0] * scale; low.y = (float)eight[1] * scale; low.z = (float)eight[2] * scale; low.w = (float)eight[3] * scale;
                high.x = (float)eight[4] * scale; high.y = (float)eight[5] * scale; high.z = (float)eight[6] * scale; high.w = (float)eight[7] * scale;
                *reinterpret_cast<float4*>(dst + i) = low;
                *reinterpret_cast<float4*>(dst + i + 4) = high;
            }
            return;
        }
    }
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = to_float(row[i]) * scale;
}

// the same from a table kept in tiles (a table that is also the output head's weight)
__global__ void embed_packed_kernel(const bf16* __restrict__ table, const int* __restrict__ ids,
                                    float* __restrict__ out, int hidden, const Packing packing, float scale) {
    const long token = blockIdx.x;
    const long row = packed_row(packing, ids[token]);
    float* dst = out + token * hidden;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = to_float(table[packed_offset(row, i / 8 * 8, hidden) + i % 8]) * scale;
}

template <typename T>
__global__ void add_kernel(float* __restrict__ residual, const T* __restrict__ delta, long count) {
    const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < count) residual[i] += to_float(delta[i]);
}

template <typename T> struct alignas(sizeof(T) * 4) Vec4 { T e[4]; };

// Rows whose length is a multiple of 4 are read once, 16 bytes per lane and all loads in flight
// together, and kept in registers between the sum and the scaling (up to CACHED * 1024 elements;
// the rest of a longer row is read twice). Other rows take the scalar path. The order of the sum
// depends only on the row length.
//
// CONV: a step in which every sequence brings one token may let this kernel also do the short convolution over time that
// reads the normed row (csrc/sequence_state.hip: xrt_short_conv, whose arithmetic this repeats term for term on the normed
// values as the norm alone would have rounded them): out = conv(normed) (+ normed), and the sequence's kept inputs move on
// by the normed row. A lane touches only its own channels of its row's sequence.
struct ConvAfterNorm {
    const void* w;          // [hidden][taps]
    int w_dtype, taps, plus_input;
    float* state;           // [slots][taps - 1][hidden]
    const int* token_slots; // [rows]: negative: padding, whose row becomes zeros
};

template <typename TO>
__device__ __forceinline__ float conv_after_norm(const ConvAfterNorm& conv, float normed, int slot, int c, int hidden) {
#pragma clang fp contract(off)      // (only the products and sums written as fmaf are fused: the same in every kernel that does this convolution)
    const float now = to_float(from_float<TO>(normed));
    float* mine = conv.state + (long)slot * (conv.taps - 1) * hidden + c;
    const long w_at = (long)c * conv.taps;
    auto weight = [&](int j) { return conv.w_dtype == XRT_F32 ? ((const float*)conv.w)[w_at + j] : to_float(((const bf16*)conv.w)[w_at + j]); };
    float y = 0.f;
    for (int m = 0; m < conv.taps - 1; ++m) {
        const float kept = mine[(long)m * hidden];
        y = fmaf(weight(m), kept, y);
        if (m > 0) mine[(long)(m - 1) * hidden] = kept;
    }
    y = fmaf(weight(conv.taps - 1), now, y);
    if (conv.plus_input) y += now;
    if (conv.taps >= 2) mine[(long)(conv.taps - 2) * hidden] = now;
    return y;
}

// The same for four neighbouring channels 4 q .. 4 q + 3 at once (hidden a multiple of 4), the number of taps known when the
// kernel is compiled: everything is fetched, sixteen bytes a load, before anything is written, so that the loads are in flight together.
constexpr int CONV_AFTER_NORM_MOST_TAPS = 8;

template <typename TO, int TAPS>
__device__ __forceinline__ void conv_after_norm4(const ConvAfterNorm& conv, float (&normed)[4], int slot, int q, int hidden) {
#pragma clang fp contract(off)      // (only the products and sums written as fmaf are fused: the same in every kernel that does this convolution)
    float4* mine = reinterpret_cast<float4*>(conv.state + (long)slot * (TAPS - 1) * hidden) + q;      // row m: + m * hidden / 4
    const int quads = hidden / 4;
    float4 kept[TAPS > 1 ? TAPS - 1 : 1];
    float w[4 * TAPS];                                      // of channel 4 q + e: w[e * TAPS ..]
#pragma unroll
    for (int m = 0; m < TAPS - 1; ++m) kept[m] = mine[(long)m * quads];
#pragma unroll
    for (int i = 0; i < 4 * TAPS; ++i) {
        const long at = (long)4 * q * TAPS + i;
        w[i] = conv.w_dtype == XRT_F32 ? ((const float*)conv.w)[at] : to_float(((const bf16*)conv.w)[at]);
    }
    float now[4], y[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) now[e] = to_float(from_float<TO>(normed[e]));
#pragma unroll
    for (int m = 0; m < TAPS - 1; ++m) {
        y[0] = fmaf(w[0 * TAPS + m], kept[m].x, y[0]);
        y[1] = fmaf(w[1 * TAPS + m], kept[m].y, y[1]);
        y[2] = fmaf(w[2 * TAPS + m], kept[m].z, y[2]);
        y[3] = fmaf(w[3 * TAPS + m], kept[m].w, y[3]);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        y[e] = fmaf(w[e * TAPS + TAPS - 1], now[e], y[e]);
        if (conv.plus_input) y[e] += now[e];
    }
#pragma unroll
    for (int m = 1; m < TAPS - 1; ++m) mine[(long)(m - 1) * quads] = kept[m];
    if constexpr (TAPS >= 2) mine[(long)(TAPS - 2) * quads] = make_float4(now[0], now[1], now[2], now[3]);
#pragma unroll
    for (int e = 0; e < 4; ++e) normed[e] = y[e];
}

// TAPS: 0 for the norm alone, else the taps of the convolution that follows it
template <typename TW, typename TO, int TAPS>
__global__ void __launch_bounds__(256) rmsnorm_kernel(const float* __restrict__ x, const TW* __restrict__ weight,
                                                      float eps, TO* __restrict__ out,
                                                      const int* __restrict__ rows, int hidden, const ConvAfterNorm conv) {
    constexpr int CACHED = 8;
    constexpr bool CONV = TAPS > 0;
    __shared__ float scratch[32];
    const long src = rows ? rows[blockIdx.x] : blockIdx.x;
    const float* row = x + src * hidden;
    TO* dst = out + (long)blockIdx.x * hidden;
    int slot = 0;
    if constexpr (CONV) {
        slot = conv.token_slots[blockIdx.x];
        if (slot < 0) {
            for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = from_float<TO>(0.f);
            return;
        }
    }
    // what is written for channel c, whose normed value is given
    auto finished = [&](float normed, int c) {
        if constexpr (CONV) return from_float<TO>(conv_after_norm<TO>(conv, normed, slot, c, hidden));
        else return from_float<TO>(normed);
    };
    if (hidden % 4 == 0) {
        const int quads = hidden / 4;
        const float4* row4 = reinterpret_cast<const float4*>(row);
        float4 kept[CACHED];
        Vec4<TW> gain[CACHED];                                  // asked for now, so that they arrive under the sum
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < CACHED; ++i) {
            const int q = threadIdx.x + i * 256;
            kept[i] = q < quads ? row4[q] : make_float4(0.f, 0.f, 0.f, 0.f);
            gain[i] = q < quads ? *reinterpret_cast<const Vec4<TW>*>(weight + 4 * q) : Vec4<TW>{};
        }
#pragma unroll
        for (int i = 0; i < CACHED; ++i)
            sum = fmaf(kept[i].x, kept[i].x, fmaf(kept[i].y, kept[i].y, fmaf(kept[i].z, kept[i].z, fmaf(kept[i].w, kept[i].w, sum))));
        for (int q = threadIdx.x + CACHED * 256; q < quads; q += 256) {
            const float4 v = row4[q];
            sum = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, sum))));
        }
        sum = block_sum(sum, scratch);
        const float inv_rms = 1.0f / sqrtf(sum / (float)hidden + eps);
        auto emit = [&](int q, const float4& v, const Vec4<TW>& w) {
            Vec4<TO> r;
            float four[4] = {(v.x * inv_rms) * to_float(w.e[0]), (v.y * inv_rms) * to_float(w.e[1]),
                             (v.z * inv_rms) * to_float(w.e[2]), (v.w * inv_rms) * to_float(w.e[3])};
            if constexpr (CONV) conv_after_norm4<TO, TAPS>(conv, four, slot, q, hidden);
#pragma unroll
            for (int e = 0; e < 4; ++e) r.e[e] = from_float<TO>(four[e]);
            *reinterpret_cast<Vec4<TO>*>(dst + 4 * q) = r;
        };
#pragma unroll
        for (int i = 0; i < CACHED; ++i) {
            const int q = threadIdx.x + i * 256;
            if (q < quads) emit(q, kept[i], gain[i]);
        }
        for (int q = threadIdx.x + CACHED * 256; q < quads; q += 256) emit(q, row4[q], *reinterpret_cast<const Vec4<TW>*>(weight + 4 * q));
        return;
    }
    float sum = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) sum = fmaf(row[i], row[i], sum);
    sum = block_sum(sum, scratch);
    const float inv_rms = 1.0f / sqrtf(sum / (float)hidden + eps);
    for (int i = threadIdx.x; i < hidden; i += blockDim.x)
        dst[i] = finished((row[i] * inv_rms) * to_float(weight[i]), i);
}

// Two norms of the same rows that differ in their gains, a workgroup a row (the arithmetic and the order of rmsnorm_kernel's sums).
template <typename TW, typename TO>
__global__ void __launch_bounds__(256) rmsnorm_two_kernel(const float* __restrict__ x, const TW* __restrict__ weight_a, const TW* __restrict__ weight_b,
                                                          float eps, TO* __restrict__ out_a, TO* __restrict__ out_b, int hidden) {
    constexpr int CACHED = 8;
    __shared__ float scratch[32];
    const float* row = x + (long)blockIdx.x * hidden;
    TO* dst_a = out_a + (long)blockIdx.x * hidden;
    TO* dst_b = out_b + (long)blockIdx.x * hidden;
    float sum = 0.f;
    if (hidden % 4 == 0) {
        const int quads = hidden / 4;
        const float4* row4 = reinterpret_cast<const float4*>(row);
        float4 kept[CACHED];
#pragma unroll
        for (int i = 0; i < CACHED; ++i) {
            const int q = threadIdx.x + i * 256;
            kept[i] = q < quads ? row4[q] : make_float4(0.f, 0.f, 0.f, 0.f);
        }
#pragma unroll
        for (int i = 0; i < CACHED; ++i)
            sum = fmaf(kept[i].x, kept[i].x, fmaf(kept[i].y, kept[i].y, fmaf(kept[i].z, kept[i].z, fmaf(kept[i].w, kept[i].w, sum))));
        for (int q = threadIdx.x + CACHED * 256; q < quads; q += 256) {
            const float4 v = row4[q];
            sum = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, sum))));
        }
        const float inv_rms = 1.0f / sqrtf(block_sum(sum, scratch) / (float)hidden + eps);
        auto emit = [&](int q, const float4& v) {
            const Vec4<TW> a = *reinterpret_cast<const Vec4<TW>*>(weight_a + 4 * q), b = *reinterpret_cast<const Vec4<TW>*>(weight_b + 4 * q);
            const float four[4] = {v.x * inv_rms, v.y * inv_rms, v.z * inv_rms, v.w * inv_rms};
            Vec4<TO> of_a, of_b;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                of_a.e[e] = from_float<TO>(four[e] * to_float(a.e[e]));
                of_b.e[e] = from_float<TO>(four[e] * to_float(b.e[e]));
            }
            *reinterpret_cast<Vec4<TO>*>(dst_a + 4 * q) = of_a;
            *reinterpret_cast<Vec4<TO>*>(dst_b + 4 * q) = of_b;
        };
#pragma unroll
        for (int i = 0; i < CACHED; ++i) {
            const int q = threadIdx.x + i * 256;
            if (q < quads) emit(q, kept[i]);
        }
        for (int q = threadIdx.x + CACHED * 256; q < quads; q += 256) emit(q, row4[q]);
        return;
    }
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) sum = fmaf(row[i], row[i], sum);
    const float inv_rms = 1.0f / sqrtf(block_sum(sum, scratch) / (float)hidden + eps);
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float v = row[i] * inv_rms;
        dst_a[i] = from_float<TO>(v * to_float(weight_a[i]));
        dst_b[i] = from_float<TO>(v * to_float(weight_b[i]));
    }
}

// copy = x in another element type, then x = base; four numbers a thread where the count allows it
template <typename TO>
__global__ void __launch_bounds__(256) replace_rows_kernel(float* __restrict__ x, const float* __restrict__ base, TO* __restrict__ copy, long count, int step) {
    const long i = ((long)blockIdx.x * blockDim.x + threadIdx.x) * step;
    if (i >= count) return;
    if (step == 4) {
        const float4 old = *reinterpret_cast<const float4*>(x + i);
        Vec4<TO> rounded;
        rounded.e[0] = from_float<TO>(old.x); rounded.e[1] = from_float<TO>(old.y); rounded.e[2] = from_float<TO>(old.z); rounded.e[3] = from_float<TO>(old.w);
        *reinterpret_cast<Vec4<TO>*>(copy + i) = rounded;
        *reinterpret_cast<float4*>(x + i) = *reinterpret_cast<const float4*>(base + i);
        return;
    }
    copy[i] = from_float<TO>(x[i]);
    x[i] = base[i];
}

extern "C" int xrt_rmsnorm_two(const float* x, const void* weight_a, const void* weight_b, int weight_dtype, float eps, void* out_a, void* out_b,
                               int out_dtype, int n_rows, int hidden, void* stream) {
    XRT_REQUIRE(x && weight_a && weight_b && out_a && out_b && n_rows >= 0 && hidden > 0, "rmsnorm_two: bad operands rows=%d hidden=%d", n_rows, hidden);
    XRT_REQUIRE((weight_dtype == XRT_F32 || weight_dtype == XRT_BF16) && (out_dtype == XRT_F32 || out_dtype == XRT_BF16),
                "rmsnorm_two: unknown dtype weight=%d out=%d", weight_dtype, out_dtype);
    if (n_rows == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
#define XRT_RMS(TW, TO) rmsnorm_two_kernel<TW, TO><<<n_rows, 256, 0, s>>>(x, (const TW*)weight_a, (const TW*)weight_b, eps, (TO*)out_a, (TO*)out_b, hidden)
    if (weight_dtype == XRT_F32 && out_dtype == XRT_F32) XRT_RMS(float, float);
    else if (weight_dtype == XRT_F32) XRT_RMS(float, bf16);
    else if (out_dtype == XRT_F32) XRT_RMS(bf16, float);
    else XRT_RMS(bf16, bf16);
#undef XRT_RMS
    XRT_LAUNCH_CHECK("rmsnorm_two");
    return 0;
}

extern "C" int xrt_replace_rows(float* x, const float* base, void* copy, int copy_dtype, long count, void* stream) {
    XRT_REQUIRE(x && base && copy && count >= 0 && (copy_dtype == XRT_F32 || copy_dtype == XRT_BF16), "replace_rows: bad operands");
    if (count == 0) return 0;
    const int step = count % 4 == 0 && ((uintptr_t)x | (uintptr_t)base | (uintptr_t)copy) % 16 == 0 ? 4 : 1;
    const long blocks = (count / step + 255) / 256;
    XRT_REQUIRE(blocks < (1L << 31), "replace_rows: too many elements");
    if (copy_dtype == XRT_F32) replace_rows_kernel<float><<<(unsigned)blocks, 256, 0, (hipStream_t)stream>>>(x, base, (float*)copy, count, step);
    else replace_rows_kernel<bf16><<<(unsigned)blocks, 256, 0, (hipStream_t)stream>>>(x, base, (bf16*)copy, count, step);
    XRT_LAUNCH_CHECK("replace_rows");
    return 0;
}

extern "C" int xrt_embed(const void* table, int table_dtype, const xrt_packing* packing, const int* ids, float* out, int tokens,
                         int hidden, int vocab, float scale, void* stream) {
    XRT_REQUIRE(tokens >= 0 && hidden > 0 && vocab > 0, "embed: bad sizes tokens=%d hidden=%d vocab=%d", tokens, hidden, vocab);
    XRT_REQUIRE(table_dtype == XRT_F32 || table_dtype == XRT_BF16, "embed: unknown dtype %d", table_dtype);
    if (tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    if (packing && is_packed(*packing)) {
        XRT_REQUIRE(packing->kind == XRT_PACK_TILES && table_dtype == XRT_BF16 && hidden % 32 == 0,
                    "embed: a packed table is bfloat16 in plain tiles with a width that is a multiple of 32");
        embed_packed_kernel<<<tokens, 256, 0, s>>>((const bf16*)table, ids, out, hidden, *packing, scale);
        XRT_LAUNCH_CHECK("embed (packed)");
        return 0;
    }
    if (table_dtype == XRT_F32)
        embed_kernel<float><<<tokens, 256, 0, s>>>((const float*)table, ids, out, hidden, scale);
    else
        embed_kernel<bf16><<<tokens, 256, 0, s>>>((const bf16*)table, ids, out, hidden, scale);
    XRT_LAUNCH_CHECK("embed");
    return 0;
}

extern "C" int xrt_add(float* residual, const void* delta, int delta_dtype, long count, void* stream) {
    XRT_REQUIRE(count >= 0, "add: negative count");
    XRT_REQUIRE(delta_dtype == XRT_F32 || delta_dtype == XRT_BF16, "add: unknown dtype %d", delta_dtype);
    if (count == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const unsigned blocks = (unsigned)((count + 255) / 256);
    if (delta_dtype == XRT_F32)
        add_kernel<float><<<blocks, 256, 0, s>>>(residual, (const float*)delta, count);
    else
        add_kernel<bf16><<<blocks, 256, 0, s>>>(residual, (const bf16*)delta, count);
    XRT_LAUNCH_CHECK("add");
    return 0;
}

extern "C" int xrt_rmsnorm(const float* x, const void* weight, int weight_dtype, float eps, void* out,
                           int out_dtype, const int* rows, int n_rows, int hidden, void* stream) {
    XRT_REQUIRE(n_rows >= 0 && hidden > 0, "rmsnorm: bad sizes rows=%d hidden=%d", n_rows, hidden);
    XRT_REQUIRE((weight_dtype == XRT_F32 || weight_dtype == XRT_BF16) && (out_dtype == XRT_F32 || out_dtype == XRT_BF16),
                "rmsnorm: unknown dtype weight=%d out=%d", weight_dtype, out_dtype);
    if (n_rows == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
#define XRT_RMS(TW, TO) rmsnorm_kernel<TW, TO, 0><<<n_rows, 256, 0, s>>>(x, (const TW*)weight, eps, (TO*)out, rows, hidden, ConvAfterNorm{})
    if (weight_dtype == XRT_F32 && out_dtype == XRT_F32) XRT_RMS(float, float);
    else if (weight_dtype == XRT_F32) XRT_RMS(float, bf16);
    else if (out_dtype == XRT_F32) XRT_RMS(bf16, float);
    else XRT_RMS(bf16, bf16);
#undef XRT_RMS
    XRT_LAUNCH_CHECK("rmsnorm");
    return 0;
}

extern "C" int xrt_rmsnorm_conv_step(const float* x, const void* weight, int weight_dtype, float eps, void* out, int out_dtype, int n_rows,
                                     int hidden, const void* conv_w, int conv_w_dtype, int taps, int plus_input, float* state,
                                     const int* token_slots, void* stream) {
    XRT_REQUIRE(n_rows >= 0 && hidden > 0, "rmsnorm_conv_step: bad sizes rows=%d hidden=%d", n_rows, hidden);
    XRT_REQUIRE((weight_dtype == XRT_F32 || weight_dtype == XRT_BF16) && (out_dtype == XRT_F32 || out_dtype == XRT_BF16) &&
                (conv_w_dtype == XRT_F32 || conv_w_dtype == XRT_BF16), "rmsnorm_conv_step: unknown dtype");
    XRT_REQUIRE(x && weight && out && conv_w && token_slots && (state || taps == 1) && taps >= 1, "rmsnorm_conv_step: null operand");
    XRT_REQUIRE(taps <= CONV_AFTER_NORM_MOST_TAPS, "rmsnorm_conv_step: %d taps, up to %d are served", taps, CONV_AFTER_NORM_MOST_TAPS);
    if (n_rows == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const ConvAfterNorm conv{conv_w, conv_w_dtype, taps, plus_input, state, token_slots};
#define XRT_RMS(TW, TO, TAPS_) rmsnorm_kernel<TW, TO, TAPS_><<<n_rows, 256, 0, s>>>(x, (const TW*)weight, eps, (TO*)out, nullptr, hidden, conv)
#define XRT_RMS_TYPES(TAPS_)                                                                 \
    do {                                                                                     \
        if (weight_dtype == XRT_F32 && out_dtype == XRT_F32) XRT_RMS(float, float, TAPS_);   \
        else if (weight_dtype == XRT_F32) XRT_RMS(float, bf16, TAPS_);                       \
        else if (out_dtype == XRT_F32) XRT_RMS(bf16, float, TAPS_);                          \
        else XRT_RMS(bf16, bf16, TAPS_);                                                     \
    } while (0)
    switch (taps) {
        case 1: XRT_RMS_TYPES(1); break;
        case 2: XRT_RMS_TYPES(2); break;
        case 3: XRT_RMS_TYPES(3); break;
        case 4: XRT_RMS_TYPES(4); break;
        case 5: XRT_RMS_TYPES(5); break;
        case 6: XRT_RMS_TYPES(6); break;
        case 7: XRT_RMS_TYPES(7); break;
        default: XRT_RMS_TYPES(8); break;
    }
#undef XRT_RMS_TYPES
#undef XRT_RMS
    XRT_LAUNCH_CHECK("rmsnorm_conv_step");
    return 0;
}
