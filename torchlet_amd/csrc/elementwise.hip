// Row-wise kernels: embedding gather, residual add + RMSNorm, rotary position
// encoding fused with the write of keys and values into cache pages, SwiGLU gate.
// Each is templated on the activation type (float or bfloat16); all arithmetic is float.
#include "common.h"

// ------------------------------------------------------------------ embedding
// out[c, t, :] = float(table[ids[t], :]) * scale (+ float(pos_table[positions[t], :])) for every copy c; the residual stream is 32-bit.
template <typename T>
__global__ void embedding_kernel(const int* __restrict__ ids, const T* __restrict__ table,
                                 float* __restrict__ out, int hidden, int vocab, float scale,
                                 const int* __restrict__ positions, const void* __restrict__ pos_table, int pos_f32, int pos_rows,
                                 int copies, size_t copy_stride) {
    const int t = blockIdx.x;
    int id = ids[t];
    if (id < 0 || id >= vocab) id = 0;  // ids are checked on the host; never read out of bounds
    const T* src = table + (size_t)id * hidden;
    float* dst = out + (size_t)t * hidden;
    int p = pos_table ? positions[t] : 0;
    if (p < 0 || p >= pos_rows) p = 0;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float v = to_float(src[i]) * scale;
        if (pos_table) v += load_vec(pos_table, pos_f32, (size_t)p * hidden + i);
        for (int c = 0; c < copies; ++c) dst[c * copy_stride + i] = v;
    }
}

extern "C" int tl_embedding(const void* ids, const void* table, int table_dtype, void* out,
                            int tokens, int hidden, int vocab, float scale, const void* positions, const void* pos_table,
                            int pos_dtype, int pos_rows, int copies, hipStream_t stream) {
    TL_REQUIRE(tokens >= 0 && hidden > 0 && vocab > 0 && copies > 0, "embedding: bad sizes tokens=%d hidden=%d vocab=%d copies=%d", tokens, hidden, vocab, copies);
    TL_REQUIRE(!pos_table || (positions && pos_rows > 0), "embedding: a position table needs positions and rows");
    if (tokens == 0) return TL_OK;
    dim3 grid(tokens), block(256);
    const size_t copy_stride = (size_t)tokens * hidden;
    const int pos_f32 = pos_dtype == TL_DT_F32;
    if (table_dtype == TL_DT_F32)
        embedding_kernel<float><<<grid, block, 0, stream>>>((const int*)ids, (const float*)table, (float*)out, hidden, vocab, scale,
                                                            (const int*)positions, pos_table, pos_f32, pos_rows, copies, copy_stride);
    else if (table_dtype == TL_DT_BF16)
        embedding_kernel<bf16_t><<<grid, block, 0, stream>>>((const int*)ids, (const bf16_t*)table, (float*)out, hidden, vocab, scale,
                                                             (const int*)positions, pos_table, pos_f32, pos_rows, copies, copy_stride);
    else TL_REQUIRE(false, "embedding: unknown dtype %d", table_dtype);
    TL_CHECK_LAUNCH("embedding");
    return TL_OK;
}

// ------------------------------------------------------------------ add + RMSNorm
// One block per output row.  r = residual[row] (+ pending[row]); if `update`, r is
// written back to the residual; out = r * rsqrt(mean(r^2) + eps) * weight.
// `rows` (optional) selects the source row of each output row; then nothing is written back.
// `gain` multiplies the row's scale factor (1: the plain norm; a model with a factor on its logits puts it here).
// The pending branch output comes either as one [rows, hidden] tensor of the activation type
// (parts == 0) or as `parts` float slabs [parts, total_rows, hidden] of partial sums that are
// added up here (the split-K products write such slabs).
template <typename T>
__global__ void add_rmsnorm_kernel(float* __restrict__ residual, const void* __restrict__ pending, int parts, size_t part_stride,
                                   const void* __restrict__ weight, int weight_f32, float eps, float gain,
                                   T* __restrict__ out, const int* __restrict__ rows, int hidden) {
    __shared__ float red[16];
    const int orow = blockIdx.x;
    const int srow = rows ? rows[orow] : orow;
    float* res = residual + (size_t)srow * hidden;
    const T* pen = (pending && parts == 0) ? (const T*)pending + (size_t)srow * hidden : nullptr;
    const float* pparts = (pending && parts > 0) ? (const float*)pending + (size_t)srow * hidden : nullptr;
    const bool update = (pending != nullptr) && (rows == nullptr);
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float r = res[i];
        if (pen) r += to_float(pen[i]);
        if (pparts)
            for (int p = 0; p < parts; ++p) r += pparts[p * part_stride + i];
        if (update) res[i] = r;
        ss += r * r;
    }
    ss = block_sum(ss, red);
    const float inv = rsqrtf(ss / (float)hidden + eps) * gain;
    T* dst = out + (size_t)orow * hidden;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float r = res[i];
        if (!update) {
            if (pen) r += to_float(pen[i]);
            if (pparts)
                for (int p = 0; p < parts; ++p) r += pparts[p * part_stride + i];
        }
        dst[i] = from_float<T>(r * inv * load_vec(weight, weight_f32, i));
    }
}

// The same with every element of the row held in registers between the two passes: a thread
// owns IT groups of 4 contiguous elements, loaded with one 16-byte (float) or 8-byte
// (bfloat16) access each, so the row is read from memory once and the weight load overlaps
// the reduction.  Used when hidden % 4 == 0 and hidden <= 16 * blockDim.
template <typename T> struct Vec4;
template <> struct Vec4<float> {
    static __device__ __forceinline__ void load(const float* p, float (&v)[4]) {
        const float4 t = *(const float4*)p; v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
    }
    static __device__ __forceinline__ void store(float* p, const float (&v)[4]) { *(float4*)p = make_float4(v[0], v[1], v[2], v[3]); }
};
template <> struct Vec4<bf16_t> {
    static __device__ __forceinline__ void load(const bf16_t* p, float (&v)[4]) {
        const uint2 t = *(const uint2*)p;
        v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
        v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
    }
    static __device__ __forceinline__ void store(bf16_t* p, const float (&v)[4]) {
        uint2 t;
        t.x = (uint32_t)from_float<bf16_t>(v[0]).bits | ((uint32_t)from_float<bf16_t>(v[1]).bits << 16);
        t.y = (uint32_t)from_float<bf16_t>(v[2]).bits | ((uint32_t)from_float<bf16_t>(v[3]).bits << 16);
        *(uint2*)p = t;
    }
};

// r += the N slabs' four elements at src, src + stride, ...: all requested, then added in their order.
template <int N>
__device__ __forceinline__ void add_slabs(const float* src, size_t stride, float (&r)[4]) {
    float p[N][4];
#pragma unroll
    for (int u = 0; u < N; ++u) Vec4<float>::load(src + u * stride, p[u]);
#pragma unroll
    for (int u = 0; u < N; ++u)
#pragma unroll
        for (int v = 0; v < 4; ++v) r[v] += p[u][v];
}

template <typename T, int IT>
__global__ void add_rmsnorm_reg_kernel(float* __restrict__ residual, const void* __restrict__ pending, int parts, size_t part_stride,
                                       const void* __restrict__ weight, int weight_f32, float eps, float gain,
                                       T* __restrict__ out, const int* __restrict__ rows, int hidden) {
    __shared__ float red[16];
    const int orow = blockIdx.x;
    const int srow = rows ? rows[orow] : orow;
    float* res = residual + (size_t)srow * hidden;
    const T* pen = (pending && parts == 0) ? (const T*)pending + (size_t)srow * hidden : nullptr;
    const float* pparts = (pending && parts > 0) ? (const float*)pending + (size_t)srow * hidden : nullptr;
    const bool update = (pending != nullptr) && (rows == nullptr);
    float r[IT][4], wv[IT][4];
    float ss = 0.f;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int i = (it * blockDim.x + threadIdx.x) * 4;
        if (i < hidden) {
            Vec4<float>::load(res + i, r[it]);
            if (pen) {
                float p[4];
                Vec4<T>::load(pen + i, p);
#pragma unroll
                for (int v = 0; v < 4; ++v) r[it][v] += p[v];
            }
            if (pparts) {
                // four slabs at a time, all requested before the first is added (a loop over a count known
                // only at run time fetches one slab after the other: a trip to memory each); the sums are
                // added in the order of the slabs either way.  The last two or three slabs are a group as well
                // (three slabs, as for the matrices 5120 wide, were three trips).
                int q = 0;
                for (; q + 4 <= parts; q += 4) add_slabs<4>(pparts + q * part_stride + i, part_stride, r[it]);
                if (parts - q == 3) add_slabs<3>(pparts + q * part_stride + i, part_stride, r[it]);
                else if (parts - q == 2) add_slabs<2>(pparts + q * part_stride + i, part_stride, r[it]);
                else if (parts - q == 1) add_slabs<1>(pparts + q * part_stride + i, part_stride, r[it]);
            }
            if (weight_f32) Vec4<float>::load((const float*)weight + i, wv[it]);
            else Vec4<bf16_t>::load((const bf16_t*)weight + i, wv[it]);
#pragma unroll
            for (int v = 0; v < 4; ++v) ss += r[it][v] * r[it][v];
        }
    }
    if (update) {
#pragma unroll
        for (int it = 0; it < IT; ++it) {
            const int i = (it * blockDim.x + threadIdx.x) * 4;
            if (i < hidden) Vec4<float>::store(res + i, r[it]);
        }
    }
    ss = block_sum(ss, red);
    const float inv = rsqrtf(ss / (float)hidden + eps) * gain;
    T* dst = out + (size_t)orow * hidden;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
        const int i = (it * blockDim.x + threadIdx.x) * 4;
        if (i < hidden) {
            float o[4];
#pragma unroll
            for (int v = 0; v < 4; ++v) o[v] = r[it][v] * inv * wv[it][v];
            Vec4<T>::store(dst + i, o);
        }
    }
}

template <typename T>
static void launch_add_rmsnorm(float* residual, const void* pending, int parts, size_t part_stride, const void* weight,
                               int weight_f32, float eps, float gain, T* out, const int* rows, int out_rows, int hidden, hipStream_t stream) {
    const bool aligned = hidden % 4 == 0 && ((uintptr_t)residual % 16) == 0 && ((uintptr_t)out % 16) == 0 &&
                         ((uintptr_t)pending % 16) == 0 && ((uintptr_t)weight % 16) == 0;
    dim3 grid(out_rows);
    if (aligned && hidden <= 1024)
        add_rmsnorm_reg_kernel<T, 1><<<grid, 256, 0, stream>>>(residual, pending, parts, part_stride, weight, weight_f32, eps, gain, out, rows, hidden);
    else if (aligned && hidden <= 2048)
        add_rmsnorm_reg_kernel<T, 2><<<grid, 256, 0, stream>>>(residual, pending, parts, part_stride, weight, weight_f32, eps, gain, out, rows, hidden);
    else if (aligned && hidden <= 4096)
        add_rmsnorm_reg_kernel<T, 2><<<grid, 512, 0, stream>>>(residual, pending, parts, part_stride, weight, weight_f32, eps, gain, out, rows, hidden);
    else if (aligned && hidden <= 8192)
        add_rmsnorm_reg_kernel<T, 4><<<grid, 512, 0, stream>>>(residual, pending, parts, part_stride, weight, weight_f32, eps, gain, out, rows, hidden);
    else if (aligned && hidden <= 16384)
        add_rmsnorm_reg_kernel<T, 4><<<grid, 1024, 0, stream>>>(residual, pending, parts, part_stride, weight, weight_f32, eps, gain, out, rows, hidden);
    else
        add_rmsnorm_kernel<T><<<grid, hidden >= 2048 ? 512 : 256, 0, stream>>>(residual, pending, parts, part_stride, weight, weight_f32, eps, gain, out, rows, hidden);
}

// parts == 0: `pending` is [rows, hidden] of the activation type (or null); parts > 0: `pending` is
// float [parts, part_rows, hidden], slabs of partial sums to be added up.
extern "C" int tl_add_rmsnorm(void* residual, const void* pending, int parts, int part_rows, const void* weight,
                              int weight_f32, float eps, float gain, void* out, const void* rows, int out_rows, int hidden,
                              int act_dtype, hipStream_t stream) {
    TL_REQUIRE(parts >= 0 && parts <= 64, "add_rmsnorm: %d partial slabs", parts);
    const size_t part_stride = (size_t)part_rows * hidden;
    TL_REQUIRE(out_rows >= 0 && hidden > 0, "add_rmsnorm: bad sizes rows=%d hidden=%d", out_rows, hidden);
    if (out_rows == 0) return TL_OK;
    if (act_dtype == TL_DT_F32)
        launch_add_rmsnorm<float>((float*)residual, pending, parts, part_stride, weight, weight_f32, eps, gain, (float*)out, (const int*)rows, out_rows, hidden, stream);
    else if (act_dtype == TL_DT_BF16)
        launch_add_rmsnorm<bf16_t>((float*)residual, pending, parts, part_stride, weight, weight_f32, eps, gain, (bf16_t*)out, (const int*)rows, out_rows, hidden, stream);
    else TL_REQUIRE(false, "add_rmsnorm: unknown dtype %d", act_dtype);
    TL_CHECK_LAUNCH("add_rmsnorm");
    return TL_OK;
}

// ------------------------------------------------------------------ RoPE + cache write
// One wave per token and head.  Row layout of `qkv`: [q heads | k heads | v heads], each head
// `head_dim` wide, row stride `row_stride` elements.
//   * rotate (inv_freq != null): the first `rot_heads` heads (q, then k) are rotated in
//     place with the split-half pairing (j, j + head_dim/2) by angle = float(pos) * inv_freq[j];
//     with `pairs` the two elements of frequency j are the neighbours (2j, 2j + 1) instead.
//   * write (k_plane != null): rotated k and raw v of the token go to the page
//     block_table[token_req[t]][pos / page] at offset pos % page.  The key plane is
//     [pages, kv_heads, page, head_dim]; the value plane holds each page transposed,
//     [pages, kv_heads, head_dim, page], the layout the attention kernels read.  Page 0 is the
//     sentinel that empty block-table entries point to: a token whose page is 0 (a padding row of a
//     step of fixed shape) has its keys and values dropped, so nothing ever writes that page.
// One pair turned by its angle, in a fixed sequence of roundings (one product, one fused
// multiply-add per result), so that every kernel here gives the same bits for the same input.
__device__ __forceinline__ void rope_turn(float& x1, float& x2, float c, float sn) {
    const float y1 = __fmaf_rn(x1, c, -__fmul_rn(x2, sn));
    const float y2 = __fmaf_rn(x2, c, __fmul_rn(x1, sn));
    x1 = y1;
    x2 = y2;
}

#define ROPE_HEADS_PER_GROUP 4          // one wave per head, four heads per work-group
template <typename T>
__global__ __launch_bounds__(ROPE_HEADS_PER_GROUP * TL_WAVE)
void rope_cache_write_kernel(T* __restrict__ qkv, int row_stride, int q_heads, int kv_heads,
                             int head_dim, int rot_heads, const int* __restrict__ positions,
                             const float* __restrict__ inv_freq, const int* __restrict__ token_req,
                             const int* __restrict__ block_table, int bt_stride,
                             T* __restrict__ k_plane, T* __restrict__ v_plane, int page_size, int pairs, int pair_aligned,
                             const float* __restrict__ parts, int num_parts, size_t part_stride, int parts_ld,
                             const void* __restrict__ bias, int bias_f32) {
    // A wave owns one head of one token: a query head (rotated in place), a key head (rotated in
    // place and written to its page) or a value head (written to its page, transposed).  Each wave
    // takes the cosines and sines of its own pairs, so no wave waits for another.
    const int t = blockIdx.x;
    const int head = blockIdx.y * ROPE_HEADS_PER_GROUP + threadIdx.x / TL_WAVE;
    const int lane = threadIdx.x % TL_WAVE;
    const int heads = q_heads + kv_heads + (k_plane ? kv_heads : 0);
    if (head >= heads) return;
    const int pos = positions[t];
    const int half = head_dim / 2;
    T* x = qkv + (size_t)t * row_stride + (size_t)head * head_dim;
    T* dst = nullptr;                      // this head's place in the cache, if it has one
    if (k_plane && head >= q_heads) {
        const int page = block_table[(size_t)token_req[t] * bt_stride + pos / page_size];
        const int kvh = (head - q_heads) % kv_heads;
        const size_t base = ((size_t)page * kv_heads + kvh) * page_size * head_dim;
        if (page != 0)
            dst = head < q_heads + kv_heads ? k_plane + base + (size_t)(pos % page_size) * head_dim
                                            : v_plane + base + (pos % page_size);
    }
    // With `parts` the row does not come from qkv but is the sum of float slabs of partial sums
    // [num_parts][tokens, parts_ld] plus the bias (a projection that was split over K); the rotated
    // queries then go to qkv, keys and values to their pages only.
    auto element = [&](int i) -> float {
        if (!parts) return to_float(x[i]);
        const size_t col = (size_t)head * head_dim + i;
        float sum = bias ? load_vec(bias, bias_f32, col) : 0.f;
        const float* src = parts + (size_t)t * parts_ld + col;
        int p = 0;
        for (; p + 4 <= num_parts; p += 4) {       // four slabs requested before the first is added, in their order
            float v[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) v[u] = src[(size_t)(p + u) * part_stride];
#pragma unroll
            for (int u = 0; u < 4; ++u) sum += v[u];
        }
        if (num_parts - p == 3) {                  // (and the last two or three)
            const float v0 = src[(size_t)p * part_stride], v1 = src[(size_t)(p + 1) * part_stride], v2 = src[(size_t)(p + 2) * part_stride];
            sum += v0; sum += v1; sum += v2;
        } else if (num_parts - p == 2) {
            const float v0 = src[(size_t)p * part_stride], v1 = src[(size_t)(p + 1) * part_stride];
            sum += v0; sum += v1;
        } else if (num_parts - p == 1) {
            sum += src[(size_t)p * part_stride];
        }
        return sum;
    };
    if (head >= q_heads + kv_heads) {      // value head: [head_dim, page] inside the page
        if (dst)
            for (int d = lane; d < head_dim; d += TL_WAVE) dst[(size_t)d * page_size] = from_float<T>(element(d));
        return;
    }
    const bool rotate = inv_freq && head < rot_heads;
    if (!rotate && !dst && !parts) return;
    if (pairs && pair_aligned && !parts) {
        // pair layout: the two elements of a frequency are one aligned load and one aligned store
        struct __attribute__((aligned(2 * sizeof(T)))) Two { T a, b; };
        for (int j = lane; j < half; j += TL_WAVE) {
            Two p = *(const Two*)(x + 2 * j);
            float x1 = to_float(p.a), x2 = to_float(p.b);
            if (rotate) {
                const float angle = (float)pos * inv_freq[j];
                rope_turn(x1, x2, cosf(angle), sinf(angle));
            }
            p.a = from_float<T>(x1);
            p.b = from_float<T>(x2);
            if (rotate) *(Two*)(x + 2 * j) = p;
            if (dst) *(Two*)(dst + 2 * j) = p;
        }
        return;
    }
    for (int j = lane; j < half; j += TL_WAVE) {
        // the two elements that frequency j turns: (j, j + half), or neighbours (2j, 2j + 1) in the
        // pair layout (a projection whose rows were reordered that way at load time)
        const int i1 = pairs ? 2 * j : j, i2 = pairs ? 2 * j + 1 : j + half;
        float x1 = element(i1), x2 = element(i2);
        if (rotate) {
            const float angle = (float)pos * inv_freq[j];
            rope_turn(x1, x2, cosf(angle), sinf(angle));
        }
        if (rotate || parts) {
            x[i1] = from_float<T>(x1);
            x[i2] = from_float<T>(x2);
        }
        if (dst) {
            dst[i1] = from_float<T>(x1);
            dst[i2] = from_float<T>(x2);
        }
    }
}

// The same for bfloat16 rows in the pair layout whose heads are multiples of 8 wide, 16 bytes at a
// time: a work-group owns one token, a thread one 16-byte piece (four pairs of one head) per round.
// Queries are rotated in place, keys rotated and copied to their page in whole pieces, values
// scattered to their transposed place.  (One wave per head, as above, moved 1.7 TB/s on a prompt of
// 2048 tokens; this is for steps of many tokens.)
__global__ __launch_bounds__(256)
void rope_cache_write_rows_kernel(bf16_t* __restrict__ qkv, int row_stride, int q_heads, int kv_heads, int head_dim,
                                  int rot_heads, const int* __restrict__ positions, const float* __restrict__ inv_freq,
                                  const int* __restrict__ token_req, const int* __restrict__ block_table, int bt_stride,
                                  bf16_t* __restrict__ k_plane, bf16_t* __restrict__ v_plane, int page_size) {
    const int t = blockIdx.x;
    const int pos = positions[t];
    const int heads = q_heads + kv_heads + (k_plane ? kv_heads : 0);
    const int pph = head_dim / 8;                                  // pieces per head
    bf16_t* row = qkv + (size_t)t * row_stride;
    size_t page_base = 0;
    if (k_plane) page_base = (size_t)block_table[(size_t)token_req[t] * bt_stride + pos / page_size] * kv_heads * page_size * head_dim;
    const bool stores = k_plane && page_base != 0;                 // page 0 is the sentinel: never written
    const int off = pos % page_size;
    // The token's cosines and sines are worked out once, not once a head: the same 32-bit angle and functions, read
    // back from shared memory by every head's threads (28 query heads and 4 key heads of 128: 2048 tokens 17 -> 12 us).
    __shared__ float2 turn[128];                                   // (head_dim <= 256: the host checks)
    if (inv_freq) {
        for (int j = threadIdx.x; j < head_dim / 2; j += 256) {
            const float angle = (float)pos * inv_freq[j];
            turn[j] = make_float2(cosf(angle), sinf(angle));
        }
        __syncthreads();
    }
    for (int p = threadIdx.x; p < heads * pph; p += 256) {
        const int head = p / pph, d0 = (p % pph) * 8;
        union { uint4 u; uint16_t e[8]; } piece;
        piece.u = *(const uint4*)(row + (size_t)head * head_dim + d0);
        if (head >= q_heads + kv_heads) {                          // value head: [head_dim, page] inside the page
            bf16_t* dst = v_plane + page_base + (size_t)(head - q_heads - kv_heads) * page_size * head_dim + off;
            if (stores) {
#pragma unroll
                for (int e = 0; e < 8; ++e) dst[(size_t)(d0 + e) * page_size].bits = piece.e[e];
            }
            continue;
        }
        const bool rotate = inv_freq && head < rot_heads;
        if (rotate) {
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                bf16_t a, b;
                a.bits = piece.e[2 * j];
                b.bits = piece.e[2 * j + 1];
                float x1 = to_float(a), x2 = to_float(b);
                const float2 cs = turn[d0 / 2 + j];
                rope_turn(x1, x2, cs.x, cs.y);
                piece.e[2 * j] = from_float<bf16_t>(x1).bits;
                piece.e[2 * j + 1] = from_float<bf16_t>(x2).bits;
            }
            *(uint4*)(row + (size_t)head * head_dim + d0) = piece.u;
        }
        if (head >= q_heads && stores)
            *(uint4*)(k_plane + page_base + ((size_t)(head - q_heads) * page_size + off) * head_dim + d0) = piece.u;
    }
}

extern "C" int tl_rope_cache_write(void* qkv, int row_stride, int tokens, int q_heads, int kv_heads,
                                   int head_dim, int rot_heads, const void* positions, const void* inv_freq,
                                   const void* token_req, const void* block_table, int bt_stride,
                                   void* k_plane, void* v_plane, int page_size, int pairs, int act_dtype,
                                   const void* parts, int num_parts, size_t part_stride, int parts_ld,
                                   const void* bias, int bias_f32, hipStream_t stream) {
    TL_REQUIRE(!parts || (num_parts > 0 && parts_ld >= (q_heads + kv_heads + (k_plane ? kv_heads : 0)) * head_dim),
               "rope_cache_write: slabs of partial sums need a count and rows as wide as the heads");
    TL_REQUIRE(tokens >= 0 && q_heads >= 0 && kv_heads >= 0 && head_dim > 0 && head_dim % 2 == 0 && head_dim <= 256,
               "rope_cache_write: bad sizes tokens=%d q_heads=%d kv_heads=%d head_dim=%d (even, at most 256)", tokens, q_heads, kv_heads, head_dim);
    TL_REQUIRE(rot_heads <= q_heads + kv_heads, "rope_cache_write: rot_heads %d exceeds q+k heads", rot_heads);
    TL_REQUIRE((k_plane == nullptr) == (v_plane == nullptr), "rope_cache_write: give both planes or none");
    TL_REQUIRE(!k_plane || (block_table && token_req && page_size > 0 && bt_stride > 0),
               "rope_cache_write: cache write needs block table, token_req and page size");
    TL_REQUIRE(row_stride >= (q_heads + (k_plane ? 2 * kv_heads : kv_heads)) * head_dim,
               "rope_cache_write: row stride %d too small", row_stride);
    if (tokens == 0) return TL_OK;
    const int heads = q_heads + kv_heads + (k_plane ? kv_heads : 0);
    // pairs as one access: rows and planes start on a multiple of two elements (eight bytes covers both dtypes)
    const int pair_aligned = row_stride % 2 == 0 && ((uintptr_t)qkv % 8) == 0 && ((uintptr_t)k_plane % 8) == 0;
    if (act_dtype == TL_DT_BF16 && pairs && !parts && tokens >= 64 && head_dim % 8 == 0 && row_stride % 8 == 0 &&
        ((uintptr_t)qkv % 16) == 0 && ((uintptr_t)k_plane % 16) == 0 && (!inv_freq || ((uintptr_t)inv_freq % 16) == 0)) {
        rope_cache_write_rows_kernel<<<dim3(tokens), dim3(256), 0, stream>>>((bf16_t*)qkv, row_stride, q_heads, kv_heads, head_dim, rot_heads,
            (const int*)positions, (const float*)inv_freq, (const int*)token_req, (const int*)block_table, bt_stride,
            (bf16_t*)k_plane, (bf16_t*)v_plane, page_size);
        TL_CHECK_LAUNCH("rope_cache_write");
        return TL_OK;
    }
    dim3 grid(tokens, (heads + ROPE_HEADS_PER_GROUP - 1) / ROPE_HEADS_PER_GROUP), block(ROPE_HEADS_PER_GROUP * TL_WAVE);
    if (act_dtype == TL_DT_F32)
        rope_cache_write_kernel<float><<<grid, block, 0, stream>>>((float*)qkv, row_stride, q_heads, kv_heads, head_dim, rot_heads,
            (const int*)positions, (const float*)inv_freq, (const int*)token_req, (const int*)block_table, bt_stride,
            (float*)k_plane, (float*)v_plane, page_size, pairs, pair_aligned, (const float*)parts, num_parts, part_stride, parts_ld, bias, bias_f32);
    else if (act_dtype == TL_DT_BF16)
        rope_cache_write_kernel<bf16_t><<<grid, block, 0, stream>>>((bf16_t*)qkv, row_stride, q_heads, kv_heads, head_dim, rot_heads,
            (const int*)positions, (const float*)inv_freq, (const int*)token_req, (const int*)block_table, bt_stride,
            (bf16_t*)k_plane, (bf16_t*)v_plane, page_size, pairs, pair_aligned, (const float*)parts, num_parts, part_stride, parts_ld, bias, bias_f32);
    else TL_REQUIRE(false, "rope_cache_write: unknown dtype %d", act_dtype);
    TL_CHECK_LAUNCH("rope_cache_write");
    return TL_OK;
}

// ------------------------------------------------------------------ SwiGLU gate
// out[t, i] = act(gu[t, i]) * gu[t, inter + i]; act 0: silu(g) = g / (1 + exp(-g)), act 1: relu, act 2: the tanh form of gelu.
template <typename T>
__global__ void swiglu_kernel(const T* __restrict__ gu, T* __restrict__ out, int inter, size_t total, int act) {
    const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= total) return;
    const size_t t = idx / inter;
    const int i = (int)(idx % inter);
    const float g = to_float(gu[t * 2 * inter + i]);
    const float u = to_float(gu[t * 2 * inter + inter + i]);
    out[idx] = from_float<T>((act == 1 ? fmaxf(g, 0.f) : act == 2 ? gelu_tanh(g) : g / (1.f + expf(-g))) * u);
}

extern "C" int tl_swiglu(const void* gu, void* out, int tokens, int inter, int act_dtype, int act, hipStream_t stream) {
    TL_REQUIRE(tokens >= 0 && inter > 0 && act >= 0 && act <= 2, "swiglu: bad sizes tokens=%d inter=%d, or an unknown gate %d", tokens, inter, act);
    const size_t total = (size_t)tokens * inter;
    if (total == 0) return TL_OK;
    dim3 block(256), grid((unsigned)((total + 255) / 256));
    if (act_dtype == TL_DT_F32)
        swiglu_kernel<float><<<grid, block, 0, stream>>>((const float*)gu, (float*)out, inter, total, act);
    else if (act_dtype == TL_DT_BF16)
        swiglu_kernel<bf16_t><<<grid, block, 0, stream>>>((const bf16_t*)gu, (bf16_t*)out, inter, total, act);
    else TL_REQUIRE(false, "swiglu: unknown dtype %d", act_dtype);
    TL_CHECK_LAUNCH("swiglu");
    return TL_OK;
}

// ------------------------------------------------------------------ streaming read (a yardstick)
// Reads `bytes` of memory once, as fast as the machine lets a kernel read: every work-group walks a
// contiguous share in 16-byte pieces, eight requests per thread on their way, and folds what it read into one
// word per work-group (written to `sink`, so that no read can be dropped).  What it measures is the rate at
// which this GPU delivers memory to any kernel that only reads; the benchmark quotes the decode step against it.
#define STREAM_THREADS 256
#define STREAM_DEPTH 8
__global__ __launch_bounds__(STREAM_THREADS) void stream_read_kernel(const uint4* __restrict__ p, size_t pieces,
                                                                     size_t per_group, uint32_t* __restrict__ sink) {
    const size_t begin = (size_t)blockIdx.x * per_group;
    const size_t end = begin + per_group < pieces ? begin + per_group : pieces;
    uint32_t acc = 0;
    size_t i = begin + threadIdx.x;
    for (; i + (STREAM_DEPTH - 1) * STREAM_THREADS < end; i += STREAM_DEPTH * STREAM_THREADS) {
        uint4 v[STREAM_DEPTH];
#pragma unroll
        for (int u = 0; u < STREAM_DEPTH; ++u) v[u] = p[i + (size_t)u * STREAM_THREADS];
#pragma unroll
        for (int u = 0; u < STREAM_DEPTH; ++u) acc ^= v[u].x ^ v[u].y ^ v[u].z ^ v[u].w;
    }
    for (; i < end; i += STREAM_THREADS) {
        const uint4 v = p[i];
        acc ^= v.x ^ v.y ^ v.z ^ v.w;
    }
#pragma unroll
    for (int o = TL_WAVE / 2; o > 0; o >>= 1) acc ^= __shfl_xor(acc, o, TL_WAVE);
    __shared__ uint32_t part[STREAM_THREADS / TL_WAVE];
    if (threadIdx.x % TL_WAVE == 0) part[threadIdx.x / TL_WAVE] = acc;
    __syncthreads();
    if (threadIdx.x == 0) {
        uint32_t all = 0;
        for (int w = 0; w < STREAM_THREADS / TL_WAVE; ++w) all ^= part[w];
        sink[blockIdx.x] = all;
    }
}

// Work-groups the read is dealt to by default (`sink` needs one 32-bit word per work-group).
extern "C" int tl_stream_read_groups() { return 8192; }     // measured: 256 give 5.6 TB/s, 2048 6.2, 8192 6.3, 16384 6.2

extern "C" int tl_stream_read(const void* data, size_t bytes, void* sink, int groups, hipStream_t stream) {
    TL_REQUIRE(data != nullptr && sink != nullptr && bytes >= 16 && ((uintptr_t)data % 16) == 0,
               "stream_read: needs 16-byte aligned memory of at least 16 bytes and a sink");
    TL_REQUIRE(groups >= 0 && groups <= 65536, "stream_read: %d work-groups", groups);
    const size_t pieces = bytes / 16;
    if (groups == 0) groups = tl_stream_read_groups();
    const size_t per_group = (pieces + groups - 1) / groups;
    stream_read_kernel<<<dim3(groups), dim3(STREAM_THREADS), 0, stream>>>((const uint4*)data, pieces, per_group, (uint32_t*)sink);
    TL_CHECK_LAUNCH("stream_read");
    return TL_OK;
}

// ------------------------------------------------------------------ norm after the sum
// x <- norm(alpha * x + y) * weight, row by row: the layer arrangement in which the norm follows the sum and the
// sublayers read the normed stream itself.  `residual` (float) holds x and receives the result; `out` (optional)
// receives its rounding to the activation type, which the next sublayer's products read.  y comes as one tensor of
// the activation type (parts == 0), as float slabs of partial sums, or not at all.
template <typename T>
__global__ void scaled_add_rmsnorm_kernel(float* __restrict__ residual, const void* __restrict__ pending, int parts, size_t part_stride,
                                          float alpha, const void* __restrict__ weight, int weight_f32, float eps,
                                          T* __restrict__ out, int hidden) {
    __shared__ float red[16];
    const int row = blockIdx.x;
    float* res = residual + (size_t)row * hidden;
    const T* pen = (pending && parts == 0) ? (const T*)pending + (size_t)row * hidden : nullptr;
    const float* pparts = (pending && parts > 0) ? (const float*)pending + (size_t)row * hidden : nullptr;
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float r = alpha * res[i];
        if (pen) r += to_float(pen[i]);
        if (pparts) {
            float y = 0.f;
            for (int p = 0; p < parts; ++p) y += pparts[p * part_stride + i];
            r += y;
        }
        res[i] = r;                      // the same thread reads it back below
        ss = fmaf(r, r, ss);
    }
    ss = block_sum(ss, red);
    const float inv = 1.f / sqrtf(ss / (float)hidden + eps);
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float y = res[i] * inv * load_vec(weight, weight_f32, i);
        res[i] = y;
        if (out) out[(size_t)row * hidden + i] = from_float<T>(y);
    }
}

extern "C" int tl_scaled_add_rmsnorm(void* residual, const void* pending, int parts, int total_rows, float alpha, const void* weight,
                                     int weight_f32, float eps, void* out, int rows, int hidden, int dtype, hipStream_t stream) {
    TL_REQUIRE(rows >= 0 && hidden > 0 && parts >= 0, "scaled_add_rmsnorm: bad sizes rows=%d hidden=%d", rows, hidden);
    if (rows == 0) return TL_OK;
    const size_t part_stride = (size_t)total_rows * hidden;
    dim3 grid(rows), block(hidden <= 512 ? 128 : hidden <= 2048 ? 256 : 512);
    if (dtype == TL_DT_F32)
        scaled_add_rmsnorm_kernel<float><<<grid, block, 0, stream>>>((float*)residual, pending, parts, part_stride, alpha, weight, weight_f32, eps, (float*)out, hidden);
    else if (dtype == TL_DT_BF16)
        scaled_add_rmsnorm_kernel<bf16_t><<<grid, block, 0, stream>>>((float*)residual, pending, parts, part_stride, alpha, weight, weight_f32, eps, (bf16_t*)out, hidden);
    else TL_REQUIRE(false, "scaled_add_rmsnorm: unknown dtype %d", dtype);
    TL_CHECK_LAUNCH("scaled_add_rmsnorm");
    return TL_OK;
}

// ------------------------------------------------------------------ norm over several copies of the residual
// x [S, T, hidden] float: S copies of the residual (hyper-connections).  One block per output row:
//   the pending branch output p (one [T, hidden] tensor of the activation type, or `parts` float slabs of partial sums) enters
//   all copies at once, x_t <- sum_s mix[s, t] x_s + gate[t] p (mix == null: x_t <- x_t + p), written back unless `rows` selects;
//   u = sum_s read[s] x_s (read == null: the sum of the copies);
//   kind 0: out = u / sqrt(mean(u^2) + eps) * gain * weight;  kind 1: out = ((u - mean) / sqrt(mean((u - mean)^2) + eps) * weight + bias) * gain.
// u stays in shared memory between the passes (mean, squared deviations, output), so the deviations are taken from the mean itself.
#define SN_MAX 8

template <typename T>
__global__ void __launch_bounds__(256)
streams_norm_kernel(float* __restrict__ x, int S, int total_rows, int hidden, const void* __restrict__ pending, int parts,
                    const float* __restrict__ mix, const float* __restrict__ gate, const float* __restrict__ read, int kind,
                    const void* __restrict__ weight, int weight_f32, const void* __restrict__ bias, int bias_f32, float eps, float gain,
                    T* __restrict__ out, const int* __restrict__ rows) {
    extern __shared__ float u_row[];                 // [hidden]
    __shared__ float red[16];
    const int orow = blockIdx.x;
    const int srow = rows ? rows[orow] : orow;
    const size_t copy_stride = (size_t)total_rows * hidden;
    float* xr = x + (size_t)srow * hidden;
    const T* pen = (pending && parts == 0) ? (const T*)pending + (size_t)srow * hidden : nullptr;
    const float* slabs = (pending && parts > 0) ? (const float*)pending + (size_t)srow * hidden : nullptr;
    const bool update = pending != nullptr && rows == nullptr;
    float m[SN_MAX][SN_MAX], g[SN_MAX], rd[SN_MAX];
#pragma unroll
    for (int a = 0; a < SN_MAX; ++a) {
        g[a] = (gate && a < S) ? gate[a] : 1.f;
        rd[a] = a < S ? (read ? read[a] : 1.f) : 0.f;
#pragma unroll
        for (int b = 0; b < SN_MAX; ++b) m[a][b] = (mix && a < S && b < S) ? mix[a * S + b] : (a == b ? 1.f : 0.f);
    }
    float sum = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float xs[SN_MAX];
#pragma unroll
        for (int a = 0; a < SN_MAX; ++a) xs[a] = a < S ? xr[a * copy_stride + i] : 0.f;
        float u = 0.f;
        if (pending) {
            float p = 0.f;
            if (pen) p = to_float(pen[i]);
            else
                for (int q = 0; q < parts; ++q) p += slabs[q * copy_stride + i];
#pragma unroll
            for (int b = 0; b < SN_MAX; ++b) {
                if (b < S) {
                    float nb = 0.f;
#pragma unroll
                    for (int a = 0; a < SN_MAX; ++a)
                        if (a < S) nb = fmaf(m[a][b], xs[a], nb);
                    nb = fmaf(g[b], p, nb);
                    if (update) xr[b * copy_stride + i] = nb;
                    u = fmaf(rd[b], nb, u);
                }
            }
        } else {
#pragma unroll
            for (int b = 0; b < SN_MAX; ++b)
                if (b < S) u = fmaf(rd[b], xs[b], u);
        }
        u_row[i] = u;
        sum += u;
    }
    float mean = 0.f;
    if (kind == 1) mean = block_sum(sum, red) / (float)hidden;
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float d = u_row[i] - mean;
        ss = fmaf(d, d, ss);
    }
    ss = block_sum(ss, red);
    const float inv = 1.f / sqrtf(ss / (float)hidden + eps);
    T* dst = out + (size_t)orow * hidden;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float d = (u_row[i] - mean) * inv;
        const float w = load_vec(weight, weight_f32, i);
        dst[i] = from_float<T>(kind == 1 ? (d * w + load_vec(bias, bias_f32, i)) * gain : d * gain * w);
    }
}

extern "C" int tl_streams_norm(void* x, int streams, int total_rows, int hidden, const void* pending, int parts, const void* mix,
                               const void* gate, const void* read, int kind, const void* weight, int weight_f32, const void* bias,
                               int bias_f32, float eps, float gain, void* out, const void* rows, int n_out, int act_dtype, hipStream_t stream) {
    TL_REQUIRE(streams >= 1 && streams <= SN_MAX && total_rows >= 0 && hidden > 0 && n_out >= 0, "streams_norm: bad sizes");
    TL_REQUIRE(kind == 0 || (kind == 1 && bias), "streams_norm: kind %d (a layer norm needs its bias)", kind);
    TL_REQUIRE((size_t)hidden * sizeof(float) <= 60 * 1024, "streams_norm: rows of %d numbers do not fit the shared memory", hidden);
    TL_REQUIRE((mix == nullptr) == (gate == nullptr), "streams_norm: mix and gate come together");
    if (n_out == 0) return TL_OK;
    dim3 grid(n_out), block(256);
    const size_t smem = (size_t)hidden * sizeof(float);
    if (act_dtype == TL_DT_F32)
        streams_norm_kernel<float><<<grid, block, smem, stream>>>((float*)x, streams, total_rows, hidden, pending, parts, (const float*)mix, (const float*)gate,
                                                                  (const float*)read, kind, weight, weight_f32, bias, bias_f32, eps, gain, (float*)out, (const int*)rows);
    else if (act_dtype == TL_DT_BF16)
        streams_norm_kernel<bf16_t><<<grid, block, smem, stream>>>((float*)x, streams, total_rows, hidden, pending, parts, (const float*)mix, (const float*)gate,
                                                                   (const float*)read, kind, weight, weight_f32, bias, bias_f32, eps, gain, (bf16_t*)out, (const int*)rows);
    else TL_REQUIRE(false, "streams_norm: unknown dtype %d", act_dtype);
    TL_CHECK_LAUNCH("streams_norm");
    return TL_OK;
}

// ------------------------------------------------------------------ embedding with a hashed bigram row
// out[c, t, :] = float(table[ids[t], :]) * scale + float(bigram[row(t), :]), row(t) = (prev * mul_prev + ids[t] * mul_cur) mod buckets with prev
// the token before t in its sequence, or row `buckets` (the table's last) for a sequence's first token (position 0).  The token before a
// step's first token of a request is read from last_token[slot] (what the step before left there); last_token_kernel moves it on.
template <typename T>
__global__ void bigram_embedding_kernel(const int* __restrict__ ids, const T* __restrict__ table, float* __restrict__ out, int hidden, int vocab,
                                        float scale, const int* __restrict__ token_req, const int* __restrict__ req_indptr,
                                        const int* __restrict__ positions, const int* __restrict__ slots, const int* __restrict__ last_token,
                                        const T* __restrict__ bigram, int buckets, long long mul_prev, long long mul_cur, int copies, size_t copy_stride) {
    const int t = blockIdx.x;
    int id = ids[t];
    if (id < 0 || id >= vocab) id = 0;
    const int r = token_req[t];
    int row = buckets;
    if (positions[t] > 0) {
        int prev = t > req_indptr[r] ? ids[t - 1] : last_token[slots[r]];
        if (prev < 0 || prev >= vocab) prev = 0;
        long long h = ((long long)prev * mul_prev + (long long)id * mul_cur) % buckets;
        if (h < 0) h += buckets;
        row = (int)h;
    }
    const T* src = table + (size_t)id * hidden;
    const T* big = bigram + (size_t)row * hidden;
    float* dst = out + (size_t)t * hidden;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float v = fmaf(to_float(src[i]), scale, to_float(big[i]));
        for (int c = 0; c < copies; ++c) dst[c * copy_stride + i] = v;
    }
}

__global__ void last_token_kernel(const int* __restrict__ ids, const int* __restrict__ req_indptr, const int* __restrict__ slots,
                                  int* __restrict__ last_token, int requests) {
    const int r = blockIdx.x * blockDim.x + threadIdx.x;
    if (r >= requests) return;
    const int a = req_indptr[r], b = req_indptr[r + 1];
    if (b > a) last_token[slots[r]] = ids[b - 1];
}

extern "C" int tl_bigram_embedding(const void* ids, const void* table, void* out, int tokens, int hidden, int vocab, float scale,
                                   const void* token_req, const void* req_indptr, int requests, const void* positions, const void* slots,
                                   void* last_token, const void* bigram, int buckets, long mul_prev, long mul_cur, int copies, int dtype,
                                   hipStream_t stream) {
    TL_REQUIRE(tokens >= 0 && hidden > 0 && vocab > 0 && copies > 0 && buckets > 0 && requests >= 0, "bigram_embedding: bad sizes");
    TL_REQUIRE(token_req && req_indptr && positions && slots && last_token && bigram, "bigram_embedding: a null operand");
    if (tokens == 0) return TL_OK;
    const size_t copy_stride = (size_t)tokens * hidden;
    if (dtype == TL_DT_F32)
        bigram_embedding_kernel<float><<<tokens, 256, 0, stream>>>((const int*)ids, (const float*)table, (float*)out, hidden, vocab, scale,
            (const int*)token_req, (const int*)req_indptr, (const int*)positions, (const int*)slots, (const int*)last_token, (const float*)bigram,
            buckets, mul_prev, mul_cur, copies, copy_stride);
    else if (dtype == TL_DT_BF16)
        bigram_embedding_kernel<bf16_t><<<tokens, 256, 0, stream>>>((const int*)ids, (const bf16_t*)table, (float*)out, hidden, vocab, scale,
            (const int*)token_req, (const int*)req_indptr, (const int*)positions, (const int*)slots, (const int*)last_token, (const bf16_t*)bigram,
            buckets, mul_prev, mul_cur, copies, copy_stride);
    else TL_REQUIRE(false, "bigram_embedding: unknown dtype %d", dtype);
    TL_CHECK_LAUNCH("bigram_embedding");
    last_token_kernel<<<(requests + 63) / 64, 64, 0, stream>>>((const int*)ids, (const int*)req_indptr, (const int*)slots, (int*)last_token, requests);
    TL_CHECK_LAUNCH("last_token");
    return TL_OK;
}

// ------------------------------------------------------------------ rows in pieces of four numbers
__device__ __forceinline__ float4 load4(const float* p) { return *(const float4*)p; }
__device__ __forceinline__ float4 load4(const bf16_t* p) {
    const uint2 t = *(const uint2*)p;
    return make_float4(__uint_as_float(t.x << 16), __uint_as_float(t.x & 0xffff0000u), __uint_as_float(t.y << 16), __uint_as_float(t.y & 0xffff0000u));
}
__device__ __forceinline__ void store4(float* p, float4 v) { *(float4*)p = v; }
__device__ __forceinline__ void store4(bf16_t* p, float4 v) {
    uint2 t;
    t.x = (uint32_t)from_float<bf16_t>(v.x).bits | ((uint32_t)from_float<bf16_t>(v.y).bits << 16);
    t.y = (uint32_t)from_float<bf16_t>(v.z).bits | ((uint32_t)from_float<bf16_t>(v.w).bits << 16);
    *(uint2*)p = t;
}
// Up to four neighbouring numbers: all four at once where rows are multiples of four (VEC 4), one otherwise.
template <int VEC, typename T> __device__ __forceinline__ void load_piece(const T* p, float (&v)[VEC]) {
    if constexpr (VEC == 4) { const float4 f = load4(p); v[0] = f.x; v[1] = f.y; v[2] = f.z; v[3] = f.w; }
    else v[0] = to_float(p[0]);
}
template <int VEC, typename T> __device__ __forceinline__ void store_piece(T* p, const float (&v)[VEC]) {
    if constexpr (VEC == 4) store4(p, make_float4(v[0], v[1], v[2], v[3]));
    else p[0] = from_float<T>(v[0]);
}

// A row of `hidden` numbers (a multiple of four) held by a work-group in registers: piece n of a thread is the four numbers from
// 4 (thread + n * threads) on.  All fetches of a row are requested before the first is used.
template <int NP> struct RowPieces {
    float v[NP][4];
};
template <int NP, typename T>
__device__ __forceinline__ void load_row(const T* p, int hidden, RowPieces<NP>& r) {
#pragma unroll
    for (int n = 0; n < NP; ++n) {
        const int i = 4 * (threadIdx.x + n * blockDim.x);
        if (i < hidden) load_piece<4>(p + i, r.v[n]);
        else { r.v[n][0] = r.v[n][1] = r.v[n][2] = r.v[n][3] = 0.f; }
    }
}
template <int NP, typename T>
__device__ __forceinline__ void store_row(T* p, int hidden, const RowPieces<NP>& r) {
#pragma unroll
    for (int n = 0; n < NP; ++n) {
        const int i = 4 * (threadIdx.x + n * blockDim.x);
        if (i < hidden) store_piece<4>(p + i, r.v[n]);
    }
}
// A branch's output: one row of the activation type, or the sum of `parts` float slabs (four requested at a time, added in their order).
template <int NP, typename T>
__device__ __forceinline__ void load_branch(const void* pending, int parts, size_t part_stride, size_t row_off, int hidden, RowPieces<NP>& y) {
    if (parts == 0) { load_row<NP>((const T*)pending + row_off, hidden, y); return; }
    const float* slab = (const float*)pending + row_off;
#pragma unroll
    for (int n = 0; n < NP; ++n) {
        const int i = 4 * (threadIdx.x + n * blockDim.x);
#pragma unroll
        for (int v = 0; v < 4; ++v) y.v[n][v] = 0.f;
        if (i >= hidden) continue;
        for (int p = 0; p < parts; p += 4) {
            float z[4][4];
#pragma unroll
            for (int u = 0; u < 4; ++u) load_piece<4>(slab + (size_t)min(p + u, parts - 1) * part_stride + i, z[u]);
#pragma unroll
            for (int u = 0; u < 4; ++u)
                if (p + u < parts) {
#pragma unroll
                    for (int v = 0; v < 4; ++v) y.v[n][v] += z[u][v];
                }
        }
    }
}
template <int NP>
__device__ __forceinline__ float row_squares(const RowPieces<NP>& r) {
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < NP; ++n)
#pragma unroll
        for (int v = 0; v < 4; ++v) ss = fmaf(r.v[n][v], r.v[n][v], ss);
    return ss;
}
// The weights of a norm: a vector, or one number for all coordinates.
template <int NP>
__device__ __forceinline__ void load_weights(const float* w, int count, int hidden, RowPieces<NP>& r) {
    if (count != 1) { load_row<NP>(w, hidden, r); return; }
    const float one = w[0];
#pragma unroll
    for (int n = 0; n < NP; ++n)
#pragma unroll
        for (int v = 0; v < 4; ++v) r.v[n][v] = one;
}
// Threads and pieces per thread for a row: up to 1024 threads, then up to three pieces each (12288 numbers).
struct RowPlan { int threads, pieces; };
static RowPlan plan_row(int hidden) {
    const int n = hidden / 4;
    const int threads = n <= 64 ? 64 : n <= 128 ? 128 : n <= 256 ? 256 : n <= 512 ? 512 : 1024;
    return RowPlan{threads, (n + threads - 1) / threads};
}

// ------------------------------------------------------------------ norm of the branch output, addition, norm of the sum
// One block per output row, the row kept in shared memory between the passes:
//   y = pending[row] (one tensor of the activation type, or `parts` float slabs added up);
//   r = residual[row] (+ extra[row]) + y * branch_gain * (post ? rsqrt(mean(y^2) + post_eps) * post[i] : 1);   written back unless `rows` selects
//   out = r * rsqrt(mean(r^2) + eps) * weight[i] * gain, or, without a `weight`, r * gain (the sum itself, in the activation type).
// `post` and `weight` are float vectors of post_n / weight_n numbers: `hidden` of them, or one for all coordinates.
template <typename T>
__global__ void sandwich_norm_kernel(float* __restrict__ residual, const void* __restrict__ pending, int parts, size_t part_stride,
                                     const float* __restrict__ post, int post_n, float post_eps, float branch_gain, const float* __restrict__ extra,
                                     const float* __restrict__ weight, int weight_n, float eps, float gain, T* __restrict__ out,
                                     const int* __restrict__ rows, int hidden) {
    extern __shared__ float sn_row[];
    __shared__ float red[16];
    const int orow = blockIdx.x;
    const int srow = rows ? rows[orow] : orow;
    float* res = residual + (size_t)srow * hidden;
    const T* pen = (pending && parts == 0) ? (const T*)pending + (size_t)srow * hidden : nullptr;
    const float* pparts = (pending && parts > 0) ? (const float*)pending + (size_t)srow * hidden : nullptr;
    const float* ex = extra ? extra + (size_t)srow * hidden : nullptr;
    float inv_y = branch_gain;
    if (pending) {
        float ss = 0.f;
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
            float y = 0.f;
            if (pen) y = to_float(pen[i]);
            if (pparts)
                for (int p = 0; p < parts; ++p) y += pparts[p * part_stride + i];
            sn_row[i] = y;
            ss = fmaf(y, y, ss);
        }
        if (post) inv_y = rsqrtf(block_sum(ss, red) / (float)hidden + post_eps) * branch_gain;
    }
    const bool update = (pending != nullptr || ex != nullptr) && rows == nullptr;
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float r = res[i];
        if (ex) r += ex[i];
        if (pending) r += post ? sn_row[i] * inv_y * post[post_n == 1 ? 0 : i] : sn_row[i] * inv_y;
        if (update) res[i] = r;
        sn_row[i] = r;
        ss = fmaf(r, r, ss);
    }
    T* dst = out + (size_t)orow * hidden;
    if (!weight) {
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = from_float<T>(sn_row[i] * gain);
        return;
    }
    const float inv = rsqrtf(block_sum(ss, red) / (float)hidden + eps) * gain;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = from_float<T>(sn_row[i] * inv * weight[weight_n == 1 ? 0 : i]);
}

// The same with the row in registers (hidden a multiple of four, aligned rows): what the residual, the weights and the branch's slabs hold is
// requested at once, so a decode step's few rows pay one trip to memory.
template <typename T, int NP>
__global__ void __launch_bounds__(1024)
sandwich_norm_rows_kernel(float* __restrict__ residual, const void* __restrict__ pending, int parts, size_t part_stride,
                          const float* __restrict__ post, int post_n, float post_eps, float branch_gain, const float* __restrict__ extra,
                          const float* __restrict__ weight, int weight_n, float eps, float gain, T* __restrict__ out,
                          const int* __restrict__ rows, int hidden) {
    __shared__ float red[16];
    const int srow = rows ? rows[blockIdx.x] : blockIdx.x;
    const size_t at = (size_t)srow * hidden;
    RowPieces<NP> r, y, pw, w, ex;
    load_row<NP>(residual + at, hidden, r);
    if (pending) load_branch<NP, T>(pending, parts, part_stride, at, hidden, y);
    if (pending && post) load_weights<NP>(post, post_n, hidden, pw);
    if (extra) load_row<NP>(extra + at, hidden, ex);
    if (weight) load_weights<NP>(weight, weight_n, hidden, w);
    const float inv_y = branch_gain * (pending && post ? rsqrtf(block_sum(row_squares(y), red) / (float)hidden + post_eps) : 1.f);
#pragma unroll
    for (int n = 0; n < NP; ++n)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            if (extra) r.v[n][v] += ex.v[n][v];
            if (pending) r.v[n][v] += post ? y.v[n][v] * inv_y * pw.v[n][v] : y.v[n][v] * inv_y;
        }
    if ((pending || extra) && !rows) store_row<NP>(residual + at, hidden, r);
    const float inv = weight ? rsqrtf(block_sum(row_squares(r), red) / (float)hidden + eps) * gain : gain;
#pragma unroll
    for (int n = 0; n < NP; ++n)
#pragma unroll
        for (int v = 0; v < 4; ++v) r.v[n][v] = weight ? r.v[n][v] * inv * w.v[n][v] : r.v[n][v] * inv;
    store_row<NP>(out + (size_t)blockIdx.x * hidden, hidden, r);
}

extern "C" int tl_sandwich_norm(void* residual, const void* pending, int parts, int part_rows, const void* post, int post_n, float post_eps,
                                float branch_gain, const void* extra, const void* weight, int weight_n, float eps, float gain, void* out, const void* rows,
                                int out_rows, int hidden, int act_dtype, hipStream_t stream) {
    TL_REQUIRE(parts >= 0 && parts <= 64 && out_rows >= 0 && hidden > 0 && hidden <= 12288, "sandwich_norm: bad sizes rows=%d hidden=%d parts=%d", out_rows, hidden, parts);
    TL_REQUIRE((!weight || weight_n == 1 || weight_n == hidden) && (!post || post_n == 1 || post_n == hidden), "sandwich_norm: weights of one number or of %d", hidden);
    if (out_rows == 0) return TL_OK;
    const size_t part_stride = (size_t)part_rows * hidden, smem = sizeof(float) * hidden;
    TL_REQUIRE(act_dtype == TL_DT_F32 || act_dtype == TL_DT_BF16, "sandwich_norm: unknown dtype %d", act_dtype);
    const uintptr_t bits = (uintptr_t)residual | (uintptr_t)pending | (uintptr_t)post | (uintptr_t)extra | (uintptr_t)weight | (uintptr_t)out;
    if (hidden % 4 == 0 && bits % 16 == 0) {
        const RowPlan plan = plan_row(hidden);
#define TL_SN(T, N)                                                                                                                               \
    sandwich_norm_rows_kernel<T, N><<<out_rows, plan.threads, 0, stream>>>((float*)residual, pending, parts, part_stride, (const float*)post, post_n, post_eps, \
        branch_gain, (const float*)extra, (const float*)weight, weight_n, eps, gain, (T*)out, (const int*)rows, hidden)
#define TL_SN_T(T) if (plan.pieces == 1) TL_SN(T, 1); else if (plan.pieces == 2) TL_SN(T, 2); else TL_SN(T, 3)
        if (act_dtype == TL_DT_F32) { TL_SN_T(float); } else { TL_SN_T(bf16_t); }
#undef TL_SN_T
#undef TL_SN
        TL_CHECK_LAUNCH("sandwich_norm");
        return TL_OK;
    }
    const int threads = hidden >= 2048 ? 512 : 256;
    if (act_dtype == TL_DT_F32)
        sandwich_norm_kernel<float><<<out_rows, threads, smem, stream>>>((float*)residual, pending, parts, part_stride, (const float*)post, post_n, post_eps,
            branch_gain, (const float*)extra, (const float*)weight, weight_n, eps, gain, (float*)out, (const int*)rows, hidden);
    else if (act_dtype == TL_DT_BF16)
        sandwich_norm_kernel<bf16_t><<<out_rows, threads, smem, stream>>>((float*)residual, pending, parts, part_stride, (const float*)post, post_n, post_eps,
            branch_gain, (const float*)extra, (const float*)weight, weight_n, eps, gain, (bf16_t*)out, (const int*)rows, hidden);
    else TL_REQUIRE(false, "sandwich_norm: unknown dtype %d", act_dtype);
    TL_CHECK_LAUNCH("sandwich_norm");
    return TL_OK;
}

// ------------------------------------------------------------------ sum of normed branches
// out[t, :] = sum_b x[b, t, :] * rsqrt(mean(x[b, t, :]^2) + eps) * w[b, :] over `branches` tensors side by side; one block per row, float sums.
#define NS_MAX_BRANCHES 8
template <typename T>
__global__ void normed_sum_kernel(const T* __restrict__ x, int branches, size_t branch_stride, const float* __restrict__ w, float eps,
                                  T* __restrict__ out, int hidden) {
    __shared__ float red[16];
    const int row = blockIdx.x;
    float inv[NS_MAX_BRANCHES];
    for (int b = 0; b < branches; ++b) {
        const T* src = x + b * branch_stride + (size_t)row * hidden;
        float ss = 0.f;
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) { const float v = to_float(src[i]); ss = fmaf(v, v, ss); }
        inv[b] = rsqrtf(block_sum(ss, red) / (float)hidden + eps);
    }
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float y = 0.f;
        for (int b = 0; b < branches; ++b) y = fmaf(to_float(x[b * branch_stride + (size_t)row * hidden + i]) * inv[b], w[(size_t)b * hidden + i], y);
        out[(size_t)row * hidden + i] = from_float<T>(y);
    }
}

extern "C" int tl_normed_sum(const void* x, int branches, int rows, int hidden, const void* w, float eps, void* out, int dtype, hipStream_t stream) {
    TL_REQUIRE(branches > 0 && branches <= NS_MAX_BRANCHES && rows >= 0 && hidden > 0, "normed_sum: bad sizes (up to %d branches)", NS_MAX_BRANCHES);
    if (rows == 0) return TL_OK;
    const size_t stride = (size_t)rows * hidden;
    if (dtype == TL_DT_F32) normed_sum_kernel<float><<<rows, 256, 0, stream>>>((const float*)x, branches, stride, (const float*)w, eps, (float*)out, hidden);
    else if (dtype == TL_DT_BF16) normed_sum_kernel<bf16_t><<<rows, 256, 0, stream>>>((const bf16_t*)x, branches, stride, (const float*)w, eps, (bf16_t*)out, hidden);
    else TL_REQUIRE(false, "normed_sum: unknown dtype %d", dtype);
    TL_CHECK_LAUNCH("normed_sum");
    return TL_OK;
}

// ------------------------------------------------------------------ embedding rows, normed
// out[t, :] = r * rsqrt(mean(r^2) + eps) * weight[:] with r = float(table[ids[t], :]) * scale: a token's row enters the 32-bit stream through a
// root-mean-square norm (weight: `hidden` floats).  One block per token, the row kept in shared memory between the two passes.
template <typename T>
__global__ void embedding_norm_kernel(const int* __restrict__ ids, const T* __restrict__ table, float* __restrict__ out, int hidden, int vocab,
                                      float scale, const float* __restrict__ weight, float eps) {
    extern __shared__ float en_row[];
    __shared__ float red[16];
    const int t = blockIdx.x;
    int id = ids[t];
    if (id < 0 || id >= vocab) id = 0;
    const T* src = table + (size_t)id * hidden;
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float v = to_float(src[i]) * scale;
        en_row[i] = v;
        ss = fmaf(v, v, ss);
    }
    const float inv = rsqrtf(block_sum(ss, red) / (float)hidden + eps);
    float* dst = out + (size_t)t * hidden;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = en_row[i] * inv * weight[i];
}

extern "C" int tl_embedding_norm(const void* ids, const void* table, int table_dtype, void* out, int tokens, int hidden, int vocab, float scale,
                                 const void* weight, float eps, hipStream_t stream) {
    TL_REQUIRE(tokens >= 0 && hidden > 0 && hidden <= 12288 && vocab > 0 && weight, "embedding_norm: bad sizes tokens=%d hidden=%d vocab=%d", tokens, hidden, vocab);
    if (tokens == 0) return TL_OK;
    const size_t smem = sizeof(float) * hidden;
    if (table_dtype == TL_DT_F32)
        embedding_norm_kernel<float><<<tokens, 256, smem, stream>>>((const int*)ids, (const float*)table, (float*)out, hidden, vocab, scale, (const float*)weight, eps);
    else if (table_dtype == TL_DT_BF16)
        embedding_norm_kernel<bf16_t><<<tokens, 256, smem, stream>>>((const int*)ids, (const bf16_t*)table, (float*)out, hidden, vocab, scale, (const float*)weight, eps);
    else TL_REQUIRE(false, "embedding_norm: unknown dtype %d", table_dtype);
    TL_CHECK_LAUNCH("embedding_norm");
    return TL_OK;
}

// ------------------------------------------------------------------ the sum, and mixes of neighbouring tokens
// x_t = residual[t] + y_t * (post ? rsqrt(mean(y_t^2) + post_eps) * post[i] : 1), y_t the pending output (the activation type, or `parts`
// float slabs added up; null: x_t = residual[t]), written to `settled` (another place than the residual: a work-group also reads the row
// before its own first one).  Then, with x' the token before's (of the request's slot, `tail`, for the first token that a request brings),
//   mixes[s][t][i] = x_t[i] + (x'[i] - x_t[i]) * mu[s][i],   s < count.
// A work-group takes `run` neighbouring tokens, row after row, and makes the row before the first of them a second time.  All in float, one
// rounding of the mixes.  Rows of a multiple of four numbers are held in registers; others in shared memory, where a row's numbers stay with
// the threads that made them, so that they need no barrier of their own.
struct ShiftArgs {
    const float* residual;
    float* settled;
    const void* pending;
    int parts;
    size_t part_stride;
    const float* post;
    int post_n;
    float post_eps;
    const float* state;            // the slots: the row of the token before at slot * slot_stride + tail_off
    size_t slot_stride, tail_off;
    const int *slots, *req_indptr, *token_req;
    const float* mu;
    int count, tokens, hidden, run;
};

template <typename T, int NP>
__global__ void __launch_bounds__(1024)
settle_shift_rows_kernel(ShiftArgs a, T* __restrict__ mixes) {
    __shared__ float red[16];
    const int first = blockIdx.x * a.run, last = min(first + a.run, a.tokens) - 1, hidden = a.hidden;
    RowPieces<NP> pw;
    if (a.pending && a.post) load_weights<NP>(a.post, a.post_n, hidden, pw);
    auto settle = [&](int t, RowPieces<NP>& r) {
        const size_t at = (size_t)t * hidden;
        load_row<NP>(a.residual + at, hidden, r);
        if (!a.pending) return;
        RowPieces<NP> y;
        load_branch<NP, T>(a.pending, a.parts, a.part_stride, at, hidden, y);
        const float inv = a.post ? rsqrtf(block_sum(row_squares(y), red) / (float)hidden + a.post_eps) : 1.f;
#pragma unroll
        for (int n = 0; n < NP; ++n)
#pragma unroll
            for (int v = 0; v < 4; ++v) r.v[n][v] += a.post ? y.v[n][v] * inv * pw.v[n][v] : y.v[n][v];
    };
    RowPieces<NP> before, x;
    bool have = false;                                 // `before` holds the row ahead of the one at hand
    for (int t = first; t <= last; ++t) {
        const int req = a.token_req[t];
        if (t == a.req_indptr[req]) {                  // the request's first token of the step: its slot has the row before (anywhere in memory)
            const float* tail = a.state + (size_t)a.slots[req] * a.slot_stride + a.tail_off;
#pragma unroll
            for (int n = 0; n < NP; ++n)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    const int i = 4 * (threadIdx.x + n * blockDim.x) + v;
                    before.v[n][v] = i < hidden ? tail[i] : 0.f;
                }
        } else if (!have) settle(t - 1, before);
        settle(t, x);
        if (a.pending) store_row<NP>(a.settled + (size_t)t * hidden, hidden, x);
        for (int s = 0; s < a.count; ++s) {
            RowPieces<NP> m;
            load_row<NP>(a.mu + (size_t)s * hidden, hidden, m);
#pragma unroll
            for (int n = 0; n < NP; ++n)
#pragma unroll
                for (int v = 0; v < 4; ++v) m.v[n][v] = fmaf(before.v[n][v] - x.v[n][v], m.v[n][v], x.v[n][v]);
            store_row<NP>(mixes + ((size_t)s * a.tokens + t) * hidden, hidden, m);
        }
        before = x;
        have = true;
    }
}

template <typename T>
__global__ void __launch_bounds__(256)
settle_shift_kernel(ShiftArgs a, T* __restrict__ mixes) {
    extern __shared__ float ss_rows[];                 // two rows
    __shared__ float red[16];
    const int first = blockIdx.x * a.run, last = min(first + a.run, a.tokens) - 1, hidden = a.hidden;
    auto settle = [&](int t, float* buf) {
        const size_t at = (size_t)t * hidden;
        float inv = 1.f;
        if (a.pending) {
            float ss = 0.f;
            for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
                float y = 0.f;
                if (a.parts == 0) y = to_float(((const T*)a.pending)[at + i]);
                for (int p = 0; p < a.parts; ++p) y += ((const float*)a.pending)[p * a.part_stride + at + i];
                ss = fmaf(y, y, ss);
                buf[i] = y;
            }
            if (a.post) inv = rsqrtf(block_sum(ss, red) / (float)hidden + a.post_eps);
        }
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
            float r = a.residual[at + i];
            if (a.pending) r += a.post ? buf[i] * inv * a.post[a.post_n == 1 ? 0 : i] : buf[i];
            buf[i] = r;
        }
    };
    float *cur = ss_rows, *before = ss_rows + hidden;
    bool have = false;
    for (int t = first; t <= last; ++t) {
        const int req = a.token_req[t];
        const float* tail = t == a.req_indptr[req] ? a.state + (size_t)a.slots[req] * a.slot_stride + a.tail_off : nullptr;
        if (!tail && !have) settle(t - 1, before);
        settle(t, cur);
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
            const float x = cur[i], b = tail ? tail[i] : before[i];
            if (a.pending) a.settled[(size_t)t * hidden + i] = x;
            for (int s = 0; s < a.count; ++s)
                mixes[((size_t)s * a.tokens + t) * hidden + i] = from_float<T>(fmaf(b - x, a.mu[(size_t)s * hidden + i], x));
        }
        float* other = cur; cur = before; before = other;
        have = true;
    }
}

extern "C" int tl_settle_shift(const void* residual, void* settled, const void* pending, int parts, const void* post, int post_n, float post_eps,
                               const void* state, long slot_stride, long tail_off, const void* slots, const void* req_indptr, const void* token_req,
                               const void* mu, void* mixes, int count, int tokens, int hidden, int act_dtype, hipStream_t stream) {
    TL_REQUIRE(parts >= 0 && parts <= 64 && tokens >= 0 && hidden > 0 && hidden <= 12288 && count > 0, "settle_shift: bad sizes tokens=%d hidden=%d", tokens, hidden);
    TL_REQUIRE(!post || post_n == 1 || post_n == hidden, "settle_shift: a norm weight of one number or of %d", hidden);
    TL_REQUIRE(!pending || settled != residual, "settle_shift: the sum goes to another place than the residual it is made from");
    TL_REQUIRE(tail_off >= 0 && slot_stride >= tail_off + hidden, "settle_shift: the slots do not hold a row of %d numbers", hidden);
    TL_REQUIRE(hidden % 4 == 0 || hidden <= 8000, "settle_shift: rows of a multiple of four numbers, or of up to 8000, not %d", hidden);
    TL_REQUIRE(act_dtype == TL_DT_F32 || act_dtype == TL_DT_BF16, "settle_shift: unknown dtype %d", act_dtype);
    if (tokens == 0) return TL_OK;
    const int run = tokens >= 2048 ? 4 : (tokens >= 768 ? 2 : 1);
    const ShiftArgs a{(const float*)residual, (float*)settled, pending, parts, (size_t)tokens * hidden, (const float*)post, post_n, post_eps,
                      (const float*)state, (size_t)slot_stride, (size_t)tail_off, (const int*)slots, (const int*)req_indptr, (const int*)token_req,
                      (const float*)mu, count, tokens, hidden, run};
    const int grid = (tokens + run - 1) / run;
    const uintptr_t bits = (uintptr_t)residual | (uintptr_t)settled | (uintptr_t)pending | (uintptr_t)post | (uintptr_t)mu | (uintptr_t)mixes;
    if (hidden % 4 == 0 && bits % 16 == 0) {
        const RowPlan plan = plan_row(hidden);
#define TL_SS(T, N) settle_shift_rows_kernel<T, N><<<grid, plan.threads, 0, stream>>>(a, (T*)mixes)
#define TL_SS_T(T) if (plan.pieces == 1) TL_SS(T, 1); else if (plan.pieces == 2) TL_SS(T, 2); else TL_SS(T, 3)
        if (act_dtype == TL_DT_F32) { TL_SS_T(float); } else { TL_SS_T(bf16_t); }
#undef TL_SS_T
#undef TL_SS
    } else {
        const size_t smem = sizeof(float) * 2 * hidden;
        if (act_dtype == TL_DT_F32) settle_shift_kernel<float><<<grid, 256, smem, stream>>>(a, (float*)mixes);
        else settle_shift_kernel<bf16_t><<<grid, 256, smem, stream>>>(a, (bf16_t*)mixes);
    }
    TL_CHECK_LAUNCH("settle_shift");
    return TL_OK;
}
