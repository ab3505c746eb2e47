// Per-head q/k RMSNorm, rotate-half rotation and the write of new keys and values into their
// pages, for all tokens of the step (portions of prompts and decoded tokens alike).
//
// rotary_table: cos and sin of position * inv_freq, times a constant, for every token of the step, once per step
//   (the angles depend on the token and the pair of dimensions only, not on the layer or head).
// qk_norm_rope_kv_write: d / 16 lanes per (token, head), vector accesses throughout.  q heads are
//   normalised, rotated and written back in place into the projection buffer; k heads are
//   normalised, rotated and stored at keys[page][kv_head][slot][:]; v heads are stored transposed
//   at values[page][kv_head][:][slot].  The page of a token is table[row][position / page_size];
//   nothing is allocated here.
//   For long portions, the v heads go through LDS in tiles of 64 tokens so that the transposed stores of
//   neighbouring tokens (neighbouring slots of a page) coalesce: further workgroups of the same launch.
// Norm sums, angles, cos/sin and the rotation are 32-bit; results are rounded once.
#include "common.hpp"

using namespace lsa;

__global__ void rotary_table_kernel(const int* __restrict__ positions, const float* __restrict__ inv_freq,
                                    float* __restrict__ cos_sin, int half, int n_tokens, float amplitude) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n_tokens * half) return;
    const int token = i / half, pair = i % half;
    const float angle = (float)positions[token] * inv_freq[pair];
    cos_sin[(size_t)token * 2 * half + pair] = amplitude * cosf(angle);
    cos_sin[(size_t)token * 2 * half + half + pair] = amplitude * sinf(angle);
}

// A (token, head) pair is handled by d / 16 neighbouring lanes: lane j of them owns dimensions
// [8j, 8j + 8) of the first half and their rotation partners [d/2 + 8j, d/2 + 8j + 8), both as one
// vector load, so a wavefront covers 64 / (d / 16) pairs at once and every access is 16 bytes or more.
template <typename T> struct Eight {
    float v[8];
};
template <typename T>
__device__ inline Eight<T> load8(const T* p) {
    Eight<T> r;
    if (sizeof(T) == 2) {
        const Vec16<T> x = load_vec16(p);
#pragma unroll
        for (int e = 0; e < 8; ++e) r.v[e] = (float)x.v[e];
    } else {
        const Vec16<T> x = load_vec16(p), y = load_vec16(p + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            r.v[e] = (float)x.v[e];
            r.v[4 + e] = (float)y.v[e];
        }
    }
    return r;
}
template <typename T>
__device__ inline void store8(T* p, const float (&v)[8]) {
    if (sizeof(T) == 2) {
        Vec16<T> x;
#pragma unroll
        for (int e = 0; e < 8; ++e) x.v[e] = (T)v[e];
        store_vec16(p, x);
    } else {
        Vec16<T> x, y;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            x.v[e] = (T)v[e];
            y.v[e] = (T)v[4 + e];
        }
        store_vec16(p, x);
        store_vec16(p + 4, y);
    }
}

template <typename T>
__device__ __forceinline__ void qk_norm_rope_kv_write_block(
    const int block,
    T* __restrict__ qkv,                 // [tokens, (Hq + 2 Hkv) * d]
    T* __restrict__ keys,                // [pages, Hkv, page_size, d]
    T* __restrict__ values,              // [pages, Hkv, d, page_size]
    const int* __restrict__ table, int table_stride,
    const int* __restrict__ token_row, const int* __restrict__ positions,
    const float* __restrict__ q_weight, const float* __restrict__ k_weight, float eps,
    const float* __restrict__ cos_sin,   // [tokens, d] (cos of the d/2 pairs, then sin) or nullptr
    int page_size, int n_q, int n_kv, int d, int write_cache, int n_heads, int n_tokens) {
    const int lanes_per_pair = d >> 4, pairs_per_wave = 64 / lanes_per_pair;
    const int lane = threadIdx.x & 63, wave = block * 4 + (threadIdx.x >> 6);
    const int slot_in_wave = lane / lanes_per_pair, j = lane % lanes_per_pair;
    const long pair = (long)wave * pairs_per_wave + slot_in_wave;
    const bool active = slot_in_wave < pairs_per_wave && pair < (long)n_tokens * n_heads;
    const int token = active ? (int)(pair / n_heads) : 0, head = active ? (int)(pair % n_heads) : 0;
    const int half = d >> 1;
    const bool is_q = head < n_q, is_k = !is_q && head < n_q + n_kv;
    T* src = qkv + (size_t)token * (n_q + 2 * n_kv) * d + (size_t)head * d;
    const Eight<T> lo = load8(src + 8 * j), hi = load8(src + half + 8 * j);
    // Sum of squares of the head over its lanes (every lane of the wavefront takes part in the shuffles).
    float sq = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) sq += lo.v[e] * lo.v[e] + hi.v[e] * hi.v[e];
    float total = 0.f;
    const int first_lane = lane - j;
    for (int other = 0; other < lanes_per_pair; ++other) total += __shfl(sq, first_lane + other, 64);
    if (!active || (!is_q && !write_cache)) return;
    size_t page = 0;
    int slot = 0;
    if (!is_q) {
        const int pos = positions[token];
        const int p = table[(size_t)token_row[token] * table_stride + pos / page_size];
        if (p < 0) return;               // the host never schedules a token without a page
        page = (size_t)p;
        slot = pos % page_size;
    }
    if (!is_q && !is_k) {                // value head: copy, transposed
        T* dst = values + ((page * n_kv + (head - n_q - n_kv)) * d) * page_size + slot;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            dst[(size_t)(8 * j + e) * page_size] = (T)lo.v[e];
            dst[(size_t)(half + 8 * j + e) * page_size] = (T)hi.v[e];
        }
        return;
    }
    const float* w = is_q ? q_weight : k_weight;
    float x1[8], x2[8];
    if (w) {
        const float rstd = rsqrtf(total / (float)d + eps);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            x1[e] = lo.v[e] * rstd * w[8 * j + e];
            x2[e] = hi.v[e] * rstd * w[half + 8 * j + e];
        }
    } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            x1[e] = lo.v[e];
            x2[e] = hi.v[e];
        }
    }
    if (cos_sin) {
        const float* cs = cos_sin + (size_t)token * d + 8 * j;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float c = cs[e], s = cs[half + e];
            const float r1 = x1[e] * c - x2[e] * s, r2 = x2[e] * c + x1[e] * s;
            x1[e] = r1;
            x2[e] = r2;
        }
    }
    T* dst = is_q ? src : keys + ((page * n_kv + (head - n_q)) * page_size + slot) * d;
    store8(dst + 8 * j, x1);
    store8(dst + half + 8 * j, x2);
}

// Values of long portions: a workgroup takes 64 consecutive tokens of one KV head through LDS, reads
// them from the projection in 16-byte pieces and writes them transposed (store_value_tile).
template <typename T>
__device__ __forceinline__ void value_tiles_block(
    const int tile_index, const int kv_head, unsigned char* tile_bytes,          // tile_bytes: [VT_TOKENS][d + VEC] elements of T in LDS
    const T* __restrict__ qkv, T* __restrict__ values, const int* __restrict__ table, int table_stride,
    const int* __restrict__ token_row, const int* __restrict__ positions, int page_size, int n_q, int n_kv, int d, int n_tokens) {
    constexpr int VEC = Elem<T>::kVec;
    T* tile = reinterpret_cast<T*>(tile_bytes);
    const int token0 = tile_index * VT_TOKENS;
    const int pitch = d + VEC;
    const int width = (n_q + 2 * n_kv) * d;
    const int pieces = d / VEC;
    for (int e = threadIdx.x; e < VT_TOKENS * pieces; e += 256) {
        const int t = e / pieces, part = e % pieces;
        if (token0 + t < n_tokens)
            store_vec16(tile + t * pitch + part * VEC,
                        load_vec16(qkv + (size_t)(token0 + t) * width + (size_t)(n_q + n_kv + kv_head) * d + part * VEC));
    }
    store_value_tile(tile, pitch, token0, kv_head, d, values, table, table_stride, token_row, positions, page_size, n_kv, d, n_tokens);
}

// One launch for both: the first `qk_blocks` workgroups take the (token, head) pairs of the q and k heads (and of the v
// heads, unless these go in tiles), the others a tile of 64 tokens of one KV head's values each.
template <typename T>
__global__ __launch_bounds__(256) void qk_norm_rope_kv_write_kernel(
    T* __restrict__ qkv, T* __restrict__ keys, T* __restrict__ values, const int* __restrict__ table, int table_stride,
    const int* __restrict__ token_row, const int* __restrict__ positions, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, float eps, const float* __restrict__ cos_sin, int page_size, int n_q, int n_kv, int d,
    int write_cache, int n_heads, int n_tokens, int qk_blocks) {
    extern __shared__ unsigned char tile_bytes[];          // (none unless values go in tiles)
    if ((int)blockIdx.x < qk_blocks) {
        qk_norm_rope_kv_write_block<T>((int)blockIdx.x, qkv, keys, values, table, table_stride, token_row, positions, q_weight, k_weight, eps,
                                       cos_sin, page_size, n_q, n_kv, d, write_cache, n_heads, n_tokens);
        return;
    }
    const int tile = ((int)blockIdx.x - qk_blocks) / n_kv, kv_head = ((int)blockIdx.x - qk_blocks) % n_kv;
    value_tiles_block<T>(tile, kv_head, tile_bytes, qkv, values, table, table_stride, token_row, positions, page_size, n_q, n_kv, d, n_tokens);
}

template <typename T>
static int launch(void* qkv, void* keys, void* values, const int* table, int table_stride, const int* token_row,
                  const int* positions, const float* q_weight, const float* k_weight, float eps, const float* cos_sin,
                  int page_size, int n_q, int n_kv, int d, int write_cache, int n_tokens, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    // Long portions: the v heads take the tiled path, the main kernel then covers q and k heads only.
    const bool tiled_values = write_cache && n_tokens >= 4 * VT_TOKENS;
    const int n_heads = tiled_values ? n_q + n_kv : n_q + 2 * n_kv;
    if (d % 16 != 0 || d > 1024) return -1;
    const long pairs = (long)n_tokens * n_heads;
    const int pairs_per_block = 4 * (64 / (d / 16));
    const long qk_blocks = (pairs + pairs_per_block - 1) / pairs_per_block;
    const long value_blocks = tiled_values ? (long)((n_tokens + VT_TOKENS - 1) / VT_TOKENS) * n_kv : 0;
    if (qk_blocks + value_blocks > 0x7fffffffL) return -1;
    const size_t tile_bytes = tiled_values ? (size_t)VT_TOKENS * (d + Elem<T>::kVec) * sizeof(T) : 0;
    qk_norm_rope_kv_write_kernel<T><<<dim3((unsigned)(qk_blocks + value_blocks)), 256, tile_bytes, stream>>>(
        (T*)qkv, (T*)keys, (T*)values, table, table_stride, token_row, positions, q_weight, k_weight, eps, cos_sin, page_size,
        n_q, n_kv, d, write_cache, n_heads, n_tokens, (int)qk_blocks);
    LSA_LAUNCH_CHECK();
}

LSA_EXPORT int lsa_rotary_table(const int* positions, const float* inv_freq, float* cos_sin, int half, int n_tokens, float amplitude, hipStream_t stream) {
    const int total = n_tokens * half;
    if (total <= 0) return 0;
    rotary_table_kernel<<<(total + 255) / 256, 256, 0, stream>>>(positions, inv_freq, cos_sin, half, n_tokens, amplitude);
    LSA_LAUNCH_CHECK();
}

LSA_EXPORT int lsa_qk_norm_rope_kv_write(int dtype, void* qkv, void* keys, void* values, const int* table, int table_stride,
                                         const int* token_row, const int* positions, const float* q_weight,
                                         const float* k_weight, float eps, const float* cos_sin, int page_size, int n_q,
                                         int n_kv, int d, int write_cache, int n_tokens, hipStream_t stream) {
    return dtype ? launch<bf16_t>(qkv, keys, values, table, table_stride, token_row, positions, q_weight, k_weight, eps,
                                  cos_sin, page_size, n_q, n_kv, d, write_cache, n_tokens, stream)
                 : launch<float>(qkv, keys, values, table, table_stride, token_row, positions, q_weight, k_weight, eps,
                                 cos_sin, page_size, n_q, n_kv, d, write_cache, n_tokens, stream);
}

// ------------------------------------------------------------------------------------------
// The general way of preparing queries, keys and values: heads of any size, values of another size than the keys,
// a rotation of neighbouring pairs (2i, 2i + 1) on the first 2 * pairs dimensions of a head, rows filled up with zeros
// to the head size D of the pages and the attention kernels.  grid (tokens, n_q + n_kv), one wavefront per (token,
// head): a query head writes its row of out_q, a key/value head its key row and its value row (transposed) into the
// token's place in the pages.  qkv row: n_q x dim queries, n_kv x dim keys, n_kv x value_dim values.
template <typename T>
__global__ __launch_bounds__(64) void qkv_prepare_kernel(const T* __restrict__ qkv, long stride, T* __restrict__ keys, T* __restrict__ values,
                                                         const int* __restrict__ table, int table_stride, const int* __restrict__ token_row,
                                                         const int* __restrict__ positions, const float* __restrict__ q_weight,
                                                         const float* __restrict__ k_weight, float eps, const float* __restrict__ cos_sin,
                                                         int pairs, int page_size, int n_q, int n_kv, int dim, int value_dim, int D,
                                                         T* __restrict__ out_q, int write_cache, int halves, int value_share) {
    const int t = blockIdx.x, head = blockIdx.y, lane = threadIdx.x;
    const bool is_query = head < n_q;
    if (!is_query && !write_cache) return;
    const T* src = qkv + (size_t)t * stride + (size_t)head * dim;             // (keys follow the queries, head by head)
    const float* weight = is_query ? q_weight : k_weight;
    float inv = 1.f;
    if (weight) {
        float sq = 0.f;
        for (int e = lane; e < dim; e += 64) {
            const float v = (float)src[e];
            sq += v * v;
        }
        inv = rsqrtf(wave_sum(sq) / (float)dim + eps);
    }
    const float* cs = cos_sin ? cos_sin + (size_t)t * 2 * pairs : nullptr;
    auto prepared = [&](int e) -> float {
        if (e >= dim) return 0.f;
        auto normed = [&](int i) { return weight ? (float)src[i] * inv * weight[i] : (float)src[i]; };
        if (!cs || e >= 2 * pairs) return normed(e);
        if (halves) {                                      // dimension i turns with dimension i + pairs
            const int pair = e < pairs ? e : e - pairs;
            const float u = normed(pair), w = normed(pair + pairs), c = cs[pair], s = cs[pairs + pair];
            return e < pairs ? u * c - w * s : w * c + u * s;
        }
        const int pair = e >> 1;
        const float u = normed(2 * pair), w = normed(2 * pair + 1), c = cs[pair], s = cs[pairs + pair];
        return (e & 1) ? w * c + u * s : u * c - w * s;
    };
    if (is_query) {
        T* o = out_q + ((size_t)t * n_q + head) * D;
        for (int e = lane; e < D; e += 64) o[e] = (T)prepared(e);
        return;
    }
    const int kv = head - n_q;
    const int position = positions[t];
    const int page = table[(size_t)token_row[t] * table_stride + position / page_size], slot = position % page_size;
    if (page < 0) return;
    T* key = keys + (((size_t)page * n_kv + kv) * page_size + slot) * D;
    T* value = values + ((size_t)page * n_kv + kv) * D * page_size + slot;
    // (value_share neighbouring key heads read one value head: the projection has n_kv / value_share of them)
    const T* v = qkv + (size_t)t * stride + (size_t)(n_q + n_kv) * dim + (size_t)(kv / value_share) * value_dim;
    for (int e = lane; e < D; e += 64) {
        key[e] = (T)prepared(e);
        value[(size_t)e * page_size] = e < value_dim ? v[e] : (T)0.f;
    }
}

LSA_EXPORT int lsa_qkv_prepare(int dtype, const void* qkv, long stride, void* keys, void* values, const int* table, int table_stride,
                               const int* token_row, const int* positions, const float* q_weight, const float* k_weight, float eps,
                               const float* cos_sin, int pairs, int page_size, int n_q, int n_kv, int dim, int value_dim, int D,
                               void* out_q, int write_cache, int n_tokens, int halves, int value_share, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (value_share < 1 || n_kv % value_share) return -1;
    if (dim > D || value_dim > D || 2 * pairs > dim || page_size <= 0 || (q_weight == nullptr) != (k_weight == nullptr)) return -1;
    dim3 grid(n_tokens, n_q + n_kv);
#define LSA_LAUNCH(T) qkv_prepare_kernel<T><<<grid, 64, 0, stream>>>((const T*)qkv, stride, (T*)keys, (T*)values, table, table_stride, token_row, \
        positions, q_weight, k_weight, eps, cos_sin, pairs, page_size, n_q, n_kv, dim, value_dim, D, (T*)out_q, write_cache, halves, value_share)
    if (dtype) LSA_LAUNCH(bf16_t); else LSA_LAUNCH(float);
#undef LSA_LAUNCH
    LSA_LAUNCH_CHECK();
}
