// Shared helpers of the gfx950 kernels: element types, conversions, wavefront reductions.
// Wavefronts are 64 lanes wide; every reduction below is written for that width.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace lsa {

typedef __bf16 bf16_t;

template <typename T> struct Elem;
template <> struct Elem<float> {
    static constexpr int kVec = 4;                       // elements per 16-byte vector
    __device__ static inline float load(const float* p) { return *p; }
    __device__ static inline void store(float* p, float v) { *p = v; }
    __device__ static inline float round(float v) { return v; }
};
template <> struct Elem<bf16_t> {
    static constexpr int kVec = 8;
    __device__ static inline float load(const bf16_t* p) { return (float)(*p); }
    __device__ static inline void store(bf16_t* p, float v) { *p = (bf16_t)v; }
    __device__ static inline float round(float v) { return (float)((bf16_t)v); }
};

// A 16-byte vector of T, loaded and stored as one transaction.
template <typename T> struct alignas(16) Vec16 {
    T v[Elem<T>::kVec];
};

template <typename T>
__device__ inline Vec16<T> load_vec16(const T* p) {
    return *reinterpret_cast<const Vec16<T>*>(p);
}
template <typename T>
__device__ inline void store_vec16(T* p, const Vec16<T>& x) {
    *reinterpret_cast<Vec16<T>*>(p) = x;
}

__device__ inline float wave_sum(float v) {
#pragma unroll
    for (int offset = 32; offset > 0; offset >>= 1) v += __shfl_xor(v, offset, 64);
    return v;
}
__device__ inline float wave_max(float v) {
#pragma unroll
    for (int offset = 32; offset > 0; offset >>= 1) v = fmaxf(v, __shfl_xor(v, offset, 64));
    return v;
}

// Sum over a block of up to 1024 threads; every thread gets the result. `scratch` holds 16 floats.
__device__ inline float block_sum(float v, float* scratch) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = (blockDim.x + 63) >> 6;
    v = wave_sum(v);
    __syncthreads();                      // scratch may still be read from an earlier call
    if (lane == 0) scratch[wave] = v;
    __syncthreads();
    float total = 0.f;
    for (int w = 0; w < waves; ++w) total += scratch[w];   // same order in every thread
    return total;
}

// Puts 64 consecutive tokens of one KV head, staged in LDS as [VT_TOKENS][pitch] with `filled` numbers a token, into their
// pages values[page][kv_head][:][slot], zeros for the dimensions from `filled` to d.  Four slots of one dimension go out at
// a time (8 or 16 bytes) where four tokens are neighbours in one page, which is the rule inside a portion; a page's
// [d][page_size] block is contiguous, so these stores coalesce.  At least 64 threads; whoever wrote the tile need not have waited.
constexpr int VT_TOKENS = 64;
template <typename T>
__device__ __forceinline__ void store_value_tile(const T* tile, int pitch, int token0, int kv_head, int filled, T* __restrict__ values,
                                                 const int* __restrict__ table, int table_stride, const int* __restrict__ token_row,
                                                 const int* __restrict__ positions, int page_size, int n_kv, int d, int n_tokens) {
    __shared__ long group_base[VT_TOKENS / 4];             // element offset of the group's first slot in `values`, or -1
    __shared__ unsigned char covered[VT_TOKENS];           // token goes out with its group
    // Four tokens go out together if they are one request's neighbours starting at a position that is a multiple
    // of four; the groups are laid so that this holds when the tile lies inside one portion.
    const int shift = (4 - (positions[min(token0, n_tokens - 1)] & 3)) & 3;
    if (threadIdx.x < VT_TOKENS) covered[threadIdx.x] = 0;
    __syncthreads();
    if (threadIdx.x < VT_TOKENS / 4) {
        const int local = shift + 4 * threadIdx.x, first = token0 + local;
        long base = -1;
        if (local + 3 < VT_TOKENS && first + 3 < n_tokens) {
            const int row = token_row[first], pos = positions[first];
            bool together = (pos & 3) == 0;
            for (int r = 1; r < 4; ++r) together = together && token_row[first + r] == row && positions[first + r] == pos + r;
            const int p = table[(size_t)row * table_stride + pos / page_size];
            if (together && p >= 0) {
                base = (((long)p * n_kv + kv_head) * d) * page_size + pos % page_size;
                for (int r = 0; r < 4; ++r) covered[local + r] = 1;
            }
        }
        group_base[threadIdx.x] = base;
    }
    __syncthreads();
    for (int e = threadIdx.x; e < (VT_TOKENS / 4) * d; e += blockDim.x) {
        const int g = e & (VT_TOKENS / 4 - 1), i = e / (VT_TOKENS / 4);      // neighbouring threads: neighbouring groups of slots
        const long base = group_base[g];
        if (base < 0) continue;
        T four[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) four[r] = i < filled ? tile[(shift + 4 * g + r) * pitch + i] : (T)0.f;
        T* dst = values + base + (size_t)i * page_size;
        if (sizeof(T) == 2) *reinterpret_cast<uint2*>(dst) = *reinterpret_cast<const uint2*>(four);
        else *reinterpret_cast<uint4*>(dst) = *reinterpret_cast<const uint4*>(four);
    }
    for (int e = threadIdx.x; e < VT_TOKENS * d; e += blockDim.x) {                  // the tokens that are in no such group
        const int t = e & (VT_TOKENS - 1), i = e / VT_TOKENS;
        const int token = token0 + t;
        if (covered[t] || token >= n_tokens) continue;
        const int pos = positions[token];
        const int p = table[(size_t)token_row[token] * table_stride + pos / page_size];
        if (p >= 0) values[(((size_t)p * n_kv + kv_head) * d + i) * page_size + pos % page_size] = i < filled ? tile[t * pitch + i] : (T)0.f;
    }
}

}  // namespace lsa

#define LSA_EXPORT extern "C" __attribute__((visibility("default")))
#define LSA_LAUNCH_CHECK() return (int)hipGetLastError()
