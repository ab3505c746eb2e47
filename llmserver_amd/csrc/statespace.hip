// What stands around a recurrence with one decay per head: in front of it the short convolution with bias and the step
// sizes of a state-space mixer, or the rotation of queries and keys; behind it the skip, the gate and the norm in parts.
// Step sizes, decays, angles, rotated rows and norms are float32; a convolution's result is rounded once to the
// activations' type.
#include "common.hpp"

using namespace lsa;

namespace {

__device__ inline float silu_of(float z) { return z / (1.f + expf(-z)); }
__device__ inline float softplus_of(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// grid (tiles of TT tokens, blocks of 256 channels and, last, one more).  A channel block: out[t][c] = silu(bias[c] + sum_j
// w[c][j] x[t - TAPS + 1 + j][c]); a thread has one channel of TT tokens, and the rows in front of a token come from the step
// where the step brings them, from state[slot][k][channel] (the request's last TAPS - 1 inputs, oldest first) where it does not,
// and are zeros before the sequence.  TAPS 0: any number of taps (`taps`), read one by one.  keep (steps of one token a row): the
// thread that has read a channel's state moves it on.  The last block: every head's step size dt = softplus(z + dt_bias) and
// log_keep = -exp(A_log) dt.
template <typename T, int TAPS, int TT>
__global__ __launch_bounds__(256) void ssd_prepare_kernel(const T* __restrict__ x, long x_stride, const float* __restrict__ w, int taps,
                                                          const float* __restrict__ bias, float* state, long state_stride,
                                                          const int* __restrict__ slots, const int* __restrict__ token_row,
                                                          const int* __restrict__ positions, const int* __restrict__ row_start,
                                                          T* __restrict__ out, int channels, int keep, const T* __restrict__ dt, long dt_stride,
                                                          const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                                                          float* __restrict__ steps, float* __restrict__ log_keep, int heads, int n_tokens) {
    const int t0 = blockIdx.x * TT;
    if (blockIdx.y == gridDim.y - 1) {
        for (int i = threadIdx.x; i < TT * heads; i += blockDim.x) {
            const int t = t0 + i / heads, head = i % heads;
            if (t >= n_tokens) break;
            const float step = softplus_of((float)dt[(size_t)t * dt_stride + head] + dt_bias[head]);
            steps[(size_t)t * heads + head] = step;
            log_keep[(size_t)t * heads + head] = -expf(a_log[head]) * step;
        }
        return;
    }
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= channels) return;
    const int count = TAPS > 0 ? TAPS : taps, kept = count - 1;
    constexpr int AHEAD = TAPS > 0 ? TAPS - 1 : 0;
    float own[TT + AHEAD], tap[TAPS > 0 ? TAPS : 1];
    // (every load is of a row that is there, so that none stands under a condition and all are on their way together)
#pragma unroll
    for (int i = 0; i < TT + AHEAD; ++i) {
        const int t = min(max(t0 - AHEAD + i, 0), n_tokens - 1);
        own[i] = (float)x[(size_t)t * x_stride + c];
    }
    if constexpr (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) tap[j] = w[(size_t)c * TAPS + j];
    }
    const float shift = bias ? bias[c] : 0.f;
#pragma unroll
    for (int i = 0; i < TT; ++i) {
        const int t = t0 + i;
        if (t >= n_tokens) break;
        const int row = token_row[t], position = positions[t], first = row_start[row];
        float* mine = kept ? state + (size_t)slots[row] * state_stride + c : nullptr;
        float acc = shift;
        auto before = [&](int back) {                    // an input from in front of the row's first token of this step
            return position - back >= 0 ? mine[(size_t)(kept - (first - (t - back))) * channels] : 0.f;
        };
        if constexpr (TAPS > 0) {
            float value[TAPS];
#pragma unroll
            for (int j = 0; j < TAPS; ++j) {
                const int back = TAPS - 1 - j;
                value[j] = own[i + j];
                if (t - back < first) value[j] = before(back);
            }
#pragma unroll
            for (int j = 0; j < TAPS; ++j) acc = __builtin_fmaf(tap[j], value[j], acc);
        } else {
            for (int j = 0; j < count; ++j) {
                const int back = count - 1 - j;
                const float value = t - back >= first ? (float)x[(size_t)(t - back) * x_stride + c] : before(back);
                acc = __builtin_fmaf(w[(size_t)c * count + j], value, acc);
            }
        }
        out[(size_t)t * channels + c] = (T)silu_of(acc);
        if (keep) {
            for (int k = 0; k + 1 < kept; ++k) mine[(size_t)k * channels] = position > 0 ? mine[(size_t)(k + 1) * channels] : 0.f;
            if (kept) mine[(size_t)(kept - 1) * channels] = own[i + AHEAD];
        }
    }
}

// grid (tokens, groups): out = u / rms(u) * weight over each of `groups` equal parts of a token's row, with
// u = (y + skip[head] x) * silu(gate), head = channel / value_dim; y float32.  Parts of up to 256 * COLS channels keep their
// u in registers between the sum of squares and the result; longer ones (COLS 0) form them twice.
template <typename T, int COLS>
__global__ __launch_bounds__(256) void gated_group_norm_kernel(const float* __restrict__ y, const T* __restrict__ x, long x_stride,
                                                               const float* __restrict__ skip, const T* __restrict__ gate, long gate_stride,
                                                               const float* __restrict__ weight, float eps, T* __restrict__ out, int part,
                                                               int value_dim, int width) {
    __shared__ float scratch[16];
    const size_t t = blockIdx.x;
    const int base = blockIdx.y * part;
    auto gated = [&](int c) {
        const float z = (float)gate[t * gate_stride + c];
        return (y[t * width + c] + skip[c / value_dim] * (float)x[t * x_stride + c]) * silu_of(z);
    };
    float sq = 0.f;
    if constexpr (COLS > 0) {
        float u[COLS], w[COLS];
#pragma unroll
        for (int n = 0; n < COLS; ++n) {
            const int c = base + min((int)threadIdx.x + 256 * n, part - 1);
            u[n] = gated(c);
            w[n] = weight[c];
        }
#pragma unroll
        for (int n = 0; n < COLS; ++n)
            if ((int)threadIdx.x + 256 * n < part) sq += u[n] * u[n];
        const float inv = rsqrtf(block_sum(sq, scratch) / (float)part + eps);
#pragma unroll
        for (int n = 0; n < COLS; ++n) {
            const int c = threadIdx.x + 256 * n;
            if (c < part) out[t * width + base + c] = (T)(u[n] * inv * w[n]);
        }
        return;
    }
    for (int c = threadIdx.x; c < part; c += 256) {
        const float u = gated(base + c);
        sq += u * u;
    }
    const float inv = rsqrtf(block_sum(sq, scratch) / (float)part + eps);
    for (int c = threadIdx.x; c < part; c += 256) out[t * width + base + c] = (T)(gated(base + c) * inv * weight[base + c]);
}

// grid (tokens, blocks of 256 of a token's 2 * width numbers: its queries, then its keys).  Dimension i < pairs of every head turns
// with dimension i + pairs by the token's angle (cos_sin [T][cosines, sines]; pairs 0: nothing turns), dimensions from
// 2 * pairs on pass unchanged; keys are multiplied by key_scale afterwards.  The results are float32.
template <typename T>
__global__ __launch_bounds__(256) void rotate_heads_kernel(const T* __restrict__ q, long q_stride, const T* __restrict__ k, long k_stride,
                                                           const float* __restrict__ cos_sin, int pairs, float key_scale,
                                                           float* __restrict__ out_q, float* __restrict__ out_k, int dim, int width) {
    const size_t t = blockIdx.x;
    const int i = blockIdx.y * 256 + threadIdx.x;
    if (i >= 2 * width) return;
    const bool key = i >= width;
    const int c = key ? i - width : i, e = c % dim;
    const T* row = (key ? k + t * k_stride : q + t * q_stride) + c;
    float value = (float)row[0];
    if (e < 2 * pairs) {
        const bool low = e < pairs;
        const int pair = low ? e : e - pairs;
        const float other = (float)row[low ? pairs : -pairs];
        const float cosine = cos_sin[t * 2 * pairs + pair], sine = cos_sin[t * 2 * pairs + pairs + pair];
        value = low ? value * cosine - other * sine : value * cosine + other * sine;
    }
    (key ? out_k : out_q)[t * width + c] = key ? value * key_scale : value;
}

}  // namespace

LSA_EXPORT int lsa_ssd_prepare(int code, const void* x, long x_stride, const float* w, int taps, const float* bias, float* state,
                               long state_stride, const int* slots, const int* token_row, const int* positions, const int* row_start, void* out,
                               int channels, int keep, const void* dt, long dt_stride, const float* dt_bias, const float* a_log, float* steps,
                               float* log_keep, int heads, int n_tokens, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (taps < 1 || channels < 1 || heads < 1 || (taps > 1 && (state == nullptr || slots == nullptr))) return -1;
    const bool tiles = n_tokens >= 512;                  // (few tokens: a token a workgroup, which waits for memory once)
    const unsigned blocks = (channels + 255) / 256 + 1;
#define LSA_LAUNCH(T, TAPS, TT) ssd_prepare_kernel<T, TAPS, TT><<<dim3((n_tokens + TT - 1) / TT, blocks), 256, 0, stream>>>((const T*)x, x_stride, w, taps, \
        bias, state, state_stride, slots, token_row, positions, row_start, (T*)out, channels, keep, (const T*)dt, dt_stride, dt_bias, a_log, steps, \
        log_keep, heads, n_tokens)
#define LSA_BY_TAPS(T, TT) switch (taps) { case 1: LSA_LAUNCH(T, 1, TT); break; case 2: LSA_LAUNCH(T, 2, TT); break; case 3: LSA_LAUNCH(T, 3, TT); break; \
        case 4: LSA_LAUNCH(T, 4, TT); break; default: LSA_LAUNCH(T, 0, TT); }
    if (code) { if (tiles) LSA_BY_TAPS(bf16_t, 8) else LSA_BY_TAPS(bf16_t, 1) }
    else { if (tiles) LSA_BY_TAPS(float, 8) else LSA_BY_TAPS(float, 1) }
#undef LSA_BY_TAPS
#undef LSA_LAUNCH
    LSA_LAUNCH_CHECK();
}

LSA_EXPORT int lsa_gated_group_norm(int code, const float* y, const void* x, long x_stride, const float* skip, const void* gate, long gate_stride,
                                    const float* weight, float eps, void* out, int groups, int value_dim, int width, int n_tokens,
                                    hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (groups < 1 || width % groups || value_dim < 1) return -1;
    const int part = width / groups;
#define LSA_LAUNCH(T, COLS) gated_group_norm_kernel<T, COLS><<<dim3(n_tokens, groups), 256, 0, stream>>>(y, (const T*)x, x_stride, skip, (const T*)gate, \
        gate_stride, weight, eps, (T*)out, part, value_dim, width)
#define LSA_BY_COLS(T) do { if (part <= 256) LSA_LAUNCH(T, 1); else if (part <= 512) LSA_LAUNCH(T, 2); else if (part <= 1024) LSA_LAUNCH(T, 4); else if (part <= 2048) LSA_LAUNCH(T, 8); \
        else if (part <= 4096) LSA_LAUNCH(T, 16); else LSA_LAUNCH(T, 0); } while (0)
    if (code) LSA_BY_COLS(bf16_t); else LSA_BY_COLS(float);
#undef LSA_BY_COLS
#undef LSA_LAUNCH
    LSA_LAUNCH_CHECK();
}

LSA_EXPORT int lsa_rotate_heads(int code, const void* q, long q_stride, const void* k, long k_stride, const float* cos_sin, int pairs,
                                float key_scale, float* out_q, float* out_k, int heads, int dim, int n_tokens, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (pairs < 0 || 2 * pairs > dim || (pairs > 0 && cos_sin == nullptr) || heads < 1) return -1;
    const int width = heads * dim;
    const dim3 grid(n_tokens, (2 * width + 255) / 256);
    if (code) rotate_heads_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)q, q_stride, (const bf16_t*)k, k_stride, cos_sin, pairs, key_scale, out_q, out_k, dim, width);
    else rotate_heads_kernel<float><<<grid, 256, 0, stream>>>((const float*)q, q_stride, (const float*)k, k_stride, cos_sin, pairs, key_scale, out_q, out_k, dim, width);
    LSA_LAUNCH_CHECK();
}
