// From the product of a step's tokens to what attention reads, where more than a norm and a rotation per head lies between:
// a causal convolution over time on every channel of queries, keys and values, a norm over each head or over the whole
// projection, a rotation, and values that are mixed with those of another layer.  Rows of queries and keys stay in LDS in
// float32 between the convolution, the norm and the rotation; results are rounded once when they are stored.
//
// qkv_compose: workgroups 0 .. 2 T - 1 take a token's queries (even) or keys (odd): pass 1 forms the convolved row in LDS and
// its sum(s) of squares, pass 2 normalises, turns and stores eight outputs a thread, zeros behind a head's dimensions up to the
// pages' head size.  The workgroups behind those take values: a token's row each, stored where it belongs number by number
// (steps of few tokens), or 64 tokens of one KV head each, through LDS, so that neighbouring slots of a page go out together.
#include "common.hpp"

using namespace lsa;

namespace {

// Where a token stands: its request's row, its place in it, and the request's last inputs of earlier steps.
struct Place {
    int row, position, behind;          // behind: tokens of the same row that this step brings before it
    float* state;                       // [taps - 1][channels], oldest first, or nullptr
};

struct Taps {
    const float* w;                     // [taps][channels], or nullptr: no convolution
    int taps, channels;
    float* state;
    long state_stride;
    const int* slots;
    const int* token_row;
    const int* positions;
    const int* row_start;
    int keep;                           // a step of one token a row: the thread that has read a channel's state moves it on
};

__device__ __forceinline__ Place place_of(const Taps& c, int t) {
    Place p;
    p.row = c.token_row[t];
    p.position = c.positions[t];
    p.behind = t - c.row_start[p.row];
    p.state = c.w && c.taps > 1 ? c.state + (size_t)c.slots[p.row] * c.state_stride : nullptr;
    return p;
}

template <typename T, int V> struct alignas(V * sizeof(T)) Piece { T v[V]; };
template <int V> struct alignas(V * 4 > 16 ? 16 : V * 4) Floats { float v[V]; };

// V neighbouring channels from `c` on of token t, convolved over the token's request.
template <typename T, int V>
__device__ __forceinline__ void convolved(const T* __restrict__ qkv, long stride, int t, int c, const Taps& conv, const Place& place, float (&out)[V]) {
    const Piece<T, V> own = *reinterpret_cast<const Piece<T, V>*>(qkv + (size_t)t * stride + c);
    if (!conv.w) {
#pragma unroll
        for (int v = 0; v < V; ++v) out[v] = (float)own.v[v];
        return;
    }
    const int kept = conv.taps - 1;
    const Floats<V> last = *reinterpret_cast<const Floats<V>*>(conv.w + (size_t)kept * conv.channels + c);
#pragma unroll
    for (int v = 0; v < V; ++v) out[v] = last.v[v] * (float)own.v[v];
    const int in_step = min(kept, place.behind);
#pragma unroll 3
    for (int back = 1; back <= in_step; ++back) {
        const Floats<V> w = *reinterpret_cast<const Floats<V>*>(conv.w + (size_t)(kept - back) * conv.channels + c);
        const Piece<T, V> u = *reinterpret_cast<const Piece<T, V>*>(qkv + (size_t)(t - back) * stride + c);
#pragma unroll
        for (int v = 0; v < V; ++v) out[v] = __builtin_fmaf(w.v[v], (float)u.v[v], out[v]);
    }
    const int before = min(kept, place.position);                      // (places before the sequence are zeros)
#pragma unroll 3
    for (int back = in_step + 1; back <= before; ++back) {
        const Floats<V> w = *reinterpret_cast<const Floats<V>*>(conv.w + (size_t)(kept - back) * conv.channels + c);
        const Floats<V> u = *reinterpret_cast<const Floats<V>*>(place.state + (size_t)(kept - (back - place.behind)) * conv.channels + c);
#pragma unroll
        for (int v = 0; v < V; ++v) out[v] = __builtin_fmaf(w.v[v], u.v[v], out[v]);
    }
    if (conv.keep && kept) {
        for (int k = 0; k + 1 < kept; ++k)
            *reinterpret_cast<Floats<V>*>(place.state + (size_t)k * conv.channels + c) =
                *reinterpret_cast<const Floats<V>*>(place.state + (size_t)(k + 1) * conv.channels + c);
        Floats<V> mine;
#pragma unroll
        for (int v = 0; v < V; ++v) mine.v[v] = (float)own.v[v];
        *reinterpret_cast<Floats<V>*>(place.state + (size_t)(kept - 1) * conv.channels + c) = mine;
    }
}

struct Heads {
    int n_q, n_kv, dim, value_dim, D, page_size, table_stride;
    const int* table;
    const float* q_weight;              // [dim] or [heads * dim] (`whole`), or nullptr
    const float* k_weight;
    float eps;
    int normed, whole;                  // a norm over each head, or over the whole projection
    const float* cos_sin;               // [tokens][2 * pairs], cosines then sines, or nullptr
    int pairs, halves;
    float mix;
    long first_stride;
};

constexpr int MOST_HEADS = 512, MOST_WIDTH = 14336;       // heads of a token, and numbers of their rows, that are kept in LDS
constexpr size_t MOST_BYTES = 4 * MOST_WIDTH;

template <typename T, int V>
__global__ __launch_bounds__(256) void qkv_compose_kernel(const T* __restrict__ qkv, long stride, Taps conv, Heads h, T* __restrict__ keys,
                                                          T* __restrict__ values, T* __restrict__ out_q, const T* __restrict__ first,
                                                          T* __restrict__ own_values, int n_tokens, int tiled_values) {
    extern __shared__ __align__(16) unsigned char lds_bytes[];
    __shared__ float scratch[16];
    __shared__ float inverse[MOST_HEADS];
    const int q_width = h.n_q * h.dim, k_width = h.n_kv * h.dim, v_width = h.n_kv * h.value_dim, at_values = q_width + k_width;
    const int block = blockIdx.x, threads = blockDim.x;
    if (block < 2 * n_tokens) {
        const int t = block >> 1, is_key = block & 1;
        const int base = is_key ? q_width : 0, width = is_key ? k_width : q_width, heads = is_key ? h.n_kv : h.n_q;
        float* row = reinterpret_cast<float*>(lds_bytes);
        const Place place = place_of(conv, t);
        T* target = out_q + (size_t)t * h.n_q * h.D;
        if (is_key) {
            const int page = h.table[(size_t)place.row * h.table_stride + place.position / h.page_size];
            target = page < 0 ? nullptr : keys + ((size_t)page * h.n_kv * h.page_size + place.position % h.page_size) * h.D;
        }
        float sq = 0.f;
        for (int c = threadIdx.x * V; c < width; c += threads * V) {
            float x[V];
            convolved<T, V>(qkv, stride, t, base + c, conv, place, x);
#pragma unroll
            for (int v = 0; v < V; ++v) sq += x[v] * x[v];
            Floats<V> piece;
#pragma unroll
            for (int v = 0; v < V; ++v) piece.v[v] = x[v];
            *reinterpret_cast<Floats<V>*>(row + c) = piece;
        }
        float all = 1.f;
        if (h.whole) all = rsqrtf(block_sum(sq, scratch) / (float)width + h.eps);
        __syncthreads();                                               // the row is whole
        if (h.normed && !h.whole) {
            const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = threads >> 6;
            for (int head = wave; head < heads; head += waves) {
                float s = 0.f;
                for (int e = lane; e < h.dim; e += 64) s += row[head * h.dim + e] * row[head * h.dim + e];
                s = wave_sum(s);
                if (lane == 0) inverse[head] = rsqrtf(s / (float)h.dim + h.eps);
            }
            __syncthreads();
        }
        if (!target) return;                                           // the host never schedules a token without a page
        const float* weight = is_key ? h.k_weight : h.q_weight;
        const float* cs = h.cos_sin ? h.cos_sin + (size_t)t * 2 * h.pairs : nullptr;
        const size_t head_step = is_key ? (size_t)h.page_size * h.D : (size_t)h.D;
        for (int e = threadIdx.x * 8; e < heads * h.D; e += threads * 8) {
            const int head = e / h.D, d0 = e - head * h.D;             // (D is a multiple of 16: eight outputs lie in one head)
            const float* x = row + head * h.dim;
            const float* w = weight ? weight + (h.whole ? head * h.dim : 0) : nullptr;
            const float inv = h.whole ? all : h.normed ? inverse[head] : 1.f;
            auto normed = [&](int i) { return w ? x[i] * inv * w[i] : x[i] * inv; };
            Piece<T, 8> piece;
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const int d = d0 + i;
                float y = 0.f;
                if (d < h.dim) {
                    y = normed(d);
                    if (cs && d < 2 * h.pairs) {
                        const int pair = h.halves ? (d < h.pairs ? d : d - h.pairs) : d >> 1;
                        const bool second = h.halves ? d >= h.pairs : (d & 1) != 0;
                        const float other = normed(h.halves ? (second ? d - h.pairs : d + h.pairs) : d ^ 1);
                        const float co = cs[pair], si = cs[h.pairs + pair];
                        y = second ? y * co + other * si : y * co - other * si;
                    }
                }
                piece.v[i] = (T)y;
            }
            *reinterpret_cast<Piece<T, 8>*>(target + head * head_step + d0) = piece;
        }
        return;
    }
    const int index = block - 2 * n_tokens;
    // V channels of token t's values from `c` on: convolved, kept for other layers, mixed.
    auto value_piece = [&](int t, int c, const Place& place, float (&v)[V]) {
        convolved<T, V>(qkv, stride, t, at_values + c, conv, place, v);
        if (own_values) {
            Piece<T, V> piece;
#pragma unroll
            for (int i = 0; i < V; ++i) piece.v[i] = (T)v[i];
            *reinterpret_cast<Piece<T, V>*>(own_values + (size_t)t * v_width + c) = piece;
        }
        if (first) {
            const Piece<T, V> other = *reinterpret_cast<const Piece<T, V>*>(first + (size_t)t * h.first_stride + c);
#pragma unroll
            for (int i = 0; i < V; ++i) v[i] = (1.f - h.mix) * v[i] + h.mix * (float)other.v[i];
        }
    };
    if (!tiled_values) {
        const int t = index;
        const Place place = place_of(conv, t);
        const int page = h.table[(size_t)place.row * h.table_stride + place.position / h.page_size];
        T* slot = page < 0 ? nullptr : values + (size_t)page * h.n_kv * h.D * h.page_size + place.position % h.page_size;
        for (int c = threadIdx.x * V; c < v_width; c += threads * V) {
            float v[V];
            value_piece(t, c, place, v);
            if (!slot) continue;
#pragma unroll
            for (int i = 0; i < V; ++i) {
                const int head = (c + i) / h.value_dim, d = (c + i) - head * h.value_dim;
                slot[((size_t)head * h.D + d) * h.page_size] = (T)v[i];
            }
        }
        const int rest = h.D - h.value_dim;
        if (slot && rest)
            for (int i = threadIdx.x; i < h.n_kv * rest; i += threads)
                slot[((size_t)(i / rest) * h.D + h.value_dim + i % rest) * h.page_size] = (T)0.f;
        return;
    }
    const int tile_index = index / h.n_kv, head = index - tile_index * h.n_kv, token0 = tile_index * VT_TOKENS;
    T* tile = reinterpret_cast<T*>(lds_bytes);
    const int pieces = h.value_dim / V, pitch = h.value_dim + 16 / (int)sizeof(T);
    for (int e = threadIdx.x; e < VT_TOKENS * pieces; e += threads) {
        const int i = e / pieces, c = (e - i * pieces) * V, t = token0 + i;
        if (t >= n_tokens) continue;
        const Place place = place_of(conv, t);
        float v[V];
        value_piece(t, head * h.value_dim + c, place, v);
#pragma unroll
        for (int k = 0; k < V; ++k) tile[i * pitch + c + k] = (T)v[k];
    }
    store_value_tile(tile, pitch, token0, head, h.value_dim, values, h.table, h.table_stride, conv.token_row, conv.positions, h.page_size, h.n_kv,
                     h.D, n_tokens);
}

template <typename T, int V>
int launch(const T* qkv, long stride, const Taps& conv, const Heads& h, T* keys, T* values, T* out_q, const T* first, T* own_values, int n_tokens,
           hipStream_t stream) {
    // Long portions: values in tiles of 64 tokens and one KV head (a piece must not reach into the next head's values).
    const size_t tile = (size_t)VT_TOKENS * (h.value_dim + 16 / sizeof(T)) * sizeof(T);
    const bool tiled = n_tokens >= 4 * VT_TOKENS && h.value_dim % V == 0 && h.page_size % 4 == 0 && tile <= MOST_BYTES;
    const int widest = (h.n_q > h.n_kv ? h.n_q : h.n_kv) * h.dim;
    size_t lds = (size_t)widest * sizeof(float);
    if (tiled && tile > lds) lds = tile;
    const long blocks = 2L * n_tokens + (tiled ? (long)((n_tokens + VT_TOKENS - 1) / VT_TOKENS) * h.n_kv : n_tokens);
    if (blocks > 0x7fffffffL || lds > MOST_BYTES || h.n_q > MOST_HEADS || h.n_kv > MOST_HEADS) return -1;
    qkv_compose_kernel<T, V><<<dim3((unsigned)blocks), 256, lds, stream>>>(qkv, stride, conv, h, keys, values, out_q, first, own_values, n_tokens,
                                                                          tiled ? 1 : 0);
    LSA_LAUNCH_CHECK();
}

template <typename T>
int dispatch(const void* qkv, long stride, const Taps& conv, const Heads& h, void* keys, void* values, void* out_q, const void* first, void* own_values,
             int n_tokens, hipStream_t stream) {
    // Pieces of eight channels where every row they touch begins at a multiple of sixteen bytes and has whole pieces.
    constexpr int V = 8;
    auto aligned = [](const void* p) { return (reinterpret_cast<size_t>(p) & 15) == 0; };
    const bool wide = h.n_q * h.dim % V == 0 && h.n_kv * h.dim % V == 0 && h.n_kv * h.value_dim % V == 0 && stride % V == 0 && aligned(qkv) &&
                      (!conv.w || (aligned(conv.w) && (conv.taps < 2 || (aligned(conv.state) && conv.state_stride % 4 == 0)))) &&
                      (!first || (aligned(first) && h.first_stride % V == 0)) && (!own_values || aligned(own_values));
    if (wide) return launch<T, V>((const T*)qkv, stride, conv, h, (T*)keys, (T*)values, (T*)out_q, (const T*)first, (T*)own_values, n_tokens, stream);
    return launch<T, 1>((const T*)qkv, stride, conv, h, (T*)keys, (T*)values, (T*)out_q, (const T*)first, (T*)own_values, n_tokens, stream);
}

}  // namespace

// The widest row of queries or keys (all heads of a token) that the kernel keeps in LDS.
LSA_EXPORT int lsa_compose_most_width() { return MOST_WIDTH; }
LSA_EXPORT int lsa_compose_most_heads() { return MOST_HEADS; }

// span 0: no norm; 1: over each head; 2: over the whole projection.
LSA_EXPORT int lsa_qkv_compose(int dtype, const void* qkv, long stride, const float* taps, int n_taps, float* state, long state_stride, const int* slots,
                               const int* token_row, const int* positions, const int* row_start, int keep, const float* q_weight,
                               const float* k_weight, int span, float eps, const float* cos_sin, int pairs, int halves, void* keys, void* values,
                               const int* table, int table_stride, int page_size, int n_q, int n_kv, int dim, int value_dim, int D, void* out_q,
                               float mix, const void* first, long first_stride, void* own_values, int n_tokens, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (dim < 1 || value_dim < 1 || dim > D || value_dim > D || D % 16 || page_size < 1 || span < 0 || span > 2 || 2 * pairs > dim) return -1;
    if (taps && (n_taps < 1 || (n_taps > 1 && (!state || !slots)))) return -1;
    const int channels = (n_q + n_kv) * dim + n_kv * value_dim;
    if (stride < channels) return -1;
    const Taps conv = {taps, n_taps, channels, state, state_stride, slots, token_row, positions, row_start, keep};
    const Heads h = {n_q, n_kv, dim, value_dim, D, page_size, table_stride, table, q_weight, k_weight, eps, span > 0, span == 2, cos_sin, pairs, halves,
                     mix, first_stride};
    return dtype ? dispatch<bf16_t>(qkv, stride, conv, h, keys, values, out_q, first, own_values, n_tokens, stream)
                 : dispatch<float>(qkv, stride, conv, h, keys, values, out_q, first, own_values, n_tokens, stream);
}
