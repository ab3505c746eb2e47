// From the product of a step's tokens to what attention reads, where more than a norm and a rotation per head lies between:
// a causal convolution over time on every channel of queries, keys and values, a norm over each head or over the whole
// projection, a rotation, and values that are mixed with those of another layer.  Between the convolution, the norm and the
// rotation everything is float32; results are rounded once when they are stored.
//
// The first workgroups of a launch take values: a token's row each, stored where it belongs number by number (steps of few
// tokens), or 64 tokens of one KV head each, through LDS, so that neighbouring slots of a page go out together.  The others
// take queries and keys by turns, a token each with the row in LDS (any sizes), or, where heads are whole pieces of eight
// numbers, one token or four with a thread's piece of each in registers from the load to the store.
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
__device__ __forceinline__ Floats<V> convolved(const T* __restrict__ qkv, long stride, int t, int c, const Taps& conv, const Place place) {
    Floats<V> out;
    const Piece<T, V> own = *reinterpret_cast<const Piece<T, V>*>(qkv + (size_t)t * stride + c);
    if (!conv.w) {
#pragma unroll
        for (int v = 0; v < V; ++v) out.v[v] = (float)own.v[v];
        return out;
    }
    const int kept = conv.taps - 1;
    const Floats<V> last = *reinterpret_cast<const Floats<V>*>(conv.w + (size_t)kept * conv.channels + c);
#pragma unroll
    for (int v = 0; v < V; ++v) out.v[v] = last.v[v] * (float)own.v[v];
    const int in_step = min(kept, place.behind);
#pragma unroll 3
    for (int back = 1; back <= in_step; ++back) {
        const Floats<V> w = *reinterpret_cast<const Floats<V>*>(conv.w + (size_t)(kept - back) * conv.channels + c);
        const Piece<T, V> u = *reinterpret_cast<const Piece<T, V>*>(qkv + (size_t)(t - back) * stride + c);
#pragma unroll
        for (int v = 0; v < V; ++v) out.v[v] = __builtin_fmaf(w.v[v], (float)u.v[v], out.v[v]);
    }
    const int before = min(kept, place.position);                      // (places before the sequence are zeros)
#pragma unroll 3
    for (int back = in_step + 1; back <= before; ++back) {
        const Floats<V> w = *reinterpret_cast<const Floats<V>*>(conv.w + (size_t)(kept - back) * conv.channels + c);
        const Floats<V> u = *reinterpret_cast<const Floats<V>*>(place.state + (size_t)(kept - (back - place.behind)) * conv.channels + c);
#pragma unroll
        for (int v = 0; v < V; ++v) out.v[v] = __builtin_fmaf(w.v[v], u.v[v], out.v[v]);
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
    return out;
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

template <typename T> struct Rows {
    const T* qkv;
    long stride;
    T* keys;
    T* values;
    T* out_q;
    const T* first;                     // the values these are mixed with, or nullptr
    T* own_values;
    int n_tokens;
};

// A workgroup's share of the values: token `index`'s row (tiled 0), or 64 tokens of one KV head through LDS.
template <typename T, int V>
__device__ __forceinline__ void values_block(int index, int tiled, const Taps& conv, const Heads& h, const Rows<T>& rows, unsigned char* lds_bytes) {
    const int v_width = h.n_kv * h.value_dim, at_values = (h.n_q + h.n_kv) * h.dim, threads = blockDim.x;
    // V channels of token t's values from `c` on: convolved, kept for other layers, mixed.
    auto value_piece = [&](int t, int c, const Place place) {
        Floats<V> v = convolved<T, V>(rows.qkv, rows.stride, t, at_values + c, conv, place);
        if (rows.own_values) {
            Piece<T, V> piece;
#pragma unroll
            for (int i = 0; i < V; ++i) piece.v[i] = (T)v.v[i];
            *reinterpret_cast<Piece<T, V>*>(rows.own_values + (size_t)t * v_width + c) = piece;
        }
        if (rows.first) {
            const Piece<T, V> other = *reinterpret_cast<const Piece<T, V>*>(rows.first + (size_t)t * h.first_stride + c);
#pragma unroll
            for (int i = 0; i < V; ++i) v.v[i] = (1.f - h.mix) * v.v[i] + h.mix * (float)other.v[i];
        }
        return v;
    };
    if (!tiled) {
        const int t = index;
        const Place place = place_of(conv, t);
        const int page = h.table[(size_t)place.row * h.table_stride + place.position / h.page_size];
        T* slot = page < 0 ? nullptr : rows.values + (size_t)page * h.n_kv * h.D * h.page_size + place.position % h.page_size;
        for (int c = threadIdx.x * V; c < v_width; c += threads * V) {
            const Floats<V> v = value_piece(t, c, place);
            if (!slot) continue;                                       // (the host never schedules a token without a page)
#pragma unroll
            for (int i = 0; i < V; ++i) {
                const int head = (c + i) / h.value_dim, d = (c + i) - head * h.value_dim;
                slot[((size_t)head * h.D + d) * h.page_size] = (T)v.v[i];
            }
        }
        const int rest = h.D - h.value_dim;
        if (slot && rest)
            for (int i = threadIdx.x; i < h.n_kv * rest; i += threads)
                slot[((size_t)(i / rest) * h.D + h.value_dim + i % rest) * h.page_size] = (T)0.f;
        return;
    }
    __shared__ Place places[VT_TOKENS];
    const int tile_index = index / h.n_kv, head = index - tile_index * h.n_kv, token0 = tile_index * VT_TOKENS;
    if (threadIdx.x < VT_TOKENS) places[threadIdx.x] = place_of(conv, min(token0 + (int)threadIdx.x, rows.n_tokens - 1));
    __syncthreads();
    T* tile = reinterpret_cast<T*>(lds_bytes);
    const int pieces = h.value_dim / V, pitch = h.value_dim + 16 / (int)sizeof(T);
    for (int e = threadIdx.x; e < VT_TOKENS * pieces; e += threads) {
        const int i = e / pieces, c = (e - i * pieces) * V, t = token0 + i;
        if (t >= rows.n_tokens) continue;
        const Floats<V> v = value_piece(t, head * h.value_dim + c, places[i]);
        Piece<T, V> piece;
#pragma unroll
        for (int k = 0; k < V; ++k) piece.v[k] = (T)v.v[k];
        *reinterpret_cast<Piece<T, V>*>(tile + i * pitch + c) = piece;
    }
    store_value_tile(tile, pitch, token0, head, h.value_dim, rows.values, h.table, h.table_stride, conv.token_row, conv.positions, h.page_size, h.n_kv,
                     h.D, rows.n_tokens);
}

// Where a token's queries or keys go: its row of out_q, or its slot in its page (heads then lie page_size * D apart), or nullptr.
template <typename T>
__device__ __forceinline__ T* target_of(const Heads& h, const Rows<T>& rows, const Place& place, int t, int is_key) {
    if (!is_key) return rows.out_q + (size_t)t * h.n_q * h.D;
    const int page = h.table[(size_t)place.row * h.table_stride + place.position / h.page_size];
    return page < 0 ? nullptr : rows.keys + ((size_t)page * h.n_kv * h.page_size + place.position % h.page_size) * h.D;
}

// Any sizes: a workgroup a token's queries or keys, the row in LDS.
template <typename T, int V>
__global__ __launch_bounds__(256) void qkv_compose_kernel(Taps conv, Heads h, Rows<T> rows, int value_blocks, int tiled_values) {
    extern __shared__ __align__(16) unsigned char lds_bytes[];
    __shared__ float scratch[16];
    __shared__ float inverse[MOST_HEADS];
    if ((int)blockIdx.x < value_blocks) {
        values_block<T, V>(blockIdx.x, tiled_values, conv, h, rows, lds_bytes);
        return;
    }
    const int block = (int)blockIdx.x - value_blocks, threads = blockDim.x, t = block >> 1, is_key = block & 1;
    const int base = is_key ? h.n_q * h.dim : 0, heads = is_key ? h.n_kv : h.n_q, width = heads * h.dim;
    float* row = reinterpret_cast<float*>(lds_bytes);
    const Place place = place_of(conv, t);
    T* target = target_of(h, rows, place, t, is_key);
    float sq = 0.f;
    for (int c = threadIdx.x * V; c < width; c += threads * V) {
        const Floats<V> piece = convolved<T, V>(rows.qkv, rows.stride, t, base + c, conv, place);
#pragma unroll
        for (int v = 0; v < V; ++v) sq += piece.v[v] * piece.v[v];
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
}

// Heads of whole pieces of eight numbers (and, for a norm over each head, of 1, 2, 4, ... 32 pieces), dimensions turned as
// neighbours, no convolution or one of TAPS taps: a thread keeps its piece of TT consecutive tokens in registers from the load
// to the store.  All rows that its convolutions can read in this step are asked for at once, each once (TT + TAPS - 1 rows for TT
// tokens), at places that are there; the state is read where a row's first tokens need it.
template <typename T, int TAPS, int TT>
__global__ __launch_bounds__(TT > 1 ? 512 : 1024) void qkv_compose_pieces_kernel(Taps conv, Heads h, Rows<T> rows, int value_blocks, int tiled_values) {
    extern __shared__ __align__(16) unsigned char lds_bytes[];
    if ((int)blockIdx.x < value_blocks) {
        values_block<T, 8>(blockIdx.x, tiled_values, conv, h, rows, lds_bytes);
        return;
    }
    constexpr int KEPT = TAPS > 0 ? TAPS - 1 : 0;
    __shared__ float sums[TT][16];
    const int block = (int)blockIdx.x - value_blocks, is_key = block & 1, t0 = (block >> 1) * TT;
    const int base = is_key ? h.n_q * h.dim : 0, heads = is_key ? h.n_kv : h.n_q, width = heads * h.dim;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6;
    const bool active = (int)threadIdx.x * 8 < width;
    const int c = min((int)threadIdx.x * 8, width - 8), head = c / h.dim, d0 = c - head * h.dim;
    Piece<T, 8> raw[TT + KEPT];
#pragma unroll
    for (int i = 0; i < TT + KEPT; ++i)
        raw[i] = *reinterpret_cast<const Piece<T, 8>*>(rows.qkv + (size_t)min(max(t0 - KEPT + i, 0), rows.n_tokens - 1) * rows.stride + base + c);
    Floats<8> tap[TAPS > 0 ? TAPS : 1];
    if constexpr (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) tap[j] = *reinterpret_cast<const Floats<8>*>(conv.w + (size_t)j * conv.channels + base + c);
    }
    const float* weight = is_key ? h.k_weight : h.q_weight;
    Floats<8> w;
    if (weight) w = *reinterpret_cast<const Floats<8>*>(weight + (h.whole ? c : d0));
    else
#pragma unroll
        for (int e = 0; e < 8; ++e) w.v[e] = 1.f;
    Place place[TT];
#pragma unroll
    for (int i = 0; i < TT; ++i) place[i] = place_of(conv, min(t0 + i, rows.n_tokens - 1));
    float x[TT][8];
#pragma unroll
    for (int i = 0; i < TT; ++i) {
        if constexpr (TAPS == 0) {
#pragma unroll
            for (int e = 0; e < 8; ++e) x[i][e] = (float)raw[i].v[e];
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) x[i][e] = tap[KEPT].v[e] * (float)raw[i + KEPT].v[e];
            // (the same for all lanes)
            if (place[i].behind >= KEPT) {
#pragma unroll
                for (int back = 1; back <= KEPT; ++back)
#pragma unroll
                    for (int e = 0; e < 8; ++e) x[i][e] = __builtin_fmaf(tap[KEPT - back].v[e], (float)raw[i + KEPT - back].v[e], x[i][e]);
            } else {
                float* mine = place[i].state + base + c;
                Floats<8> before[KEPT > 0 ? KEPT : 1];
#pragma unroll
                for (int k = 0; k < KEPT; ++k) before[k] = *reinterpret_cast<const Floats<8>*>(mine + (size_t)k * conv.channels);
#pragma unroll
                for (int back = 1; back <= KEPT; ++back) {
                    // the input `back` places before the token: a row of this step, a row of the state, or a zero before the sequence
                    const bool in_step = back <= place[i].behind, there = back <= place[i].position;
#pragma unroll
                    for (int e = 0; e < 8; ++e) {
                        float u = (float)raw[i + KEPT - back].v[e];
#pragma unroll
                        for (int k = 0; k < KEPT; ++k)
                            if (!in_step && k == KEPT - (back - place[i].behind)) u = before[k].v[e];
                        x[i][e] = __builtin_fmaf(tap[KEPT - back].v[e], there ? u : 0.f, x[i][e]);
                    }
                }
                if (TT == 1 && conv.keep && active) {
#pragma unroll
                    for (int k = 0; k + 1 < KEPT; ++k) *reinterpret_cast<Floats<8>*>(mine + (size_t)k * conv.channels) = before[k + 1];
                    Floats<8> last;
#pragma unroll
                    for (int e = 0; e < 8; ++e) last.v[e] = (float)raw[KEPT].v[e];
                    *reinterpret_cast<Floats<8>*>(mine + (size_t)(KEPT - 1) * conv.channels) = last;
                }
            }
        }
    }
    float inv[TT];
#pragma unroll
    for (int i = 0; i < TT; ++i) inv[i] = 1.f;
    if (h.normed) {
        float sq[TT];
#pragma unroll
        for (int i = 0; i < TT; ++i) {
            sq[i] = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) sq[i] += x[i][e] * x[i][e];
            if (!active) sq[i] = 0.f;
        }
        const int span = h.whole ? 64 : h.dim / 8;                    // lanes that share a sum
        for (int offset = 1; offset < span; offset <<= 1)
#pragma unroll
            for (int i = 0; i < TT; ++i) sq[i] += __shfl_xor(sq[i], offset, 64);
        if (h.whole) {
            if (lane == 0)
#pragma unroll
                for (int i = 0; i < TT; ++i) sums[i][wave] = sq[i];
            __syncthreads();
#pragma unroll
            for (int i = 0; i < TT; ++i) {
                sq[i] = 0.f;
                for (int other = 0; other < waves; ++other) sq[i] += sums[i][other];
            }
        }
        const float count = h.whole ? (float)width : (float)h.dim;
#pragma unroll
        for (int i = 0; i < TT; ++i) inv[i] = rsqrtf(sq[i] / count + h.eps);
    }
    const size_t head_step = is_key ? (size_t)h.page_size * h.D : (size_t)h.D;
#pragma unroll
    for (int i = 0; i < TT; ++i) {
        const int t = t0 + i;
        if (t >= rows.n_tokens) break;
        T* target = target_of(h, rows, place[i], t, is_key);
        if (!target) continue;
        if (active) {
#pragma unroll
            for (int e = 0; e < 8; ++e) x[i][e] *= inv[i] * w.v[e];
            if (h.cos_sin && d0 < 2 * h.pairs) {
                const float* cs = h.cos_sin + (size_t)t * 2 * h.pairs;
#pragma unroll
                for (int e = 0; e < 8; e += 2) {
                    const int pair = (d0 + e) >> 1, there = min(pair, h.pairs - 1);
                    const float co = cs[there], si = cs[h.pairs + there], u = x[i][e], v = x[i][e + 1];
                    if (pair < h.pairs) {
                        x[i][e] = u * co - v * si;
                        x[i][e + 1] = v * co + u * si;
                    }
                }
            }
            Piece<T, 8> piece;
#pragma unroll
            for (int e = 0; e < 8; ++e) piece.v[e] = (T)x[i][e];
            *reinterpret_cast<Piece<T, 8>*>(target + head * head_step + d0) = piece;
        }
        const int pads = (h.D - h.dim) / 8;
        for (int p = threadIdx.x; p < heads * pads; p += blockDim.x) {
            Piece<T, 8> zeros;
#pragma unroll
            for (int e = 0; e < 8; ++e) zeros.v[e] = (T)0.f;
            *reinterpret_cast<Piece<T, 8>*>(target + (p / pads) * head_step + h.dim + 8 * (p % pads)) = zeros;
        }
    }
}

template <typename T, int V>
int launch(const Taps& conv, const Heads& h, const Rows<T>& rows, bool pieces, hipStream_t stream) {
    const int n_tokens = rows.n_tokens;
    // Long portions: values in tiles of 64 tokens and one KV head (a piece must not reach into the next head's values).
    const size_t tile = (size_t)VT_TOKENS * (h.value_dim + 16 / sizeof(T)) * sizeof(T);
    const bool tiled = n_tokens >= 4 * VT_TOKENS && h.value_dim % V == 0 && h.page_size % 4 == 0 && tile <= MOST_BYTES;
    const int widest = (h.n_q > h.n_kv ? h.n_q : h.n_kv) * h.dim;
    const long value_blocks = tiled ? (long)((n_tokens + VT_TOKENS - 1) / VT_TOKENS) * h.n_kv : n_tokens;
    if (value_blocks + 2L * n_tokens > 0x7fffffffL || h.n_q > MOST_HEADS || h.n_kv > MOST_HEADS) return -1;
    if constexpr (V == 8) {
        if (pieces && widest <= 8192) {
            int threads = (widest / 8 + 63) / 64 * 64;
            if (threads < 128) threads = 128;
            const bool many = n_tokens >= 256 && !conv.keep && threads <= 512;
            const long blocks = value_blocks + 2L * (many ? (n_tokens + 3) / 4 : n_tokens);
#define LSA_LAUNCH(TAPS) do { \
            if (many) qkv_compose_pieces_kernel<T, TAPS, 4><<<dim3((unsigned)blocks), threads, tiled ? tile : 0, stream>>>(conv, h, rows, (int)value_blocks, tiled ? 1 : 0); \
            else qkv_compose_pieces_kernel<T, TAPS, 1><<<dim3((unsigned)blocks), threads, tiled ? tile : 0, stream>>>(conv, h, rows, (int)value_blocks, tiled ? 1 : 0); \
            LSA_LAUNCH_CHECK(); } while (0)
            if (!conv.w) LSA_LAUNCH(0);
            if (conv.taps == 2) LSA_LAUNCH(2);
            if (conv.taps == 3) LSA_LAUNCH(3);
            if (conv.taps == 4) LSA_LAUNCH(4);
#undef LSA_LAUNCH
        }
    }
    size_t lds = (size_t)widest * sizeof(float);
    if (tiled && tile > lds) lds = tile;
    if (lds > MOST_BYTES) return -1;
    qkv_compose_kernel<T, V><<<dim3((unsigned)(value_blocks + 2L * n_tokens)), 256, lds, stream>>>(conv, h, rows, (int)value_blocks, tiled ? 1 : 0);
    LSA_LAUNCH_CHECK();
}

template <typename T>
int dispatch(const Taps& conv, const Heads& h, const void* qkv, long stride, void* keys, void* values, void* out_q, const void* first, void* own_values,
             int n_tokens, hipStream_t stream) {
    const Rows<T> rows = {(const T*)qkv, stride, (T*)keys, (T*)values, (T*)out_q, (const T*)first, (T*)own_values, n_tokens};
    // Pieces of eight channels where every row they touch begins at a multiple of sixteen bytes and has whole pieces.
    constexpr int V = 8;
    auto aligned = [](const void* p) { return (reinterpret_cast<size_t>(p) & 15) == 0; };
    const bool wide = h.n_q * h.dim % V == 0 && h.n_kv * h.dim % V == 0 && h.n_kv * h.value_dim % V == 0 && stride % V == 0 && aligned(qkv) &&
                      (!conv.w || (aligned(conv.w) && (conv.taps < 2 || (aligned(conv.state) && conv.state_stride % 4 == 0)))) &&
                      (!first || (aligned(first) && h.first_stride % V == 0)) && (!own_values || aligned(own_values));
    if (!wide) return launch<T, 1>(conv, h, rows, false, stream);
    const int per_head = h.dim / 8;
    const bool powers = per_head > 0 && per_head <= 32 && (per_head & (per_head - 1)) == 0;
    const bool pieces = h.dim % 8 == 0 && (!h.cos_sin || !h.halves) && (!h.normed || h.whole || powers) &&
                        (!h.q_weight || (aligned(h.q_weight) && aligned(h.k_weight)));
    return launch<T, V>(conv, h, rows, pieces, stream);
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
    return dtype ? dispatch<bf16_t>(conv, h, qkv, stride, keys, values, out_q, first, own_values, n_tokens, stream)
                 : dispatch<float>(conv, h, qkv, stride, keys, values, out_q, first, own_values, n_tokens, stream);
}
