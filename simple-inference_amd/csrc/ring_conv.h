// A short causal convolution whose kept inputs lie in a ring: the input of position p of a sequence is ring row p % taps
// of the sequence's state, taps rows of ``channels`` floats.
//
//   c[t] = sum_j w[j] * u[t - (taps - 1) + j],   u = a column of the projected rows plus the projection's bias
//
// A step's tokens read the ring for the inputs before the step's first token.  In a step in which every sequence brings
// one token, the token's own input goes into a row that no token of the step reads (the rows read are those of the taps - 1
// positions before it), so whoever has the channel may write it at once, whatever other workgroups still read.  After a
// step of runs of tokens a kernel of its own (``ring_keep``) writes the rows of each run's last taps - 1 inputs.
#pragma once

#include "common.h"

#define RING_MAX_TAPS 16

// Up to three runs of columns of the projected rows that together are the convolution's channels.
struct RingColumns {
    int col[3], size[3];
    __device__ __host__ __forceinline__ int channels() const { return size[0] + size[1] + size[2]; }
    __device__ __forceinline__ int column(int c) const {
        if (c < size[0]) return col[0] + c;
        c -= size[0];
        if (c < size[1]) return col[1] + c;
        return col[2] + c - size[1];
    }
};

// V consecutive channels from channel c on (column ``at`` of the rows), of token t at position pos, whose sequence's first
// token of the step is ``first``; w is [taps][channels], ring the sequence's rows.  own: the token's own input.
template <typename T, int V>
__device__ __forceinline__ void ring_conv(const T* __restrict__ proj, int row_stride, int at, int c, int channels,
                                          const float* __restrict__ bias, const float* __restrict__ w, int taps,
                                          const float* __restrict__ ring, int t, int first, int pos, float (&acc)[V],
                                          float (&own)[V]) {
    float add[V];
#pragma unroll
    for (int e = 0; e < V; ++e) {
        add[e] = bias ? bias[c + e] : 0.f;
        acc[e] = 0.f;
    }
    for (int j = 0; j < taps; ++j) {
        const int back = taps - 1 - j, src = t - back;
        if (back > pos) continue;      // before the sequence
        float u[V];
        if (src >= first) {
            if constexpr (V == 8) {
                Vec8<T> v;
                v.load(proj + (size_t)src * row_stride + at);
                v.get(u);
            } else {
#pragma unroll
                for (int e = 0; e < V; ++e) u[e] = to_float(proj[(size_t)src * row_stride + at + e]);
            }
#pragma unroll
            for (int e = 0; e < V; ++e) u[e] += add[e];
        } else {
            const float* row = ring + (size_t)((pos - back) % taps) * channels + c;
#pragma unroll
            for (int e = 0; e < V; ++e) u[e] = row[e];
        }
#pragma unroll
        for (int e = 0; e < V; ++e) {
            acc[e] += (w ? w[(size_t)j * channels + c + e] : 1.f) * u[e];
            if (back == 0) own[e] = u[e];
        }
    }
}

// The same for a token that is its sequence's only one in the step, with the number of taps known: the inputs before it all
// lie in the ring, so every load is issued before the first is used (rows of positions before the sequence are read and
// weigh nothing).
template <typename T, int V, int TAPS>
__device__ __forceinline__ void ring_conv_single(const T* __restrict__ proj, int row_stride, int at, int c, int channels,
                                                 const float* __restrict__ bias, const float* __restrict__ w,
                                                 const float* __restrict__ ring, int t, int pos, float (&acc)[V],
                                                 float (&own)[V]) {
    if constexpr (V == 8) {
        Vec8<T> v;
        Vec8<float> vb, vw[TAPS], vr[TAPS > 1 ? TAPS - 1 : 1];
        v.load(proj + (size_t)t * row_stride + at);
        vb.load(bias + c);
#pragma unroll
        for (int j = 0; j < TAPS; ++j) vw[j].load(w + (size_t)j * channels + c);
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j) {
            const int back = TAPS - 1 - j;
            vr[j].load(ring + (size_t)((pos - back + TAPS) % TAPS) * channels + c);      // pos - back >= -TAPS
        }
        float b[8], k[8], u[8];
        v.get(own);
        vb.get(b);
        vw[TAPS - 1].get(k);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            own[e] += b[e];
            acc[e] = 0.f;
        }
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j) {
            const bool live = TAPS - 1 - j <= pos;
            float m[8];
            vw[j].get(m);
            vr[j].get(u);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[e] += live ? m[e] * u[e] : 0.f;
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] += k[e] * own[e];
    } else {
        ring_conv<T, V>(proj, row_stride, at, c, channels, bias, w, TAPS, ring, t, t, pos, acc, own);
    }
}

// All of a step's tokens, four tokens of V channels a thread (whatever sequences they belong to): a window of the last
// inputs stays in registers, so that an input is read once and the weights once a thread.  out [tokens][out_stride] holds
// the channels without gaps, plus ``add`` if given.
#define RING_TILE 4
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(128) void ring_conv_tile_kernel(const T* __restrict__ proj, int row_stride, RingColumns cols,
                                                             const float* __restrict__ bias, const float* __restrict__ w,
                                                             const float* __restrict__ add, const float* __restrict__ state,
                                                             long long state_stride, int state_offset,
                                                             const int* __restrict__ cu_q,
                                                             const int* __restrict__ seq_of_token,
                                                             const int* __restrict__ positions,
                                                             const int* __restrict__ slots, T* __restrict__ out,
                                                             int out_stride, int n_tokens) {
    const int t0 = blockIdx.x * RING_TILE, c = (blockIdx.y * blockDim.x + threadIdx.x) * V, channels = cols.channels();
    if (c >= channels) return;
    const int at = cols.column(c);
    auto load = [&](int t, float (&x)[V]) {
        if constexpr (V == 8) {
            Vec8<T> v;
            v.load(proj + (size_t)t * row_stride + at);
            v.get(x);
        } else {
            x[0] = to_float(proj[(size_t)t * row_stride + at]);
        }
    };
    auto vector = [&](const float* from, float (&x)[V]) {
        if constexpr (V == 8) {
            Vec8<float> v;
            v.load(from);
            v.get(x);
        } else {
            x[0] = from[0];
        }
    };
    float x[RING_TILE][V], b[V] = {}, k[TAPS][V], plus[V] = {};
#pragma unroll
    for (int i = 0; i < RING_TILE; ++i) load(min(t0 + i, n_tokens - 1), x[i]);
    if (bias) vector(bias + c, b);
    if (add) vector(add + c, plus);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) vector(w + (size_t)j * channels + c, k[j]);
    float past[TAPS > 1 ? TAPS - 1 : 1][V];      // past[0]: the input before, past[1]: the one before that, ...
    int first = -1, last = -1;      // the current token's sequence
#pragma unroll
    for (int i = 0; i < RING_TILE; ++i) {
        const int t = t0 + i;
        if (t >= n_tokens) break;
        if (t >= last) {      // the tile's first token, or a sequence's: what lies before it comes from memory
            const int seq = seq_of_token[t], pos = positions[t];
            first = cu_q[seq];
            last = cu_q[seq + 1];
            const float* ring = state + (size_t)slots[seq] * state_stride + state_offset;
#pragma unroll
            for (int j = 0; j + 1 < TAPS; ++j) {
                const int src = t - 1 - j;
                if (src >= first) {
                    load(src, past[j]);
#pragma unroll
                    for (int e = 0; e < V; ++e) past[j][e] += b[e];
                } else {
#pragma unroll
                    for (int e = 0; e < V; ++e)
                        past[j][e] = j + 1 <= pos ? ring[(size_t)((pos - 1 - j) % TAPS) * channels + c + e] : 0.f;
                }
            }
        }
        float y[V];
#pragma unroll
        for (int e = 0; e < V; ++e) {
            x[i][e] += b[e];
            y[e] = 0.f;
#pragma unroll
            for (int j = 0; j + 1 < TAPS; ++j) y[e] += k[j][e] * past[TAPS - 2 - j][e];
            y[e] += k[TAPS - 1][e] * x[i][e];
            y[e] += plus[e];
#pragma unroll
            for (int j = TAPS - 2; j > 0; --j) past[j][e] = past[j - 1][e];
            past[0][e] = x[i][e];
        }
        T* dst = out + (size_t)t * out_stride + c;
        if constexpr (V == 8) {
            Vec8<T> v;
            v.set(y);
            v.store(dst);
        } else {
            dst[0] = from_float<T>(y[0]);
        }
    }
}

// Any number of taps, a token a thread.
template <typename T>
__global__ __launch_bounds__(256) void ring_conv_token_kernel(const T* __restrict__ proj, int row_stride, RingColumns cols,
                                                              const float* __restrict__ bias, const float* __restrict__ w,
                                                              const float* __restrict__ add, const float* __restrict__ state,
                                                              long long state_stride, int state_offset, int taps,
                                                              const int* __restrict__ cu_q,
                                                              const int* __restrict__ seq_of_token,
                                                              const int* __restrict__ positions,
                                                              const int* __restrict__ slots, T* __restrict__ out,
                                                              int out_stride) {
    const int n = blockIdx.x, c = blockIdx.y * blockDim.x + threadIdx.x, channels = cols.channels();
    if (c >= channels) return;
    const int seq = seq_of_token[n];
    float acc[1], own[1];
    ring_conv<T, 1>(proj, row_stride, cols.column(c), c, channels, bias, w, taps,
                    state + (size_t)slots[seq] * state_stride + state_offset, n, cu_q[seq], positions[n], acc, own);
    out[(size_t)n * out_stride + c] = from_float<T>(acc[0] + (add ? add[c] : 0.f));
}

// The convolution of a whole step into ``out``.  vec: rows, columns and sizes of the runs of columns are multiples of 8.
template <typename T>
static void launch_ring_conv(const T* proj, int row_stride, const RingColumns& cols, const float* bias, const float* w,
                             const float* add, const float* state, long long state_stride, int state_offset, int taps,
                             const int* cu_q, const int* seq_of_token, const int* positions, const int* slots, T* out,
                             int out_stride, int n_tokens, bool vec, hipStream_t stream) {
    const int channels = cols.channels();
    if (taps > 4) {
        dim3 grid(n_tokens, (channels + 255) / 256), block(256);
        hipLaunchKernelGGL(ring_conv_token_kernel<T>, grid, block, 0, stream, proj, row_stride, cols, bias, w, add, state,
                           state_stride, state_offset, taps, cu_q, seq_of_token, positions, slots, out, out_stride);
        return;
    }
    const int pieces = vec ? channels / 8 : channels;
    dim3 grid((n_tokens + RING_TILE - 1) / RING_TILE, (pieces + 127) / 128), block(128);
#define RING_TILE_AS(V, TAPS)                                                                                        \
    hipLaunchKernelGGL((ring_conv_tile_kernel<T, V, TAPS>), grid, block, 0, stream, proj, row_stride, cols, bias, w, add, \
                       state, state_stride, state_offset, cu_q, seq_of_token, positions, slots, out, out_stride, n_tokens)
#define RING_TILE_TAPS(TAPS)                                                                                         \
    do {                                                                                                             \
        if (vec) RING_TILE_AS(8, TAPS);                                                                              \
        else RING_TILE_AS(1, TAPS);                                                                                  \
    } while (0)
    if (taps == 1) RING_TILE_TAPS(1);
    else if (taps == 2) RING_TILE_TAPS(2);
    else if (taps == 3) RING_TILE_TAPS(3);
    else RING_TILE_TAPS(4);
#undef RING_TILE_TAPS
#undef RING_TILE_AS
}

// The rows of each run's last taps - 1 inputs (a run shorter than that leaves older rows as they are).
template <typename T>
__global__ __launch_bounds__(256) void ring_keep_kernel(const T* __restrict__ proj, int row_stride, RingColumns cols,
                                                        const float* __restrict__ bias, float* __restrict__ state,
                                                        long long state_stride, int state_offset, int taps,
                                                        const int* __restrict__ cu_q, const int* __restrict__ positions,
                                                        const int* __restrict__ slots) {
    const int seq = blockIdx.x, c = blockIdx.y * blockDim.x + threadIdx.x, channels = cols.channels();
    if (c >= channels) return;
    const int first = cu_q[seq], last = cu_q[seq + 1];
    const int at = cols.column(c);
    float* ring = state + (size_t)slots[seq] * state_stride + state_offset;
    for (int t = max(first, last - (taps - 1)); t < last; ++t)
        ring[(size_t)(positions[t] % taps) * channels + c] = to_float(proj[(size_t)t * row_stride + at]) + (bias ? bias[c] : 0.f);
}

template <typename T>
static void launch_ring_keep(const T* proj, int row_stride, const RingColumns& cols, const float* bias, float* state,
                             long long state_stride, int state_offset, int taps, const int* cu_q, const int* positions,
                             const int* slots, int n_seqs, hipStream_t stream) {
    if (taps <= 1) return;
    dim3 grid(n_seqs, (cols.channels() + 255) / 256), block(256);
    hipLaunchKernelGGL(ring_keep_kernel<T>, grid, block, 0, stream, proj, row_stride, cols, bias, state, state_stride,
                       state_offset, taps, cu_q, positions, slots);
}
