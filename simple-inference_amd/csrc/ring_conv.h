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
