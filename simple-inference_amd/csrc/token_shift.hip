// Several mixtures of each token's row with the row of the token before it:
//
//   out[s][n] = h[n] + (h[n - 1] - h[n]) * mu[s]        s = 0 .. mixtures - 1; float, one rounding
//
// The row before a step's first token of a sequence is kept in the sequence's state (width floats, zeros before its first
// token).  The threads of that first token are the only ones that read it; each then leaves its columns of the step's last
// row of the sequence there.
#include "common.h"

template <typename T, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(const T* __restrict__ h, const float* __restrict__ mu,
                                                          int mixtures, float* __restrict__ state, long long state_stride,
                                                          int state_offset, const int* __restrict__ cu_q,
                                                          const int* __restrict__ seq_of_token,
                                                          const int* __restrict__ slots, T* __restrict__ out,
                                                          int n_tokens, int width) {
    const int n = blockIdx.x, c = (blockIdx.y * blockDim.x + threadIdx.x) * V;
    if (c >= width) return;
    const int seq = seq_of_token[n], first = cu_q[seq];
    float own[V], before[V];
    auto load = [&](int t, float (&x)[V]) {
        if constexpr (V == 8) {
            Vec8<T> v;
            v.load(h + (size_t)t * width + c);
            v.get(x);
        } else {
            x[0] = to_float(h[(size_t)t * width + c]);
        }
    };
    load(n, own);
    if (n == first) {
        float* kept = state + (size_t)slots[seq] * state_stride + state_offset + c;
        float last[V];
        load(cu_q[seq + 1] - 1, last);
#pragma unroll
        for (int e = 0; e < V; ++e) {
            before[e] = kept[e];
            kept[e] = last[e];
        }
    } else {
        load(n - 1, before);
    }
    for (int s = 0; s < mixtures; ++s) {
        const float* m = mu + (size_t)s * width + c;
        T* dst = out + ((size_t)s * n_tokens + n) * width + c;
        float x[V];
#pragma unroll
        for (int e = 0; e < V; ++e) x[e] = own[e] + (before[e] - own[e]) * m[e];
        if constexpr (V == 8) {
            Vec8<T> v;
            v.set(x);
            v.store(dst);
        } else {
            dst[0] = from_float<T>(x[0]);
        }
    }
}

SIA_EXPORT int sia_token_shift(const void* h, const float* mu, int mixtures, float* state, long long state_stride,
                               int state_offset, const int* cu_q, const int* seq_of_token, const int* slots, void* out,
                               int n_tokens, int width, int dtype, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (width <= 0 || mixtures <= 0 || !h || !mu || !state || !out || state_offset < 0 ||
        (long long)state_offset + width > state_stride || (dtype != SIA_F32 && dtype != SIA_BF16))
        return SIA_BAD_ARGUMENT;
    const bool vec = width % 8 == 0;
    // few tokens: smaller workgroups, so that a row is more than one of them
    dim3 block(n_tokens <= 64 ? 64 : 256), grid(n_tokens, ((vec ? width / 8 : width) + block.x - 1) / block.x);
#define LAUNCH(T)                                                                                                    \
    do {                                                                                                             \
        if (vec) hipLaunchKernelGGL((token_shift_kernel<T, 8>), grid, block, 0, stream, (const T*)h, mu, mixtures, state, \
                                    state_stride, state_offset, cu_q, seq_of_token, slots, (T*)out, n_tokens, width); \
        else hipLaunchKernelGGL((token_shift_kernel<T, 1>), grid, block, 0, stream, (const T*)h, mu, mixtures, state, \
                                state_stride, state_offset, cu_q, seq_of_token, slots, (T*)out, n_tokens, width);    \
    } while (0)
    if (dtype == SIA_F32) LAUNCH(float);
    else LAUNCH(bf16_t);
#undef LAUNCH
    return SIA_LAUNCH_CHECK();
}
