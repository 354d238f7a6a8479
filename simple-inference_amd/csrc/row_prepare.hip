// What lies between the q/k/v product and attention for heads that need a token's whole row at once:
//
//   u  = projected q, k, v + bias
//   c  = a short causal convolution of u per channel (ring_conv.h), if weights are given
//   q  = q * rsqrt(mean(q^2) + eps) * gain     over all of a token's q elements at once (gain of that size), or per head
//   k  likewise                                 (one gain of head_dim for all heads); none if no gains are given
//   (a, b) <- (a cos - b sin, b cos + a sin)   for the first rotary_dim elements of a head, neighbours (2i, 2i + 1) or
//                                               halves (i, i + rotary_dim / 2) paired, at the token's absolute position
//
// all in float with one rounding; q goes to a matrix of its own (heads q_head_stride apart, zeros between them), k and v to
// the token's place in its page (layout as in qk_prepare.hip).  q, k and v are runs of columns of the projected rows that
// start anywhere; the channels of bias, convolution and ring are [q | k | v] without gaps.
//
// In a step of single tokens the convolution is part of this kernel (the ring holds what it needs); a step of runs of tokens
// is convolved first, by ring_conv.h's kernel into rows of their own (rounded once more, as a convolution's result may be).
//
// A workgroup takes a token's q and k.  Where neighbours turn together, a piece of eight elements is a thread's and the norm is
// over the row (or absent), everything stays in registers and all loads are issued before the row's sums are taken
// (``row_pieces_kernel``); else the elements meet in LDS as floats, where norm and rotation find their
// partners.  The values are further workgroups' (16 tokens each, or one in a step of single tokens): where 8 or 16 consecutive
// tokens of a sequence fill an aligned run of a page, the run's positions of a channel (innermost in a page) are written at
// once.
#include "ring_conv.h"

#define ROWP_MAX_ELEMENTS 15000       // q and k elements of a token (LDS)

struct RowPrepare {
    const void* proj;
    int row_stride;
    RingColumns cols;              // q, k, v
    const float *bias, *conv;      // [channels], [taps][channels]
    int taps;
    const float *q_gain, *k_gain;
    float eps;
    int over_row;
    const float *cos_table, *sin_table;
    int rotary_dim, neighbours;
    const int *positions, *seq_of_token, *cu_q, *slots, *block_table;
    int table_width;
    float* state;
    long long state_stride;
    void *k_pages, *v_pages, *q_out;
    int n_tokens, n_heads, n_kv, head_dim, value_dim, page_size, k_row, v_rows, q_head_stride;
    int v_group, v_tile, single;
};

// TAPS: 0 the rows are convolved already (or there is no convolution); 1 to 4, or -1 for any number, the convolution of a
// step of single tokens.
template <typename T, int V, int TAPS>
__device__ __forceinline__ void elements(const RowPrepare& p, int n, int pos, int at, int c, float* ring, float (&x)[V]) {
    const T* proj = (const T*)p.proj;
    if constexpr (TAPS == 0) {
        if constexpr (V == 8) {
            Vec8<T> v;
            v.load(proj + (size_t)n * p.row_stride + at);
            v.get(x);
        } else {
            x[0] = to_float(proj[(size_t)n * p.row_stride + at]);
        }
        if (p.bias) {
#pragma unroll
            for (int e = 0; e < V; ++e) x[e] += p.bias[c + e];
        }
    } else {
        float own[V];
        const int channels = p.cols.channels();
        if constexpr (TAPS > 0)
            ring_conv_single<T, V, TAPS>(proj, p.row_stride, at, c, channels, p.bias, p.conv, ring, n, pos, x, own);
        else
            ring_conv<T, V>(proj, p.row_stride, at, c, channels, p.bias, p.conv, p.taps, ring, n, n, pos, x, own);
        if (p.taps > 1) {
            float* row = ring + (size_t)(pos % p.taps) * channels + c;      // nobody reads this row in this step
#pragma unroll
            for (int e = 0; e < V; ++e) row[e] = own[e];
        }
    }
}

template <typename T, int V, int TAPS>
__device__ __forceinline__ void prepare_values(const RowPrepare& p, int n) {
    const T* proj = (const T*)p.proj;
    T* pages = (T*)p.v_pages;
    const int pos = p.positions[n], seq = p.seq_of_token[n];
    const int page = p.block_table[(size_t)seq * p.table_width + pos / p.page_size], off = pos % p.page_size;
    if (page < 0) return;
    const int c0 = p.cols.size[0] + p.cols.size[1], rows = p.cols.size[2];
    auto at_page = [&](int i) {
        return pages + (((size_t)page * p.n_kv + i / p.value_dim) * p.v_rows + i % p.value_dim) * p.page_size;
    };
    if (TAPS == 0 && p.v_group > 0) {
        const int place = off % p.v_group, begin = n - place;
        if (begin >= p.cu_q[seq] && begin + p.v_group <= p.cu_q[seq + 1]) {      // a whole run: its first token writes it
            if (place != 0) return;
            constexpr int MAX = 16, PER = 16 / sizeof(T);
            for (int i = threadIdx.x; i < rows; i += blockDim.x) {
                const float add = p.bias ? p.bias[c0 + i] : 0.f;
                __attribute__((aligned(16))) T vals[MAX];
#pragma unroll
                for (int m = 0; m < MAX; ++m)
                    vals[m] = m < p.v_group ? from_float<T>(to_float(proj[(size_t)(n + m) * p.row_stride + p.cols.col[2] + i]) + add) : T(0);
                T* dst = at_page(i) + off;
#pragma unroll
                for (int m = 0; m < MAX; m += PER)
                    if (m < p.v_group) *reinterpret_cast<uint4*>(dst + m) = *reinterpret_cast<const uint4*>(vals + m);
            }
            return;
        }
    }
    float* ring = p.taps > 1 ? p.state + (size_t)p.slots[seq] * p.state_stride : nullptr;
    for (int i = threadIdx.x * V; i < rows; i += blockDim.x * V) {
        float x[V];
        elements<T, V, TAPS>(p, n, pos, p.cols.col[2] + i, c0 + i, ring, x);
#pragma unroll
        for (int e = 0; e < V; ++e) at_page(i + e)[off] = from_float<T>(x[e]);
    }
}

// The values of the tokens of value workgroup ``g``.
template <typename T, int V, int TAPS>
__device__ __forceinline__ void values_of(const RowPrepare& p, int g) {
    for (int n = g * p.v_tile; n < min(p.n_tokens, (g + 1) * p.v_tile); ++n) prepare_values<T, V, TAPS>(p, n);
}

// Sums of two values over a workgroup, in one pass (``scratch``: 32 floats).
__device__ __forceinline__ void block_sums(float& a, float& b, float* scratch) {
    a = wave_sum(a);
    b = wave_sum(b);
    const int wave = threadIdx.x / SIA_WAVE, n_waves = blockDim.x / SIA_WAVE;
    if (threadIdx.x % SIA_WAVE == 0) {
        scratch[wave] = a;
        scratch[16 + wave] = b;
    }
    __syncthreads();
    a = b = 0.f;
    for (int w = 0; w < n_waves; ++w) {
        a += scratch[w];
        b += scratch[16 + w];
    }
}

// A thread a piece of eight q or k elements (at most 1,024 pieces): neighbours turn together, rotary_dim % 8 == 0.
template <typename T, int TAPS>
__global__ __launch_bounds__(1024) void row_pieces_kernel(const RowPrepare p) {
    __shared__ float scratch[32];
    const int n = blockIdx.x, tid = threadIdx.x;
    if (n >= p.n_tokens) {
        values_of<T, 8, TAPS>(p, n - p.n_tokens);
        return;
    }
    const int nq = p.cols.size[0], nqk = nq + p.cols.size[1], D = p.head_dim, c = tid * 8;
    const bool live = c < nqk, is_q = c < nq;
    const int h = c / D, d0 = c % D;
    const int pos = p.positions[n], seq = p.seq_of_token[n];
    float* ring = p.taps > 1 ? p.state + (size_t)p.slots[seq] * p.state_stride : nullptr;
    float x[8] = {};
    Vec8<float> vg;
    float4 vc, vs;
    const bool turns = live && d0 < p.rotary_dim;
    if (live) {
        if (p.q_gain) vg.load(is_q ? p.q_gain + c : p.k_gain + c - nq);
        if (turns) {
            const size_t at = (size_t)pos * (p.rotary_dim / 2) + d0 / 2;
            vc = *reinterpret_cast<const float4*>(p.cos_table + at);
            vs = *reinterpret_cast<const float4*>(p.sin_table + at);
        }
        elements<T, 8, TAPS>(p, n, pos, is_q ? p.cols.col[0] + c : p.cols.col[1] + c - nq, c, ring, x);
    }
    if (p.q_gain) {      // uniform
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
        float sq = is_q ? ss : 0.f, sk = is_q ? 0.f : ss;
        block_sums(sq, sk, scratch);
        if (live) {
            const float inv = is_q ? rsqrtf(sq / (float)nq + p.eps) : rsqrtf(sk / (float)(nqk - nq) + p.eps);
            float gain[8];
            vg.get(gain);
#pragma unroll
            for (int e = 0; e < 8; ++e) x[e] *= inv * gain[e];
        }
    }
    if (!live) return;
    if (turns) {
        const float co[4] = {vc.x, vc.y, vc.z, vc.w}, si[4] = {vs.x, vs.y, vs.z, vs.w};
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float a = x[2 * i], b = x[2 * i + 1];
            x[2 * i] = a * co[i] - b * si[i];
            x[2 * i + 1] = b * co[i] + a * si[i];
        }
    }
    Vec8<T> v;
    v.set(x);
    if (is_q) {
        T* head = (T*)p.q_out + ((size_t)n * p.n_heads + h) * p.q_head_stride;
        v.store(head + d0);
        if (d0 + 8 == D) {      // zeros between the heads
            const float zero[8] = {};
            v.set(zero);
            for (int d = D; d < p.q_head_stride; d += 8) v.store(head + d);
        }
    } else {
        const int page = p.block_table[(size_t)seq * p.table_width + pos / p.page_size];
        if (page >= 0)
            v.store((T*)p.k_pages + (((size_t)page * p.n_kv + h - p.n_heads) * p.page_size + pos % p.page_size) * p.k_row + d0);
    }
}

template <typename T, int V, int TAPS>
__global__ __launch_bounds__(1024) void row_prepare_kernel(const RowPrepare p) {
    extern __shared__ float row_s[];      // q and k elements
    __shared__ float scratch[16];
    const int n = blockIdx.x, tid = threadIdx.x, threads = blockDim.x;
    if (n >= p.n_tokens) {
        values_of<T, V, TAPS>(p, n - p.n_tokens);
        return;
    }
    const int pos = p.positions[n], seq = p.seq_of_token[n];
    const int nq = p.cols.size[0], nqk = nq + p.cols.size[1], D = p.head_dim;
    float* ring = p.taps > 1 ? p.state + (size_t)p.slots[seq] * p.state_stride : nullptr;
    float ss_q = 0.f, ss_k = 0.f;
    for (int c = tid * V; c < nqk; c += threads * V) {
        float x[V];
        elements<T, V, TAPS>(p, n, pos, c < nq ? p.cols.col[0] + c : p.cols.col[1] + c - nq, c, ring, x);
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < V; ++e) {
            row_s[c + e] = x[e];
            ss += x[e] * x[e];
        }
        if (c < nq) ss_q += ss;
        else ss_k += ss;
    }
    if (p.q_gain && p.over_row) {
        ss_q = block_sum(ss_q, scratch);
        ss_k = block_sum(ss_k, scratch);
        const float iq = rsqrtf(ss_q / (float)nq + p.eps), ik = rsqrtf(ss_k / (float)(nqk - nq) + p.eps);
        for (int c = tid * V; c < nqk; c += threads * V)      // a thread's own elements
#pragma unroll
            for (int e = 0; e < V; ++e) row_s[c + e] *= c < nq ? iq * p.q_gain[c + e] : ik * p.k_gain[c + e - nq];
    } else if (p.q_gain) {
        __syncthreads();
        const int wave = tid / SIA_WAVE, lane = tid % SIA_WAVE;
        for (int h = wave; h < p.n_heads + p.n_kv; h += threads / SIA_WAVE) {
            float ss = 0.f;
            for (int d = lane; d < D; d += SIA_WAVE) ss += row_s[h * D + d] * row_s[h * D + d];
            const float inv = rsqrtf(wave_sum(ss) / (float)D + p.eps);
            const float* gain = h < p.n_heads ? p.q_gain : p.k_gain;
            for (int d = lane; d < D; d += SIA_WAVE) row_s[h * D + d] *= inv * gain[d];
        }
    }
    __syncthreads();
    const int page = p.block_table[(size_t)seq * p.table_width + pos / p.page_size], off = pos % p.page_size;
    const int half = p.rotary_dim / 2;
    const float *cs = p.cos_table + (size_t)pos * half, *sn = p.sin_table + (size_t)pos * half;
    for (int c = tid * V; c < nqk; c += threads * V) {
        const int h = c / D, d0 = c % D;      // V divides D: a piece lies in one head
        float x[V];
#pragma unroll
        for (int e = 0; e < V; ++e) {
            const int d = d0 + e;
            const float own = row_s[c + e];
            if (d >= p.rotary_dim) {
                x[e] = own;
            } else if (p.neighbours) {
                const float other = row_s[c - d0 + (d ^ 1)];
                const int i = d >> 1;
                x[e] = (d & 1) ? own * cs[i] + other * sn[i] : own * cs[i] - other * sn[i];
            } else if (d < half) {
                x[e] = own * cs[d] - row_s[c + e + half] * sn[d];
            } else {
                x[e] = own * cs[d - half] + row_s[c + e - half] * sn[d - half];
            }
        }
        T* dst;
        if (h < p.n_heads) dst = (T*)p.q_out + ((size_t)n * p.n_heads + h) * p.q_head_stride + d0;
        else if (page >= 0) dst = (T*)p.k_pages + (((size_t)page * p.n_kv + h - p.n_heads) * p.page_size + off) * p.k_row + d0;
        else continue;
        if constexpr (V == 8) {
            Vec8<T> v;
            v.set(x);
            v.store(dst);
        } else {
            dst[0] = from_float<T>(x[0]);
        }
    }
    const int gap = p.q_head_stride - D;      // zeros between the heads of q
    if (gap > 0)
        for (int i = tid; i < p.n_heads * gap; i += threads)
            ((T*)p.q_out)[((size_t)n * p.n_heads + i / gap) * p.q_head_stride + D + i % gap] = from_float<T>(0.f);
}

SIA_EXPORT int sia_row_prepare_max_elements() { return ROWP_MAX_ELEMENTS; }

// q_col, k_col, v_col: where the three runs of columns start; state: ring of taps rows of [q | k | v] channels (null with
// one tap); conv [taps][channels] or null (taps must then be 1), bias must come with it; neighbours: which elements the
// rotation pairs; convolved: room for the convolved rows of a step of runs of tokens, [tokens][channels, rounded up to 8].
SIA_EXPORT int sia_row_prepare(const void* proj, int row_stride, int q_col, int k_col, int v_col, const float* bias,
                               const float* conv, int taps, const float* q_gain, const float* k_gain, float eps,
                               int over_row, const float* cos_table, const float* sin_table, int rotary_dim,
                               int neighbours, const int* positions, const int* seq_of_token, const int* cu_q,
                               const int* slots, const int* block_table, int table_width, float* state,
                               long long state_stride, void* k_pages, void* v_pages, void* q_out, int n_tokens,
                               int n_seqs, int max_q_len, int n_heads, int n_kv, int head_dim, int value_dim,
                               int page_size, int k_row, int v_rows, int q_head_stride, void* convolved, int dtype,
                               hipStream_t stream) {
    if (n_tokens <= 0 || n_seqs <= 0) return 0;
    RowPrepare p{};
    p.cols = RingColumns{{q_col, k_col, v_col}, {n_heads * head_dim, n_kv * head_dim, n_kv * value_dim}};
    const int nqk = p.cols.size[0] + p.cols.size[1];
    if (n_heads <= 0 || n_kv <= 0 || head_dim <= 0 || value_dim <= 0 || nqk > ROWP_MAX_ELEMENTS || taps < 1 ||
        taps > RING_MAX_TAPS || (conv && (!bias || (max_q_len > 1 && !convolved))) || (taps > 1 && (!conv || !state || state_stride < (long long)taps * p.cols.channels())) ||
        rotary_dim < 0 || rotary_dim > head_dim || (rotary_dim & 1) || (rotary_dim > 0 && (!cos_table || !sin_table)) ||
        (q_gain == nullptr) != (k_gain == nullptr) || !k_pages || !v_pages || !q_out || !block_table || page_size <= 0 ||
        k_row < head_dim || v_rows < value_dim || q_head_stride < head_dim || (dtype != SIA_F32 && dtype != SIA_BF16))
        return SIA_BAD_ARGUMENT;
    for (int i = 0; i < 3; ++i)
        if (p.cols.col[i] < 0 || p.cols.col[i] + p.cols.size[i] > row_stride) return SIA_BAD_ARGUMENT;
    p.proj = proj;
    p.row_stride = row_stride;
    p.bias = bias;
    p.conv = conv;
    p.taps = taps;
    p.q_gain = q_gain;
    p.k_gain = k_gain;
    p.eps = eps;
    p.over_row = over_row;
    p.cos_table = cos_table;
    p.sin_table = sin_table;
    p.rotary_dim = rotary_dim;
    p.neighbours = neighbours;
    p.positions = positions;
    p.seq_of_token = seq_of_token;
    p.cu_q = cu_q;
    p.slots = slots;
    p.block_table = block_table;
    p.table_width = table_width;
    p.state = state;
    p.state_stride = state_stride;
    p.k_pages = k_pages;
    p.v_pages = v_pages;
    p.q_out = q_out;
    p.n_tokens = n_tokens;
    p.n_heads = n_heads;
    p.n_kv = n_kv;
    p.head_dim = head_dim;
    p.value_dim = value_dim;
    p.page_size = page_size;
    p.k_row = k_row;
    p.v_rows = v_rows;
    p.q_head_stride = q_head_stride;
    p.single = max_q_len <= 1;
    p.v_group = p.single ? 0 : page_size % 16 == 0 ? 16 : page_size % 8 == 0 ? 8 : 0;
    bool vec = head_dim % 8 == 0 && value_dim % 8 == 0 && row_stride % 8 == 0 && q_col % 8 == 0 && k_col % 8 == 0 &&
               v_col % 8 == 0 && k_row % 8 == 0 && q_head_stride % 8 == 0 && ((uintptr_t)proj % 16) == 0;
    if (conv && !p.single) {      // convolved first, the projection's bias included
        const int channels = p.cols.channels(), wide = (channels + 7) / 8 * 8;
#define CONVOLVE(T)                                                                                                  \
    do {                                                                                                             \
        launch_ring_conv<T>((const T*)proj, row_stride, p.cols, bias, conv, nullptr, state, state_stride, 0, taps, cu_q, \
                            seq_of_token, positions, slots, (T*)convolved, wide, n_tokens, vec, stream);             \
        launch_ring_keep<T>((const T*)proj, row_stride, p.cols, bias, state, state_stride, 0, taps, cu_q, positions, \
                            slots, n_seqs, stream);                                                                  \
    } while (0)
        if (dtype == SIA_F32) CONVOLVE(float);
        else CONVOLVE(bf16_t);
#undef CONVOLVE
        p.proj = convolved;
        p.row_stride = wide;
        p.cols.col[0] = 0;
        p.cols.col[1] = p.cols.size[0];
        p.cols.col[2] = nqk;
        p.bias = nullptr;
        p.conv = nullptr;
        p.taps = 1;
    } else if (conv && taps > 1 && (state_stride % 4 != 0 || ((uintptr_t)state % 16) != 0)) {
        vec = false;      // the ring's rows are read in 16-byte pieces
    }
    const int pieces = vec ? nqk / 8 : nqk;
    int threads = (pieces + SIA_WAVE - 1) / SIA_WAVE * SIA_WAVE;
    threads = threads > 1024 ? 1024 : threads;
    if (!p.single && threads > 512) threads = 512;
    // the form that stays in registers
    const bool pieces_fit = vec && pieces <= 1024 && (rotary_dim == 0 || neighbours) && rotary_dim % 8 == 0 && (!q_gain || over_row) &&
                            (rotary_dim == 0 || (((uintptr_t)cos_table % 16) == 0 && ((uintptr_t)sin_table % 16) == 0));
    if (pieces_fit) threads = (pieces + SIA_WAVE - 1) / SIA_WAVE * SIA_WAVE;
    p.v_tile = p.single ? 1 : 16;
    dim3 grid(n_tokens + (n_tokens + p.v_tile - 1) / p.v_tile), block(threads);
    const size_t lds = (size_t)nqk * sizeof(float);
#define LAUNCH_AS(T, TAPS)                                                                             \
    do {                                                                                               \
        if (pieces_fit) hipLaunchKernelGGL((row_pieces_kernel<T, TAPS>), grid, block, 0, stream, p);   \
        else if (vec) hipLaunchKernelGGL((row_prepare_kernel<T, 8, TAPS>), grid, block, lds, stream, p); \
        else hipLaunchKernelGGL((row_prepare_kernel<T, 1, TAPS>), grid, block, lds, stream, p);        \
    } while (0)
#define LAUNCH(T)                                                                                      \
    do {                                                                                               \
        if (!p.conv) LAUNCH_AS(T, 0);                                                                  \
        else if (taps == 1) LAUNCH_AS(T, 1);                                                           \
        else if (taps == 2) LAUNCH_AS(T, 2);                                                           \
        else if (taps == 3) LAUNCH_AS(T, 3);                                                           \
        else if (taps == 4) LAUNCH_AS(T, 4);                                                           \
        else LAUNCH_AS(T, -1);                                                                         \
    } while (0)
    if (dtype == SIA_F32) LAUNCH(float);
    else LAUNCH(bf16_t);
#undef LAUNCH
#undef LAUNCH_AS
    return SIA_LAUNCH_CHECK();
}
