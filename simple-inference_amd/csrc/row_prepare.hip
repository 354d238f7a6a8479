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
// A workgroup takes a token's q and k: their convolved elements meet in LDS as floats, where norm and rotation find their
// partners.  A second workgroup a token takes the values: where 8 or 16 consecutive tokens of a sequence fill an aligned run of a page, the
// run's workgroups share its channels and each walks its channels over all the run's tokens, a window of inputs in
// registers, and writes the run's positions (innermost in a page) at once.
#include "ring_conv.h"

#define ROWP_THREADS 256
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
    int v_group, single;
};

// the run's values of one channel, position by position
template <typename T>
__device__ __forceinline__ void prepare_values(const RowPrepare& p, int n) {
    const T* proj = (const T*)p.proj;
    T* pages = (T*)p.v_pages;
    const int pos = p.positions[n], seq = p.seq_of_token[n], first = p.cu_q[seq];
    const int page = p.block_table[(size_t)seq * p.table_width + pos / p.page_size], off = pos % p.page_size;
    if (page < 0) return;
    const int channels = p.cols.channels(), c0 = p.cols.size[0] + p.cols.size[1], rows = p.cols.size[2];
    float* ring = p.taps > 1 ? p.state + (size_t)p.slots[seq] * p.state_stride : nullptr;
    auto at_page = [&](int i) {
        return pages + (((size_t)page * p.n_kv + i / p.value_dim) * p.v_rows + i % p.value_dim) * p.page_size;
    };
    int place = 0, begin = n;
    bool whole = false;
    if (p.v_group > 0) {
        place = off % p.v_group;
        begin = n - place;
        whole = begin >= first && begin + p.v_group <= p.cu_q[seq + 1];
    }
    if (!whole) {
        for (int i = threadIdx.x; i < rows; i += ROWP_THREADS) {
            float acc[1], own[1];
            ring_conv<T, 1>(proj, p.row_stride, p.cols.col[2] + i, c0 + i, channels, p.bias, p.conv, p.taps, ring, n, first, pos, acc, own);
            at_page(i)[off] = from_float<T>(acc[0]);
            if (p.single && ring) ring[(size_t)(pos % p.taps) * channels + c0 + i] = own[0];
        }
        return;
    }
    constexpr int MAX = 16, PER = 16 / sizeof(T);
    const int slice = (rows + p.v_group - 1) / p.v_group;
    for (int i = place * slice + threadIdx.x; i < min(rows, (place + 1) * slice); i += ROWP_THREADS) {
        const int c = c0 + i;
        const float add = p.bias ? p.bias[c] : 0.f;
        float acc[MAX];
#pragma unroll
        for (int m = 0; m < MAX; ++m) acc[m] = 0.f;
        for (int j = 0; j < p.taps; ++j) {
            const int back = p.taps - 1 - j;
            const float w = p.conv ? p.conv[(size_t)j * channels + c] : 1.f;
#pragma unroll
            for (int m = 0; m < MAX; ++m) {
                if (m >= p.v_group) continue;
                const int src = begin + m - back, at = pos - place + m - back;
                if (src >= first) acc[m] += w * (to_float(proj[(size_t)src * p.row_stride + p.cols.col[2] + i]) + add);
                else if (at >= 0) acc[m] += w * ring[(size_t)(at % p.taps) * channels + c];
            }
        }
        __attribute__((aligned(16))) T vals[MAX];
#pragma unroll
        for (int m = 0; m < MAX; ++m) vals[m] = from_float<T>(acc[m]);
        T* dst = at_page(i) + (off - place);
#pragma unroll
        for (int m = 0; m < MAX; m += PER)
            if (m < p.v_group) *reinterpret_cast<uint4*>(dst + m) = *reinterpret_cast<const uint4*>(vals + m);
    }
}

template <typename T, int V>
__global__ __launch_bounds__(ROWP_THREADS) void row_prepare_kernel(const RowPrepare p) {
    extern __shared__ float row_s[];      // q and k elements; behind them a factor per head
    __shared__ float scratch[16];
    const int n = blockIdx.x, tid = threadIdx.x;
    if (blockIdx.y == 1) {
        prepare_values<T>(p, n);
        return;
    }
    const T* proj = (const T*)p.proj;
    const int pos = p.positions[n], seq = p.seq_of_token[n], first = p.cu_q[seq];
    const int channels = p.cols.channels(), nq = p.cols.size[0], nqk = nq + p.cols.size[1], D = p.head_dim;
    float* ring = p.taps > 1 ? p.state + (size_t)p.slots[seq] * p.state_stride : nullptr;
    float ss_q = 0.f, ss_k = 0.f;
    for (int c = tid * V; c < nqk; c += ROWP_THREADS * V) {
        float acc[V], own[V];
        const int at = c < nq ? p.cols.col[0] + c : p.cols.col[1] + c - nq;
        ring_conv<T, V>(proj, p.row_stride, at, c, channels, p.bias, p.conv, p.taps, ring, n, first, pos, acc, own);
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < V; ++e) {
            row_s[c + e] = acc[e];
            ss += acc[e] * acc[e];
            if (p.single && ring) ring[(size_t)(pos % p.taps) * channels + c + e] = own[e];
        }
        if (c < nq) ss_q += ss;
        else ss_k += ss;
    }
    if (p.q_gain && p.over_row) {
        ss_q = block_sum(ss_q, scratch);
        ss_k = block_sum(ss_k, scratch);
        const float iq = rsqrtf(ss_q / (float)nq + p.eps), ik = rsqrtf(ss_k / (float)(nqk - nq) + p.eps);
        for (int c = tid * V; c < nqk; c += ROWP_THREADS * V)      // a thread's own elements
#pragma unroll
            for (int e = 0; e < V; ++e) row_s[c + e] *= c < nq ? iq * p.q_gain[c + e] : ik * p.k_gain[c + e - nq];
    } else if (p.q_gain) {
        __syncthreads();
        const int wave = tid / SIA_WAVE, lane = tid % SIA_WAVE;
        for (int h = wave; h < p.n_heads + p.n_kv; h += ROWP_THREADS / SIA_WAVE) {
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
    for (int c = tid * V; c < nqk; c += ROWP_THREADS * V) {
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
        for (int i = tid; i < p.n_heads * gap; i += ROWP_THREADS)
            ((T*)p.q_out)[((size_t)n * p.n_heads + i / gap) * p.q_head_stride + D + i % gap] = from_float<T>(0.f);
}

SIA_EXPORT int sia_row_prepare_max_elements() { return ROWP_MAX_ELEMENTS; }

// q_col, k_col, v_col: where the three runs of columns start; state: ring of taps rows of [q | k | v] channels (null with
// one tap); conv [taps][channels] or null (taps must then be 1); neighbours: which elements the rotation pairs.
SIA_EXPORT int sia_row_prepare(const void* proj, int row_stride, int q_col, int k_col, int v_col, const float* bias,
                               const float* conv, int taps, const float* q_gain, const float* k_gain, float eps,
                               int over_row, const float* cos_table, const float* sin_table, int rotary_dim,
                               int neighbours, const int* positions, const int* seq_of_token, const int* cu_q,
                               const int* slots, const int* block_table, int table_width, float* state,
                               long long state_stride, void* k_pages, void* v_pages, void* q_out, int n_tokens,
                               int n_seqs, int max_q_len, int n_heads, int n_kv, int head_dim, int value_dim,
                               int page_size, int k_row, int v_rows, int q_head_stride, int dtype, hipStream_t stream) {
    if (n_tokens <= 0 || n_seqs <= 0) return 0;
    RowPrepare p{};
    p.cols = RingColumns{{q_col, k_col, v_col}, {n_heads * head_dim, n_kv * head_dim, n_kv * value_dim}};
    const int nqk = p.cols.size[0] + p.cols.size[1];
    if (n_heads <= 0 || n_kv <= 0 || head_dim <= 0 || value_dim <= 0 || nqk > ROWP_MAX_ELEMENTS || taps < 1 ||
        taps > RING_MAX_TAPS || (taps > 1 && (!conv || !state || state_stride < (long long)taps * p.cols.channels())) ||
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
    const bool vec = head_dim % 8 == 0 && row_stride % 8 == 0 && q_col % 8 == 0 && k_col % 8 == 0 && k_row % 8 == 0 &&
                     q_head_stride % 8 == 0 && ((uintptr_t)proj % 16) == 0;
    dim3 grid(n_tokens, 2), block(ROWP_THREADS);
    const size_t lds = (size_t)nqk * sizeof(float);
#define LAUNCH(T)                                                                                      \
    do {                                                                                               \
        if (vec) hipLaunchKernelGGL((row_prepare_kernel<T, 8>), grid, block, lds, stream, p);          \
        else hipLaunchKernelGGL((row_prepare_kernel<T, 1>), grid, block, lds, stream, p);              \
        if (!p.single)                                                                                 \
            launch_ring_keep<T>((const T*)proj, row_stride, p.cols, bias, state, state_stride, 0, taps, cu_q, positions, \
                                slots, n_seqs, stream);                                                \
    } while (0)
    if (dtype == SIA_F32) LAUNCH(float);
    else LAUNCH(bf16_t);
#undef LAUNCH
    return SIA_LAUNCH_CHECK();
}
