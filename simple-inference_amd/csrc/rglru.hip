// The recurrent block of a real-gated linear recurrent unit: a diagonal recurrence of width W whose decay the input decides.
//
//   u     = conv(x + x_bias) + conv_bias                  causal, per channel, inputs kept in a ring (ring_conv.h)
//   r, i  = sigmoid(R_b u_b + r_bias), sigmoid(I_b u_b + i_bias)       per block b of bs channels, R, I [blocks, bs, bs]
//   log a = -r * rate                                     rate = 8 softplus(lam), from the host
//   S_t   = a S_(t-1) + sqrt(1 - a^2) i u                 float, kept in the sequence's state row, S first, then the ring
//   out   = S_t * gelu(y + y_bias)                        tanh form
//
// x and y are columns of the projected rows.
//
// Steps of single tokens in bfloat16 are one kernel: a workgroup takes 16 channels of a block for up to 16 tokens,
// makes the block's u in LDS (every workgroup of a block makes it anew: taps loads an element), takes both gate products with
// v_mfma_f32_16x16x32_bf16 (four waves: two matrices by two halves of the block's width) and advances its channels.
//
// Other steps cut each run into chunks of 64 tokens.  Inside a chunk the recurrence from zero and the product of the
// decays are taken where the gates are made (64 tokens by 64 channels a workgroup, a scan through LDS, four segments of 16
// tokens each): S_t = local_t + product_t * carry.  Then one thread a channel walks the chunks' ends and leaves every
// chunk's carry and the sequence's state, and the last kernel puts the pieces together behind the other branch's gate.
// A thread a channel does the gates' products where the matrix cores cannot (float32, odd block sizes), the scan then has a
// kernel of its own.
#include "ring_conv.h"

#define RG_CHUNK 64
#define RG_MAX_BLOCK 1024      // channels of a block that the one-kernel form holds in LDS

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 rg_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float rg_floatx4;

struct LinearUnit {
    const void* proj;
    int row_stride, y_col, x_col;
    const float *y_bias, *x_bias, *conv, *conv_bias;     // conv [taps][W]
    const void *ra, *ri;
    const float *ra_bias, *ri_bias, *rate;
    float* state;
    long long state_stride;
    const int *positions, *seq_of_token, *cu_q, *slots;
    void* out;
    int n_tokens, n_seqs, width, blocks, bs, taps;
};

__device__ __forceinline__ float rg_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }

// decay and what is written, from the two gates' logits
__device__ __forceinline__ void rg_terms(float zr, float zi, float rate, float u, float& a, float& b) {
    const float log_a = -rg_sigmoid(zr) * rate;
    a = expf(log_a);
    b = sqrtf(-expm1f(2.f * log_a)) * rg_sigmoid(zi) * u;
}

// A chunk's place in the summaries: runs of a step get disjoint ranges (a run of n tokens has at most
// (begin + n) / 64 - begin / 64 + 1 chunks).
__device__ __forceinline__ int rg_chunk_id(int run_begin, int seq, int chunk) { return run_begin / RG_CHUNK + seq + chunk; }

// The run that chunk ``id`` belongs to: the last one whose range starts at or before it (the ranges' starts grow strictly).
__device__ __forceinline__ int rg_run_of(int id, const int* __restrict__ cu_q, int n_seqs) {
    int lo = 0, hi = n_seqs - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) / 2;
        if (cu_q[mid] / RG_CHUNK + mid <= id) lo = mid;
        else hi = mid - 1;
    }
    return lo;
}

// ---------------------------------------------------------------------------------------------------------------
// A thread a channel, eight tokens a workgroup.
#define RG_TOKENS 8
template <typename T>
__global__ __launch_bounds__(256) void rg_gates_kernel(const LinearUnit p, const T* __restrict__ u, float* __restrict__ prod,
                                                       float* __restrict__ local) {
    const int n0 = blockIdx.x * RG_TOKENS, c = blockIdx.y * blockDim.x + threadIdx.x;
    if (c >= p.width) return;
    const int nt = min(RG_TOKENS, p.n_tokens - n0), first = c / p.bs * p.bs;
    const T *wr = (const T*)p.ra + (size_t)c * p.bs, *wi = (const T*)p.ri + (size_t)c * p.bs;
    float zr[RG_TOKENS], zi[RG_TOKENS];
#pragma unroll
    for (int t = 0; t < RG_TOKENS; ++t) {
        zr[t] = p.ra_bias[c];
        zi[t] = p.ri_bias[c];
    }
    for (int k = 0; k < p.bs; ++k) {
        const float a = to_float(wr[k]), b = to_float(wi[k]);
#pragma unroll
        for (int t = 0; t < RG_TOKENS; ++t) {
            const float x = to_float(u[(size_t)(n0 + min(t, nt - 1)) * p.width + first + k]);
            zr[t] += a * x;
            zi[t] += b * x;
        }
    }
#pragma unroll
    for (int t = 0; t < RG_TOKENS; ++t) {
        if (t >= nt) continue;
        const size_t at = (size_t)(n0 + t) * p.width + c;
        rg_terms(zr[t], zi[t], p.rate[c], to_float(u[at]), prod[at], local[at]);
    }
}

// In place: decays become their running product from the chunk's start, what is written the chunk's own recurrence.
__global__ __launch_bounds__(256) void rg_scan_kernel(const LinearUnit p, float* __restrict__ prod, float* __restrict__ local,
                                                      float* __restrict__ end_prod, float* __restrict__ end_local) {
    const int c = blockIdx.y * blockDim.x + threadIdx.x;
    const int seq = rg_run_of(blockIdx.x, p.cu_q, p.n_seqs), begin = p.cu_q[seq], chunk = blockIdx.x - rg_chunk_id(begin, seq, 0);
    const int t0 = begin + chunk * RG_CHUNK, t1 = min(t0 + RG_CHUNK, p.cu_q[seq + 1]);
    if (c >= p.width || t0 >= t1) return;
    float A = 1.f, S = 0.f;
    for (int t = t0; t < t1; ++t) {
        const size_t at = (size_t)t * p.width + c;
        A *= prod[at];
        S = prod[at] * S + local[at];
        prod[at] = A;
        local[at] = S;
    }
    const size_t id = (size_t)rg_chunk_id(begin, seq, chunk) * p.width + c;
    end_prod[id] = A;
    end_local[id] = S;
}

// Gates on the matrix cores with the chunk's scan behind them: 64 tokens of a run by 64 channels of a block.
#define RG_PAD 68
__global__ __launch_bounds__(256) void rg_gates_mfma_kernel(const LinearUnit p, const bf16_t* __restrict__ u,
                                                            float* __restrict__ prod, float* __restrict__ local,
                                                            float* __restrict__ end_prod, float* __restrict__ end_local,
                                                            int tiles) {
    __shared__ __attribute__((aligned(16))) float a_s[RG_CHUNK][RG_PAD];
    __shared__ __attribute__((aligned(16))) float b_s[RG_CHUNK][RG_PAD];
    __shared__ float seg_a[4][64], seg_b[4][64];
    const int seq = rg_run_of(blockIdx.x, p.cu_q, p.n_seqs), begin = p.cu_q[seq], chunk = blockIdx.x - rg_chunk_id(begin, seq, 0);
    const int t0 = begin + chunk * RG_CHUNK, nt = min(RG_CHUNK, p.cu_q[seq + 1] - t0);
    if (nt <= 0) return;      // uniform
    const int block = blockIdx.y / tiles, j0 = (blockIdx.y % tiles) * 64;      // channels j0 .. of the block
    const int wave = threadIdx.x / SIA_WAVE, lane = threadIdx.x % SIA_WAVE, r = lane & 15, g = lane >> 4;
    const int jw = j0 + wave * 16;      // this wave's 16 channels
    const size_t row = (size_t)block * p.bs + min(jw + r, p.bs - 1);
    const bf16_t *wr = (const bf16_t*)p.ra + row * p.bs + g * 8, *wi = (const bf16_t*)p.ri + row * p.bs + g * 8;
    const bf16_t* x[4];
#pragma unroll
    for (int mb = 0; mb < 4; ++mb) x[mb] = u + (size_t)(t0 + min(mb * 16 + r, nt - 1)) * p.width + block * p.bs + g * 8;
    rg_floatx4 acc[2][4];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int mb = 0; mb < 4; ++mb) acc[m][mb] = rg_floatx4{0.f, 0.f, 0.f, 0.f};
    const rg_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll 2
    for (int k = 0; k < p.bs; k += 32) {
        const bool live = k + g * 8 < p.bs;      // bs is a multiple of 8: a lane's piece is inside or outside
        const rg_bf16x8 fr = live ? *reinterpret_cast<const rg_bf16x8*>(wr + k) : zero;
        const rg_bf16x8 fi = live ? *reinterpret_cast<const rg_bf16x8*>(wi + k) : zero;
        rg_bf16x8 b[4];
#pragma unroll
        for (int mb = 0; mb < 4; ++mb) b[mb] = live ? *reinterpret_cast<const rg_bf16x8*>(x[mb] + k) : zero;
#pragma unroll
        for (int mb = 0; mb < 4; ++mb) {
            acc[0][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fr, b[mb], acc[0][mb], 0, 0, 0);
            acc[1][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fi, b[mb], acc[1][mb], 0, 0, 0);
        }
    }
    // acc[.][mb][i]: channel jw + 4g + i of token t0 + mb * 16 + r
    const int jl = jw + 4 * g;
    if (jl < p.bs) {      // bs % 8 == 0: four channels are inside or outside together
        const int c = block * p.bs + jl;
        float br[4], bi[4], rate[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            br[i] = p.ra_bias[c + i];
            bi[i] = p.ri_bias[c + i];
            rate[i] = p.rate[c + i];
        }
#pragma unroll
        for (int mb = 0; mb < 4; ++mb) {
            const int t = mb * 16 + r;
            const uint2 uw = *reinterpret_cast<const uint2*>(u + (size_t)(t0 + min(t, nt - 1)) * p.width + c);
            const float uv[4] = {__uint_as_float(uw.x << 16), __uint_as_float(uw.x & 0xffff0000u),
                                 __uint_as_float(uw.y << 16), __uint_as_float(uw.y & 0xffff0000u)};
            float a[4], b[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                rg_terms(acc[0][mb][i] + br[i], acc[1][mb][i] + bi[i], rate[i], uv[i], a[i], b[i]);
                if (t >= nt) { a[i] = 1.f; b[i] = 0.f; }      // beyond the run: nothing changes
            }
            *reinterpret_cast<float4*>(&a_s[t][jl - j0]) = make_float4(a[0], a[1], a[2], a[3]);
            *reinterpret_cast<float4*>(&b_s[t][jl - j0]) = make_float4(b[0], b[1], b[2], b[3]);
        }
    }
    __syncthreads();
    const bool live = j0 + lane < p.bs;      // from here on: lane = channel, wave = segment of 16 tokens
    float A = 1.f, S = 0.f;
    if (live) {
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            const float a = a_s[wave * 16 + t][lane];
            A *= a;
            S = a * S + b_s[wave * 16 + t][lane];
            a_s[wave * 16 + t][lane] = A;
            b_s[wave * 16 + t][lane] = S;
        }
        seg_a[wave][lane] = A;
        seg_b[wave][lane] = S;
    }
    __syncthreads();
    if (!live) return;
    float Ap = 1.f, Sp = 0.f;      // the segments before this one
    for (int w = 0; w < wave; ++w) {
        Sp = seg_a[w][lane] * Sp + seg_b[w][lane];
        Ap *= seg_a[w][lane];
    }
    const int c = block * p.bs + j0 + lane;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
        if (wave * 16 + t >= nt) break;
        const float a = a_s[wave * 16 + t][lane];
        const size_t at = (size_t)(t0 + wave * 16 + t) * p.width + c;
        prod[at] = a * Ap;
        local[at] = b_s[wave * 16 + t][lane] + a * Sp;
    }
    if (wave == 3) {
        const size_t id = (size_t)rg_chunk_id(begin, seq, chunk) * p.width + c;
        end_prod[id] = A * Ap;
        end_local[id] = S + A * Sp;
    }
}

// Every chunk's carry (into end_local) and the sequence's state after the step.
__global__ __launch_bounds__(64) void rg_carry_kernel(const LinearUnit p, const float* __restrict__ end_prod,
                                                      float* __restrict__ end_local) {
    const int seq = blockIdx.x, c = blockIdx.y * blockDim.x + threadIdx.x;
    const int begin = p.cu_q[seq], n = p.cu_q[seq + 1] - begin;
    if (c >= p.width || n <= 0) return;
    float* st = p.state + (size_t)p.slots[seq] * p.state_stride + c;
    float S = *st;
    const size_t base = (size_t)rg_chunk_id(begin, seq, 0) * p.width + c;
    const int chunks = (n + RG_CHUNK - 1) / RG_CHUNK;
    constexpr int AHEAD = 8;
    for (int k = 0; k < chunks; k += AHEAD) {
        float A[AHEAD], B[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            const size_t at = base + (size_t)min(k + i, chunks - 1) * p.width;
            A[i] = end_prod[at];
            B[i] = end_local[at];
        }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            if (k + i >= chunks) break;
            end_local[base + (size_t)(k + i) * p.width] = S;
            S = A[i] * S + B[i];
        }
    }
    *st = S;
}

template <typename T, int V>
__global__ __launch_bounds__(256) void rg_finish_kernel(const LinearUnit p, const float* __restrict__ prod,
                                                        const float* __restrict__ local, const float* __restrict__ carry) {
    const int n = blockIdx.x, c = (blockIdx.y * blockDim.x + threadIdx.x) * V;
    if (c >= p.width) return;
    const int seq = p.seq_of_token[n], begin = p.cu_q[seq];
    const size_t at = (size_t)n * p.width + c;
    const size_t id = (size_t)rg_chunk_id(begin, seq, (n - begin) / RG_CHUNK) * p.width + c;
    const T* yp = (const T*)p.proj + (size_t)n * p.row_stride + p.y_col + c;
    float A[V], S[V], C[V], y[V];
    if constexpr (V == 8) {
        Vec8<float> a, s, k;
        Vec8<T> v;
        a.load(prod + at);
        s.load(local + at);
        k.load(carry + id);
        v.load(yp);
        a.get(A);
        s.get(S);
        k.get(C);
        v.get(y);
    } else {
        A[0] = prod[at];
        S[0] = local[at];
        C[0] = carry[id];
        y[0] = to_float(yp[0]);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) S[e] = (S[e] + A[e] * C[e]) * activate(y[e] + p.y_bias[c + e], SIA_GELU_TANH);
    T* dst = (T*)p.out + at;
    if constexpr (V == 8) {
        Vec8<T> v;
        v.set(S);
        v.store(dst);
    } else {
        dst[0] = from_float<T>(S[0]);
    }
}

// A step of single tokens, bfloat16: 16 channels of a block for up to 16 tokens.
template <int TAPS>      // 0: any number
__global__ __launch_bounds__(256) void rg_decode_kernel(const LinearUnit p, int tiles) {
    extern __shared__ __attribute__((aligned(16))) bf16_t u_s[];      // [16][bs + 8]
    __shared__ float part[4][16][17];
    const int block = blockIdx.x / tiles, j0 = (blockIdx.x % tiles) * 16, m0 = blockIdx.y * 16;
    const int M = min(16, p.n_tokens - m0), tid = threadIdx.x, pitch = p.bs + 8, pieces = p.bs / 8;
    const bf16_t* proj = (const bf16_t*)p.proj;
    for (int idx = tid; idx < 16 * pieces; idx += 256) {
        const int m = idx / pieces, j = (idx % pieces) * 8, c = block * p.bs + j;
        float acc[8] = {}, own[8];
        if (m < M) {
            const int n = m0 + m, pos = p.positions[n];
            float* ring = p.state + (size_t)p.slots[p.seq_of_token[n]] * p.state_stride + p.width;
            if constexpr (TAPS > 0)
                ring_conv_single<bf16_t, 8, TAPS>(proj, p.row_stride, p.x_col + c, c, p.width, p.x_bias, p.conv, ring, n, pos, acc, own);
            else
                ring_conv<bf16_t, 8>(proj, p.row_stride, p.x_col + c, c, p.width, p.x_bias, p.conv, p.taps, ring, n, n, pos, acc, own);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[e] += p.conv_bias[c + e];
            // this workgroup's own channels: the input goes into the ring row that no token of the step reads
            if (p.taps > 1 && j >= j0 && j < j0 + 16) {
#pragma unroll
                for (int e = 0; e < 8; ++e) ring[(size_t)(pos % p.taps) * p.width + c + e] = own[e];
            }
        }
        Vec8<bf16_t> v;
        v.set(acc);
        v.store(u_s + m * pitch + j);
    }
    __syncthreads();
    const int wave = tid / SIA_WAVE, lane = tid % SIA_WAVE, r = lane & 15, g = lane >> 4;
    const size_t row = (size_t)block * p.bs + min(j0 + r, p.bs - 1);
    const bf16_t* w = (const bf16_t*)((wave & 1) ? p.ri : p.ra) + row * p.bs + g * 8;
    const bf16_t* x = u_s + r * pitch + g * 8;
    rg_floatx4 acc = {0.f, 0.f, 0.f, 0.f};
    const rg_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll 2
    for (int k = (wave >> 1) * 32; k < p.bs; k += 64) {
        const bool live = k + g * 8 < p.bs;
        const rg_bf16x8 a = live ? *reinterpret_cast<const rg_bf16x8*>(w + k) : zero;
        const rg_bf16x8 b = live ? *reinterpret_cast<const rg_bf16x8*>(x + k) : zero;
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave][4 * g + i][r] = acc[i];      // channel 4g + i of token r
    __syncthreads();
    const int m = tid / 16, j = j0 + tid % 16, c = block * p.bs + j, n = m0 + m;
    if (m >= M || j >= p.bs) return;
    float a, b;
    rg_terms(part[0][tid % 16][m] + part[2][tid % 16][m] + p.ra_bias[c],
             part[1][tid % 16][m] + part[3][tid % 16][m] + p.ri_bias[c], p.rate[c], bf16_to_float(u_s[m * pitch + j]), a, b);
    float* st = p.state + (size_t)p.slots[p.seq_of_token[n]] * p.state_stride + c;
    const float S = a * *st + b;
    *st = S;
    const float y = bf16_to_float(proj[(size_t)n * p.row_stride + p.y_col + c]) + p.y_bias[c];
    ((bf16_t*)p.out)[(size_t)n * p.width + c] = float_to_bf16(S * activate(y, SIA_GELU_TANH));
}

SIA_EXPORT int sia_linear_unit_max_taps() { return RING_MAX_TAPS; }

// Floats of workspace of a step: the convolved inputs (as floats' worth of room), running products, local states, and two
// summaries a chunk.
SIA_EXPORT long long sia_linear_unit_workspace(int n_tokens, int n_seqs, int width) {
    const long long w8 = (width + 7) / 8 * 8;
    return w8 * (3LL * n_tokens + 2LL * (n_tokens / RG_CHUNK + n_seqs + 1)) + 32;
}

SIA_EXPORT int sia_linear_unit(const void* proj, int row_stride, int y_col, int x_col, const float* y_bias,
                               const float* x_bias, const float* conv, const float* conv_bias, const void* ra,
                               const float* ra_bias, const void* ri, const float* ri_bias, const float* rate, float* state,
                               long long state_stride, const int* positions, const int* seq_of_token, const int* cu_q,
                               const int* slots, void* out, int n_tokens, int n_seqs, int max_q_len, int width, int blocks,
                               int taps, int dtype, float* workspace, hipStream_t stream) {
    if (n_tokens <= 0 || n_seqs <= 0) return 0;
    if (width <= 0 || blocks <= 0 || width % blocks || taps < 1 || taps > RING_MAX_TAPS || !proj || !y_bias || !x_bias ||
        !conv || !conv_bias || !ra || !ri || !ra_bias || !ri_bias || !rate || !state || !out || !workspace || y_col < 0 ||
        x_col < 0 || y_col + width > row_stride || x_col + width > row_stride ||
        state_stride < (long long)width * (1 + (taps > 1 ? taps : 0)) || (dtype != SIA_F32 && dtype != SIA_BF16))
        return SIA_BAD_ARGUMENT;
    const int bs = width / blocks;
    LinearUnit p{proj, row_stride, y_col, x_col, y_bias, x_bias, conv, conv_bias, ra, ri, ra_bias, ri_bias, rate, state,
                 state_stride, positions, seq_of_token, cu_q, slots, out, n_tokens, n_seqs, width, blocks, bs, taps};
    const bool rows8 = width % 8 == 0 && row_stride % 8 == 0 && x_col % 8 == 0 && y_col % 8 == 0 && ((uintptr_t)proj % 16) == 0;
    const bool cores = dtype == SIA_BF16 && rows8 && bs % 8 == 0 && ((uintptr_t)ra % 16) == 0 && ((uintptr_t)ri % 16) == 0;
    if (cores && max_q_len <= 1 && bs <= RG_MAX_BLOCK) {
        const int tiles = (bs + 15) / 16;
        dim3 grid(blocks * tiles, (n_tokens + 15) / 16), block(256);
        const size_t lds = (size_t)16 * (bs + 8) * sizeof(bf16_t);
        const bool wide = state_stride % 4 == 0 && ((uintptr_t)state % 16) == 0;      // rows in 16-byte pieces
        if (taps == 1) hipLaunchKernelGGL(rg_decode_kernel<1>, grid, block, lds, stream, p, tiles);
        else if (taps == 2 && wide) hipLaunchKernelGGL(rg_decode_kernel<2>, grid, block, lds, stream, p, tiles);
        else if (taps == 3 && wide) hipLaunchKernelGGL(rg_decode_kernel<3>, grid, block, lds, stream, p, tiles);
        else if (taps == 4 && wide) hipLaunchKernelGGL(rg_decode_kernel<4>, grid, block, lds, stream, p, tiles);
        else hipLaunchKernelGGL(rg_decode_kernel<0>, grid, block, lds, stream, p, tiles);
        return SIA_LAUNCH_CHECK();
    }
    const size_t w8 = (width + 7) / 8 * 8, chunks = (size_t)n_tokens / RG_CHUNK + n_seqs + 1;
    float* u = workspace;
    float* prod = u + w8 * n_tokens;
    float* local = prod + w8 * n_tokens;
    float* end_prod = local + w8 * n_tokens;
    float* end_local = end_prod + w8 * chunks;
    const dim3 block(256), by8(n_tokens, (width / 8 + 255) / 256), by1(n_tokens, (width + 255) / 256);
    const RingColumns cols{{x_col, 0, 0}, {width, 0, 0}};
#define RUN(T)                                                                                                       \
    do {                                                                                                             \
        launch_ring_conv<T>((const T*)proj, row_stride, cols, x_bias, conv, conv_bias, state, state_stride, width, taps, \
                            cu_q, seq_of_token, positions, slots, (T*)u, width, n_tokens, rows8, stream);            \
        launch_ring_keep<T>((const T*)proj, row_stride, cols, x_bias, state, state_stride, width, taps, cu_q,        \
                            positions, slots, n_seqs, stream);                                                       \
        if (cores) {                                                                                                 \
            const int tiles = (bs + 63) / 64;                                                                        \
            hipLaunchKernelGGL(rg_gates_mfma_kernel, dim3((unsigned)chunks, blocks * tiles), block, 0, stream, p,    \
                               (const bf16_t*)u, prod, local, end_prod, end_local, tiles);                           \
        } else {                                                                                                     \
            hipLaunchKernelGGL(rg_gates_kernel<T>, dim3((n_tokens + RG_TOKENS - 1) / RG_TOKENS, (width + 255) / 256), \
                               block, 0, stream, p, (const T*)u, prod, local);                                       \
            hipLaunchKernelGGL(rg_scan_kernel, dim3((unsigned)chunks, (width + 255) / 256), block, 0, stream, p,     \
                               prod, local, end_prod, end_local);                                                    \
        }                                                                                                            \
        hipLaunchKernelGGL(rg_carry_kernel, dim3(n_seqs, (width + 63) / 64), dim3(64), 0, stream, p, end_prod, end_local); \
        if (rows8) hipLaunchKernelGGL((rg_finish_kernel<T, 8>), by8, block, 0, stream, p, prod, local, end_local);   \
        else hipLaunchKernelGGL((rg_finish_kernel<T, 1>), by1, block, 0, stream, p, prod, local, end_local);         \
    } while (0)
    if (dtype == SIA_F32) RUN(float);
    else RUN(bf16_t);
#undef RUN
    return SIA_LAUNCH_CHECK();
}
