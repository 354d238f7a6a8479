// The second products of two low-rank pairs, with what a recurrence makes of their results, all in float:
//
//   decay[n, h, c] = exp(-exp(A_log[h]) * softplus(sum_m a[n, m] * A2[h * D + c, m] + dt_bias[h * D + c]))
//   gate[n, j]     = sigmoid(sum_m g[n, m] * G2[j, m])
//
// or, for a recurrence whose decay goes through one pair with a tanh inside (``sia_low_rank_decay``),
//
//   decay[n, c]    = exp(-exp(sum_m tanh(a[n, m]) * W2[c, m] + w0[c]))
//
// a [rank_a] and g [rank_g] are columns of the projected rows (row_stride apart), A2 [H * D, rank_a] and G2
// [gates, rank_g] the pairs' second matrices; both results are float, [tokens, H * D] and [tokens, gates].  They do not
// depend on the recurrence's state, so a step's tokens are thousands of independent little products: one launch makes
// both (blockIdx.z says which).
//
// In bfloat16, where the 16-byte pieces of rows are aligned: v_mfma_f32_16x16x32_bf16 with the matrix's rows as first
// operand and the tokens' as second, a wave NB * 16 outputs by MB * 16 tokens; what lies beyond the rank in the last
// step of 32 is zero.  The tanh's results, floats, go in as two bfloat16 numbers each (the value and what its rounding
// left), so that nothing of the decay is rounded to 8 bits.  Otherwise (float32, odd ranks) a thread an output, eight tokens a workgroup.
#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 lr_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float lr_floatx4;

struct LowRankSide {
    const void* w;      // [outputs, rank]
    float* out;         // [tokens, outputs]
    int column, rank, outputs;
};

struct LowRankPair {
    LowRankSide side[2];            // 0: decays, 1: gates
    const float *a_log, *dt_bias;   // [outputs / per_head], [outputs] of the decays
    int per_head;                   // outputs that share an A_log
};

__device__ __forceinline__ float gate_of(float z) { return 1.f / (1.f + expf(-z)); }

// rate = exp(A_log), z with its bias
__device__ __forceinline__ float decay_of(float z, float rate) {
    return expf(-rate * (fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)))));
}

// FORM: what the second product's results become.
enum LowRankForm { LR_PAIR = 0, LR_TANH_DECAY = 1 };

#define LR_TOKENS 8
template <typename T, int FORM>
__global__ __launch_bounds__(256) void low_rank_kernel(const T* __restrict__ proj, int row_stride, const LowRankPair p,
                                                       int n_tokens) {
    extern __shared__ float in_s[];   // [LR_TOKENS][rank]
    const int which = blockIdx.z;
    const LowRankSide s = p.side[which];
    const int n0 = blockIdx.x * LR_TOKENS, nt = min(LR_TOKENS, n_tokens - n0);
    if ((int)(blockIdx.y * blockDim.x) >= s.outputs) return;   // uniform
    for (int idx = threadIdx.x; idx < nt * s.rank; idx += blockDim.x)
    {
        const float x = to_float(proj[(size_t)(n0 + idx / s.rank) * row_stride + s.column + idx % s.rank]);
        in_s[idx] = FORM == LR_TANH_DECAY ? tanhf(x) : x;
    }
    __syncthreads();
    const int o = blockIdx.y * blockDim.x + threadIdx.x;
    if (o >= s.outputs) return;
    const T* w = (const T*)s.w + (size_t)o * s.rank;
    const float bias = which ? 0.f : p.dt_bias[o], rate = which || FORM == LR_TANH_DECAY ? 0.f : expf(p.a_log[o / p.per_head]);
    float z[LR_TOKENS] = {};
    for (int m = 0; m < s.rank; ++m) {
        const float wm = to_float(w[m]);
#pragma unroll
        for (int t = 0; t < LR_TOKENS; ++t) z[t] += in_s[min(t, nt - 1) * s.rank + m] * wm;
    }
#pragma unroll
    for (int t = 0; t < LR_TOKENS; ++t)
        if (t < nt) 
            s.out[(size_t)(n0 + t) * s.outputs + o] = FORM == LR_TANH_DECAY ? expf(-expf(z[t] + bias))
                                                      : which ? gate_of(z[t]) : decay_of(z[t] + bias, rate);
}

// A workgroup four waves side by side along the outputs, all on the same MB * 16 tokens.
template <int NB, int MB, int FORM>
__global__ __launch_bounds__(256) void low_rank_mfma_kernel(const bf16_t* __restrict__ proj, int row_stride,
                                                            const LowRankPair p, int n_tokens) {
    const int which = blockIdx.z;
    const LowRankSide s = p.side[which];
    const int wave = threadIdx.x / SIA_WAVE, lane = threadIdx.x % SIA_WAVE, r = lane & 15, g = lane >> 4;
    const int t0 = blockIdx.x * MB * 16, o0 = (blockIdx.y * 4 + wave) * NB * 16;
    if (o0 >= s.outputs) return;
    const bf16_t* w = (const bf16_t*)s.w;
    const bf16_t *xp[MB], *wp[NB];
#pragma unroll
    for (int mb = 0; mb < MB; ++mb)
        xp[mb] = proj + (size_t)min(t0 + mb * 16 + r, n_tokens - 1) * row_stride + s.column + g * 8;
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) wp[nb] = w + (size_t)min(o0 + nb * 16 + r, s.outputs - 1) * s.rank + g * 8;
    // the four outputs a lane ends up with, o .. o + 3, lie in one head or reach into the next
    float bias[NB][4], rate[NB][4];
    if (which == 0) {   // uniform
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
            const int o = o0 + nb * 16 + 4 * g, head = min(o, s.outputs - 1) / p.per_head;
            const float own = FORM == LR_TANH_DECAY ? 0.f : expf(p.a_log[head]);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int c = min(o + i, s.outputs - 1);
                bias[nb][i] = p.dt_bias[c];
                rate[nb][i] = FORM == LR_TANH_DECAY || c < (head + 1) * p.per_head ? own : expf(p.a_log[c / p.per_head]);
            }
        }
    }
    lr_floatx4 acc[NB][MB];
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
        for (int mb = 0; mb < MB; ++mb) acc[nb][mb] = lr_floatx4{0.f, 0.f, 0.f, 0.f};
    const lr_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll 4
    for (int k = 0; k < s.rank; k += 32) {
        const bool live = k + g * 8 < s.rank;     // the rank is a multiple of 8: a lane's piece is inside or outside
        lr_bf16x8 a[NB], b[MB], rest[MB];
#pragma unroll
        for (int mb = 0; mb < MB; ++mb) b[mb] = live ? *reinterpret_cast<const lr_bf16x8*>(xp[mb] + k) : zero;
        if (FORM == LR_TANH_DECAY) {
#pragma unroll
            for (int mb = 0; mb < MB; ++mb) {
                Vec8<bf16_t> v, hi, lo;
                v.u = __builtin_bit_cast(uint4, b[mb]);
                float x[8], h[8];
                v.get(x);
#pragma unroll
                for (int i = 0; i < 8; ++i) x[i] = tanhf(x[i]);
                hi.set(x);
                hi.get(h);
#pragma unroll
                for (int i = 0; i < 8; ++i) x[i] -= h[i];
                lo.set(x);
                b[mb] = __builtin_bit_cast(lr_bf16x8, hi.u);
                rest[mb] = __builtin_bit_cast(lr_bf16x8, lo.u);
            }
        }
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) a[nb] = live ? *reinterpret_cast<const lr_bf16x8*>(wp[nb] + k) : zero;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb)
#pragma unroll
            for (int mb = 0; mb < MB; ++mb) {
                acc[nb][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[nb], b[mb], acc[nb][mb], 0, 0, 0);
                if (FORM == LR_TANH_DECAY)
                    acc[nb][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[nb], rest[mb], acc[nb][mb], 0, 0, 0);
            }
    }
    // acc[nb][mb][i]: output o0 + nb * 16 + 4g + i of token t0 + mb * 16 + r
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) {
        const int n = t0 + mb * 16 + r;
        if (n >= n_tokens) continue;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
            const int o = o0 + nb * 16 + 4 * g;
            float* dst = s.out + (size_t)n * s.outputs + o;
            float v[4];
#pragma unroll
            for (int i = 0; i < 4; ++i)
                v[i] = FORM == LR_TANH_DECAY ? expf(-expf(acc[nb][mb][i] + bias[nb][i]))
                       : which ? gate_of(acc[nb][mb][i]) : decay_of(acc[nb][mb][i] + bias[nb][i], rate[nb][i]);
            if (s.outputs % 4 == 0) {   // uniform; the row's pieces are whole and aligned
                if (o < s.outputs) *reinterpret_cast<float4*>(dst) = make_float4(v[0], v[1], v[2], v[3]);
                continue;
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (o + i < s.outputs) dst[i] = v[i];
        }
    }
}

// most: the larger of the sides' outputs; sides: how many there are.
template <int FORM>
static int launch_low_rank(const void* proj, int row_stride, const LowRankPair& p, int most, int sides, int most_rank,
                           bool aligned, int n_tokens, int dtype, hipStream_t stream) {
    if (dtype == SIA_BF16 && aligned) {
        const bool few = n_tokens <= 64;
        const int tokens = few ? 16 : 32, outs = few ? 64 : 128;
        dim3 grid((n_tokens + tokens - 1) / tokens, (most + outs - 1) / outs, sides), block(256);
        if (grid.y > 65535) return SIA_BAD_ARGUMENT;
        if (few)
            hipLaunchKernelGGL((low_rank_mfma_kernel<1, 1, FORM>), grid, block, 0, stream, (const bf16_t*)proj, row_stride, p, n_tokens);
        else
            hipLaunchKernelGGL((low_rank_mfma_kernel<2, 2, FORM>), grid, block, 0, stream, (const bf16_t*)proj, row_stride, p, n_tokens);
        return SIA_LAUNCH_CHECK();
    }
    dim3 grid((n_tokens + LR_TOKENS - 1) / LR_TOKENS, (most + 255) / 256, sides), block(256);
    if (grid.y > 65535) return SIA_BAD_ARGUMENT;
    const size_t lds = (size_t)LR_TOKENS * most_rank * sizeof(float);
    if (lds > 60 * 1024) return SIA_BAD_ARGUMENT;
    if (dtype == SIA_F32)
        hipLaunchKernelGGL((low_rank_kernel<float, FORM>), grid, block, lds, stream, (const float*)proj, row_stride, p, n_tokens);
    else
        hipLaunchKernelGGL((low_rank_kernel<bf16_t, FORM>), grid, block, lds, stream, (const bf16_t*)proj, row_stride, p, n_tokens);
    return SIA_LAUNCH_CHECK();
}

SIA_EXPORT int sia_low_rank_pair(const void* proj, int row_stride, int a_col, int rank_a, const void* a2,
                                 const float* a_log, const float* dt_bias, int channels, int per_head, float* decay,
                                 int g_col, int rank_g, const void* g2, int gates, float* gate, int n_tokens, int dtype,
                                 hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (rank_a <= 0 || rank_g <= 0 || rank_a > 4096 || rank_g > 4096 || channels <= 0 || gates <= 0 || per_head <= 0 ||
        channels % per_head || a_col < 0 || g_col < 0 || a_col + rank_a > row_stride || g_col + rank_g > row_stride ||
        !a2 || !g2 || !a_log || !dt_bias || !decay || !gate || (dtype != SIA_F32 && dtype != SIA_BF16))
        return SIA_BAD_ARGUMENT;
    LowRankPair p{};
    p.side[0] = LowRankSide{a2, decay, a_col, rank_a, channels};
    p.side[1] = LowRankSide{g2, gate, g_col, rank_g, gates};
    p.a_log = a_log;
    p.dt_bias = dt_bias;
    p.per_head = per_head;
    const int most = channels > gates ? channels : gates;
    const bool aligned = rank_a % 8 == 0 && rank_g % 8 == 0 && a_col % 8 == 0 && g_col % 8 == 0 && row_stride % 8 == 0 &&
                         ((uintptr_t)proj % 16) == 0 && ((uintptr_t)a2 % 16) == 0 && ((uintptr_t)g2 % 16) == 0 &&
                         ((uintptr_t)decay % 16) == 0 && ((uintptr_t)gate % 16) == 0;
    return launch_low_rank<LR_PAIR>(proj, row_stride, p, most, 2, rank_a > rank_g ? rank_a : rank_g, aligned, n_tokens, dtype,
                                    stream);
}

// decay[n, c] = exp(-exp(sum_m tanh(low[n, m]) * w2[c, m] + w0[c])), float; low rows row_stride apart.
SIA_EXPORT int sia_low_rank_decay(const void* low, int row_stride, int rank, const void* w2, const float* w0, int channels,
                                  float* decay, int n_tokens, int dtype, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (rank <= 0 || rank > 4096 || rank > row_stride || channels <= 0 || !low || !w2 || !w0 || !decay ||
        (dtype != SIA_F32 && dtype != SIA_BF16))
        return SIA_BAD_ARGUMENT;
    LowRankPair p{};
    p.side[0] = LowRankSide{w2, decay, 0, rank, channels};
    p.dt_bias = w0;
    p.per_head = channels;
    const bool aligned = rank % 8 == 0 && row_stride % 8 == 0 && ((uintptr_t)low % 16) == 0 && ((uintptr_t)w2 % 16) == 0 &&
                         ((uintptr_t)decay % 16) == 0;
    return launch_low_rank<LR_TANH_DECAY>(low, row_stride, p, channels, 1, rank, aligned, n_tokens, dtype, stream);
}
