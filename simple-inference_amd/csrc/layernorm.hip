// The residual sum with a layer norm behind it, in one kernel, and the sum alone:
//
//   x   = residual[row] + d            d = delta[row], or with a post gain  delta[row] * rsqrt(mean(delta[row]^2) + post_eps) * post
//   out = (x - mean(x)) * rsqrt(mean((x - mean(x))^2) + eps) * w + b         (with w, b)
//   out = x rounded to T                                                     (without)
//
// The post gain belongs to a result that passes an RMS norm of its own on its way into the residual.  All of it is
// float with one rounding of out; the variance is the mean of the squared deviations, taken after the mean.  Without
// ``rows`` x goes back into residual[row]; with ``rows`` only those rows are normed and the residual stays as it was.
// Every sum is reduced in a fixed order that depends on the row length only.
#include "common.h"

template <typename T>
__global__ void add_layernorm_kernel(float* __restrict__ residual, const T* __restrict__ delta,
                                     const float* __restrict__ post, float post_eps, const float* __restrict__ weight,
                                     const float* __restrict__ bias, T* __restrict__ out, const int* __restrict__ rows,
                                     int hidden, float eps) {
    __shared__ float scratch[16];
    const int i_out = blockIdx.x;
    const int row = rows ? rows[i_out] : i_out;
    float* res = residual + (size_t)row * hidden;
    const T* del = delta ? delta + (size_t)row * hidden : nullptr;
    T* dst = out ? out + (size_t)i_out * hidden : nullptr;
    float scale = 1.f;
    if (del && post) {   // uniform
        float ss = 0.f;
        for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
            const float d = to_float(del[i]);
            ss += d * d;
        }
        scale = rsqrtf(block_sum(ss, scratch) / (float)hidden + post_eps);
    }
    // the sum of element i: read again in every pass where the residual is not written
    auto sum_at = [&](int i) { return del ? res[i] + (post ? to_float(del[i]) * scale * post[i] : to_float(del[i])) : res[i]; };
    float total = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float x = sum_at(i);
        total += x;
        if (!rows && del) res[i] = x;    // an element is this thread's alone in every pass
        if (!weight && dst) dst[i] = from_float<T>(x);
    }
    if (!weight) return;   // uniform
    auto x_at = [&](int i) { return rows ? sum_at(i) : res[i]; };
    const float mean = block_sum(total, scratch) / (float)hidden;
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        const float d = x_at(i) - mean;
        ss += d * d;
    }
    const float inv = rsqrtf(block_sum(ss, scratch) / (float)hidden + eps);
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = from_float<T>((x_at(i) - mean) * inv * weight[i] + bias[i]);
}

// The same for rows that one workgroup holds in registers (hidden % 8 == 0, hidden <= 8 * 1024): 8 elements a thread,
// every input read once and requested before the first is used.
template <typename T>
__global__ void add_layernorm_row_kernel(float* __restrict__ residual, const T* __restrict__ delta,
                                         const float* __restrict__ post, float post_eps,
                                         const float* __restrict__ weight, const float* __restrict__ bias,
                                         T* __restrict__ out, const int* __restrict__ rows, int hidden, float eps) {
    __shared__ float scratch[16];
    const int i_out = blockIdx.x;
    const int row = rows ? rows[i_out] : i_out;
    const int i0 = threadIdx.x * 8;
    const bool live = i0 < hidden;
    float x[8] = {}, d[8] = {}, p[8] = {}, w[8] = {}, b[8] = {};
    Vec8<float> vr;
    if (live) {
        Vec8<float> vp, vw, vb;
        Vec8<T> vd;
        vr.load(residual + (size_t)row * hidden + i0);
        if (delta) vd.load(delta + (size_t)row * hidden + i0);
        if (delta && post) vp.load(post + i0);
        if (weight) {
            vw.load(weight + i0);
            vb.load(bias + i0);
        }
        vr.get(x);
        if (delta) vd.get(d);
        if (delta && post) vp.get(p);
        if (weight) {
            vw.get(w);
            vb.get(b);
        }
    }
    if (delta && post) {   // uniform
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += d[i] * d[i];
        const float scale = rsqrtf(block_sum(ss, scratch) / (float)hidden + post_eps);
#pragma unroll
        for (int i = 0; i < 8; ++i) d[i] = d[i] * scale * p[i];
    }
    float total = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        x[i] += d[i];      // lanes beyond the row hold zeros
        total += x[i];
    }
    if (live && delta && !rows) {
        vr.set(x);
        vr.store(residual + (size_t)row * hidden + i0);
    }
    Vec8<T> vo;
    if (!weight) {   // uniform
        if (live && out) {
            vo.set(x);
            vo.store(out + (size_t)i_out * hidden + i0);
        }
        return;
    }
    const float mean = block_sum(total, scratch) / (float)hidden;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        x[i] = live ? x[i] - mean : 0.f;
        ss += x[i] * x[i];
    }
    const float inv = rsqrtf(block_sum(ss, scratch) / (float)hidden + eps);
    if (!live) return;
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = x[i] * inv * w[i] + b[i];
    vo.set(x);
    vo.store(out + (size_t)i_out * hidden + i0);
}

// weight and bias come together or not at all; without them (the sum alone) rows must be absent and out may be.
SIA_EXPORT int sia_add_layernorm(float* residual, const void* delta, const float* post, float post_eps,
                                 const float* weight, const float* bias, void* out, const int* rows, int n_out,
                                 int hidden, float eps, int dtype, hipStream_t stream) {
    if (n_out <= 0) return 0;
    if ((dtype != SIA_F32 && dtype != SIA_BF16) || !residual || hidden <= 0 || (weight != nullptr) != (bias != nullptr) ||
        (weight && !out) || (!weight && rows) || (!delta && post))
        return SIA_BAD_ARGUMENT;
    const bool row_form = hidden % 8 == 0 && hidden <= 8 * 1024;
    dim3 grid(n_out), block(row_form ? ((hidden / 8 + SIA_WAVE - 1) / SIA_WAVE) * SIA_WAVE : hidden >= 2048 ? 512 : 256);
#define LAUNCH(KERNEL, T)                                                                                            \
    hipLaunchKernelGGL(KERNEL<T>, grid, block, 0, stream, residual, (const T*)delta, post, post_eps, weight, bias,   \
                       (T*)out, rows, hidden, eps)
    if (row_form && dtype == SIA_F32) LAUNCH(add_layernorm_row_kernel, float);
    else if (row_form) LAUNCH(add_layernorm_row_kernel, bf16_t);
    else if (dtype == SIA_F32) LAUNCH(add_layernorm_kernel, float);
    else LAUNCH(add_layernorm_kernel, bf16_t);
#undef LAUNCH
    return SIA_LAUNCH_CHECK();
}
