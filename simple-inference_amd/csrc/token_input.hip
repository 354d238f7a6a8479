// What a layer takes of the token itself:  out[n, i] = act(z[n, i]) * table[ids[n], first + i]   (i < dim; 0 beyond)
//
// z are the products of the stream with the layer's gate matrix, rows of ``width`` >= dim elements; the table's rows
// are table_width apart.  Float, one rounding.  (For few rows the same is the epilogue of the product's own kernel.)
#include "common.h"

template <typename T>
__global__ __launch_bounds__(256) void embedding_gate_kernel(const T* __restrict__ z, T* __restrict__ out,
                                                             const T* __restrict__ table, int table_width, int first,
                                                             int dim, const int* __restrict__ ids, int width, int kind) {
    const int n = blockIdx.x;
    const T* e = table + (size_t)ids[n] * table_width + first;
    for (int i = blockIdx.y * blockDim.x + threadIdx.x; i < width; i += gridDim.y * blockDim.x)
        out[(size_t)n * width + i] =
            i < dim ? from_float<T>(activate(to_float(z[(size_t)n * width + i]), kind) * to_float(e[i])) : from_float<T>(0.f);
}

SIA_EXPORT int sia_embedding_gate(const void* z, void* out, const void* table, int table_width, int first, int dim,
                                  const int* ids, int n_tokens, int width, int activation, int dtype, hipStream_t stream) {
    if (n_tokens <= 0) return 0;
    if (!z || !out || !table || !ids || dim <= 0 || width < dim || first < 0 || first + dim > table_width ||
        (activation != SIA_RELU2 && activation != SIA_GELU_TANH && activation != SIA_GELU))
        return SIA_BAD_ARGUMENT;
    const int across = (width + 255) / 256;
    dim3 grid(n_tokens, across < 65535 ? across : 65535), block(256);
    if (dtype == SIA_F32)
        hipLaunchKernelGGL(embedding_gate_kernel<float>, grid, block, 0, stream, (const float*)z, (float*)out,
                           (const float*)table, table_width, first, dim, ids, width, activation);
    else if (dtype == SIA_BF16)
        hipLaunchKernelGGL(embedding_gate_kernel<bf16_t>, grid, block, 0, stream, (const bf16_t*)z, (bf16_t*)out,
                           (const bf16_t*)table, table_width, first, dim, ids, width, activation);
    else
        return SIA_BAD_ARGUMENT;
    return SIA_LAUNCH_CHECK();
}
