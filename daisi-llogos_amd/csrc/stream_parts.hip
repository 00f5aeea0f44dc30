// Kernels for parts that stand between a layer's sublayers and transform the float32 residual stream: sums that
// join it, and the product of a gated projection with a row of a table chosen by the token.
#include "common.h"

// ---------------------------------------------------------------- sums into the stream
// x[t, :] += (sum of the parts of delta)[t, :] + again[t, :] + vec   (each may be absent), and the new rows also in the type
// of `rows` (or null).  delta float or bfloat16.  A thread owns VEC neighbouring values.
template <typename TD, typename TR, int VEC>
__global__ void stream_add_kernel(float* __restrict__ x, const TD* __restrict__ delta, int parts, size_t part_stride,
                                  const float* __restrict__ again, const float* __restrict__ vec, TR* __restrict__ rows, size_t n, int W) {
    const size_t i = ((size_t)blockIdx.x * blockDim.x + threadIdx.x) * VEC;
    if (i >= n) return;
    const int c = (int)(i % W);
    float v[VEC], add[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) { v[e] = x[i + e]; add[e] = 0.f; }
    if (delta) {
        for (int q = 0; q < parts; ++q)
#pragma unroll
            for (int e = 0; e < VEC; ++e) add[e] += load_f32(delta + q * part_stride + i + e);
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] += add[e];
    }
    if (again) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] += again[i + e];
    }
    if (vec) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] += vec[c + e];
    }
    if (delta || again || vec) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) x[i + e] = v[e];
    }
    if (rows) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) store_f32(rows + i + e, v[e]);
    }
}

LLOGOS_EXPORT int llogos_stream_add(float* x, const void* delta, int delta_dtype, int parts, long long part_stride, const float* again,
                                    const float* vec, void* rows, int rows_dtype, int T, int W, hipStream_t stream) {
    if (T <= 0 || W <= 0 || parts < 1) return LLOGOS_BAD_ARGUMENT;
    const size_t n = (size_t)T * W;
    const bool v4 = W % 4 == 0;
    const unsigned blocks = (unsigned)((n / (v4 ? 4 : 1) + 255) / 256);
#define SA(TD, TR) do { \
        if (v4) stream_add_kernel<TD, TR, 4><<<blocks, 256, 0, stream>>>(x, (const TD*)delta, parts, (size_t)part_stride, again, vec, (TR*)rows, n, W); \
        else stream_add_kernel<TD, TR, 1><<<blocks, 256, 0, stream>>>(x, (const TD*)delta, parts, (size_t)part_stride, again, vec, (TR*)rows, n, W); } while (0)
    if (delta_dtype == DT_F32 && rows_dtype == DT_F32) SA(float, float);
    else if (delta_dtype == DT_F32 && rows_dtype == DT_BF16) SA(float, bf16_t);
    else if (delta_dtype == DT_BF16 && rows_dtype == DT_F32) SA(bf16_t, float);
    else if (delta_dtype == DT_BF16 && rows_dtype == DT_BF16) SA(bf16_t, bf16_t);
    else return LLOGOS_BAD_ARGUMENT;
#undef SA
    return LLOGOS_LAUNCH_CHECK();
}

// ---------------------------------------------------------------- gelu(z) times a row of a table
// out[t, j] = gelu_tanh(sum of the parts of z[t, j]) * table[ids[t], j]
template <typename TO, typename TZ, typename TT>
__global__ void gated_lookup_kernel(TO* __restrict__ out, const TZ* __restrict__ z, int parts, size_t part_stride,
                                    const TT* __restrict__ table, const int* __restrict__ ids, int T, int N) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= T * N) return;
    const int t = i / N, j = i % N;
    const float e = load_f32(table + (size_t)ids[t] * N + j);
    float v = load_f32(z + i);
    for (int q = 1; q < parts; ++q) v += load_f32(z + q * part_stride + i);
    const float g = 0.5f * v * (1.0f + tanhf(0.7978845608028654f * (v + 0.044715f * v * v * v)));
    store_f32(out + i, g * e);
}

LLOGOS_EXPORT int llogos_gated_lookup(void* out, int dtype, const void* z, int z_dtype, int parts, long long part_stride,
                                      const void* table, int table_dtype, const int* ids, int T, int N, hipStream_t stream) {
    if (T <= 0 || N <= 0 || parts < 1 || (long long)T * N > 0x7fffffffLL) return LLOGOS_BAD_ARGUMENT;
    const unsigned blocks = (unsigned)(((size_t)T * N + 255) / 256);
#define GL(TO, TZ, TT) gated_lookup_kernel<TO, TZ, TT><<<blocks, 256, 0, stream>>>((TO*)out, (const TZ*)z, parts, (size_t)part_stride, (const TT*)table, ids, T, N)
    if (dtype == DT_F32 && z_dtype == DT_F32 && table_dtype == DT_F32) GL(float, float, float);
    else if (dtype == DT_BF16 && z_dtype == DT_F32 && table_dtype == DT_BF16) GL(bf16_t, float, bf16_t);
    else if (dtype == DT_BF16 && z_dtype == DT_BF16 && table_dtype == DT_BF16) GL(bf16_t, bf16_t, bf16_t);
    else return LLOGOS_BAD_ARGUMENT;
#undef GL
    return LLOGOS_LAUNCH_CHECK();
}
