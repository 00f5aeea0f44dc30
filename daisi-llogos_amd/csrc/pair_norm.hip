// Two sublayers that read the same rows close together:
//     v = a / sqrt(mean(a^2) + eps) * wa + b / sqrt(mean(b^2) + eps) * wb;   x <- x + v;   h = x / sqrt(mean(x^2) + eps_n) * wn
// a and b [T, H] (float or bfloat16, each maybe in float parts of a k-split product); x the float residual stream,
// written back; h the rows that the norm which reads the stream next makes (or none, without wn).  Without x the
// sum v itself is left in `delta`, float [T, H].  A factor on the sum belongs into wa and wb.  All arithmetic is 32-bit.
#include "common.h"

constexpr int kPairParts = 8;          // parts of a product whose loads are in flight together, where either comes in parts

// One block a row; a thread keeps its ITEMS values of the row in registers from pass to pass.  PARTS: 1 or kPairParts.
template <typename TA, typename TB, typename TH, int ITEMS, int PARTS>
__global__ __launch_bounds__(1024) void pair_norm_kernel(float* __restrict__ x, const TA* __restrict__ a, int a_parts, size_t a_stride,
                                                         const TB* __restrict__ b, int b_parts, size_t b_stride,
                                                         const float* __restrict__ wa, const float* __restrict__ wb, float eps,
                                                         const float* __restrict__ wn, float eps_n, TH* __restrict__ h,
                                                         float* __restrict__ delta, int H) {
    __shared__ float red[16];
    const size_t r = blockIdx.x;
    float va[ITEMS], vb[ITEMS], xv[ITEMS], fa[ITEMS], fb[ITEMS], fn[ITEMS];
    float pa[ITEMS][PARTS], pb[ITEMS][PARTS];
#pragma unroll
    for (int it = 0; it < ITEMS; ++it) {
        const int i = it * blockDim.x + threadIdx.x;
        const bool ok = i < H;
        xv[it] = (ok && x) ? x[r * H + i] : 0.f;
        fa[it] = ok ? wa[i] : 0.f;
        fb[it] = ok ? wb[i] : 0.f;
        fn[it] = (ok && wn) ? wn[i] : 0.f;
#pragma unroll
        for (int q = 0; q < PARTS; ++q) {
            pa[it][q] = (ok && q < a_parts) ? load_f32(a + q * a_stride + r * H + i) : 0.f;
            pb[it][q] = (ok && q < b_parts) ? load_f32(b + q * b_stride + r * H + i) : 0.f;
        }
    }
    float sa = 0.f, sb = 0.f;
#pragma unroll
    for (int it = 0; it < ITEMS; ++it) {
        const int i = it * blockDim.x + threadIdx.x;
        float ta = pa[it][0], tb = pb[it][0];
#pragma unroll
        for (int q = 1; q < PARTS; ++q) { ta += pa[it][q]; tb += pb[it][q]; }       // ascending order
        if (i < H) {
            for (int q = PARTS; q < a_parts; ++q) ta += load_f32(a + q * a_stride + r * H + i);
            for (int q = PARTS; q < b_parts; ++q) tb += load_f32(b + q * b_stride + r * H + i);
        }
        va[it] = ta;
        vb[it] = tb;
        sa = fmaf(ta, ta, sa);
        sb = fmaf(tb, tb, sb);
    }
    const float ia = 1.0f / sqrtf(block_sum(sa, red) / (float)H + eps);
    const float ib = 1.0f / sqrtf(block_sum(sb, red) / (float)H + eps);
    float ss = 0.f;
#pragma unroll
    for (int it = 0; it < ITEMS; ++it) {
        const int i = it * blockDim.x + threadIdx.x;
        const float t = xv[it] + (va[it] * ia * fa[it] + vb[it] * ib * fb[it]);
        if (i < H) {
            if (x) x[r * H + i] = t;
            else delta[r * H + i] = t;
        }
        va[it] = t;
        ss = fmaf(t, t, ss);
    }
    if (!wn) return;
    const float in = 1.0f / sqrtf(block_sum(ss, red) / (float)H + eps_n);
#pragma unroll
    for (int it = 0; it < ITEMS; ++it) {
        const int i = it * blockDim.x + threadIdx.x;
        if (i < H) store_f32(h + r * H + i, va[it] * in * fn[it]);
    }
}

LLOGOS_EXPORT int llogos_pair_norm(float* x, const void* a, int a_dtype, int a_parts, long long a_stride, const void* b, int b_dtype,
                                   int b_parts, long long b_stride, const float* wa, const float* wb, float eps, const float* wn,
                                   float eps_n, void* h, int h_dtype, float* delta, int T, int H, hipStream_t stream) {
    if (T <= 0 || H <= 0 || H > 16384 || a_parts < 1 || b_parts < 1 || !wa || !wb || (!x && !delta) || (wn && (!h || !x))) return LLOGOS_BAD_ARGUMENT;
    int items = T >= 256 ? 4 : 1;
    while ((H + items - 1) / items > 1024) items *= 2;
    const int threads = ((H + items - 1) / items + kWave - 1) / kWave * kWave;
#define PNP(TA, TB, TH, IT, PARTS) pair_norm_kernel<TA, TB, TH, IT, PARTS><<<T, threads, 0, stream>>>(x, (const TA*)a, a_parts, (size_t)a_stride, \
        (const TB*)b, b_parts, (size_t)b_stride, wa, wb, eps, wn, eps_n, (TH*)h, delta, H)
#define PN(TA, TB, TH, IT) do { if (a_parts == 1 && b_parts == 1) PNP(TA, TB, TH, IT, 1); else PNP(TA, TB, TH, IT, kPairParts); } while (0)
#define PNI(TA, TB, TH) do { if (items == 1) PN(TA, TB, TH, 1); else if (items == 2) PN(TA, TB, TH, 2); else if (items == 4) PN(TA, TB, TH, 4); \
        else if (items == 8) PN(TA, TB, TH, 8); else PN(TA, TB, TH, 16); } while (0)
    if (h && h_dtype != DT_F32 && h_dtype != DT_BF16) return LLOGOS_BAD_ARGUMENT;
    const bool hb = h && h_dtype == DT_BF16;
    if (a_dtype == DT_F32 && b_dtype == DT_F32) { if (hb) PNI(float, float, bf16_t); else PNI(float, float, float); }
    else if (a_dtype == DT_BF16 && b_dtype == DT_BF16) { if (hb) PNI(bf16_t, bf16_t, bf16_t); else PNI(bf16_t, bf16_t, float); }
    else if (a_dtype == DT_F32 && b_dtype == DT_BF16) { if (hb) PNI(float, bf16_t, bf16_t); else PNI(float, bf16_t, float); }
    else if (a_dtype == DT_BF16 && b_dtype == DT_F32) { if (hb) PNI(bf16_t, float, bf16_t); else PNI(bf16_t, float, float); }
    else return LLOGOS_BAD_ARGUMENT;
#undef PNI
#undef PN
#undef PNP
    return LLOGOS_LAUNCH_CHECK();
}
